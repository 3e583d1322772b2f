"""Sandwich layers of the token language models on a machine without a GPU: the oracle against closed forms, the layout,
configuration, native argument checks."""
import ctypes as C
import json
import math

import pytest
import torch

from oracle import lm_oracle as O
from tests import lm_util as U
from tests.test_lm_host import _lib


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- oracle ----
def test_grouped_norm_norms_every_part_alone():
    x = torch.tensor([[3.0, 4.0, 30.0, 40.0]], dtype=torch.float64)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=torch.float64)
    r = math.sqrt(12.5 + 0.5), math.sqrt(1250 + 0.5)
    assert torch.allclose(O.grouped_norm(x, w, 2, 0.5), torch.tensor([[3 / r[0], 8 / r[0], 90 / r[1], 160 / r[1]]], dtype=torch.float64))
    assert torch.allclose(O.grouped_norm(x, w, 1, 0.5), O.rms_unit(x, 0.5) * w)


def test_gated_linear_attention_is_a_decayed_sum():
    cfg = U.sandwich([(U.gla(tau=2.0), None)])
    mx = cfg["layers"][0]["mixer"]
    w = {k: v.double() for k, v in U.sandwich_weights(cfg, 1).items()}
    h, p = rnd(7, cfg["width"], seed=2), "l0.mix."
    H, dim, vdim = mx["heads"], mx["dim"], mx["vdim"]
    q, k = ((h @ w[p + n].T).reshape(7, H, dim) for n in "qk")
    v = (h @ w[p + "v"].T).reshape(7, H, vdim)
    la = torch.log(torch.sigmoid((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"])).reshape(7, H, dim) / 2.0
    out = torch.zeros(7, H, vdim, dtype=torch.float64)
    for t in range(7):
        for s in range(t + 1):
            share = (q[t] / math.sqrt(dim) * k[s] * torch.exp(la[s + 1:t + 1].sum(0))).sum(1)
            out[t] += share[:, None] * v[s]
    out = O.rms_unit(out, 3e-5) * w[p + "norm"]
    ref = (out.reshape(7, -1) * torch.nn.functional.silu(h @ w[p + "g"].T)) @ w[p + "o"].T
    assert (O.gated_linear_attention(h, w, p, mx, 3e-5) - ref).abs().max() < 1e-11


def test_sigmoid_attention_sums_what_it_sees():
    """Every weight pushed to one: the plain sum of the values; to zero: the output bias."""
    cfg = U.sandwich([(U.sig(), None)])
    mx, p = cfg["layers"][0]["mixer"], "l0.mix."
    w = {k: v.double() for k, v in U.sandwich_weights(cfg, 3).items()}
    h = rnd(6, cfg["width"], seed=4)
    w[p + "pb"] = torch.full_like(w[p + "pb"], 200.0)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(6, 2, 40).cumsum(0).repeat_interleave(2, dim=1)
    gate = torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    ref = (v * gate).reshape(6, -1) @ w[p + "o"].T + w[p + "o.b"]
    assert (O.sigmoid_attention(h, w, p, mx, 1e-5) - ref).abs().max() < 1e-11
    w[p + "pb"] = torch.full_like(w[p + "pb"], -200.0)
    assert (O.sigmoid_attention(h, w, p, mx, 1e-5) - w[p + "o.b"]).abs().max() < 1e-11


def test_distance_buckets():
    """Eight buckets up to 64: one each below 4, then four steps of the logarithm from 4 to 64, each a factor of two."""
    got = [O.distance_bucket(n, 8, 64) for n in range(100)]
    assert got[:4] == [0, 1, 2, 3]
    assert [got.index(b) for b in range(4, 8)] == [4, 8, 16, 32] and got[63] == got[99] == 7
    assert sorted(got) == got
    from vui_amd.lm_layout import distance_buckets

    for buckets, far in ((8, 64), (12, 50), (32, 128), (32, 257), (6, 2), (2, 10), (1, 5), (20, 160), (16, 9)):
        assert distance_buckets(400, buckets, far) == [O.distance_bucket(n, buckets, far) for n in range(400)], (buckets, far)


def test_xielu_and_experts_closed_forms():
    z = torch.tensor([-3.0, -1e-4, 0.0, 1e-4, 2.0], dtype=torch.float64)
    p, q = torch.tensor([0.3, -1.2], dtype=torch.float64)
    a, b = math.log(1 + math.exp(0.3)), 0.5 + math.log(1 + math.exp(-1.2))
    y = O.xielu(z, p, q)
    assert abs(y[0] - (b * (math.exp(-3) - 1 + 3) - 1.5)) < 1e-12 and abs(y[4] - (4 * a + 1)) < 1e-12
    assert abs((y[3] - y[1]) / 2e-4 - 0.5) < 1e-3 and y[2] == 0
    E, W, f = 4, 6, 5
    w = {f"e{e}.{n}": rnd(*s, seed=10 * e + k) for e in range(E) for k, (n, s) in enumerate((("up", (f, W)), ("down", (W, f))))}
    w["router"], w["router.b"] = rnd(E, W, seed=50), rnd(E, seed=51)
    h = rnd(3, W, seed=52)
    one = [torch.relu(h @ w[f"e{e}.up"].T) ** 2 @ w[f"e{e}.down"].T for e in range(E)]
    z = h @ w["router"].T + w["router.b"]
    full = sum(torch.softmax(z, 1)[:, e:e + 1] * one[e] for e in range(E))
    m = []
    assert torch.allclose(O.expert_mlp(h, w, "", {"top": E}, m), full) and torch.isinf(m[0]).all()
    best = z.argmax(1)
    assert torch.allclose(O.expert_mlp(h, w, "", {"top": 1}), torch.stack([one[e][t] for t, e in enumerate(best.tolist())]))


def test_layer_passes_and_the_products_runs_agree():
    from vui_amd.config import LMConfig

    for loop in (None, (0, 5, 2), (1, 4, 2), (2, 3, 4), (4, 5, 1)):
        cfg = U.sandwich_mixed(loop=loop)
        assert O.layer_passes(cfg) == LMConfig.from_dict(cfg).runs()
    assert O.layer_passes(U.sandwich_mixed(loop=(1, 3, 2))) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]


# ---- layout ----
@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
def test_matrices_land_where_the_header_says(dt):
    from vui_amd import lm_layout as LL
    from vui_amd.config import LMConfig
    from vui_amd.lm import TokenLM

    L, lib = _lib()
    cfg = U.sandwich_mixed()
    W = cfg["width"]
    sd = {k: v.to(dt) for k, v in U.sandwich_weights(cfg, 5).items()}
    m = TokenLM(LMConfig.from_dict(cfg), sd, device="cpu", dtype=dt, max_seqlen=40)
    for i, (layer, d, parts) in enumerate(zip(cfg["layers"], m.dims, m.parts)):
        mx, p = layer["mixer"], f"l{i}.mix."
        H, dim, vdim = mx["heads"], mx["dim"], mx["vdim"]
        assert d.in_rows % 32 == 0 and d.out_k % 64 == 0 and (d.dim16 % 16, d.vdim16 % 16) == (0, 0)
        w_in = LL.untile(parts["w_in"], d.in_rows, d.w64)
        assert not w_in[:, W:].any()
        r = 0
        attn = layer["type"] == "attention"
        for n, heads, size, rows in (("q", H, dim, d.dim16), ("k", mx.get("kv_heads", H), dim, d.dim16), ("v", mx.get("kv_heads", H), vdim, d.vdim16)):
            for h in range(heads):
                assert torch.equal(w_in[r:r + size, :W], sd[p + n][h * size:(h + 1) * size]) and not w_in[r + size:r + rows].any()
                if attn:
                    assert torch.equal(parts["in_bias"][r:r + size], sd[p + n + ".b"][h * size:(h + 1) * size].float())
                r += rows
        if attn:
            assert torch.equal(w_in[r:r + H, :W], sd[p + "g"])
            t = parts["dist_bias"]
            for n in (0, 1, 5, 39):
                k = min(n, t.shape[1] - 1)
                assert torch.equal(t[:, k], sd[p + "rel"][O.distance_bucket(n, mx["_buckets"], mx["bias_max"])].float() + sd[p + "pb"].float())
        else:
            for h in range(H):
                assert torch.equal(w_in[r:r + vdim, :W], sd[p + "g"][h * vdim:(h + 1) * vdim])
                r += d.vdim16
            assert torch.equal(w_in[r:r + mx["_rank"], :W], sd[p + "a1"]) and parts["rank"] == mx["_rank"]
            assert torch.equal(parts["w_a2"].reshape(H, d.dim16, -1)[:, :dim], sd[p + "a2"].float().reshape(H, dim, -1))
        w_out = LL.untile(parts["w_out"], d.out_rows, d.out_k)
        for h in range(H):
            assert torch.equal(w_out[:W, h * d.vdim16:h * d.vdim16 + vdim], sd[p + "o"][:, h * vdim:(h + 1) * vdim])
        q = f"l{i}.mlp."
        if layer["mlp"] is None:
            assert "w_up" not in parts
        elif layer["mlp"]["kind"] == "dense":
            f = layer["mlp"]["ff"]
            assert torch.equal(LL.untile(parts["w_up"], d.ff16, d.w64)[:f, :W], sd[q + "up"])
            assert torch.equal(LL.untile(parts["w_down"], d.out_rows, d.ff64)[:W, :f], sd[q + "down"])
            assert abs(parts["act_pos"] - math.log1p(math.exp(float(sd[q + "act"][0])))) < 1e-6
        else:
            E, f = layer["mlp"]["router"]["experts"], layer["mlp"]["expert"]["ff"]
            up = parts["w_up"].reshape(E, -1)
            for e in range(E):
                assert torch.equal(LL.untile(up[e], d.ff16, d.w64)[:f, :W], sd[f"{q}e{e}.up"])
    mix = LL.untile(m.loop_in, m.dims[0].out_rows, 2 * m.dims[0].w64)
    assert torch.equal(mix[:W, :W], sd["loop.in"][:, :W]) and torch.equal(mix[:W, m.dims[0].w64:m.dims[0].w64 + W], sd["loop.in"][:, W:])


# ---- configuration ----
def test_config_reads_every_key_and_refuses_what_it_does_not_know():
    from vui_amd.config import ExpertsMLPConfig, GatedLinearAttentionConfig, LMConfig, SigmoidAttentionConfig

    cfg = U.sandwich_mixed(eps=7e-4, groups=5)
    c = LMConfig.from_dict(json.loads(json.dumps(cfg)))
    assert (c.width, c.vocab, c.norm_eps, c.norm_groups, c.embed_scale) == (80, 301, 7e-4, 5, 2.5)
    assert isinstance(c.layers[0].mixer, SigmoidAttentionConfig) and c.layers[0].mixer.q_temp.every == 7 and c.layers[2].mixer.q_temp is None
    assert isinstance(c.layers[1].mixer, GatedLinearAttentionConfig) and c.layers[3].mixer.tau == 1.0 and c.layers[2].mlp is None
    assert c.layers[4].mlp == ExpertsMLPConfig(ff=44, experts=9, top=3) and (c.loop.start, c.loop.stop, c.loop.times) == (1, 4, 2)
    for change in (lambda d: d["layers"][0].update(type="latent_attention"), lambda d: d["layers"][0]["mlp"].update(kind="sparse"),
                   lambda d: d["layers"][0]["mixer"].update(kv_heads=3), lambda d: d["norm"].update(groups=3), lambda d: d["norm"].update(groups=0),
                   lambda d: d["layers"][4]["mlp"]["router"].update(top=10), lambda d: d["loop"].update(stop=6), lambda d: d["loop"].update(stop=1),
                   lambda d: d["loop"].update(times=0), lambda d: d["layers"][0]["mixer"]["q_temp"].update(every=0), lambda d: d.update(architecture="Vui")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            LMConfig.from_dict(bad)


def test_native_argument_errors():
    L, lib = _lib()

    def bytes_of(**kw):
        c, layer = L.LmConfigC(), L.LmLayerC()
        c.width, c.vocab, c.n_layers, c.max_seqlen, c.n_slots, c.max_rows, c.norm_eps, c.norm_groups = 80, 301, 1, 64, 2, 64, 1e-5, 4
        layer.mixer, layer.kv_from, layer.heads, layer.kv_heads, layer.dim, layer.vdim, layer.bias_len = L.LM_SIGMOID_ATTENTION, -1, 4, 2, 8, 8, 9
        for k, v in kw.items():
            setattr(c if hasattr(c, k) else layer, k, v)
        return lib.vui_lm_workspace_bytes(C.byref(c), C.byref(layer))

    assert bytes_of() > 0 and bytes_of(ff=40, experts=8, top=2) > bytes_of(ff=40)
    for kw, text in ((dict(norm_groups=3), "equal parts"), (dict(kv_heads=3), "kv_heads"), (dict(bias_len=0), "bias_len"), (dict(mixer=L.LM_GLA), "rank"),
                     (dict(mixer=L.LM_MINGRU), "does not go"), (dict(ff=40, experts=8, top=9), "feed-forward"), (dict(experts=8, top=2), "feed-forward"),
                     (dict(temp_coef=1.0), "temp_every"), (dict(vdim=4096), "sizes")):
        assert bytes_of(**kw) < 0 and text in L.last_error(), kw


def test_command_line_info(tmp_path, capsys):
    from vui_amd.__main__ import main

    (tmp_path / "config.json").write_text(json.dumps(U.sandwich_mixed()))
    assert main(["info", str(tmp_path)]) == 0
    info = json.loads(capsys.readouterr().out)
    assert info["layers"] == ["sigmoid_attention", "gla", "sigmoid_attention", "gla", "gla", "sigmoid_attention", "gla", "sigmoid_attention"]
    assert info["cached_values_per_token"] == 2 * 64 + 2 * 28 + 2 * 90
    assert info["state_bytes_per_row"] == 2 * 4 * (3 * 20 * 36 + 2 * 33 * 8)
