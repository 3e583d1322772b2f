"""Token language models on a machine without a GPU: the oracle against closed forms, the operand layout, configuration
and registry, the scheduler's and the trace replay's bookkeeping."""
import ctypes as C
import json
import math
import os

import pytest
import torch

from oracle import lm_oracle as O
from tests import lm_util as U


# ---- oracle ----
def test_rotate_half_pairs_and_relative_positions():
    x, y = torch.randn(2, 7, generator=torch.Generator().manual_seed(0), dtype=torch.float64)
    r = O.rotate_half(x, 5, 6, 100.0)
    for i in range(3):
        a = 5 * 100.0 ** (-2 * i / 6)
        z = complex(x[i], x[i + 3]) * complex(math.cos(a), math.sin(a))
        assert abs(r[i] - z.real) < 1e-12 and abs(r[i + 3] - z.imag) < 1e-12
    assert r[6] == x[6]  # beyond the rotated dims
    d = [float(O.rotate_half(x, p, 6, 100.0) @ O.rotate_half(y, p + 9, 6, 100.0)) for p in (0, 4, 77)]
    assert max(d) - min(d) < 1e-10


def test_mingru_is_a_convex_average_of_candidates():
    cfg = U.config([U.gru(11)], ff=None)
    w = {k: v.double() for k, v in U.weights(cfg, 1).items()}
    h = torch.randn(9, cfg["width"], generator=torch.Generator().manual_seed(2), dtype=torch.float64)
    got = O.mingru(h, w, "l0.mix.", cfg["layers"][0]["mixer"])
    z = torch.sigmoid(h @ w["l0.mix.z"].T + w["l0.mix.z.b"])
    u = h @ w["l0.mix.x"].T + w["l0.mix.x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S = torch.stack([sum(cand[s] * z[s] * torch.prod(1 - z[s + 1:t + 1], dim=0) for s in range(t + 1)) for t in range(9)])
    ref = (S * torch.nn.functional.silu(h @ w["l0.mix.g"].T)) @ w["l0.mix.o"].T
    assert (got - ref).abs().max() < 1e-12


def test_latent_attention_equals_its_latent_space_form():
    """Scores through W_uk^T and values through W_uv after the average: the same sums."""
    cfg = U.config([U.attn()], ff=None)
    mx = cfg["layers"][0]["mixer"]
    w = {k: v.double() for k, v in U.weights(cfg, 3).items()}
    h = torch.randn(6, cfg["width"], generator=torch.Generator().manual_seed(4), dtype=torch.float64)
    c, kr = O.latent_entries(h, w, "l0.mix.", mx, 1e-5)
    ref = O.latent_attention(h, c, kr, w, "l0.mix.", mx)
    H, dim, rot, vdim = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    t = 5
    q = (h[t] @ w["l0.mix.q"].T).reshape(H, dim + rot)
    out = []
    for a in range(H):
        ql = q[a, :dim] @ w["l0.mix.uk"][a * dim:(a + 1) * dim]
        s = (c @ ql + kr @ O.rotate_half(q[a, dim:], t, rot, mx["rot"]["base"])) * mx["scale"]
        out.append(w["l0.mix.uv"][a * vdim:(a + 1) * vdim] @ (torch.softmax(s, 0) @ c) * torch.sigmoid(w["l0.mix.g"][a] @ h[t]))
    assert (torch.cat(out) @ w["l0.mix.o"].T - ref[t]).abs().max() < 1e-12


def test_norm_and_feed_forward_closed_forms():
    x = torch.tensor([[3.0, 4.0]], dtype=torch.float64)
    assert torch.allclose(O.scalar_norm(x, torch.tensor(2.0), 0.5), x * 2 / math.sqrt(12.5 + 0.5))
    w = {"gate": torch.tensor([[1.0], [1.0]]).double(), "up": torch.tensor([[1.0], [-1.0]]).double(), "down": torch.eye(2).double()}
    y = O.clamped_mlp(torch.tensor([[9.0], [-9.0]], dtype=torch.float64), w, "", 1.5)
    s = 1.5 / (1 + math.exp(-1.702 * 1.5))
    n = -9.0 / (1 + math.exp(1.702 * 9.0))  # the gate has no lower clamp
    assert torch.allclose(y, torch.tensor([[s * 2.5, s * -0.5], [n * -0.5, n * 2.5]], dtype=torch.float64))


# ---- layout ----
def test_tile_places_what_the_kernels_read():
    from vui_amd import lm_layout as LL

    for dt, ep in ((torch.bfloat16, 8), (torch.float32, 4)):
        for block in (64, 32):
            W = torch.arange(48 * 128).reshape(48, 128).to(torch.int32).float()
            W = (W % 251).to(dt)
            flat = LL.tile(W, block)
            lc = block // 4
            for r, k in ((0, 0), (5, 17), (17, 63), (40, 64), (47, 127), (31, 100)):
                kb, c = k % block, (k % block) % lc
                off = ((r >> 4) * (128 // block) + k // block) * 16 * block + (c // ep) * 64 * ep + ((r & 15) + 16 * (kb // lc)) * ep + c % ep
                assert flat[off] == W[r, k]
            assert torch.equal(LL.untile(flat, 48, 128, block), W)
    with pytest.raises(ValueError):
        LL.tile(torch.zeros(15, 64))


def test_pair_order_and_rotation_table():
    from vui_amd import lm_layout as LL

    assert LL.pair_order(7, 4).tolist() == [0, 2, 1, 3, 4, 5, 6]
    t = LL.rotation_table(4000, 6, 777.0)
    assert t.shape == (4000, 3, 2) and t.dtype == torch.float32
    for p, i in ((0, 0), (3, 1), (3999, 0), (3999, 2)):
        a = p * 777.0 ** (-2 * i / 6)
        assert abs(t[p, i, 0] - math.cos(a)) < 1e-7 and abs(t[p, i, 1] - math.sin(a)) < 1e-7


def _lib():
    from vui_amd import _lib as L

    if not os.path.exists(L.LIB_PATH):
        pytest.skip("libvui_amd.so not built")
    return L, L.load()


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
def test_projection_rows_land_where_the_header_says(dt):
    """w_in row by row against the checkpoint, for a layer of every kind."""
    from vui_amd import lm_layout as LL
    from vui_amd.config import LMConfig
    from vui_amd.lm import TokenLM

    L, lib = _lib()
    cfg = U.mixed()
    sd = {k: v.to(dt) for k, v in U.weights(cfg, 5).items()}
    m = TokenLM(LMConfig.from_dict(cfg), sd, device="cpu", dtype=dt, max_seqlen=40)
    for i, (layer, d, parts) in enumerate(zip(cfg["layers"], m.dims, m.parts)):
        mx, p = layer["mixer"], f"l{i}."
        assert d.w64 % 64 == 0 and d.out_k % 64 == 0 and d.mix_rows % 16 == 0
        w_in = LL.untile(parts["w_in"], d.in_rows, d.w64)
        assert torch.equal(w_in[:, cfg["width"]:], torch.zeros_like(w_in[:, cfg["width"]:]))
        w_in = w_in[:, :cfg["width"]]
        w_out = LL.untile(parts["w_out"], d.out_rows, d.out_k)[:cfg["width"]]
        if layer["type"] == "latent_attention":
            H, dim, rot = mx["heads"], mx["dim"], mx["rot_dim"]
            q = sd[p + "mix.q"].reshape(H, dim + rot, -1)
            r = 0
            for h in range(H):
                assert torch.equal(w_in[r:r + dim], q[h, :dim]) and not w_in[r + dim:r + d.dim16].any()
                r += d.dim16
            for h in range(H):
                assert torch.equal(w_in[r], q[h, dim]) and torch.equal(w_in[r + 1], q[h, dim + rot // 2])
                r += d.rot16
            if mx.get("kv_from") is None:
                assert torch.equal(w_in[r:r + mx["kv_rank"]], sd[p + "mix.dkv"][:mx["kv_rank"]])
                r += d.rank16 + d.rot16
            assert torch.equal(w_in[r:r + H], sd[p + "mix.g"])
            o = sd[p + "mix.o"].reshape(-1, H, mx["vdim"])
            for h in range(H):
                assert torch.equal(w_out[:, h * d.vdim16:h * d.vdim16 + mx["vdim"]], o[:, h])
            uk = LL.untile(parts["w_uk"], H * d.dim64, d.rank64).reshape(H, d.dim64, d.rank64)
            ukt = LL.untile(parts["w_uk_t"], H * d.rank16, d.dim64).reshape(H, d.rank16, d.dim64)
            assert torch.equal(uk[:, :dim, :d.rank16], ukt[:, :, :dim].transpose(1, 2))
        else:
            for ch in (0, 15, 16, mx["width"] - 1):
                for k, name in enumerate("zxg"):
                    assert torch.equal(w_in[(ch // 16) * 48 + 16 * k + ch % 16], sd[p + "mix." + name][ch])
            assert torch.equal(w_out[:, :mx["width"]], sd[p + "mix.o"])
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"] - 1
            assert torch.equal(w_in[d.mix_rows + 2 * f], sd[p + "mlp.gate"][f]) and torch.equal(w_in[d.mix_rows + 2 * f + 1], sd[p + "mlp.up"][f])
            assert torch.equal(w_out[:, d.ff_off + f], sd[p + "mlp.down"][:, f])
        else:
            assert d.in_rows == d.mix_rows and d.out_k == d.ff_off


def test_native_argument_errors():
    L, lib = _lib()
    c, layer, d = L.LmConfigC(), L.LmLayerC(), L.LmDimsC()
    c.dtype, c.width, c.vocab, c.n_layers, c.max_seqlen, c.n_slots, c.max_rows, c.norm_eps = 0, 80, 301, 1, 64, 2, 64, 1e-5
    layer.mixer, layer.kv_from, layer.rnn_width = L.LM_MINGRU, -1, 33
    assert lib.vui_lm_workspace_bytes(C.byref(c), C.byref(layer)) > 0
    layer.rnn_width = 0
    assert lib.vui_lm_workspace_bytes(C.byref(c), C.byref(layer)) < 0 and "recurrence width" in L.last_error()
    layer.mixer, layer.heads, layer.dim, layer.rot_dim, layer.rot_pairs, layer.vdim, layer.kv_rank = L.LM_LATENT_ATTENTION, 2, 8, 4, 3, 8, 16
    assert lib.vui_lm_workspace_bytes(C.byref(c), C.byref(layer)) < 0 and "latent attention sizes" in L.last_error()
    layer.rot_pairs, layer.kv_from = 2, 0
    assert lib.vui_lm_workspace_bytes(C.byref(c), C.byref(layer)) < 0 and "kv_from" in L.last_error()
    assert lib.vui_lm_decode(None, None, None, None, None, 1, None, None) == -22
    assert lib.vui_lm_prefill(None, None, 1, 0, 0, None, None, 0, None, None) == -22


# ---- configuration, registry ----
def test_config_reads_every_key_and_refuses_what_it_does_not_know():
    from vui_amd.config import LatentAttentionConfig, LMConfig, MinGRUConfig

    cfg = U.mixed(eps=7e-4)
    c = LMConfig.from_dict(json.loads(json.dumps(cfg)))
    assert (c.width, c.vocab, c.norm_eps, len(c.layers)) == (80, 301, 7e-4, 6)
    assert isinstance(c.layers[0].mixer, LatentAttentionConfig) and c.layers[0].mixer.rot.base == 9000.0
    assert c.layers[2].mixer.kv_from == 0 and c.layers[2].mlp is None and c.layers[3].mlp.ff == 7
    assert isinstance(c.layers[3].mixer, MinGRUConfig) and c.layers[3].mixer.width == 33
    for change in (lambda d: d["layers"][0].update(type="ring"), lambda d: d["layers"][0]["mlp"].update(kind="sparse"),
                   lambda d: d["layers"][2]["mixer"].update(kv_from=1), lambda d: d["layers"][2]["mixer"].update(kv_from=4),
                   lambda d: d["layers"][5]["mixer"].update(kv_from=2), lambda d: d["layers"][2]["mixer"].update(kv_rank=48),
                   lambda d: d["layers"][0]["mixer"]["rot"].update(dims=10), lambda d: d["layers"][0]["mixer"]["rot"].update(dims=3)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            LMConfig.from_dict(bad)


def test_registry_chooses_by_config(tmp_path):
    from safetensors.torch import save_file

    from vui_amd import registry
    from vui_amd.lm import TokenLM
    from vui_amd.model import Vui

    assert {"Sakupel", "Vui"} <= set(registry.registered())
    (tmp_path / "config.json").write_text(json.dumps(U.mixed()))
    assert registry.model_class(registry.read_architecture(str(tmp_path))) is TokenLM
    assert registry.model_class(registry.read_architecture({"config": {"model": {}}, "model": {}})) is Vui
    f = str(tmp_path / "v.safetensors")
    save_file({"a": torch.zeros(1)}, f, metadata={"config": json.dumps({"model": {}})})
    assert registry.read_architecture(f) == "Vui"
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.model_class("Nobody")
    with pytest.raises(FileNotFoundError):
        registry.read_architecture(str(tmp_path / "missing"))


# ---- command line ----
def test_command_line_without_a_gpu(tmp_path, capsys):
    from vui_amd.__main__ import main

    assert main(["models"]) == 0
    assert {ln.split("\t")[0] for ln in capsys.readouterr().out.splitlines()} == {"Mabidra", "Sakupel", "Vui"}
    (tmp_path / "config.json").write_text(json.dumps(U.mixed()))
    assert main(["info", str(tmp_path)]) == 0
    info = json.loads(capsys.readouterr().out)
    assert info["architecture"] == "Sakupel" and info["layers"][2] == "latent_attention<-0" and info["layers"][1] == "mingru"
    assert info["cached_values_per_token"] == 56 + 8 + 30 + 4 and info["state_bytes_per_row"] == 4 * (72 + 33)
    assert main(["generate", "--model", str(tmp_path)]) == 2
    with pytest.raises(SystemExit):
        main(["trace", "--help"])


# ---- trace replay ----
def test_trace_replay_bookkeeping(tmp_path):
    from vui_amd.trace import replay

    log = []

    class Row:
        def __init__(self, n):
            self.n, self.seen = n, 0

        def extend(self, toks, want):
            self.seen += len(toks)
            return torch.tensor([[self.n, toks[k], self.seen] for k in want], dtype=torch.float32).reshape(len(want), 3)

        def close(self):
            log.append(("close", self.n))

    class Eng:
        made = 0

        def new_row(self):
            Eng.made += 1
            return Row(Eng.made)

    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [2, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": [9], "want": [0]}, {"id": "c", "tokens": [1, 2], "want": [1]}], "end": ["b", "c"]},
             {"step": 3, "entries": [{"id": "a", "tokens": [4], "want": [0]}], "end": []}]
    said = []
    replay(Eng(), (json.dumps(s) for s in steps), str(tmp_path), said.append)
    assert said == [f"done {i}" for i in range(4)]
    assert log == [("close", 1), ("close", 2), ("close", 3)]

    def read(i):
        import numpy as np

        return np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, 3).tolist()

    assert read(0) == [[1, 7, 3], [1, 5, 3]] and not (tmp_path / "1.f32").exists()
    assert read(2) == [[2, 9, 1], [3, 2, 2]] and read(3) == [[4, 4, 1]]  # 'a' ended: the name starts anew
