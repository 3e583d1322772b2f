"""Small configurations and random weights of token language models for the tests."""
import math

import torch


def attn(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, base=9000.0, dims=None, scale=None, kv_from=None):
    mx = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, rot=dict(dims=rot_dim if dims is None else dims, base=base),
              scale=1.0 / math.sqrt(dim + rot_dim) if scale is None else scale)
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mx)


def gru(width=72):
    return dict(type="mingru", mixer=dict(width=width))


def config(layers, width=80, vocab=301, ff=100, limit=2.5, eps=3e-5):
    """ff: one number for all layers, or a list with one entry per layer (None: no feed-forward)."""
    out = []
    for i, layer in enumerate(layers):
        f = ff[i] if isinstance(ff, (list, tuple)) else ff
        out.append(dict(layer, mlp=None if f is None else dict(kind="dense", ff=f, limit=limit)))
    return dict(architecture="Sakupel", width=width, vocab=vocab, norm=dict(eps=eps), layers=out)


def mixed(**kw):
    """Every kind of layer, a shared latent two layers away, unequal sizes."""
    return config([attn(), gru(), attn(heads=2, dim=10, vdim=18, kv_rank=56, kv_from=0), gru(33), attn(heads=5, dim=16, rot_dim=4, vdim=8, kv_rank=30),
                   attn(heads=1, dim=40, rot_dim=4, vdim=50, kv_rank=30, kv_from=4)], ff=[100, 60, None, 7, 100, 41], **kw)


def weights(cfg, seed=0, q_gain=1.0):
    """bf16-representable weights under the checkpoint's names; q_gain sharpens the attention."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    sd = {}

    def mat(name, n, k, gain=1.0):
        sd[name] = (gain * torch.randn(n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)

    def one(name):
        sd[name] = (0.5 + torch.rand((), generator=g)).to(torch.bfloat16)

    sd["embed"] = torch.randn(cfg["vocab"], W, generator=g).to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        one(p + "norm1")
        if layer["type"] == "latent_attention":
            H = mx["heads"]
            mat(p + "mix.q", H * (mx["dim"] + mx["rot_dim"]), W, q_gain)
            if mx.get("kv_from") is None:
                mat(p + "mix.dkv", mx["kv_rank"] + mx["rot_dim"], W)
                sd[p + "mix.dkv.norm"] = (0.5 + torch.rand(mx["kv_rank"], generator=g)).to(torch.bfloat16)
            mat(p + "mix.uk", H * mx["dim"], mx["kv_rank"])
            mat(p + "mix.uv", H * mx["vdim"], mx["kv_rank"])
            mat(p + "mix.g", H, W)
            mat(p + "mix.o", W, H * mx["vdim"], 2.0)
        else:
            n = mx["width"]
            for k in ("z", "x", "g"):
                mat(p + "mix." + k, n, W)
            sd[p + "mix.z.b"] = (torch.randn(n, generator=g) - 2.0).to(torch.bfloat16)
            sd[p + "mix.x.b"] = torch.randn(n, generator=g).to(torch.bfloat16)
            mat(p + "mix.o", W, n, 2.0)
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            mat(p + "mlp.gate", f, W, 2.0)
            mat(p + "mlp.up", f, W, 2.0)
            mat(p + "mlp.down", W, f)
    one("final.norm")
    mat("head", cfg["vocab"], W)
    return sd


# ---- sandwich layers (Mabidra); keys with an underscore are tensor shapes that no configuration names ----
def sig(heads=4, kv_heads=2, dim=24, vdim=40, bias_max=50, buckets=12, scale=0.4, q_temp=(0.4, 7)):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, bias_max=bias_max, scale=scale, _buckets=buckets)
    if q_temp is not None:
        mx["q_temp"] = dict(coef=q_temp[0], every=q_temp[1])
    return dict(type="attention", mixer=mx)


def gla(heads=3, dim=20, vdim=36, tau=5.0, rank=7):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau, _rank=rank))


def dense(ff=100):
    return dict(kind="dense", ff=ff)


def moe(ff=44, experts=9, top=3):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def sandwich(layers, width=80, vocab=301, groups=4, eps=3e-5, scale=2.5, loop=None):
    """layers: (mixer, feed-forward or None) pairs; loop: (start, stop, times)."""
    out = dict(architecture="Mabidra", width=width, vocab=vocab, norm=dict(eps=eps, groups=groups), embedding=dict(scale=scale),
               layers=[dict(m, mlp=f) for m, f in layers])
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def sandwich_mixed(**kw):
    """Every kind of layer, unequal sizes, a loop in the middle; the experts come last, so that a choice another
    rounding would have made differently stays in its own position."""
    return sandwich([(sig(), dense()), (gla(), dense(60)), (sig(heads=6, kv_heads=1, dim=10, vdim=18, bias_max=9, buckets=8, q_temp=None), None),
                     (gla(heads=2, dim=33, vdim=8, tau=1.0, rank=3), dense(41)), (sig(heads=2, kv_heads=2, dim=40, vdim=50), moe())],
                    loop=kw.pop("loop", (1, 4, 2)), **kw)


def sandwich_weights(cfg, seed=0):
    """bf16-representable weights under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    sd = {}

    def mat(name, n, k, gain=1.0):
        sd[name] = (gain * torch.randn(n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)

    def vec(name, n, gain=1.0, at=0.0):
        sd[name] = (at + gain * torch.randn(n, generator=g)).to(torch.bfloat16)

    def norm(name, n):
        sd[name] = (0.5 + torch.rand(n, generator=g)).to(torch.bfloat16)

    sd["embed"] = torch.randn(cfg["vocab"], W, generator=g).to(torch.bfloat16)
    if cfg.get("loop"):
        mat("loop.in", W, 2 * W)
        sd["loop.step"] = (0.5 * torch.randn(cfg["loop"]["times"], W, generator=g)).to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp is not None else ()):
            norm(p + n, W)
        H, dim, vdim = mx["heads"], mx["dim"], mx["vdim"]
        if layer["type"] == "attention":
            for n, rows in (("q", H * dim), ("k", mx["kv_heads"] * dim), ("v", mx["kv_heads"] * vdim)):
                mat(p + "mix." + n, rows, W)
                vec(p + "mix." + n + ".b", rows, 0.3)
            for n in ("q.norm", "k.norm"):
                norm(p + "mix." + n, dim)
            sd[p + "mix.rel"] = (1.5 * torch.randn(mx["_buckets"], H, generator=g)).to(torch.bfloat16)
            vec(p + "mix.pb", H, 0.5, -2.0)
            mat(p + "mix.g", H, W)
            mat(p + "mix.o", W, H * vdim)
            vec(p + "mix.o.b", W, 0.3)
        else:
            for n, rows in (("q", H * dim), ("k", H * dim), ("v", H * vdim), ("g", H * vdim)):
                mat(p + "mix." + n, rows, W)
            mat(p + "mix.a1", mx["_rank"], W)
            mat(p + "mix.a2", H * dim, mx["_rank"])
            vec(p + "mix.a2.b", H * dim, 2.0)
            norm(p + "mix.norm", vdim)
            mat(p + "mix.o", W, H * vdim)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            mat(p + "mlp.up", mlp["ff"], W)
            mat(p + "mlp.down", W, mlp["ff"])
            vec(p + "mlp.act", 2)
        else:
            E, f = mlp["router"]["experts"], mlp["expert"]["ff"]
            for e in range(E):
                mat(f"{p}mlp.e{e}.up", f, W)
                mat(f"{p}mlp.e{e}.down", W, f)
            mat(p + "mlp.router", E, W)
            vec(p + "mlp.router.b", E, 0.5)
    norm("final.norm", W)
    mat("head", cfg["vocab"], W)
    return sd


def tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def engine(cfg, sd, dtype=torch.float32, max_rows=2, max_seq=256):
    from vui_amd.lm import TokenLM
    from vui_amd.lm_engine import TokenEngine

    return TokenEngine(model=TokenLM.from_config(cfg, sd, dtype=dtype, max_seqlen=max_seq), max_rows=max_rows)


# Largest error of a position's logits, as a fraction of their root mean square.  fp32: sums of some hundred products
# in another order.  bf16: operands rounded to 8 bits, a handful of layers deep.
TOL = {torch.float32: 2e-5, torch.bfloat16: 0.04}


def err(got, ref):
    """Per position: root mean square of the difference over that of the reference."""
    got, ref = got.double().cpu(), ref.double().cpu()
    return ((got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt()).max().item()


def err_clear(got, ref, margins, least=0.05):
    """err() over the positions whose experts were no close call (bf16: a choice may fall differently)."""
    ok = torch.stack([m >= least for m in margins]).all(0) if margins else torch.ones(len(ref), dtype=torch.bool)
    assert ok.float().mean() > 0.3
    return err(got.cpu()[ok], ref[ok])
