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
