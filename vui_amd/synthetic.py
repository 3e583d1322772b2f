"""Random-init checkpoints of a given architecture (there is no trained checkpoint offline): the
state-dict keys and shapes of the reference model (src/vui/model.py:1076-1136, 577-663) filled
with per-key seeded N(0, std) values, norm weights 1, eos bias 0.  Used by the benchmark."""
from __future__ import annotations

import torch
from torch import Tensor

from .config import Config, DataConfig, VuiConfig, nano_config


def state_dict_shapes(m: VuiConfig) -> dict[str, tuple[int, ...]]:
    H, KV, hd, d = m.n_heads, m.kv_heads, m.head_dim, m.d_model
    sh: dict[str, tuple[int, ...]] = {}
    sh["token_emb.weight"] = (m.vocab_size, d)
    sh["audio_emb.embedding.weight"] = (m.n_quantizers * m.codebook_size, d)
    sh["codec_head.weight"] = (m.codebook_size, d)
    sh["eos_head.weight"] = (1, d)
    sh["eos_head.bias"] = (1,)
    for i in range(m.n_layers):
        p = f"decoder.blocks.{i}."
        sh[p + "attn_norm.weight"] = (d,)
        sh[p + "attn.Wqkv.weight"] = ((H + 2 * KV) * hd, d)
        sh[p + "attn.out_proj.weight"] = (d, d)
        sh[p + "mlp_norm.weight"] = (d,)
        sh[p + "mlp.w1.weight"] = (m.ffn, d)
        sh[p + "mlp.w3.weight"] = (m.ffn, d)
        sh[p + "mlp.w2.weight"] = (d, m.ffn)
    sh["decoder.norm.weight"] = (d,)
    R = m.rq_d_model
    if R != d:
        sh["rq_transformer.backbone_proj.weight"] = (R, d)
    sh["rq_transformer.code_emb.embedding.weight"] = ((m.n_quantizers - 1) * m.codebook_size, R)
    sh["rq_transformer.pos_emb.weight"] = (m.n_quantizers, R)
    sh["rq_transformer.head_W"] = (m.n_quantizers - 1, m.codebook_size, R)
    sh["rq_transformer.norm.weight"] = (R,)
    for i in range(m.rq_n_layers):
        p = f"rq_transformer.blocks.{i}."
        sh[p + "attn_norm.weight"] = (R,)
        sh[p + "Wqkv.weight"] = (3 * R, R)
        sh[p + "out_proj.weight"] = (R, R)
        sh[p + "mlp_norm.weight"] = (R,)
        sh[p + "w1.weight"] = (m.rq_ffn, R)
        sh[p + "w3.weight"] = (m.rq_ffn, R)
        sh[p + "w2.weight"] = (R, m.rq_ffn)
    return sh


def synthetic_state_dict(m: VuiConfig, seed: int = 0, std: float = 0.02) -> dict[str, Tensor]:
    """Each key draws from its own CPU generator seeded with (seed, key index)."""
    sd = {}
    for idx, (k, shape) in enumerate(state_dict_shapes(m).items()):
        g = torch.Generator().manual_seed(seed * 1000003 + idx)
        if k.endswith("norm.weight"):
            sd[k] = torch.ones(shape)
        elif k.endswith(".bias"):
            sd[k] = torch.zeros(shape)
        else:
            sd[k] = std * torch.randn(shape, generator=g)
    return sd


def nano_for_cache(preset: str, max_seqlen: int) -> Config:
    """Vui Nano with the backbone's position table / cache cut to max_seqlen positions
    (decoder.max_seqlen = max_text_tokens + max_audio_tokens + Q when data.max_secs gives 0,
    src/vui/model.py:1069-1073, 1127)."""
    cfg = nano_config(preset)
    cfg.data = DataConfig(max_secs=0)
    cfg.model.has_spk_proj = False
    cfg.model.max_text_tokens = max_seqlen - cfg.model.n_quantizers
    cfg.model.max_audio_tokens = 0
    return cfg


def synthetic_codec_state_dict(cfg, seed: int = 0) -> dict[str, Tensor]:
    """Deterministic fp32 vocoder weights (vui_amd.codec.CodecConfig) that keep activations O(1) through
    its ~60 layers: linear and conv weights N(0, 1/fan_in), biases N(0, 0.05), norm weights 1 + N(0, 0.1),
    snake log-rates N(0, 0.3), residual scales N(0.3, 0.1), codebooks N(0, 1); the closing 1x1 conv of every
    residual unit is scaled by 0.3 and the last conv by 0.12.  Each key draws from its own CPU generator
    seeded with (seed, key index)."""
    import math

    from .codec import codec_state_dict_shapes

    sd = {}
    for idx, (k, shape) in enumerate(codec_state_dict_shapes(cfg).items()):
        g = torch.Generator().manual_seed(seed * 1000003 + 7919 + idx)
        r = torch.randn(shape, generator=g)
        if k.endswith("embed"):
            t = r
        elif k.endswith(("alpha", "beta")):
            t = 0.3 * r
        elif k.endswith(("attn_scale", "mlp_scale", "gamma")):
            t = 0.3 + 0.1 * r
        elif k.endswith("norm.weight"):
            t = 1.0 + 0.1 * r
        elif k.endswith(".bias"):
            t = 0.05 * r
        elif len(shape) == 3 and (".block.1." in k or (k.startswith("upsample") and ".0.conv" in k)):
            stride = shape[2] if k.startswith("upsample") else shape[2] // 2
            t = r / math.sqrt(shape[0] * shape[2] / stride)
        elif len(shape) == 3:
            t = r / math.sqrt(shape[1] * shape[2])
            if "conv2.conv" in k:
                t = 0.3 * t
            elif shape[0] == 1:
                t = 0.12 * t
        else:
            t = r / math.sqrt(shape[-1])
        sd[k] = t.contiguous()
    return sd


def token_lm_config(width: int, heads: int, ff: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, n_layers: int,
                    vocab: int = 8192, rnn_width: int = 0) -> dict:
    """A Sakupel configuration whose layers repeat the pattern: attention with own latents, minGRU, attention on the
    latents of the first, attention with own latents."""
    layers = []
    own = 0
    for i in range(n_layers):
        mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
        if i % 4 == 1:
            layers.append({"type": "mingru", "mixer": {"width": rnn_width or width}, "mlp": mlp})
            continue
        mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
              "scale": (dim + rot_dim) ** -0.5, "rot": {"dims": rot_dim, "base": 10000.0}}
        if i % 4 == 2:
            mx["kv_from"] = own
        else:
            own = i
        layers.append({"type": "latent_attention", "mixer": mx, "mlp": mlp})
    return {"architecture": "Sakupel", "width": width, "vocab": vocab, "norm": {"eps": 1e-5}, "layers": layers}


def sandwich_lm_config(width: int, heads: int, kv_heads: int, dim: int, ff: int, experts: int, top: int, n_layers: int,
                       vocab: int = 8192, rank: int = 32) -> dict:
    """A Mabidra configuration whose layers repeat the pattern: gated linear attention, attention, attention, attention;
    every second feed-forward is made of experts, `top` of which have the ff features of a dense one together.  One
    pass over all layers (a loop of one time, so that its mixing product is there)."""
    layers = []
    for i in range(n_layers):
        mlp = {"kind": "dense", "ff": ff} if i % 2 == 0 else {
            "kind": "moe", "expert": {"ff": ff // top}, "router": {"experts": experts, "top": top}}
        if i % 4 == 0:
            layers.append({"type": "gla", "mixer": {"heads": heads // 2, "dim": dim, "vdim": 2 * dim, "tau": 8.0}, "mlp": mlp})
            continue
        layers.append({"type": "attention", "mlp": mlp, "mixer": {
            "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "bias_max": 1000,
            "q_temp": {"coef": 0.1, "every": 500}}})
    return {"architecture": "Mabidra", "width": width, "vocab": vocab, "norm": {"eps": 1e-5, "groups": 4}, "layers": layers,
            "embedding": {"scale": 1.0}, "loop": {"start": 0, "stop": n_layers, "times": 1}, "gla_rank": rank}


def token_lm_state_dict(cfg: dict, seed: int = 0, device="cpu") -> dict[str, Tensor]:
    """Random bf16 weights N(0, 1 / fan_in) of a token model's configuration, norm weights 1, biases 0 (`gla_rank`: rank of
    the decays of gated linear attention, which a checkpoint tells by a shape)."""
    g = torch.Generator(device=device).manual_seed(seed)
    W = cfg["width"]
    sd: dict[str, Tensor] = {}

    def mat(name: str, n: int, k: int) -> None:
        sd[name] = (torch.randn(n, k, generator=g, device=device) * k ** -0.5).to(torch.bfloat16)

    def ones(name: str, *shape: int) -> None:
        sd[name] = torch.ones(shape, dtype=torch.bfloat16, device=device)

    def zeros(name: str, *shape: int) -> None:
        sd[name] = torch.zeros(shape, dtype=torch.bfloat16, device=device)

    sandwich = cfg["architecture"] == "Mabidra"
    mat("embed", cfg["vocab"], W)
    if cfg.get("loop"):
        mat("loop.in", W, 2 * W)
        zeros("loop.step", cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        if sandwich:
            H, m = mx["heads"], p + "mix."
            G = mx.get("kv_heads", H)
            for k in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] else ()):
                ones(p + k, W)
            for k, n in (("q", H * mx["dim"]), ("k", G * mx["dim"]), ("v", G * mx["vdim"])):
                mat(m + k, n, W)
            mat(m + "o", W, H * mx["vdim"])
            if layer["type"] == "gla":
                r = cfg.get("gla_rank", 16)
                mat(m + "g", H * mx["vdim"], W)
                mat(m + "a1", r, W)
                mat(m + "a2", H * mx["dim"], r)
                zeros(m + "a2.b", H * mx["dim"])
                ones(m + "norm", mx["vdim"])
            else:
                mat(m + "g", H, W)
                for k, n in (("q", H * mx["dim"]), ("k", G * mx["dim"]), ("v", G * mx["vdim"]), ("o", W)):
                    zeros(m + k + ".b", n)
                ones(m + "q.norm", mx["dim"])
                ones(m + "k.norm", mx["dim"])
                mat(m + "rel", 32, H)
                zeros(m + "pb", H)
            mlp = layer["mlp"]
            if mlp is not None and mlp["kind"] == "moe":
                f = mlp["expert"]["ff"]
                for e in range(mlp["router"]["experts"]):
                    mat(f"{p}mlp.e{e}.up", f, W)
                    mat(f"{p}mlp.e{e}.down", W, f)
                mat(p + "mlp.router", mlp["router"]["experts"], W)
                zeros(p + "mlp.router.b", mlp["router"]["experts"])
            elif mlp is not None:
                mat(p + "mlp.up", mlp["ff"], W)
                mat(p + "mlp.down", W, mlp["ff"])
                zeros(p + "mlp.act", 2)
            continue
        ones(p + "norm1")
        if layer["type"] == "latent_attention":
            H, r = mx["heads"], mx["kv_rank"]
            mat(p + "mix.q", H * (mx["dim"] + mx["rot_dim"]), W)
            if mx.get("kv_from") is None:
                mat(p + "mix.dkv", r + mx["rot_dim"], W)
                ones(p + "mix.dkv.norm", r)
            mat(p + "mix.uk", H * mx["dim"], r)
            mat(p + "mix.uv", H * mx["vdim"], r)
            mat(p + "mix.g", H, W)
            mat(p + "mix.o", W, H * mx["vdim"])
        else:
            n = mx["width"]
            for k in ("z", "x", "g"):
                mat(p + "mix." + k, n, W)
            for k in ("z.b", "x.b"):
                zeros(p + "mix." + k, n)
            mat(p + "mix.o", W, n)
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            mat(p + "mlp.gate", f, W)
            mat(p + "mlp.up", f, W)
            mat(p + "mlp.down", W, f)
    ones("final.norm", *((W,) if sandwich else ()))
    mat("head", cfg["vocab"], W)
    return sd
