"""CPU oracle for the token language models (vui_amd.lm).  TEST INFRASTRUCTURE ONLY.

Plain, slow restatements, one function per mechanism, written from the design's equations; nothing is shared with the
product path.  Everything runs in the dtype of its inputs (the tests use float64 or float32); weights arrive under the
names of the checkpoint.  A sequence is processed as a whole: there is no cache and no state here.
"""
from __future__ import annotations

import math

import torch

Tensor = torch.Tensor


def rms_unit(x: Tensor, eps: float) -> Tensor:
    """x over its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def scalar_norm(x: Tensor, g: Tensor, eps: float) -> Tensor:
    """RMS norm with a scalar weight."""
    return rms_unit(x, eps) * g.reshape(())


def rotate_half(x: Tensor, pos: int, dims: int, base: float) -> Tensor:
    """Rotates the first dims entries of the last axis at position pos: entry i pairs with entry i + dims / 2, the
    angle of pair i is pos * base^(-2 i / dims); the rest passes."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def latent_entries(h: Tensor, w: dict, p: str, mx: dict, eps: float) -> "tuple[Tensor, Tensor]":
    """What a layer with its own down-projection contributes per position: the normed latent (T, kv_rank) and the
    rotated key part common to the heads (T, rot_dim)."""
    y = h @ w[p + "dkv"].T
    c = rms_unit(y[:, :mx["kv_rank"]], eps) * w[p + "dkv.norm"]
    kr = torch.stack([rotate_half(y[t, mx["kv_rank"]:], t, mx["rot"]["dims"], mx["rot"]["base"]) for t in range(len(y))])
    return c, kr


def latent_attention(h: Tensor, c: Tensor, kr: Tensor, w: dict, p: str, mx: dict) -> Tensor:
    """Causal softmax attention with keys and values expanded from the latent, per head and per position, with the
    per-head sigmoid gate on the output."""
    T, H, dim, rot, vdim = len(h), mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dim + rot)
    ku = (c @ w[p + "uk"].T).reshape(T, H, dim)
    v = (c @ w[p + "uv"].T).reshape(T, H, vdim)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = torch.zeros(T, H, vdim, dtype=h.dtype)
    for t in range(T):
        qr = rotate_half(q[t, :, dim:], t, mx["rot"]["dims"], mx["rot"]["base"])
        for a in range(H):
            s = (ku[:t + 1, a] @ q[t, a, :dim] + kr[:t + 1] @ qr[a]) * mx["scale"]
            e = torch.exp(s - s.max())
            out[t, a] = (e / e.sum()) @ v[:t + 1, a] * gate[t, a]
    return out.reshape(T, H * vdim) @ w[p + "o"].T


def mingru(h: Tensor, w: dict, p: str, mx: dict) -> Tensor:
    """S <- (1 - z) S + z cand, channel by channel; z and cand are functions of the token at hand alone."""
    z = torch.sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    u = h @ w[p + "x"].T + w[p + "x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    gate = h @ w[p + "g"].T
    gate = gate * torch.sigmoid(gate)
    S = torch.zeros(mx["width"], dtype=h.dtype)
    rows = []
    for t in range(len(h)):
        S = (1 - z[t]) * S + z[t] * cand[t]
        rows.append(S * gate[t])
    return torch.stack(rows) @ w[p + "o"].T


def clamped_mlp(h: Tensor, w: dict, p: str, limit: float) -> Tensor:
    """Gated feed-forward with clamped branches: g sigmoid(1.702 g) (u + 1)."""
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def forward(cfg: dict, w: dict, tokens, dtype=torch.float64, layers_out: "list | None" = None) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream behind each layer."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    entries: dict = {}
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        h = scalar_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "latent_attention":
            src = mx.get("kv_from")
            if src is None:
                src = i
                entries[i] = latent_entries(h, w, p + "mix.", mx, eps)
            y = latent_attention(h, *entries[src], w, p + "mix.", mx)
        elif layer["type"] == "mingru":
            y = mingru(h, w, p + "mix.", mx)
        else:
            raise ValueError(layer["type"])
        if layer.get("mlp") is not None:
            y = y + clamped_mlp(h, w, p + "mlp.", layer["mlp"]["limit"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return scalar_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg: dict, w: dict, tokens, n: int, dtype=torch.float64) -> "list[int]":
    """n tokens drawn greedily, the whole sequence recomputed for each."""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(forward(cfg, w, seq, dtype)[-1].argmax()))
    return seq[len(tokens):]
