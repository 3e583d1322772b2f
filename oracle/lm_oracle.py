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


# ---- mechanisms of the design Mabidra ----
def grouped_norm(x: Tensor, w: Tensor, groups: int, eps: float) -> Tensor:
    """Every one of `groups` equal consecutive parts over its own root mean square, then one weight per entry."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms_unit(parts, eps).reshape(x.shape) * w


def gated_linear_attention(h: Tensor, w: dict, p: str, mx: dict, eps: float) -> Tensor:
    """S <- diag(a) S + k v^T per head, read by q; a decays the rows of S (one number per key channel); the read is
    normed per head and multiplied by silu of a gate."""
    T, H, dim, vdim = len(h), mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dim) / math.sqrt(dim)
    k = (h @ w[p + "k"].T).reshape(T, H, dim)
    v = (h @ w[p + "v"].T).reshape(T, H, vdim)
    z = h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "a2.b"]
    a = torch.exp(torch.nn.functional.logsigmoid(z) / mx["tau"]).reshape(T, H, dim)
    g = h @ w[p + "g"].T
    S = torch.zeros(H, dim, vdim, dtype=h.dtype)
    rows = []
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o = (S * q[t][:, :, None]).sum(dim=1)
        rows.append((rms_unit(o, eps) * w[p + "norm"]).reshape(-1))
    return (torch.stack(rows) * g * torch.sigmoid(g)) @ w[p + "o"].T


def distance_bucket(n: int, buckets: int, far: int) -> int:
    """Bucket of a distance n >= 0: one each below buckets / 2, then logarithmic, full at `far`."""
    half = buckets // 2
    if n < half:
        return n
    if half < 1 or far <= half:
        return buckets - 1
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (buckets - half) + 1e-9))


def sigmoid_attention(h: Tensor, w: dict, p: str, mx: dict, eps: float) -> Tensor:
    """Causal attention whose weights are sigmoids of the scores: normed queries and keys, a temperature that grows with
    the position, a bias per distance bucket and head, a number per head, a gate per head on the output."""
    T, H, G, dim, vdim = len(h), mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = rms_unit((h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, dim), eps) * w[p + "q.norm"]
    k = rms_unit((h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, dim), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, vdim)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    rel = w[p + "rel"]
    bucket = torch.tensor([distance_bucket(n, len(rel), mx["bias_max"]) for n in range(T)])
    qt = mx.get("q_temp")
    out = torch.zeros(T, H, vdim, dtype=h.dtype)
    for t in range(T):
        temp = 1.0 + qt["coef"] * math.log((t + 1) // qt["every"] + 1) if qt else 1.0
        for a in range(H):
            b = a // (H // G)
            s = (k[:t + 1, b] @ (q[t, a] * temp)) * mx["scale"] + rel[bucket[:t + 1].flip(0), a] + w[p + "pb"][a]
            out[t, a] = torch.sigmoid(s) @ v[:t + 1, b] * gate[t, a]
    return out.reshape(T, H * vdim) @ w[p + "o"].T + w[p + "o.b"]


def xielu(z: Tensor, p: Tensor, q: Tensor) -> Tensor:
    """Quadratic above zero, exponential below, slope 1/2 at zero; p and q pass through softplus."""
    sp = torch.nn.functional.softplus
    neg = torch.clamp(z, max=0.0)
    return torch.where(z > 0, sp(p) * z * z, (0.5 + sp(q)) * (torch.expm1(neg) - neg)) + z / 2


def xielu_mlp(h: Tensor, w: dict, p: str) -> Tensor:
    return xielu(h @ w[p + "up"].T, *w[p + "act"]) @ w[p + "down"].T


def expert_mlp(h: Tensor, w: dict, p: str, router: dict, margins: "list | None" = None) -> Tensor:
    """The `top` experts with the largest router logits per token, weighed by a softmax over those; relu squared inside.
    margins, if given, receives how far every token was from another choice (T)."""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    out = torch.zeros_like(h)
    for t in range(len(h)):
        best = torch.topk(z[t], router["top"])
        share = torch.softmax(best.values, 0)
        for e, s in zip(best.indices.tolist(), share):
            out[t] += s * (torch.relu(h[t] @ w[f"{p}e{e}.up"].T).square() @ w[f"{p}e{e}.down"].T)
    if margins is not None:
        v = torch.sort(z, dim=1, descending=True).values
        margins.append(v[:, router["top"] - 1] - v[:, router["top"]] if router["top"] < v.shape[1] else torch.full_like(v[:, 0], math.inf))
    return out


def layer_passes(cfg: dict) -> "list[tuple[int, int | None]]":
    """The layers in the order they run: (layer, number of the pass it starts, or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward_sandwich(cfg: dict, w: dict, tokens, layers_out: "list | None" = None, margins: "list | None" = None) -> Tensor:
    """Mabidra: norms on both sides of every sublayer, a loop over some layers that mixes the embedding back in."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i, start in layer_passes(cfg):
        p, layer = f"l{i}.", cfg["layers"][i]
        mx = layer["mixer"]
        if start is not None:
            x = torch.cat((x, x0), dim=-1) @ w["loop.in"].T + w["loop.step"][start]
        h = grouped_norm(x, w[p + "norm1"], groups, eps)
        if layer["type"] == "gla":
            y = gated_linear_attention(h, w, p + "mix.", mx, eps)
        elif layer["type"] == "attention":
            y = sigmoid_attention(h, w, p + "mix.", mx, eps)
        else:
            raise ValueError(layer["type"])
        x = x + grouped_norm(y, w[p + "norm1b"], groups, eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = grouped_norm(x, w[p + "norm2"], groups, eps)
            y = xielu_mlp(h, w, p + "mlp.") if mlp["kind"] == "dense" else expert_mlp(h, w, p + "mlp.", mlp["router"], margins)
            x = x + grouped_norm(y, w[p + "norm2b"], groups, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return grouped_norm(x, w["final.norm"], groups, eps) @ w["head"].T


def forward(cfg: dict, w: dict, tokens, dtype=torch.float64, layers_out: "list | None" = None, margins: "list | None" = None) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream behind each layer run."""
    w = {k: v.to(dtype) for k, v in w.items()}
    if cfg["architecture"] == "Mabidra":
        return forward_sandwich(cfg, w, tokens, layers_out, margins)
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
