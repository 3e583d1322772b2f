"""Weights of the token language models in the form their kernels read: matrices that share an input side by side,
padded with zero rows and columns to the sizes of `vui_lm_layer_dims`, in the tiled operand layout.

Row order of an input projection (include/vui_lm.h, w_in), every segment padded to 16 rows:
* latent attention: per head the unrotated query rows, per head the rotated ones, the latent, the shared rotated key
  part, the head gates;
* minGRU: blocks of 16 channels, three at a time (update gate, candidate, output gate);
* then the feed-forward, gate and up rows alternating.
Sandwich layers, whose feed-forward is a matrix of its own:
* sigmoid attention: per head the query rows, per group the key rows, per group the value rows, the head gates;
* gated linear attention: per head query, per head key, per head value, per head gate rows, the low-rank part of the decay.
Rotated rows are reordered so that the two partners of a pair are neighbours (queries and keys alike, so scores do not
change) and an epilogue that holds four consecutive rows can rotate them."""
from __future__ import annotations

import math
from fractions import Fraction

import torch
from torch import Tensor


def pad_to(W: Tensor, rows: int, cols: int | None = None) -> Tensor:
    out = torch.zeros(rows, W.shape[1] if cols is None else cols, dtype=W.dtype, device=W.device)
    out[:W.shape[0], :W.shape[1]] = W
    return out


def tile(W: Tensor, block: int = 64) -> Tensor:
    """(rows, K) -> the tiled operand layout (flat): blocks of 16 rows x `block` columns, lane (row, column group of
    block / 4) owning block / 4 columns as 16-byte pieces; rows a multiple of 16, K of `block`."""
    N, K = W.shape
    if N % 16 or K % block:
        raise ValueError(f"{N} x {K} is not padded to 16 x {block}")
    ep = 16 // W.element_size()
    t = W.reshape(N // 16, 16, K // block, 4, block // 4 // ep, ep)
    return t.permute(0, 2, 4, 3, 1, 5).contiguous().reshape(-1)


def untile(flat: Tensor, rows: int, K: int, block: int = 64) -> Tensor:
    ep = 16 // flat.element_size()
    t = flat.reshape(rows // 16, K // block, block // 4 // ep, 4, 16, ep)
    return t.permute(0, 4, 1, 3, 2, 5).reshape(rows, K)


def pair_order(rot_dim: int, dims: int) -> Tensor:
    """Order of the rotated rows: (0, dims/2), (1, dims/2 + 1), ..., then what passes unrotated."""
    half = dims // 2
    first = torch.stack((torch.arange(half), torch.arange(half) + half), dim=1).reshape(-1)
    return torch.cat((first, torch.arange(dims, rot_dim)))


def rotation_table(n: int, dims: int, base: float) -> Tensor:
    """(n, dims / 2, 2) fp32 cos/sin; the angles are formed in float64 and rounded once."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    a = torch.arange(n, dtype=torch.float64)[:, None] * torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims)
    return torch.stack((a.cos(), a.sin()), dim=-1).float().contiguous()


def _ff_rows(gate: Tensor, up: Tensor, ff_pad: int) -> Tensor:
    return torch.stack((pad_to(gate, ff_pad), pad_to(up, ff_pad)), dim=1).reshape(2 * ff_pad, -1)


def latent_attention_weights(w: dict, p: str, mx, d) -> dict:
    """w: checkpoint tensors of one dtype; p: 'l<i>.'; mx: LatentAttentionConfig; d: vui_lm_dims."""
    m = p + "mix."
    H = mx.heads
    order = pair_order(mx.rot_dim, mx.rot.dims).to(w[m + "q"].device)
    q = w[m + "q"].reshape(H, mx.dim + mx.rot_dim, -1)
    parts = [pad_to(q[h, :mx.dim], d.dim16) for h in range(H)]
    parts += [pad_to(q[h, mx.dim:][order], d.rot16) for h in range(H)]
    if mx.kv_from is None:
        dkv = w[m + "dkv"]
        parts += [pad_to(dkv[:mx.kv_rank], d.rank16), pad_to(dkv[mx.kv_rank:][order], d.rot16)]
    parts.append(pad_to(w[m + "g"], d.heads16))
    uk = w[m + "uk"].reshape(H, mx.dim, mx.kv_rank)
    uv = w[m + "uv"].reshape(H, mx.vdim, mx.kv_rank)
    o = w[m + "o"].reshape(-1, H, mx.vdim)
    o_pad = torch.zeros(o.shape[0], H, d.vdim16, dtype=o.dtype, device=o.device)
    o_pad[:, :, :mx.vdim] = o
    # expanded keys get all dim64 columns: the pad columns of the query operand hold whatever another layer left there
    out = {
        "mix": torch.cat(parts), "out": o_pad.reshape(o.shape[0], H * d.vdim16),
        "w_uk_t": torch.cat([tile(pad_to(uk[h].T, d.rank16, d.dim64)) for h in range(H)]),
        "w_uk": torch.cat([tile(pad_to(uk[h], d.dim64, d.rank64)) for h in range(H)]),
        "w_uv": torch.cat([tile(pad_to(uv[h], d.vdim16, d.rank64)) for h in range(H)]),
    }
    if mx.kv_from is None:
        n = torch.zeros(d.rank16, dtype=torch.float32, device=o.device)
        n[:mx.kv_rank] = w[m + "dkv.norm"].float()
        out["latent_norm"] = n
    return out


def mingru_weights(w: dict, p: str, mx, d) -> dict:
    m = p + "mix."
    blocks = [pad_to(w[m + k], d.gru16).reshape(d.gru16 // 16, 16, -1) for k in ("z", "x", "g")]
    out = {"mix": torch.stack(blocks, dim=1).reshape(3 * d.gru16, -1), "out": w[m + "o"]}
    for name, key in (("bias_z", "z.b"), ("bias_x", "x.b")):
        b = torch.zeros(d.gru16, dtype=torch.float32, device=w[m + "z"].device)
        b[:mx.width] = w[m + key].float()
        out[name] = b
    return out


def layer_projections(w: dict, p: str, parts: dict, has_ff: bool, d) -> "tuple[Tensor, Tensor]":
    """w_in and w_out of a layer, tiled, from its mixer's rows / columns and its feed-forward."""
    w_in = pad_to(parts["mix"], d.mix_rows, d.w64)
    w_out = torch.zeros(d.out_rows, d.out_k, dtype=w_in.dtype, device=w_in.device)
    w_out[:parts["out"].shape[0], :parts["out"].shape[1]] = parts["out"]
    if has_ff:
        ff = _ff_rows(w[p + "mlp.gate"], w[p + "mlp.up"], d.ff_pad)
        w_in = torch.cat((w_in, pad_to(ff, ff.shape[0], d.w64)))
        down = w[p + "mlp.down"]
        w_out[:down.shape[0], d.ff_off:d.ff_off + down.shape[1]] = down
    return tile(w_in), tile(w_out)


# ---- sandwich layers ----
def vector(v: Tensor, n: int) -> Tensor:
    """fp32, zero beyond its own entries."""
    out = torch.zeros(n, dtype=torch.float32, device=v.device)
    out[:v.numel()] = v.float().reshape(-1)
    return out


def _heads(W: Tensor, heads: int, rows: int) -> Tensor:
    """(heads * d, K) -> (heads * rows, K): every head's rows padded."""
    t = W.reshape(heads, W.shape[0] // heads, -1)
    out = torch.zeros(heads, rows, t.shape[2], dtype=W.dtype, device=W.device)
    out[:, :t.shape[1]] = t
    return out.reshape(heads * rows, -1)


def _head_columns(W: Tensor, heads: int, vdim16: int, rows: int, cols: int) -> Tensor:
    """An output projection (width, heads * vdim) with every head's columns padded."""
    t = W.reshape(W.shape[0], heads, W.shape[1] // heads)
    out = torch.zeros(W.shape[0], heads, vdim16, dtype=W.dtype, device=W.device)
    out[:, :, :t.shape[2]] = t
    return pad_to(out.reshape(W.shape[0], -1), rows, cols)


def distance_buckets(n: int, buckets: int, far: int) -> "list[int]":
    """Buckets of the distances 0 .. n - 1: one each below buckets / 2, then equal steps of the logarithm up to `far`,
    everything beyond in the last.  The steps' borders are decided in exact arithmetic."""
    half = buckets // 2
    out = []
    for d in range(n):
        if d < half:
            out.append(d)
        elif half < 1 or far <= half:
            out.append(buckets - 1)
        else:
            steps = buckets - half
            x = math.log(d / half) / math.log(far / half) * steps
            k = round(x)
            if abs(x - k) < 1e-6:  # too close to call in floating point: (d / half)^steps against (far / half)^k
                k = k if Fraction(d, half) ** steps >= Fraction(far, half) ** k else k - 1
            else:
                k = math.floor(x)
            out.append(min(buckets - 1, half + k))
    return out


def distance_table(rel: Tensor, per_head: Tensor, far: int, max_seqlen: int) -> Tensor:
    """(heads, n) fp32: bias of every distance up to the one from which it stays the same, the heads' own numbers
    included."""
    buckets = rel.shape[0]
    n = min(max_seqlen, math.ceil(max(far, buckets)) + 1)
    index = torch.tensor(distance_buckets(n, buckets, far), device=rel.device)
    return (rel.float()[index] + per_head.float()).T.contiguous()


def sigmoid_attention_weights(w: dict, p: str, mx, d, max_seqlen: int) -> dict:
    m = p + "mix."
    parts, bias = [], []
    for name, heads, rows in (("q", mx.heads, d.dim16), ("k", mx.kv_heads, d.dim16), ("v", mx.kv_heads, d.vdim16)):
        parts.append(_heads(w[m + name], heads, rows))
        bias.append(_heads(w[m + name + ".b"][:, None], heads, rows)[:, 0])
    parts.append(pad_to(w[m + "g"], d.heads16))
    return {
        "w_in": tile(pad_to(torch.cat(parts), d.in_rows, d.w64)), "in_bias": vector(torch.cat(bias), d.in_rows),
        "w_out": tile(_head_columns(w[m + "o"], mx.heads, d.vdim16, d.out_rows, d.out_k)), "out_bias": vector(w[m + "o.b"], d.out_rows),
        "q_norm": vector(w[m + "q.norm"], d.dim16), "k_norm": vector(w[m + "k.norm"], d.dim16),
        "dist_bias": distance_table(w[m + "rel"], w[m + "pb"], mx.bias_max, max_seqlen),
    }


def gated_linear_attention_weights(w: dict, p: str, mx, d) -> dict:
    m = p + "mix."
    rank = w[m + "a1"].shape[0]
    parts = [_heads(w[m + n], mx.heads, r) for n, r in (("q", d.dim16), ("k", d.dim16), ("v", d.vdim16), ("g", d.vdim16))]
    parts.append(w[m + "a1"])
    return {
        "w_in": tile(pad_to(torch.cat(parts), d.in_rows, d.w64)),
        "w_out": tile(_head_columns(w[m + "o"], mx.heads, d.vdim16, d.out_rows, d.out_k)),
        "w_a2": _heads(w[m + "a2"], mx.heads, d.dim16).float().contiguous(), "rank": rank,
        "a2_bias": _heads(w[m + "a2.b"][:, None], mx.heads, d.dim16)[:, 0].float().contiguous(),
        "head_norm": vector(w[m + "norm"], d.vdim16),
    }


def sandwich_norms(w: dict, p: str, has_ff: bool, d) -> dict:
    return {n: vector(w[p + n], d.w64) for n in ("norm1", "norm1b") + (("norm2", "norm2b") if has_ff else ())}


def xielu_weights(w: dict, p: str, d) -> dict:
    m = p + "mlp."
    a, b = torch.nn.functional.softplus(w[m + "act"].double()).tolist()
    return {"w_up": tile(pad_to(w[m + "up"], d.ff16, d.w64)), "w_down": tile(pad_to(w[m + "down"], d.out_rows, d.ff64)),
            "act_pos": a, "act_neg": 0.5 + b}


def expert_weights(w: dict, p: str, mlp, d) -> dict:
    m = p + "mlp."
    return {
        "w_up": torch.cat([tile(pad_to(w[f"{m}e{e}.up"], d.ff16, d.w64)) for e in range(mlp.experts)]),
        "w_down": torch.cat([tile(pad_to(w[f"{m}e{e}.down"], d.out_rows, d.ff64)) for e in range(mlp.experts)]),
        "w_router": tile(pad_to(w[m + "router"], d.experts16, d.w64)), "router_bias": vector(w[m + "router.b"], d.experts16),
    }


def loop_weights(w: dict, d) -> "tuple[Tensor, Tensor]":
    """The mixing matrix of [x; embedding], either half padded, and the vector of every pass."""
    W = w["loop.in"]
    n = W.shape[1] // 2
    mix = tile(torch.cat((pad_to(W[:, :n], d.out_rows, d.w64), pad_to(W[:, n:], d.out_rows, d.w64)), dim=1))
    return mix, torch.stack([vector(s, d.w64) for s in w["loop.step"]])
