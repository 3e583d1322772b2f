"""Weights of the token language models in the form their kernels read: matrices that share an input side by side,
padded with zero rows and columns to the sizes of `vui_lm_layer_dims`, in the tiled operand layout.

Row order of an input projection (include/vui_lm.h, w_in), every segment padded to 16 rows:
* latent attention: per head the unrotated query rows, per head the rotated ones, the latent, the shared rotated key
  part, the head gates;
* minGRU: blocks of 16 channels, three at a time (update gate, candidate, output gate);
* then the feed-forward, gate and up rows alternating.
Rotated rows are reordered so that the two partners of a pair are neighbours (queries and keys alike, so scores do not
change) and an epilogue that holds four consecutive rows can rotate them."""
from __future__ import annotations

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
