"""Token language models: decoder-only models described layer by layer (config.LMConfig), on the native step of
include/vui_lm.h.  Two designs are registered.

Sakupel: parallel layers (mixer and gated feed-forward read one scalar-weight RMS norm and are added to the residual
together) whose mixer is latent attention, with latents of its own or those of an earlier layer, or a minGRU recurrence.

Mabidra: sandwich layers (grouped RMS norms before and after every sublayer) whose mixer is attention with sigmoid weights
and a learned distance bias or gated linear attention, with a dense or an expert feed-forward; some layers may run several
times in a row, each run with caches and states of its own.

The model holds the weights in the kernels' layout; `SlotCache` holds what sequences leave behind, slot by slot, and
`vui_amd.lm_engine.TokenEngine` deals slots to requests."""
from __future__ import annotations

import ctypes as C
import json
import os

import torch
from torch import Tensor

from . import _lib, lm_layout
from .config import ExpertsMLPConfig, GatedLinearAttentionConfig, GatedMLPConfig, LatentAttentionConfig, LMConfig, MinGRUConfig, SigmoidAttentionConfig
from .registry import register_model

MAX_BATCH = _lib.VUI_MAX_BATCH


class SlotCache:
    """Per-slot memory of a token model, by layer run: for every latent attention with latents of its own the latent and
    the rotated key part per position (tiled rows), for every sigmoid attention keys and values, for every recurrence one
    fp32 state; and one length per slot.

    Positions are rewound by setting a length; a recurrence cannot be, so a rewind to anything but 0 needs the states
    that `snapshot` took at that length."""

    def __init__(self, model: "TokenLM", n_slots: int):
        self.n_slots = n_slots
        self.c: "dict[int, Tensor]" = {}
        self.kr: "dict[int, Tensor]" = {}
        self.k: "dict[int, Tensor]" = {}
        self.v: "dict[int, Tensor]" = {}
        self.state: "dict[int, Tensor]" = {}
        dev, dt = model.device, model.dtype
        for i, (li, _) in enumerate(model.runs):
            mx, d = model.config.layers[li].mixer, model.dims[li]
            if isinstance(mx, MinGRUConfig):
                self.state[i] = torch.zeros(n_slots, d.gru16, dtype=torch.float32, device=dev)
            elif isinstance(mx, GatedLinearAttentionConfig):
                self.state[i] = torch.zeros(n_slots, mx.heads * d.dim16 * d.vdim16, dtype=torch.float32, device=dev)
            elif isinstance(mx, SigmoidAttentionConfig):
                self.k[i] = torch.zeros(n_slots, mx.kv_heads * d.s64 * d.dim64, dtype=dt, device=dev)
                self.v[i] = torch.zeros(n_slots, mx.kv_heads * d.s64 * d.vdim16, dtype=dt, device=dev)
            elif mx.kv_from is None:
                self.c[i] = torch.zeros(n_slots, d.s64 * d.rank64, dtype=dt, device=dev)
                self.kr[i] = torch.zeros(n_slots, d.s64 * d.rot32, dtype=dt, device=dev)
        self.seq_lens = torch.zeros(n_slots, dtype=torch.int32, device=dev)

    def bytes_per_slot(self) -> int:
        return sum(t[0].numel() * t.element_size() for g in (self.c, self.kr, self.k, self.v, self.state) for t in g.values())

    def snapshot(self, slot: int) -> "dict[int, Tensor]":
        return {i: s[slot].clone() for i, s in self.state.items()}

    def restore(self, slot: int, length: int, states: "dict[int, Tensor] | None") -> None:
        if length > 0 and self.state:
            if states is None:
                raise ValueError(f"the recurrent state of slot {slot} at position {length} was not kept")
            for i, s in states.items():
                self.state[i][slot].copy_(s)
        self.seq_lens[slot] = length


class _NativeLM:
    """Owns the native context and its workspace."""

    def __init__(self, model: "TokenLM", cache: SlotCache):
        lib = model.lib
        c = model._config_c(cache.n_slots)
        layers = (_lib.LmLayerC * len(model.runs))()
        for i, (li, start) in enumerate(model.runs):
            L, parts = layers[i], model.parts[li]
            model._layer_sizes(li, L)
            for name, v in parts.items():
                setattr(L, name, v.data_ptr() if isinstance(v, Tensor) else v)
            if start is not None:
                L.loop_in, L.loop_step = model.loop_in.data_ptr(), model.loop_step[start].data_ptr()
            if i in cache.state:
                L.state = cache.state[i].data_ptr()
            elif i in cache.k:
                L.k_cache, L.v_cache = cache.k[i].data_ptr(), cache.v[i].data_ptr()
            else:
                src = i if L.kv_from < 0 else L.kv_from
                L.c_cache, L.kr_cache = cache.c[src].data_ptr(), cache.kr[src].data_ptr()
        w = _lib.LmWeightsC()
        w.embed, w.head, w.final_norm = model.embed.data_ptr(), model.head.data_ptr(), model.final_norm.data_ptr()
        nbytes = lib.vui_lm_workspace_bytes(C.byref(c), layers)
        if nbytes < 0:
            raise RuntimeError(f"vui_lm_workspace_bytes: {_lib.last_error()}")
        self.workspace = torch.zeros(nbytes + 256, dtype=torch.uint8, device=model.device)
        base = (self.workspace.data_ptr() + 255) & ~255
        h = C.c_void_p()
        _lib.check(lib.vui_lm_create(C.byref(c), layers, C.byref(w), base, nbytes, C.byref(h)), "vui_lm_create")
        self.handle, self.lib = h, lib

    def __del__(self):
        try:
            if getattr(self, "handle", None):
                self.lib.vui_lm_destroy(self.handle)
                self.handle = None
        except Exception:
            pass


@register_model("Mabidra")
@register_model("Sakupel")
class TokenLM:
    """Decoder-only token model: weights in the kernels' layout, prefill and decode over a slot cache."""

    PREFILL_CHUNK = 1024  # most positions of one native prefill call

    def __init__(self, config: LMConfig, state_dict: "dict[str, Tensor]", device="cuda", dtype=torch.bfloat16,
                 max_seqlen: int = 4096):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("dtype must be bfloat16 or float32")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.max_seqlen = max_seqlen
        self.lib = _lib.load(lm_only=True)
        self._cap_stream = torch.cuda.Stream(device=self.device) if self.device.type == "cuda" else None
        w = {k: v.to(self.device, dtype) for k, v in state_dict.items() if v.is_floating_point()}
        self.runs = config.runs()
        self.ranks = [w[f"l{i}.mix.a1"].shape[0] if isinstance(layer.mixer, GatedLinearAttentionConfig) else 0
                      for i, layer in enumerate(config.layers)]
        self.dims = [self._dims(i) for i in range(len(config.layers))]
        self._tables: dict = {}
        load = self._sandwich_parts if config.design.sandwich else self._parallel_parts
        self.parts: "list[dict]" = [load(w, i) for i in range(len(config.layers))]
        d = self.dims[0]
        if config.loop is not None:
            self.loop_in, self.loop_step = lm_layout.loop_weights(w, d)
        self.embed = w["embed"].contiguous()
        self.head = lm_layout.tile(lm_layout.pad_to(w["head"], -(-config.vocab // 16) * 16, d.w64))
        fn = w["final.norm"].float()
        self.final_norm = lm_layout.vector(fn, d.w64) if config.design.sandwich else fn.reshape(1)
        self.cache: SlotCache | None = None
        self._native: _NativeLM | None = None

    def _parallel_parts(self, w: "dict[str, Tensor]", i: int) -> dict:
        layer, d, p = self.config.layers[i], self.dims[i], f"l{i}."
        mx = layer.mixer
        if isinstance(mx, LatentAttentionConfig):
            parts = lm_layout.latent_attention_weights(w, p, mx, d)
            key = (mx.rot.dims, mx.rot.base)
            if key not in self._tables:
                self._tables[key] = lm_layout.rotation_table(self.max_seqlen, *key).to(self.device)
            parts["rope"] = self._tables[key]
        else:
            parts = lm_layout.mingru_weights(w, p, mx, d)
        parts["w_in"], parts["w_out"] = lm_layout.layer_projections(w, p, parts, layer.mlp is not None, d)
        parts["norm"] = w[p + "norm1"].float().reshape(1)
        del parts["mix"], parts["out"]
        return parts

    def _sandwich_parts(self, w: "dict[str, Tensor]", i: int) -> dict:
        layer, d, p = self.config.layers[i], self.dims[i], f"l{i}."
        mx = layer.mixer
        if isinstance(mx, SigmoidAttentionConfig):
            parts = lm_layout.sigmoid_attention_weights(w, p, mx, d, self.max_seqlen)
            parts["bias_len"] = parts["dist_bias"].shape[1]
        else:
            parts = lm_layout.gated_linear_attention_weights(w, p, mx, d)
        parts.update(lm_layout.sandwich_norms(w, p, layer.mlp is not None, d))
        if isinstance(layer.mlp, ExpertsMLPConfig):
            parts.update(lm_layout.expert_weights(w, p, layer.mlp, d))
        elif layer.mlp is not None:
            parts.update(lm_layout.xielu_weights(w, p, d))
        return parts

    # -- construction ------------------------------------------------------------------
    @classmethod
    def from_config(cls, config: dict, state_dict: "dict[str, Tensor]", device="cuda", dtype=torch.bfloat16, **kw) -> "TokenLM":
        return cls(LMConfig.from_dict(config), state_dict, device=device, dtype=dtype, **kw)

    @classmethod
    def from_pretrained(cls, path: str, device="cuda", dtype=torch.bfloat16, **kw) -> "TokenLM":
        """A local checkpoint folder: config.json beside model.safetensors."""
        from safetensors.torch import load_file

        with open(os.path.join(path, "config.json")) as f:
            config = json.load(f)
        return cls.from_config(config, load_file(os.path.join(path, "model.safetensors")), device, dtype, **kw)

    def _config_c(self, n_slots: int):
        c = _lib.LmConfigC()
        c.dtype = _lib.DTYPE_F32 if self.dtype == torch.float32 else _lib.DTYPE_BF16
        c.width, c.vocab, c.n_layers = self.config.width, self.config.vocab, len(self.runs)
        c.max_seqlen, c.n_slots, c.norm_eps = self.max_seqlen, n_slots, self.config.norm_eps
        c.norm_groups, c.embed_scale = self.config.norm_groups, self.config.embed_scale
        c.max_rows = min(self.PREFILL_CHUNK, self.max_seqlen)
        return c

    def _layer_sizes(self, i: int, L) -> None:
        layer = self.config.layers[i]
        mx, mlp = layer.mixer, layer.mlp
        L.kv_from = -1
        if isinstance(mx, MinGRUConfig):
            L.mixer, L.rnn_width = _lib.LM_MINGRU, mx.width
        elif isinstance(mx, GatedLinearAttentionConfig):
            L.mixer = _lib.LM_GLA
            L.heads, L.dim, L.vdim, L.rank = mx.heads, mx.dim, mx.vdim, self.ranks[i]
            L.scale, L.inv_tau = mx.dim ** -0.5, 1.0 / mx.tau
        elif isinstance(mx, SigmoidAttentionConfig):
            L.mixer = _lib.LM_SIGMOID_ATTENTION
            L.heads, L.kv_heads, L.dim, L.vdim, L.scale = mx.heads, mx.kv_heads, mx.dim, mx.vdim, mx.scale
            if mx.q_temp is not None:
                L.temp_coef, L.temp_every = mx.q_temp.coef, mx.q_temp.every
        else:
            L.mixer = _lib.LM_LATENT_ATTENTION
            L.heads, L.dim, L.rot_dim, L.rot_pairs = mx.heads, mx.dim, mx.rot_dim, mx.rot.dims // 2
            L.vdim, L.kv_rank, L.scale = mx.vdim, mx.kv_rank, mx.scale
            if mx.kv_from is not None:
                L.kv_from = mx.kv_from
        if mlp is not None:
            L.ff = mlp.ff
            if isinstance(mlp, GatedMLPConfig):
                L.limit = mlp.limit
            elif isinstance(mlp, ExpertsMLPConfig):
                L.act, L.experts, L.top = _lib.LM_ACT_RELU2, mlp.experts, mlp.top
            else:
                L.act = _lib.LM_ACT_XIELU

    def _dims(self, i: int):
        L, d = _lib.LmLayerC(), _lib.LmDimsC()
        self._layer_sizes(i, L)
        _lib.check(self.lib.vui_lm_layer_dims(C.byref(self._config_c(1)), C.byref(L), C.byref(d)), "vui_lm_layer_dims")
        return d

    # -- step ----------------------------------------------------------------------------
    def allocate_cache(self, n_slots: int) -> SlotCache:
        self._native = None
        self.cache = SlotCache(self, n_slots)
        self._native = _NativeLM(self, self.cache)
        return self.cache

    def _need(self) -> _NativeLM:
        if self._native is None:
            raise RuntimeError("allocate_cache() must be called first")
        return self._native

    def decode(self, tokens: Tensor, slot_idx: "Tensor | None", seq_inc: "Tensor | None", B: int, logits_out: Tensor,
               stream: int) -> None:
        """One token for each of B rows at its slot's length; logits_out (B, vocab) fp32.  Capturable."""
        nat = self._need()
        _lib.check(nat.lib.vui_lm_decode(nat.handle, tokens.data_ptr(), _lib.ptr(slot_idx), self.cache.seq_lens.data_ptr(),
                                         _lib.ptr(seq_inc), B, logits_out.data_ptr(), stream), "vui_lm_decode")

    def prefill(self, tokens: Tensor, slot: int, pos0: int, want: "list[int]") -> Tensor:
        """tokens (T) int64 on the device, appended to `slot` at pos0 (its length); logits (len(want), vocab) fp32 of
        the positions want (indices into tokens)."""
        nat = self._need()
        T = tokens.shape[0]
        if pos0 + T > self.max_seqlen:
            raise ValueError(f"{T} positions at offset {pos0} exceed max_seqlen={self.max_seqlen}")
        if any(not 0 <= k < T for k in want):
            raise ValueError(f"wanted positions outside [0, {T})")
        st = torch.cuda.current_stream().cuda_stream
        out = torch.empty(len(want), self.config.vocab, dtype=torch.float32, device=self.device)
        step = self._config_c(1).max_rows
        order = sorted(range(len(want)), key=lambda k: want[k])
        for t0 in range(0, T, step):
            n = min(step, T - t0)
            mine = [k for k in order if t0 <= want[k] < t0 + n]
            idx = torch.tensor([want[k] - t0 for k in mine], dtype=torch.int32, device=self.device)
            part = torch.empty(len(mine), self.config.vocab, dtype=torch.float32, device=self.device)
            tk = tokens[t0:t0 + n].contiguous()
            _lib.check(nat.lib.vui_lm_prefill(nat.handle, tk.data_ptr(), n, slot, pos0 + t0, self.cache.seq_lens.data_ptr(),
                                              idx.data_ptr() if mine else None, len(mine), part.data_ptr() if mine else None, st),
                       "vui_lm_prefill")
            if mine:
                out[mine] = part
        return out
