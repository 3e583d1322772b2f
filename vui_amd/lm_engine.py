"""Serving of token language models (vui_amd.lm) on the slots, buckets, captured steps and sampler of the codec engine:
prompts are ingested row by row, then all active rows step together, and a row whose request ends is refilled from the
queue at once."""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass, field
from typing import Iterator, Sequence

import torch
from torch import Tensor

from . import _lib
from .engine import GenConfig
from .lm import TokenLM
from .model import SampleDev, make_sample_params
from .registry import load_model
from .slots import SlotEngine

# sampling settings of a token model: greedy unless asked otherwise
GREEDY = GenConfig(temperature=1.0, top_k=1, rep_penalty=1.0)


@dataclass
class TokenRequest:
    """A prompt (token ids, at least one), the most tokens to draw, and the ids that end the answer (kept as its last
    token)."""

    tokens: "Sequence[int]"
    max_new: int = 64
    stop: "frozenset[int]" = field(default_factory=frozenset)


class TokenRow:
    """One sequence in a slot of the engine's cache."""

    def __init__(self, engine: "TokenEngine", idx: int):
        self._engine, self._idx = engine, idx
        self._length = 0  # host-side count of the slot's positions
        self._mark: "tuple[int, dict] | None" = None
        self._closed = False

    @property
    def idx(self) -> int:
        return self._idx

    @property
    def offset(self) -> int:
        return self._length

    def extend(self, tokens: "Sequence[int] | Tensor", want: "Sequence[int]" = ()) -> Tensor:
        """Runs the row's next tokens from what its slot holds; logits (len(want), vocab) fp32 of the places `want`."""
        return self._engine._extend(self, tokens, list(want))

    def mark_prompt(self) -> int:
        """Keeps what a later rewind to this length needs (recurrent states; cached positions stay where they are)."""
        self._mark = (self._length, self._engine.model.cache.snapshot(self._idx))
        return self._length

    def rewind(self) -> int:
        if self._mark is None:
            return self.reset()
        self._length, states = self._mark
        self._engine.model.cache.restore(self._idx, self._length, states)
        return self._length

    def reset(self) -> int:
        self._engine.model.cache.restore(self._idx, 0, None)
        self._length = 0
        return 0

    def close(self) -> None:
        if not self._closed:
            self._engine._release_row(self)
            self._closed = True

    def __enter__(self):
        return self

    def __exit__(self, *exc):
        self.close()


@dataclass
class _Active:
    row: TokenRow
    request: int
    out: "list[int]"


class TokenEngine(SlotEngine):
    """Batched decoding of a token model over max_rows slots (plus the padding slot)."""

    STEPS_PER_READ = 8  # steps enqueued between two looks at the drawn tokens, when answers may stop early

    def __init__(self, name: "str | None" = None, *, model: "TokenLM | None" = None, max_rows: int = 1,
                 max_seq: "int | None" = None, dtype=torch.bfloat16):
        if model is None:
            if name is None:
                raise ValueError("pass model= or a local checkpoint path")
            model = load_model(name, dtype=dtype, **({"max_seqlen": max_seq} if max_seq else {}))
        if not isinstance(model, TokenLM):
            raise ValueError(f"{type(model).__name__} is not a token model")
        self._check_rows(max_rows)
        self.model, self.max_rows, self.device = model, max_rows, model.device
        self.max_seq = max_seq or model.max_seqlen
        if self.max_seq > model.max_seqlen:
            raise ValueError(f"max_seq={self.max_seq} exceeds the model's {model.max_seqlen} positions")
        self.vocab = model.config.vocab
        self.seq_lens = model.allocate_cache(max_rows + 1).seq_lens
        self._setup_slots(self.vocab, rep_rows=max_rows + 1)  # padding rows draw too, on a state of their own
        B, dev = self._buckets[-1], self.device
        self._g_tokens = torch.zeros(B, dtype=torch.long, device=dev)
        self._g_logits = torch.zeros(B, self.vocab, dtype=torch.float32, device=dev)
        self._frame_ctr = torch.zeros(1, dtype=torch.int32, device=dev)
        self._sdev = SampleDev(dev)
        self._step_graphs: dict = {}

    def _make_row(self, idx: int) -> TokenRow:
        return TokenRow(self, idx)

    def _rep_window_changed(self) -> None:
        self._step_graphs = {}

    # ------------------------------------------------------------------ steps
    def _decode_body(self, B: int, stream: int) -> None:
        self.model.decode(self._g_tokens, self._g_slot_idx, self._g_seq_inc, B, self._g_logits, stream)

    def decode_step(self, rows: "list[TokenRow]", tokens: Tensor) -> Tensor:
        """One token for each row (B) through the bucketed captured step; a view of the static logits (B, vocab)."""
        self._room(rows, 1)
        self._set_active_slots([r.idx for r in rows])
        self._g_tokens[:len(rows)] = tokens
        self._replay_bucket(len(rows), self._decode_body)
        for r in rows:
            r._length += 1
        return self._g_logits[:len(rows)]

    def _room(self, rows: "list[TokenRow]", n: int) -> None:
        for r in rows:
            if r._length + n > self.max_seq:
                raise ValueError(f"{n} positions at offset {r._length} exceed max_seq={self.max_seq}")

    def _extend(self, row: TokenRow, tokens, want: "list[int]") -> Tensor:
        t = torch.as_tensor(tokens, dtype=torch.long).to(self.device)
        if t.numel() < 1:
            raise ValueError("no tokens")
        if t.numel() == 1 and row._length > 0:
            if any(k != 0 for k in want):
                raise ValueError("wanted positions outside [0, 1)")
            return self.decode_step([row], t)[[0] * len(want)]
        self._room([row], t.numel())
        out = self.model.prefill(t, row.idx, row._length, want)
        row._length += t.numel()
        return out

    # ------------------------------------------------------------------ sampling
    def _sample(self, logits: Tensor, cfg: GenConfig, slots: Tensor, out: Tensor, B: int, stream: int, dev=None):
        """Penalise, draw and push with the state of each row's slot; returns the parameter block (kept by captures)."""
        use_rep = cfg.rep_penalty > 1.0
        win = cfg.rep_window if (use_rep and self._rep_history is not None) else 0
        sp = make_sample_params(cfg.temperature, cfg.top_k, cfg.seed, self._frame_ctr, state_rows=slots,
                                top_p=cfg.top_p or 0.0, dev=dev)
        _lib.check(self.model.lib.vui_sample_tokens(
            logits.data_ptr(), self.vocab, self._rep_counts.data_ptr() if use_rep else None,
            _lib.ptr(self._rep_history) if win else None, self._rep_pos.data_ptr() if win else None,
            float(cfg.rep_penalty), win, C.byref(sp), out.data_ptr(), B, stream), "vui_sample_tokens")
        return sp

    def _generate_step(self, B_active: int, cfg: GenConfig) -> None:
        """Decode step and draw as one captured graph; the drawn tokens are the next step's input."""
        self._sdev.set(cfg.temperature, cfg.top_k, cfg.seed)
        key = (cfg.rep_penalty, cfg.rep_window, cfg.top_p)
        graphs = self._step_graphs.setdefault(key, {})
        saved, self._bucketed_graphs = self._bucketed_graphs, graphs
        kept = []

        def body(B, st):
            self._decode_body(B, st)
            kept.append(self._sample(self._g_logits, cfg, self._g_slot_idx, self._g_tokens, B, st, dev=self._sdev))

        bucket = self._bucket(B_active)
        try:
            if bucket not in graphs:  # the capture's warm-up run draws into the token buffer (on the padding slot)
                tokens = self._g_tokens.clone()
                self._replay_bucket(B_active, body, run=False)
                graphs[bucket]._sp = kept
                self._g_tokens.copy_(tokens)
            self._replay_bucket(B_active, body)
        finally:
            self._bucketed_graphs = saved
        self._frame_ctr += 1

    @torch.inference_mode()
    def generate(self, requests: "list[TokenRequest]", cfg: GenConfig = GREEDY) -> "list[list[int]]":
        """Continuous batching: any number of requests through max_rows slots; the drawn tokens of each, in input
        order."""
        outs: "list[list[int]]" = [[] for _ in requests]
        for ri, toks in self._run(requests, cfg):
            outs[ri] = toks
        return outs

    @torch.inference_mode()
    def stream(self, request: TokenRequest, cfg: GenConfig = GREEDY) -> "Iterator[int]":
        """The tokens of one request as they are drawn."""
        self._rep_reset(cfg.rep_penalty, cfg.rep_window)
        self._frame_ctr.zero_()
        info = self._start(request, 0, cfg)
        try:
            yield info.out[-1]
            while not self._done(request, info):
                self._set_active_slots([info.row.idx])
                self._g_tokens[:1] = info.out[-1]
                self._generate_step(1, cfg)
                info.row._length += 1
                info.out.append(int(self._g_tokens[0]))
                yield info.out[-1]
        finally:
            info.row.close()

    def _start(self, req: TokenRequest, ri: int, cfg: GenConfig) -> _Active:
        """Takes a slot, ingests the prompt, draws the first token."""
        row = self.new_row()
        try:
            if len(req.tokens) < 1 or req.max_new < 1:
                raise ValueError("a request needs a token and room for one")
            self._rep_counts[row.idx].zero_()
            self._rep_pos[row.idx].zero_()
            logits = self._extend(row, req.tokens, [len(req.tokens) - 1])
            slot = torch.tensor([row.idx], dtype=torch.int32, device=self.device)
            first = torch.empty(1, dtype=torch.long, device=self.device)
            self._sample(logits.contiguous(), cfg, slot, first, 1, torch.cuda.current_stream().cuda_stream)
            self._frame_ctr += 1
            return _Active(row, ri, [int(first[0])])
        except Exception:
            row.close()
            raise

    def _done(self, req: TokenRequest, a: _Active) -> bool:
        return len(a.out) >= req.max_new or a.out[-1] in req.stop or a.row._length >= self.max_seq

    def _run(self, requests: "list[TokenRequest]", cfg: GenConfig) -> "Iterator[tuple[int, list[int]]]":
        pending = list(range(len(requests)))
        active: "dict[int, _Active]" = {}
        self._rep_reset(cfg.rep_penalty, cfg.rep_window)
        self._frame_ctr.zero_()
        prev: "list[int]" = []
        try:
            while pending or active:
                while pending and self._free:
                    a = self._start(requests[pending[0]], pending.pop(0), cfg)
                    active[a.row.idx] = a
                for slot in [s for s, a in active.items() if self._done(requests[a.request], a)]:
                    a = active.pop(slot)
                    a.row.close()
                    yield a.request, a.out
                if not active:
                    if pending and not self._free:
                        raise RuntimeError("no free rows: other rows of this engine are open")
                    continue
                if pending and self._free:
                    continue
                slots = sorted(active)
                rows = [active[s] for s in slots]
                n = min(min(requests[a.request].max_new - len(a.out), self.max_seq - a.row._length) for a in rows)
                if any(requests[a.request].stop for a in rows):
                    n = min(n, self.STEPS_PER_READ)
                if slots != prev:
                    self._set_active_slots(slots)
                    prev = slots
                self._g_tokens[:len(rows)] = torch.tensor([a.out[-1] for a in rows], dtype=torch.long, device=self.device)
                log = torch.empty(n, len(rows), dtype=torch.long, device=self.device)
                for i in range(n):
                    self._generate_step(len(rows), cfg)
                    log[i] = self._g_tokens[:len(rows)]
                drawn = log.cpu().tolist()
                for k, a in enumerate(rows):
                    stop = requests[a.request].stop
                    for i in range(n):
                        a.out.append(drawn[i][k])
                        if drawn[i][k] in stop:  # what was enqueued behind it is dropped with the slot
                            break
                    a.row._length += n
        finally:
            for a in active.values():
                a.row.close()
