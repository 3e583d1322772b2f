"""What every engine shares: slots of one cache dealt to rows, a padding slot behind them, bucketed step graphs with slot
indirection, and the rolling repetition state of the sampler.  `vui_amd.engine.Engine` (codec frames) and
`vui_amd.lm_engine.TokenEngine` (tokens) build on it.

A subclass provides `_make_row(idx)` and sets `model`, `device`, `seq_lens` (int32, one length per slot)."""
from __future__ import annotations

import torch
from torch import Tensor

from .model import MAX_BATCH, Graph


def _make_buckets(max_bs: int) -> list[int]:
    """src/vui/engine.py:134-142."""
    buckets, b = [], 1
    while b < max_bs:
        buckets.append(b)
        b *= 2
    if not buckets or buckets[-1] != max_bs:
        buckets.append(max_bs)
    return buckets


def _get_bucket(batch_size: int, buckets: list[int]) -> int:
    for b in buckets:
        if batch_size <= b:
            return b
    return buckets[-1]


class SlotEngine:
    """Rows over one shared cache of max_rows + 1 slots (the last one is the write-only target of padding rows)."""

    def _check_rows(self, max_rows: int) -> None:
        if max_rows < 1 or max_rows > MAX_BATCH:
            raise ValueError(f"max_rows must be in [1, {MAX_BATCH}]")

    def _setup_slots(self, vocab: int, rep_rows: "int | None" = None) -> None:
        """Slot bookkeeping, the bucketed steps' index tensors and the repetition state over `vocab` symbols."""
        dev = self.device
        self._pad_slot = self.max_rows
        self._buckets = _make_buckets(self.max_rows)
        self._g_slot_idx = torch.full((self._buckets[-1],), self._pad_slot, device=dev, dtype=torch.int32)
        self._g_seq_inc = torch.zeros(self.max_rows + 1, device=dev, dtype=torch.int32)
        self._bucketed_graphs: dict[int, Graph] = {}
        self._free: set[int] = set(range(self.max_rows))
        self._rows: dict = {}
        # Device-resident rolling counts (src/vui/engine.py:540-553); the ring position lives on the device too so
        # that the sampler can run inside a captured graph.
        N = self._rep_rows = rep_rows or self.max_rows
        self._rep_counts = torch.zeros(N, vocab, device=dev, dtype=torch.float32)
        self._rep_history: Tensor | None = None
        self._rep_pos = torch.zeros(N, 2, device=dev, dtype=torch.int32)
        self._rep_window_cur = 0

    # ------------------------------------------------------------------ rows
    def _make_row(self, idx: int):
        raise NotImplementedError

    def new_row(self):
        if not self._free:
            raise RuntimeError(f"No free rows (max_rows={self.max_rows} all in use)")
        idx = min(self._free)
        self._free.remove(idx)
        row = self._make_row(idx)
        self._rows[idx] = row
        self.seq_lens[idx] = 0
        return row

    def _release_row(self, row) -> None:
        self._rows.pop(row.idx, None)
        self._free.add(row.idx)

    def reset(self) -> None:
        for row in list(self._rows.values()):
            row.close()
        self.seq_lens.zero_()

    # ------------------------------------------------------------------ graphs
    def _capture(self, body) -> Graph:
        """Warm once and capture; warm-up and capture advance seq_lens, so it is restored
        (src/vui/engine.py:451-471)."""
        saved = self.seq_lens.clone()
        g = Graph(self.model, body, warmup=1)
        torch.cuda.current_stream().synchronize()
        self.seq_lens.copy_(saved)
        return g

    def _bucket(self, B_active: int) -> int:
        return _get_bucket(B_active, self._buckets)

    def _replay_bucket(self, B_active: int, body, run: bool = True) -> int:
        """src/vui/engine.py:525-534: pad the active rows up to the bucket with rows that write to the padding slot,
        replay that bucket's graph (captured on first use with every row on the padding slot).  body(B, stream)
        enqueues the step of B rows.  run=False: only the capture, where it is missing.  Returns the bucket."""
        B_bucket = self._bucket(B_active)
        self._g_slot_idx[B_active:B_bucket].fill_(self._pad_slot)
        g = self._bucketed_graphs.get(B_bucket)
        if g is None:
            saved_idx, saved_inc = self._g_slot_idx.clone(), self._g_seq_inc.clone()
            self._g_slot_idx[:B_bucket].fill_(self._pad_slot)
            self._g_seq_inc.zero_()
            g = self._capture(lambda st: body(B_bucket, st))
            self._g_slot_idx.copy_(saved_idx)
            self._g_seq_inc.copy_(saved_inc)
            self._bucketed_graphs[B_bucket] = g
        if run:
            g.replay()
        return B_bucket

    def _set_active_slots(self, slots: "list[int]") -> Tensor:
        """The rows of the next bucketed steps: their slots, and which lengths advance.  Returns the slots (int32)."""
        t = torch.tensor(slots, dtype=torch.int32, device=self.device)
        self._g_slot_idx[:len(slots)] = t
        self._g_seq_inc.zero_()
        self._g_seq_inc[t.long()] = 1
        return t

    # ------------------------------------------------------------------ repetition penalty
    def _rep_reset(self, penalty: float, window: int) -> None:
        """src/vui/engine.py:555-569."""
        self._rep_counts.zero_()
        self._rep_pos.zero_()
        if penalty <= 1.0:
            return
        if window > 0 and (self._rep_history is None or self._rep_window_cur != window):
            self._rep_history = torch.zeros(self._rep_rows, window, device=self.device, dtype=torch.int32)
            self._rep_window_cur = window
            self._rep_window_changed()
        elif window > 0:
            self._rep_history.zero_()

    def _rep_window_changed(self) -> None:
        """Captured steps that hold the old ring must go."""
