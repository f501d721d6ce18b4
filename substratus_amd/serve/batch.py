"""One engine step's worth of tokens, as the model and its kernels see it."""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Iterator, Optional

import numpy as np
import torch


@dataclass
class StepBatch:
    """Rows are packed entry by entry: first the entries of a single token,
    then portions of prompts (two tokens or more)."""
    tokens: torch.Tensor        # [rows] int32
    positions: torch.Tensor     # [rows] int32, in each request
    slots: torch.Tensor         # [rows] int32, place in the paged caches
    block_table: torch.Tensor   # [entries, max_blocks] int32
    state_slots: torch.Tensor   # [entries] int32, -1: no state (padding)
    singles: int                # entries (= rows) of one token
    seq_start: Optional[torch.Tensor]   # [portions + 1] int32, from row 0 of
                                        # the portions
    max_portion: int            # rows of the longest portion
    max_context: int            # no row has more positions than this
    want: Optional[torch.Tensor] = None  # int64 rows whose logits are needed;
                                         # None: all
    ctx_start: Optional[torch.Tensor] = None  # [portions + 1] int32, keys that
                                              # the portions see, summed up
    total_context: int = 0      # the last of those
    pairs: int = 0              # portions' rows times the keys they see
    # portions' first positions and lengths, on the host
    firsts: Optional[np.ndarray] = None
    lengths: Optional[np.ndarray] = None
    _windows: dict = field(default_factory=dict)

    def context(self, window: int = 0) -> tuple[torch.Tensor, int, int]:
        """ctx_start, total_context and pairs as they are where a row sees
        `window` keys, its own included (0: all before it)."""
        if not window:
            return self.ctx_start, self.total_context, self.pairs
        key = window, self.tokens.device
        if key not in self._windows:
            keys = np.minimum(self.firsts, window - 1) + self.lengths
            starts = np.concatenate([[0], np.cumsum(keys)]).astype(np.int32)
            seen = np.minimum(self.firsts + self.lengths, window)
            self._windows[key] = (
                torch.from_numpy(starts).to(self.tokens.device),
                int(starts[-1]), int((self.lengths * seen).sum()))
        return self._windows[key]

    def parts(self) -> Iterator[tuple[slice, slice, Optional[torch.Tensor],
                                      int]]:
        """(rows, entries, seq_start, longest) of the single-token entries and
        of the portions, whichever there are."""
        n = self.singles
        if n:
            yield slice(0, n), slice(0, n), None, 1
        if self.seq_start is not None:
            rows = self.tokens.shape[0]
            yield slice(n, rows), slice(n, self.block_table.shape[0]), \
                self.seq_start, self.max_portion

    @classmethod
    def build(cls, entries: list[tuple], block_size: int,
              device: torch.device) -> "StepBatch":
        """entries: (tokens, first position, blocks, state slot, wanted
        offsets) per request. Logits come back in the order of the entries
        and their wanted offsets, whatever the order of the rows."""
        order = sorted(range(len(entries)),
                       key=lambda i: len(entries[i][0]) > 1)
        row_of, rows = {}, 0
        for i in order:
            row_of[i] = rows
            rows += len(entries[i][0])
        singles = sum(len(e[0]) == 1 for e in entries)
        maxb = max(len(e[2]) for e in entries)
        table = np.zeros((len(entries), maxb), np.int32)
        tokens, positions, slots = (np.empty(rows, np.int32)
                                    for _ in range(3))
        starts, contexts, pairs, firsts = [0], [0], 0, []
        for at, i in enumerate(order):
            toks, first, blocks, _, _ = entries[i]
            table[at, :len(blocks)] = blocks
            r = slice(row_of[i], row_of[i] + len(toks))
            pos = np.arange(first, first + len(toks))
            tokens[r], positions[r] = toks, pos
            slots[r] = table[at, pos // block_size] * block_size \
                + pos % block_size
            if len(toks) > 1:
                starts.append(starts[-1] + len(toks))
                contexts.append(contexts[-1] + first + len(toks))
                pairs += len(toks) * (first + len(toks))
                firsts.append(first)
        state = np.array([entries[i][3] for i in order], np.int32)
        want = np.array([row_of[i] + o for i, e in enumerate(entries)
                         for o in e[4]], np.int32)
        # one host-to-device copy for everything
        parts = [tokens, positions, slots, state,
                 np.array(starts, np.int32), np.array(contexts, np.int32),
                 want, table.reshape(-1)]
        dev = torch.from_numpy(np.concatenate(parts)).to(device)
        tokens, positions, slots, state, starts_t, contexts_t, want, table = \
            dev.split([len(p) for p in parts])
        portions = len(starts) > 1
        return cls(
            tokens, positions, slots, table.view(len(entries), maxb), state,
            singles, starts_t if portions else None,
            int(np.diff(starts).max()) if portions else 0,
            maxb * block_size, want.long(),
            contexts_t if portions else None, contexts[-1], pairs,
            np.array(firsts, np.int64), np.diff(starts))
