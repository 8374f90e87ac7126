"""One packed forward batch of unequal token runs.

A step of a hybrid model runs portions of prompts beside single decoded
tokens.  Their tokens lie packed one after another; kernels find a
token's place through per-token and per-entry arrays that travel to the
GPU in a single copy.  Entries with few tokens come first, so that each
attention form finds its tokens in one run.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch

# longest entry whose queries attend one by one, as single tokens do
# (the cache read once for all heads of a query); longer ones attend in
# tiles of queries
SHORT_ENTRY = 8


@dataclass
class RaggedBatch:
    ids: torch.Tensor        # [T] token ids (all int32)
    pos: torch.Tensor        # [T] place in the sequence, from 0
    row: torch.Tensor        # [T] block-table row = state slot
    tstart: torch.Tensor     # [T] packed index of the entry's first token
    tend: torch.Tensor       # [T] packed index after the entry's last token
    e_start: torch.Tensor    # [E] per entry: first packed token,
    e_len: torch.Tensor      # [E] tokens,
    e_pos: torch.Tensor      # [E] tokens already in the cache,
    e_row: torch.Tensor      # [E] row
    block_tables: torch.Tensor   # [rows, max blocks]
    n_tok: int
    decode: bool             # every entry is one token
    # host copies of the entries, for launches sized by them
    entries: list            # [(start, length, position, row)]
    n_short: int             # packed tokens in entries <= SHORT_ENTRY
    max_keys: int            # longest context any query may see
    plans: dict = field(default_factory=dict)

    def long_plan(self, window: int):
        """Work lists of the long entries for attention over the last
        ``window`` keys: what to copy out of the pages, 64 key rows a
        block, and tiles of up to 128 queries.

        Returns (blocks, items, block count, item count); blocks are
        (row, first key position, valid keys), items (packed query,
        query position, queries, key row, key position)."""
        plan = self.plans.get(window)
        if plan is None:
            blocks, items = [], []
            for start, n, pos, row in self.entries:
                if n <= SHORT_ENTRY:
                    continue
                first, end = max(0, pos - window + 1), pos + n
                at = 64 * (len(blocks) // 3)
                for k in range(first, end, 64):
                    blocks += (row, k, min(64, end - k))
                # last queries first: they see the most keys
                for q in reversed(range(0, n, 128)):
                    items += (start + q, pos + q, min(128, n - q), at, first)
            flat = torch.tensor(blocks + items, dtype=torch.int32,
                                device=self.pos.device)
            plan = (flat[:len(blocks)], flat[len(blocks):],
                    len(blocks) // 3, len(items) // 5)
            self.plans[window] = plan
        return plan

    def query_tiles(self, size: int):
        """Work list of the long entries in tiles of up to ``size``
        queries: (items, item count), an item being (packed query, query
        position, queries, block-table row), those with the most keys
        first."""
        plan = self.plans.get(("tiles", size))
        if plan is None:
            items = []
            for start, n, pos, row in self.entries:
                if n > SHORT_ENTRY:
                    items += [(start + q, pos + q, min(size, n - q), row)
                              for q in range(0, n, size)]
            items.sort(key=lambda it: -it[1])
            plan = (torch.tensor(items, dtype=torch.int32,
                                 device=self.pos.device), len(items))
            self.plans["tiles", size] = plan
        return plan

    @staticmethod
    def int_count(n_tok: int, n_entries: int) -> int:
        return 5 * n_tok + 4 * n_entries

    @staticmethod
    def pack(runs) -> np.ndarray:
        """``runs``: [(row, position, token ids)], short ones first ->
        the flat int32 array that ``over`` splits."""
        n = np.array([len(t) for _, _, t in runs], dtype=np.int32)
        row = np.array([r for r, _, _ in runs], dtype=np.int32)
        pos = np.array([p for _, p, _ in runs], dtype=np.int32)
        end = np.cumsum(n, dtype=np.int32)
        start = end - n
        at = np.arange(end[-1], dtype=np.int32)
        return np.concatenate(
            [np.asarray(t, dtype=np.int32) for _, _, t in runs]
            + [at + np.repeat(pos - start, n), np.repeat(row, n),
               np.repeat(start, n), np.repeat(end, n), start, n, pos, row])

    @classmethod
    def over(cls, flat: torch.Tensor, runs, block_tables,
             max_keys: int | None = None) -> "RaggedBatch":
        """View a device int32 buffer filled from ``pack(runs)``.
        ``max_keys``: the bound to plan for when the buffer will be
        filled again (captured steps)."""
        T = sum(len(t) for _, _, t in runs)
        E = len(runs)
        parts = torch.split(flat, [T] * 5 + [E] * 4)
        entries, at, short = [], 0, 0
        for r, p, toks in runs:
            n = len(toks)
            entries.append((at, n, p, r))
            at += n
            if n <= SHORT_ENTRY:
                short = at
        return cls(*parts, block_tables=block_tables, n_tok=T,
                   decode=T == E, entries=entries, n_short=short,
                   max_keys=max_keys or max(p + n for _, n, p, _ in entries))

    @classmethod
    def build(cls, runs, block_tables) -> "RaggedBatch":
        dev = block_tables.device
        flat = torch.from_numpy(cls.pack(runs)).to(dev)
        return cls.over(flat, runs, block_tables)
