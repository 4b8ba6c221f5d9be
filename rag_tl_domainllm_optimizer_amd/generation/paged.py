"""Paged cache: per layer a pool of pages of 64 tokens, and one page table row per request.

The pool is sized for the tokens that live requests hold at any time (each rounded up to whole pages), not
for rows x longest sequence. Page 0 belongs to nobody: table entries without a page point at it, so a
decode graph's idle rows write there. Pools start as zeros and only ever hold finite values, so masked
keys of a reused page are harmless. Allocation is host bookkeeping; ``sync`` uploads the table.

Layers with recurrent state have one slot per row beside it: tensors [rows, ...] that belong to the row's
request and count as zero at its position 0, so a slot that is used again needs no clearing."""
from __future__ import annotations

import contextlib
from typing import List, Optional

import numpy as np
import torch

PAGE = 64


class PagedCache:
    def __init__(self, widths: List[int], rows: int, max_seq: int, tokens: Optional[int] = None, device="cpu",
                 dtype=torch.bfloat16, states=None):
        """``widths``: cached elements per token of every layer (0: no cache of its own); ``tokens``: capacity
        of the pool (default rows x max_seq); ``states``: per layer the (shape, dtype) of its state tensors'
        slots."""
        self.rows = rows
        self.max_pages = max(1, (max_seq + PAGE - 1) // PAGE)
        self.max_seq = self.max_pages * PAGE
        cap = rows * self.max_pages if tokens is None else (tokens + PAGE - 1) // PAGE
        self.n_pages = cap + 1
        self._pools = [torch.zeros(self.n_pages, PAGE, w, device=device, dtype=dtype) if w else None for w in widths]
        self._states = [tuple(torch.zeros(rows, *shape, device=device, dtype=dt) for shape, dt in s)
                        for s in (states or [()] * len(widths))]
        self._host = np.zeros((rows, self.max_pages), dtype=np.int32)
        self.table = torch.zeros(rows, self.max_pages, dtype=torch.int32, device=device)
        self.row_ids = torch.arange(rows, dtype=torch.int32, device=device)
        self.free = list(range(self.n_pages - 1, 0, -1))
        self.held = [0] * rows  # pages per row
        self._dirty = False

    def pool(self, layer: int) -> torch.Tensor:
        return self._pools[layer]

    def state(self, layer: int):
        """the layer's state tensors, [rows, ...] each"""
        return self._states[layer]

    @property
    def nbytes(self) -> int:
        held = [p for p in self._pools if p is not None] + [t for s in self._states for t in s]
        return sum(p.numel() * p.element_size() for p in held)

    @contextlib.contextmanager
    def parked(self):
        """No row takes part: a decode step of ``rows_view`` that runs inside (a graph's warm-up) neither
        appends to the pools nor advances a state."""
        self.row_ids.fill_(-1)
        try:
            yield
        finally:
            self.row_ids.copy_(torch.arange(self.rows, dtype=torch.int32))

    def free_tokens(self) -> int:
        return len(self.free) * PAGE

    def can_reserve(self, row: int, n: int) -> bool:
        need = (n + PAGE - 1) // PAGE
        return need <= self.max_pages and need - self.held[row] <= len(self.free)

    def reserve(self, row: int, n: int):
        """Pages for the first n tokens of ``row`` (keeps what it holds already)."""
        need = (n + PAGE - 1) // PAGE
        if need > self.max_pages:
            raise ValueError(f"{n} tokens exceed the cache row ({self.max_seq})")
        if need - self.held[row] > len(self.free):
            raise RuntimeError(f"cache pool exhausted: {need - self.held[row]} pages needed, {len(self.free)} free")
        for i in range(self.held[row], need):
            self._host[row, i] = self.free.pop()
            self._dirty = True
        self.held[row] = max(self.held[row], need)

    def release(self, row: int):
        n = self.held[row]
        if n:
            self.free.extend(int(p) for p in self._host[row, :n][::-1])
            self._host[row, :n] = 0
            self.held[row] = 0
            self._dirty = True

    def release_all(self):
        for r in range(self.rows):
            self.release(r)

    def sync(self):
        """Upload the page table if it changed (stream-ordered before the step that reads it)."""
        if self._dirty:
            self.table.copy_(torch.from_numpy(self._host.copy()))
            self._dirty = False

    def rows_view(self, row0: int, n: int) -> "PagedRows":
        return PagedRows(self, row0, n)


class PagedRows:
    """Rows [row0, row0 + n) of a PagedCache (a decode step's bucket)."""

    def __init__(self, cache: PagedCache, row0: int, n: int):
        self.table, self.max_seq = cache.table, cache.max_seq
        self.row_ids = cache.row_ids[row0:row0 + n]
        self.pool, self.state = cache.pool, cache.state
