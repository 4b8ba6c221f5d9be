"""Ragged batches: portions of prompts beside single decoded tokens, one step of the model for all of them.

``RaggedBatch`` is the device form of a step: token ids, cache rows and positions (single tokens first, then
short portions, then longer ones), the segment and query-tile tables of the longer ones for attention, and the
runs and chunks of everything above one token for recurrent layers. ``StepEngine`` is the step
function over a paged cache with explicit tokens: requests are admitted into rows, advanced by any
portions, and released; sampling loops (``Generator``, ``ContinuousBatcher``) drive the same model step."""
from __future__ import annotations

from typing import List, Sequence, Tuple

import numpy as np
import torch

SHORT_TOKENS = 32   # portions up to this many tokens attend token by token, like decoded ones
QUERY_TILE = 128    # query rows per workgroup of the portions' attention kernel
CHUNK = 16          # tokens per chunk of a recurrent layer's portions (csrc/kernels/delta_rule.hip)


class RaggedBatch:
    __slots__ = ("ids", "row", "pos", "n_single", "n_short", "segs", "tiles", "kv_total", "max_kv", "max_len", "offset",
                 "runs", "chunks", "first_chunk")

    def __init__(self, ids, row, pos, n_single, n_short, max_len, segs=None, tiles=None, kv_total=0, max_kv=0, offset=(),
                 runs=None, chunks=None, first_chunk=None):
        self.ids, self.row, self.pos = ids, row, pos
        self.n_single, self.n_short = n_single, n_short  # tokens of one-token entries, and with the short portions'
        self.segs, self.tiles, self.kv_total, self.max_kv = segs, tiles, kv_total, max_kv
        self.max_len = max_len      # keys of the longest short token's request (bound)
        self.offset = offset        # first token of every entry, in the order given
        # entries of two and more tokens: {row, first token, tokens, position} each, {run, chunk of the run} each,
        # every run's first chunk
        self.runs, self.chunks, self.first_chunk = runs, chunks, first_chunk

    @classmethod
    def single(cls, tokens, rows, pos, max_len: int) -> "RaggedBatch":
        """One token per row, everything on the device already (decode)."""
        return cls(tokens, rows, pos, tokens.shape[0], tokens.shape[0], max_len)

    @classmethod
    def build(cls, entries: Sequence[Tuple[int, Sequence[int], int]], device) -> "RaggedBatch":
        """``entries``: (cache row, tokens, position of the first)."""
        lens = np.array([len(t) for _, t, _ in entries], dtype=np.int64)
        order = np.argsort((lens > 1).astype(np.int64) + (lens > SHORT_TOKENS), kind="stable")
        offset = np.zeros(len(entries), dtype=np.int64)
        n, kv, max_len, n_single, n_short = 0, 0, 1, 0, 0
        segs, tiles, runs, parts_i, parts_r, parts_p = [], [], [], [], [], []
        max_kv = 0
        for e in order:
            row, toks, start = entries[e]
            L = len(toks)
            offset[e] = n
            parts_i.append(np.asarray(toks, dtype=np.int32))
            parts_r.append(np.full(L, row, dtype=np.int32))
            parts_p.append(np.arange(start, start + L, dtype=np.int32))
            if L > 1:
                runs.append((row, n, L, start))
            else:
                n_single += 1
            if L <= SHORT_TOKENS:
                n_short += L
            else:
                tiles += [(start + min(q + QUERY_TILE, L), len(segs), q // QUERY_TILE) for q in range(0, L, QUERY_TILE)]
                segs.append((row, n, L, kv, start + L, start, 0, 0))
                kv += start + L
                max_kv = max(max_kv, start + L)
            max_len = max(max_len, start + L)
            n += L
        tiles = [t[1:] for t in sorted(tiles, key=lambda t: -t[0])]  # heaviest first
        per = np.array([(r[2] + CHUNK - 1) // CHUNK for r in runs], dtype=np.int64)
        first = np.concatenate([np.zeros(1, np.int64), np.cumsum(per)])
        chunks = np.stack([np.repeat(np.arange(len(runs)), per), np.arange(int(first[-1])) - np.repeat(first[:-1], per)], 1)
        tables = [np.asarray(segs, np.int32).reshape(-1, 8), np.asarray(runs, np.int32).reshape(-1, 4),
                  np.asarray(tiles, np.int32).reshape(-1, 2), chunks.astype(np.int32), first[:-1].astype(np.int32)]
        flat = np.concatenate(parts_i + parts_r + parts_p + [np.zeros(-3 * n % 4, np.int32)] + [t.reshape(-1) for t in tables])
        buf = torch.from_numpy(flat).to(device)
        at, dev = 3 * n + -3 * n % 4, []
        for t in tables:
            dev.append(buf[at:at + t.size].view(t.shape) if t.size else None)
            at += t.size
        st, rt, tt, ct, ft = dev
        return cls(buf[:n].long(), buf[n:2 * n], buf[2 * n:3 * n], n_single, n_short, max_len, st, tt, kv, max_kv, offset, rt, ct, ft)


class StepEngine:
    """Admit requests, advance them by explicit tokens (all entries of a call are one batch), release them."""

    def __init__(self, model, rows: int, tokens: int, max_seq: int = 0):
        if not getattr(model, "ragged", False):
            raise ValueError(f"{model.cfg.arch}: this model has no ragged step")
        self.model = model
        self.device = model.embed.device
        self.cache = model.make_cache(rows, max_seq or tokens, tokens)
        self._rows = list(range(rows - 1, -1, -1))
        self.length = {}

    def admit(self) -> int:
        if not self._rows:
            raise RuntimeError("no free cache row")
        row = self._rows.pop()
        self.length[row] = 0
        return row

    def release(self, row: int):
        self.cache.release(row)
        del self.length[row]
        self._rows.append(row)

    @torch.no_grad()
    def step(self, entries: List[Tuple[int, Sequence[int], Sequence[int]]]) -> torch.Tensor:
        """``entries``: (row, next tokens, places among them whose logits are wanted) -> fp32 logits [wanted,
        vocab], in the order of the entries and their places."""
        entries = [e for e in entries if len(e[1])]
        if not entries:
            return torch.empty(0, self.model.cfg.vocab_size)
        vocab = self.model.cfg.vocab_size
        for row, toks, want in entries:
            if min(toks) < 0 or max(toks) >= vocab:
                raise ValueError("token id outside the vocabulary")
            if any(not 0 <= i < len(toks) for i in want):
                raise ValueError("wanted place outside the portion")
            self.cache.reserve(row, self.length[row] + len(toks))
        self.cache.sync()
        batch = RaggedBatch.build([(r, t, self.length[r]) for r, t, _ in entries], self.device)
        want = [int(batch.offset[e]) + i for e, (_, _, w) in enumerate(entries) for i in w]
        h = self.model.step(batch, self.cache, torch.tensor(want, dtype=torch.long).to(self.device))
        for row, toks, _ in entries:
            self.length[row] += len(toks)
        if not want:
            return torch.empty(0, vocab)
        return self.model.logits(h)
