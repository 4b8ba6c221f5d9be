"""Grouped-query attention over a sliding window plus the sequence's first tokens, on a paged cache (no grad).

A token of the batch is (cache row, position); it sees the keys j <= i of its row with i - j < ``window`` or
j < ``keep``. Tokens with short portions (listed first by ``generation.ragged.RaggedBatch``) attend one by
one, split over their visible tiles; longer portions run a flash kernel straight from the pages."""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from . import reference as ref
from ._ext import native, on_gpu


@dataclass
class WindowDims:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0   # 0: none
    window: int = 0        # 0: no limit
    keep: int = 0

    @property
    def q_cols(self) -> int:
        return self.heads * self.dim

    @property
    def cache_width(self) -> int:
        """elements per cached token"""
        return self.kv_heads * (self.dim + self.vdim)

    @property
    def in_cols(self) -> int:
        """columns of the [q | k | v] projection"""
        return self.q_cols + self.cache_width

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    def args(self):
        return ([self.heads, self.kv_heads, self.dim, self.vdim, self.window, self.keep],
                [self.scale, self.softcap])


def _np_parts(T: int, d: WindowDims, max_len: int) -> int:
    """Partitions of a token's visible tiles: enough workgroups for the chip (two per CU), at least 64 keys each."""
    keys = max_len if not d.window else min(max_len, d.window + d.keep + 64)
    groups = T * d.kv_heads
    return max(1, min((512 + groups - 1) // groups, (keys + 63) // 64, 512))


def window_attention(proj: torch.Tensor, col: int, d: WindowDims, q_norm, k_norm, eps: float, cos, sin, batch, pool, tab,
                     out: torch.Tensor, out_scale: float = 1.0):
    """``proj`` [N, ...] holds [q | k | v] from column ``col``; keys and values are appended to ``pool`` / ``tab``
    and out_scale * attention goes to ``out`` [N, heads * vdim] (strided rows). ``q_norm`` / ``k_norm``: weights
    of the RMS norms over all heads at once (or None); ``cos`` / ``sin`` [positions, rotated / 2]."""
    N = proj.shape[0]
    row, pos = batch.row, batch.pos
    if not on_gpu(proj):
        _window_cpu(proj, col, d, q_norm, k_norm, eps, cos, sin, row, pos, pool, tab, out, out_scale)
        return
    nat = native()
    dims, fs = d.args()
    nat.window_prep(proj, col, q_norm, k_norm, eps, cos, sin, row, pos, pool, tab, dims, fs)
    q = proj[:, col:col + d.q_cols]
    bf16 = proj.dtype == torch.bfloat16 and q.stride(0) % 8 == 0 and q.data_ptr() % 16 == 0
    flash = bf16 and batch.segs is not None and out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0 \
        and nat.window_prefill_ok(d.dim, d.vdim)
    n = batch.n_short if flash else N
    if n:
        if bf16 and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0 \
                and nat.window_decode_ok(d.heads, d.kv_heads, d.dim, d.vdim):
            nat.window_decode(q[:n], pool, tab, row, pos, out[:n], _np_parts(n, d, batch.max_len), out_scale, dims, fs)
        else:
            nat.window_any(q[:n], pool, tab, row, pos, out[:n], out_scale, dims, fs)
    if flash:
        nat.window_prefill(q, pool, tab, out, batch.segs, batch.tiles, out_scale, dims, fs)


def _window_cpu(proj, col, d, q_norm, k_norm, eps, cos, sin, row, pos, pool, tab, out, out_scale):
    N, dt = proj.shape[0], proj.dtype
    H, G, D, V = d.heads, d.kv_heads, d.dim, d.vdim
    q, k, v = proj[:, col:col + d.in_cols].float().split([H * D, G * D, G * V], -1)
    if q_norm is not None:
        q = ref.rms(q, q_norm, eps)
    if k_norm is not None:
        k = ref.rms(k, k_norm, eps)
    c, s = cos[pos.long()], sin[pos.long()]
    q = ref.rotate_halves(q.view(N, H, D), c, s).to(dt)
    k = ref.rotate_halves(k.view(N, G, D), c, s)
    page = pool.shape[1]
    kv = torch.cat([k, v.view(N, G, V)], -1).to(pool.dtype)
    p = pos.long()
    by_head = pool.view(pool.shape[0], G, page, D + V)  # inside a page: key head by key head
    by_head[tab[row.long(), p // page].long(), :, p % page] = kv
    size = d.window or (1 << 60)
    for r in torch.unique(row).tolist():
        t = torch.nonzero(row == r).flatten()
        n = int(pos[t].max()) + 1
        key = torch.arange(n)
        kvr = by_head[tab[r].long()[key // page], :, key % page].float()  # [n, G, D + V]
        i = p[t][:, None]
        see = (key[None] <= i) & ((i - key[None] < size) | (key[None] < d.keep))
        kh, vh = kvr[..., :D].repeat_interleave(H // G, 1), kvr[..., D:].repeat_interleave(H // G, 1)
        sc = torch.einsum("thd,nhd->htn", q[t].float(), kh) * d.scale
        if d.softcap:
            sc = d.softcap * torch.tanh(sc / d.softcap)
        pr = torch.softmax(sc.masked_fill(~see, -math.inf), -1)
        out[t] = (torch.einsum("htn,nhv->thv", pr, vh).reshape(len(t), -1) * out_scale).to(dt)
