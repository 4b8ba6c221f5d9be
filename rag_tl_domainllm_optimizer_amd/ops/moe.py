"""Mixture-of-experts feed-forward (no grad): router, pair sort and grouped expert products.

The row counts per expert stay on the device (fixed launch grids), so a decode step with experts can be
captured in a graph. Few rows per expert stream each expert's weights once (``moe_rows``); many rows
run the grouped form of the token-parallel MFMA GEMM; fp32 and odd sizes run ``gemm_any``."""
from __future__ import annotations

import torch

from . import reference as ref
from ._ext import native, on_gpu
from .linear import ROW, Glu, project
from .norm import MoePairs

# expected rows per expert from which the next form is faster (64 experts of 4096 x 1408 on one MI355X):
RING_ROWS = 5              # LDS-DMA ring instead of register streaming
TILE_ROWS_IN, TILE_ROWS_OUT = 33, 57  # 256-row MFMA tiles instead of the ring (gate / up, down)


def moe_route(logits: torch.Tensor, correction: torch.Tensor, top: int, nshared: int = 0, gate_col: int = -1,
              nslab: int = 1):
    """fp32 router logits [T, >= E] (or ``nslab`` slabs of them, stacked) -> (groups [T, top + nshared] int32,
    weights fp32): the ``top`` experts of the largest ``softmax + correction`` with their softmax values, then groups E .. E + nshared - 1 (the
    shared expert's parts) with weight sigmoid(logits[:, gate_col]) (1 without a gate column)."""
    if on_gpu(logits):
        return native().moe_route(logits, correction, top, nshared, gate_col, nslab)
    return ref.moe_route(logits, correction, top, nshared, gate_col)


def router_logits(h: torch.Tensor, router_w: torch.Tensor):
    """(fp32 logits h W^T, slabs): above 64 rows the narrow product is split over K into slabs that fill the
    chip, summed by the routing kernel."""
    T, K = h.shape
    N = router_w.shape[0]
    if on_gpu(h) and h.dtype == torch.bfloat16 and T > 64 and K % 64 == 0 and N % 8 == 0:
        ns = max(1, min(K // 256, 1024 // max(1, ((T + 63) // 64) * ((N + 63) // 64)), 16))
        if ns > 1:
            return native().gemm_small(h, router_w, ROW, ROW, 3, ns, None, 64), ns
    return project(h, router_w, out_f32=True), 1


def moe_ff(h: torch.Tensor, router_w: torch.Tensor, correction: torch.Tensor, w_gu: torch.Tensor, w_down: torch.Tensor,
           top: int, nshared: int = 0, gate_col: int = -1, glu: Glu = Glu()) -> MoePairs:
    """Experts w_gu [G, 2F, W] / w_down [G, W, F] (G = E + nshared) applied to h [T, W]."""
    T = h.shape[0]
    G, F2, W = w_gu.shape
    F = F2 // 2
    z, nslab = router_logits(h, router_w)
    idx, wt = moe_route(z, correction, top, nshared, gate_col, nslab)
    if not on_gpu(h):
        order = torch.argsort(idx.reshape(-1), stable=True)
        pos = torch.empty_like(order)
        pos[order] = torch.arange(order.numel())
        tok, grp = order // idx.shape[1], idx.reshape(-1)[order]
        y = torch.empty(order.numel(), W, dtype=h.dtype)
        for g in torch.unique(grp).tolist():
            r = torch.nonzero(grp == g).flatten()
            f = ref.glu(ref.gemm(h[tok[r]], w_gu[g]), glu.limit, glu.alpha, glu.offset)
            y[r] = ref.gemm(f, w_down[g])
        return MoePairs(y, wt, pos.int().view_as(idx))
    P = idx.numel()
    mean = (P + G - 1) // G
    bf16 = h.dtype == torch.bfloat16 and W % 8 == 0 and F % 8 == 0
    tiles = bf16 and mean >= TILE_ROWS_IN and F % 128 == 0
    srt = native().moe_sort(idx, G, 256 if tiles else 0)
    offs, tok, pos = srt[:3]
    if bf16:
        ring = mean >= RING_ROWS
        if tiles:
            f = native().gemm_grouped(h, tok, w_gu, srt[3], srt[4], P, glu.args(), 256)
        else:
            f = native().moe_rows(h, tok, w_gu, offs, P, False, mean, ring and W % 64 == 0 and F % 32 == 0, glu.args())
        if tiles and mean >= TILE_ROWS_OUT:
            y = native().gemm_grouped(f, None, w_down, srt[3], srt[4], P, [], 256)
        else:
            y = native().moe_rows(f, None, w_down, offs, P, T <= 64, mean, ring and W % 64 == 0 and F % 64 == 0, [])
    else:
        f = native().glu_any(native().gemm_any(h, w_gu, offs=offs, row_map=tok), glu.args())
        y = native().gemm_any(f, w_down, offs=offs)
    return MoePairs(y, wt, pos.view_as(idx))
