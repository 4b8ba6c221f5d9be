"""Fused residual-add + RMSNorm / LayerNorm with autograd.

``rms_norm(x, w, eps, residual)`` returns ``(y, h)`` where ``h = x + residual`` is the updated
residual stream (the vLLM-style fused_add_rms_norm pattern: the residual add of the previous
sub-layer costs no separate pass). Backward accepts gradients for both outputs.
"""
from __future__ import annotations

import torch

from . import reference as ref
from ._ext import native, on_gpu


class _NormFn(torch.autograd.Function):
    @staticmethod
    def forward(ctx, x, residual, w, b, eps, layernorm):
        xs = x.contiguous()
        rs = residual.contiguous() if residual is not None else None
        if on_gpu(x):
            y, h, rstd, mean = native().norm_fwd(layernorm, xs, rs, w, b, eps)
        else:
            y, h, rstd, mean = ref.norm(xs, w, b, eps, rs, layernorm)
        hh = h if residual is not None else xs
        ctx.layernorm = layernorm
        ctx.eps = eps
        ctx.has_res = residual is not None
        ctx.has_b = b is not None
        ctx.save_for_backward(hh, w, rstd, mean if mean is not None else torch.empty(0))
        if residual is not None:
            return y, h
        return y

    @staticmethod
    def backward(ctx, dy, dh=None):
        h, w, rstd, mean = ctx.saved_tensors
        dy = dy.contiguous()
        need_dw = ctx.needs_input_grad[2]
        need_db = ctx.has_b and ctx.needs_input_grad[3]
        dh_res = dh.contiguous() if (dh is not None and ctx.has_res) else None
        if on_gpu(dy):
            dx, dw, db = native().norm_bwd(ctx.layernorm, dy, h, w, rstd, mean if ctx.layernorm else None, dh_res,
                                           need_dw, need_db)
        else:
            with torch.enable_grad():
                hh = h.detach().float().requires_grad_(True)
                ww = w.detach().float().requires_grad_(need_dw)
                if ctx.layernorm:
                    y = torch.nn.functional.layer_norm(hh, (hh.shape[-1],), ww, None, ctx.eps)
                else:
                    y = hh * torch.rsqrt(hh.pow(2).mean(-1, keepdim=True) + ctx.eps) * ww
                grads = torch.autograd.grad(y, [hh] + ([ww] if need_dw else []), dy.float())
            dx = grads[0]
            if dh_res is not None:
                dx = dx + dh_res.float()
            dx = dx.to(dy.dtype)
            dw = grads[1] if need_dw else None
            db = dy.float().reshape(-1, dy.shape[-1]).sum(0) if need_db else None
        dw = dw.to(w.dtype) if (need_dw and dw is not None) else None
        if need_db and db is not None:
            db = db.to(w.dtype)
        else:
            db = None
        dres = dx if ctx.has_res else None
        return dx, dres, dw, db, None, None


def _norm(x, w, b, eps, residual, layernorm):
    from .linear import SplitK

    if isinstance(x, SplitK):  # the producing GEMM's split-K reduce fused into this pass
        if residual is None:
            x = x.reduce()
        else:
            return tuple(native().norm_fwd_slabs(layernorm, x.slabs, x.nsplit, x.M, x.N, residual.contiguous(), w, b,
                                                 eps))
    grad = torch.is_grad_enabled() and (x.requires_grad or w.requires_grad or (residual is not None and residual.requires_grad))
    if not grad:
        xs = x.contiguous()
        rs = residual.contiguous() if residual is not None else None
        if on_gpu(x):
            y, h, _, _ = native().norm_fwd(layernorm, xs, rs, w, b, eps)
        else:
            y, h, _, _ = ref.norm(xs, w, b, eps, rs, layernorm)
        return y, (h if residual is not None else xs)
    if residual is None:
        return _NormFn.apply(x, None, w, b, eps, layernorm), x
    return _NormFn.apply(x, residual, w, b, eps, layernorm)


def rms_norm(x, w, eps=1e-6, residual=None):
    """(y, h): h = x + residual (or x), y = RMSNorm(h) * w."""
    return _norm(x, w, None, eps, residual, False)


def layer_norm(x, w, b=None, eps=1e-5, residual=None):
    """(y, h): h = x + residual (or x), y = LayerNorm(h) * w + b."""
    return _norm(x, w, b, eps, residual, True)


class MoePairs:
    """Expert outputs of a mixture, one row of ``y`` [T * slots, H] per (token, slot) pair in expert
    order; ``w`` / ``pos`` [T, slots]: each pair's weight and its row of ``y``. The weighted sum is left to
    the consumer (:func:`branch_norm`)."""

    __slots__ = ("y", "w", "pos")

    def __init__(self, y, w, pos):
        self.y, self.w, self.pos = y, w, pos

    def combine(self) -> torch.Tensor:
        return (self.y.float()[self.pos.long().reshape(-1)].view(*self.w.shape, -1) * self.w[..., None]).sum(1)


_Y_ACT, _Y_SLABS, _Y_PAIRS, _Y_PAIRS_F32 = 1, 2, 3, 4


def embed_norm(table, ids, w_next, eps: float, w_embed=None):
    """First step of a pass with an fp32 residual stream: x = table[ids] (fp32 [T, H]; normed and weighted with
    ``w_embed`` if given) and h = rms(x) * w_next in the table's dtype (``w_next`` None: h = x, rounded).
    Returns (x, h)."""
    if on_gpu(ids):
        x = torch.empty(ids.numel(), table.shape[1], dtype=torch.float32, device=ids.device)
        h = native().branch_norm(x, 0, w_branch=w_embed, w_next=w_next, table=table, ids=ids.contiguous(), eps=eps,
                                 plain=w_next is None)
        return x, h
    x = table[ids].float()
    if w_embed is not None:
        x = ref.rms(x, w_embed, eps)
    return x, (x if w_next is None else ref.rms(x, w_next, eps)).to(table.dtype, copy=True)


def branch_norm(x, y, w_branch, w_next, eps: float, scale=None, next_mul: float = 1.0):
    """Between two sublayers with a norm after each, on the fp32 residual ``x`` (updated in place):
    ``x += rms(y) * w_branch [* scale]``; returns ``h = rms(x) * w_next * next_mul`` in the weights' dtype, or
    x itself rounded (``w_next`` None: sublayers without a norm ahead). ``y``: a tensor, unreduced split-K
    slabs (``SplitK``) or a mixture's expert outputs (:class:`MoePairs`)."""
    from .linear import SplitK

    if on_gpu(x):
        kw = dict(w_branch=w_branch, w_next=w_next, eps=eps, scale=scale, next_mul=next_mul, plain=w_next is None)
        if isinstance(y, SplitK):
            return native().branch_norm(x, _Y_SLABS, y=y.slabs, nsplit=y.nsplit, **kw)
        if isinstance(y, MoePairs):
            kind = _Y_PAIRS if y.y.dtype == w_branch.dtype else _Y_PAIRS_F32
            return native().branch_norm(x, kind, y=y.y, pair_w=y.w, pair_pos=y.pos, **kw)
        kind = _Y_ACT if y.dtype == w_branch.dtype else _Y_SLABS
        return native().branch_norm(x, kind, y=y.contiguous(), **kw)
    yf = ref.rms(y.combine() if isinstance(y, MoePairs) else y.float(), w_branch, eps)
    x.add_(yf if scale is None else yf * scale.float())
    h = x if w_next is None else ref.rms(x, w_next, eps) * next_mul
    return h.to(w_branch.dtype, copy=True)
