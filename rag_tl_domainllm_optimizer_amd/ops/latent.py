"""Latent attention over a paged latent cache (no grad).

A token of the batch is (cache row, position). ``batch`` (``generation.ragged.RaggedBatch``) lists the
tokens with short portions (decoded tokens among them) first: those run the absorbed form against the
cached latents, longer portions expand their request's keys and values and run the flash kernel."""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Optional

import torch

from . import reference as ref
from ._ext import native, on_gpu
from .linear import TransposeCache, project


def yarn_rope_tables(dims: int, base: float, max_pos: int, scaling=None, device=None):
    """cos / sin [max_pos, dims / 2] (fp32, from float64 angles) of rotary frequencies base^(-2i/dims).
    ``scaling`` (YaRN; factor, original, fast, slow): frequencies whose period fits ``slow`` .. ``fast``
    turns into the original context are blended towards frequency / factor, and both tables carry the
    multiplier 0.1 ln(factor) + 1."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = base ** (-2.0 * i / dims)
    mult = 1.0
    if scaling is not None:
        def at(turns):
            return dims * math.log(scaling.original / (2 * math.pi * turns)) / (2 * math.log(base))
        lo, hi = max(math.floor(at(scaling.fast)), 0), min(math.ceil(at(scaling.slow)), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
        f = f / scaling.factor * ramp + f * (1 - ramp)
        mult = 0.1 * math.log(scaling.factor) + 1.0
    a = torch.outer(torch.arange(max_pos, dtype=torch.float64), f)
    return (a.cos() * mult).float().to(device), (a.sin() * mult).float().to(device)


@dataclass
class LatentDims:
    heads: int
    dim: int
    rot: int
    vdim: int
    rank: int
    scale: float

    @property
    def kd(self) -> int:
        return self.rank + self.rot

    @property
    def q_cols(self) -> int:
        return self.heads * (self.dim + self.rot)


def _np_parts(T: int, heads: int, max_len: int) -> int:
    """Key partitions of the split decode attention: enough workgroups for the chip (two per CU), at least
    64 keys each."""
    groups = T * ((heads + 31) // 32 if heads > 16 else 1)
    return max(1, min((512 + groups - 1) // groups, (max_len + 63) // 64, 512))


def latent_attention(proj: torch.Tensor, d: LatentDims, kv_up: torch.Tensor, sink: torch.Tensor, cos, sin, batch, pool,
                     tab, own_kv: bool, norm_w: Optional[torch.Tensor], eps: float, uk_t: TransposeCache,
                     dense: dict, dense_key) -> torch.Tensor:
    """Gated attention output [N, heads * vdim] of one layer.

    ``proj`` [N, ...] = [q | latent + rotated key part (own_kv) | gate] projections of the layer's input;
    ``kv_up`` [heads * (dim + vdim), rank] = [W_uk; W_uv]; ``pool`` / ``tab``: the cache the layer reads (its
    own, appended here when ``own_kv``, or another layer's). ``dense``: this step's gathered cache rows
    by source layer (layers that share a cache share the gather)."""
    N = proj.shape[0]
    H, D, R, V, C = d.heads, d.dim, d.rot, d.vdim, d.rank
    kv_col = d.q_cols if own_kv else -1
    gate = proj[:, d.q_cols + (d.kd if own_kv else 0):][:, :H * V]
    uk, uv = kv_up[:H * D].view(H, D, C), kv_up[H * D:].view(H, V, C)
    row, pos = batch.row, batch.pos
    if not on_gpu(proj):
        return _latent_attention_cpu(proj, d, uk, uv, sink, cos, sin, row, pos, pool, tab, kv_col, norm_w, eps, gate)
    nat = native()
    bf16 = proj.dtype == torch.bfloat16 and d.scale > 0
    fast = bf16 and D % 8 == 0 and R % 8 == 0 and proj.stride(0) % 8 == 0 and nat.latent_decode_ok(C, d.kd)
    expand = bf16 and C % 8 == 0 and batch.segs is not None and proj.stride(0) % 8 == 0 \
        and nat.latent_prefill_ok(D, R, V)
    n_abs = batch.n_short if expand else N
    qabs = torch.empty(max(n_abs, 1), H, d.kd, dtype=proj.dtype, device=proj.device)
    nat.latent_prep(proj, kv_col, norm_w, eps, cos, sin, row, pos, pool, tab, qabs, n_abs, H, D, R, C)
    out = torch.empty(N, H * V, dtype=proj.dtype, device=proj.device)
    if n_abs:
        qabs = qabs[:n_abs]
        qn = proj[:n_abs, :d.q_cols].view(n_abs, H, D + R)[:, :, :D].transpose(0, 1)  # [H, n, dim]
        dst = qabs[:, :, :C].transpose(0, 1)
        if fast:
            nat.head_gemm(qn, uk_t.get(uk), dst)
            part, ml = nat.latent_decode(qabs, pool, tab, row, pos, C, _np_parts(n_abs, H, batch.max_len), d.scale)
            o = nat.latent_merge(part, ml, sink)
            nat.head_gemm(o.transpose(0, 1), uv, out[:n_abs].view(n_abs, H, V).transpose(0, 1), gate[:n_abs])
        else:
            nat.gemm_any(qn, uk_t.get(uk), False, dst)
            o = nat.latent_any(qabs, pool, tab, row, pos, sink, C, d.scale)
            nat.gemm_any(o.transpose(0, 1), uv, False, out[:n_abs].view(n_abs, H, V).transpose(0, 1))
            nat.gate_mul(out[:n_abs], gate[:n_abs])
    if expand:
        rows = dense.get(dense_key)
        if rows is None:
            rows = dense[dense_key] = nat.latent_gather(pool, tab, batch.segs, batch.kv_total, batch.max_kv)
        n_up = H * (D + V)
        kv = torch.empty(rows.shape[0], n_up + R, dtype=proj.dtype, device=proj.device)
        project(rows[:, :C], kv_up, out=kv[:, :n_up])
        kv[:, n_up:] = rows[:, C:]
        nat.latent_prefill(proj[:, :d.q_cols], kv, sink, gate, out, batch.segs, batch.tiles, H, D, R, V, d.scale)
    return out


def _latent_attention_cpu(proj, d, uk, uv, sink, cos, sin, row, pos, pool, tab, kv_col, norm_w, eps, gate):
    N, dt = proj.shape[0], proj.dtype
    p = pos.long()
    c, s = cos[p], sin[p]
    if kv_col >= 0:
        lat = ref.rms(proj[:, kv_col:kv_col + d.rank], norm_w, eps)
        kr = ref.rotate_pairs(proj[:, kv_col + d.rank:kv_col + d.kd], c, s)
        page = pool.shape[1]
        slot = tab[row.long(), p // page].long()
        pool[slot, p % page] = torch.cat([lat, kr], -1).to(pool.dtype)
    q = proj[:, :d.q_cols].view(N, d.heads, d.dim + d.rot)
    qa = torch.cat([torch.einsum("nhd,hdc->nhc", q[..., :d.dim].float(), uk.float()),
                    ref.rotate_pairs(q[..., d.dim:], c, s)], -1).to(dt)
    o = ref.latent_attend(qa, pool, tab, row, pos, sink, d.rank, d.scale, pool.shape[1]).to(dt)
    y = torch.einsum("nhc,hvc->nhv", o.float(), uv.float()).reshape(N, -1)
    return (y * torch.sigmoid(gate.float())).to(dt)
