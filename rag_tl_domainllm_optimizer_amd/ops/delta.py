"""Gated delta rule over a ragged batch with per-row recurrent state (no grad).

Per head a state S [D, V]: S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with q, k, v through
a short causal convolution and silu, q and k unit vectors. A cache row's state is S (fp32) and a ring of its
last projections; at position 0 both count as zero."""
from __future__ import annotations

import torch

from ._ext import native, on_gpu


def delta_rule(x, b, a, z, conv, A_log, dt, norm_w, eps: float, batch, state, ring, out, out_scale: float, kv_heads: int,
               silu_gate: bool):
    """``x`` [N, C] projections q | k (``kv_heads`` heads) | v, ``b`` [N, H] (beta), ``a`` [N, H] or [N, H * D]
    (decay per head or per key channel), ``z`` [N, H * V] (output gate: silu, or sigmoid); ``conv`` [C, taps];
    ``state`` [rows, H, D, V], ``ring`` [rows, taps, C]. Writes out_scale * gated, normed read-outs to ``out``
    [N, H * V] (strided rows) and advances the state of the batch's rows."""
    if on_gpu(x):
        native().delta_rule(x, b, a, z, conv, A_log, dt, norm_w, eps, batch.row, batch.pos, state, ring, out, out_scale,
                            kv_heads, silu_gate, batch.n_single, batch.runs, batch.chunks, batch.first_chunk)
        return
    _delta_cpu(x, b, a, z, conv, A_log, dt, norm_w, eps, batch, state, ring, out, out_scale, kv_heads, silu_gate)


def _delta_cpu(x, b, a, z, conv, A_log, dt, norm_w, eps, batch, state, ring, out, out_scale, K, silu_gate):
    H, D, V = state.shape[1:]
    taps = conv.shape[1]
    cw, n = conv.float(), K * D
    beta = torch.sigmoid(b.float())
    g = a.float() + dt
    g = -torch.exp(A_log)[:, None] * torch.nn.functional.softplus(g.view(-1, H, g.shape[1] // H))
    g = torch.exp(g).expand(-1, H, D)
    gate = z.float()
    gate = torch.nn.functional.silu(gate) if silu_gate else torch.sigmoid(gate)
    for r in torch.unique(batch.row).tolist():
        toks = torch.nonzero(batch.row == r).flatten()
        toks = toks[torch.argsort(batch.pos[toks])].tolist()
        for t in toks:
            p = int(batch.pos[t])
            S = state[r] if p else torch.zeros_like(state[r])
            ring[r, p % taps] = x[t]
            hist = torch.zeros(taps, x.shape[1])
            for j in range(taps):
                if p - j >= 0:
                    hist[taps - 1 - j] = ring[r, (p - j) % taps].float()
            y = torch.nn.functional.silu((hist * cw.t()).sum(0))
            q, k, v = y[:n].view(K, D), y[n:2 * n].view(K, D), y[2 * n:].view(H, V)
            q = (q * torch.rsqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * D ** -0.5).repeat_interleave(H // K, 0)
            k = (k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)).repeat_interleave(H // K, 0)
            S = S * g[t][..., None]
            u = beta[t][:, None] * (v - (S * k[..., None]).sum(1))
            S = S + k[..., None] * u[:, None]
            o = (S * q[..., None]).sum(1)
            state[r] = S
            o = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eps) * norm_w.float()
            out[t] = (o.reshape(-1) * gate[t] * out_scale).to(out.dtype)
