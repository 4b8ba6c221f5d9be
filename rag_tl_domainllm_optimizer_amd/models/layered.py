"""Layered decoders: every layer names its own mixer and feed-forward (``ModelConfig.layers``); the Vezatar
design. A norm stands before and after each sublayer, the residual stream is fp32.

Serving runs one step function, :meth:`LayeredLM.step`, over a ragged batch (portions of prompts beside
single decoded tokens) against a paged cache (``generation.paged.PagedCache``). ``decode`` is its
graph-capturable form for one token per row: no host sync, fixed launch grids. Per layer:

  [q | latent | gate] GEMM -> latent norm + rotation + cache append -> attention (sink, value expansion,
  output gate fused into its last kernel) -> o GEMM -> [branch norm + residual + next norm] ->
  gate/up GEMM with the gated unit in its epilogue (or router, sort, grouped expert GEMMs) -> down GEMM
  -> [branch norm (+ weighted expert sum) + residual + next norm].

The model is inference-only (no autograd, no adapters); fp32 models run the same code on fp32 operands.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from .config import FeedForwardSpec, LatentAttentionSpec, ModelConfig

CLAMPED_GLU_ALPHA, CLAMPED_GLU_OFFSET = 1.702, 1.0  # the dense feed-forward's gated unit


class LatentAttention(nn.Module):
    def __init__(self, index: int, spec: LatentAttentionSpec, width: int, eps: float, device, dtype):
        super().__init__()
        self.index, self.spec, self.eps = index, spec, eps
        self.own_kv = spec.kv_from is None
        self.source = index if self.own_kv else spec.kv_from
        d = self.dims = ops.LatentDims(spec.heads, spec.dim, spec.rot_dim, spec.vdim, spec.kv_rank, spec.scale)
        kw = dict(device=device, dtype=dtype)
        self.in_w = nn.Parameter(torch.empty(d.q_cols + (d.kd if self.own_kv else 0) + d.heads * d.vdim, width, **kw),
                                 requires_grad=False)
        self.kv_up_w = nn.Parameter(torch.empty(d.heads * (d.dim + d.vdim), d.rank, **kw), requires_grad=False)
        self.o_w = nn.Parameter(torch.empty(width, d.heads * d.vdim, **kw), requires_grad=False)
        self.sink = nn.Parameter(torch.zeros(d.heads, device=device, dtype=torch.float32), requires_grad=False)
        self.latent_norm_w = nn.Parameter(torch.ones(d.rank, **kw), requires_grad=False) if self.own_kv else None
        self._uk_t = ops.TransposeCache()
        self._shuf = {"in": ops.ShufCache(), "o": ops.ShufCache()}

    def cache_width(self) -> int:
        """elements per cached token (0: the layer reads another layer's cache)"""
        return self.dims.kd if self.own_kv else 0

    def forward(self, h, batch, cache, tables, dense):
        cos, sin = tables(self.spec.rot)
        proj = ops.project(h, self.in_w, shuf=self._shuf["in"])
        return ops.latent_attention(proj, self.dims, self.kv_up_w, self.sink, cos, sin, batch, cache.pool(self.source),
                                    cache.table, self.own_kv, self.latent_norm_w, self.eps, self._uk_t, dense,
                                    self.source)

    def out(self, a):
        return ops.branch_project(a, self.o_w, self._shuf["o"])

    def refresh(self):
        d = self.dims
        self._uk_t.get(self.kv_up_w[:d.heads * d.dim].view(d.heads, d.dim, d.rank))
        for c, w in ((self._shuf["in"], self.in_w), (self._shuf["o"], self.o_w)):
            if "key" in c:
                c.get(w)


class DenseFF(nn.Module):
    def __init__(self, spec: FeedForwardSpec, width: int, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        self.glu = ops.Glu(spec.limit, CLAMPED_GLU_ALPHA, CLAMPED_GLU_OFFSET)
        self.gate_up_w = nn.Parameter(torch.empty(2 * spec.ff, width, **kw), requires_grad=False)
        self.down_w = nn.Parameter(torch.empty(width, spec.ff, **kw), requires_grad=False)
        self._shuf = {"gate_up": ops.ShufCache(), "down": ops.ShufCache()}

    def forward(self, h):
        return ops.branch_project(ops.glu_project(h, self.gate_up_w, self.glu, self._shuf["gate_up"]), self.down_w,
                                  self._shuf["down"])

    def refresh(self):
        for c, w in ((self._shuf["gate_up"], self.gate_up_w), (self._shuf["down"], self.down_w)):
            if "key" in c:
                c.get(w)


class MoEFF(nn.Module):
    """Routed experts plus a gated shared expert. The shared expert is held as parts of an expert's width
    (the last one zero-padded) behind the routed ones, so one grouped product runs all of them."""

    def __init__(self, spec: FeedForwardSpec, width: int, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        self.spec, self.width = spec, width
        self.nshared = (spec.shared_ff + spec.ff - 1) // spec.ff
        g = spec.experts + self.nshared
        rows = spec.experts + (1 if spec.shared_ff else 0)
        # router rows, the shared expert's gate row behind them, padded to the GEMM's column multiple
        self.router_w = nn.Parameter(torch.zeros((rows + 7) // 8 * 8, width, **kw), requires_grad=False)
        self.correction = nn.Parameter(torch.zeros(spec.experts, device=device, dtype=torch.float32), requires_grad=False)
        self.gate_up_w = nn.Parameter(torch.zeros(g * 2 * spec.ff, width, **kw), requires_grad=False)
        self.down_w = nn.Parameter(torch.zeros(g * width, spec.ff, **kw), requires_grad=False)

    def forward(self, h):
        s = self.spec
        g = s.experts + self.nshared
        return ops.moe_ff(h, self.router_w, self.correction, self.gate_up_w.view(g, 2 * s.ff, self.width),
                          self.down_w.view(g, self.width, s.ff), s.top, self.nshared, s.experts if self.nshared else -1)

    def refresh(self):
        pass


class LayeredLayer(nn.Module):
    def __init__(self, index, spec, width, eps, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)

        def norm():
            return nn.Parameter(torch.ones(width, **kw), requires_grad=False)
        self.norm1_w, self.norm1b_w = norm(), norm()
        self.mix = LatentAttention(index, spec.mixer, width, eps, device, dtype)
        self.mlp = None
        if spec.mlp is not None:
            self.norm2_w, self.norm2b_w = norm(), norm()
            self.mlp = (DenseFF if spec.mlp.kind == "dense" else MoEFF)(spec.mlp, width, device, dtype)


class LayeredLM(nn.Module):
    ragged = True  # served by ragged steps over a paged cache

    def __init__(self, cfg: ModelConfig, device=None, dtype=torch.bfloat16, init: bool = True, seed: int = 0):
        super().__init__()
        assert cfg.is_layered, cfg.arch
        self.cfg, self.dtype = cfg, dtype
        kw = dict(device=device, dtype=dtype)
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size, **kw), requires_grad=False)
        self.norm_w = nn.Parameter(torch.ones(cfg.hidden_size, **kw), requires_grad=False)
        self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size, **kw), requires_grad=False)
        self.layers = nn.ModuleList([LayeredLayer(i, s, cfg.hidden_size, cfg.norm_eps, device, dtype)
                                     for i, s in enumerate(cfg.layers)])
        self._tables, self._old_tables = {}, []
        self._head_shuf = ops.ShufCache()
        if init:
            self.reset_parameters(seed)

    @torch.no_grad()
    def reset_parameters(self, seed: int = 0):
        from .decoder import _normal_

        g = torch.Generator(device="cpu").manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if "norm" in leaf:
                p.fill_(1.0)
            elif leaf in ("sink", "correction"):
                p.zero_()
            else:
                _normal_(p, self.cfg.initializer_range, g)
        self._zero_padding()

    @torch.no_grad()
    def _zero_padding(self):
        """The unused tail of a shared expert that is no multiple of an expert's width stays zero."""
        for layer in self.layers:
            m = layer.mlp
            if isinstance(m, MoEFF) and m.spec.shared_ff % m.spec.ff:
                s, c = m.spec, m.spec.shared_ff % m.spec.ff
                e = s.experts + m.nshared - 1
                gu, dn = m.gate_up_w.view(-1, 2, s.ff, m.width), m.down_w.view(-1, m.width, s.ff)
                gu[e, :, c:] = 0
                dn[e, :, c:] = 0

    # ------------------------------------------------------------------ cache and positions
    def make_cache(self, rows: int, max_seq: int, tokens: Optional[int] = None, device=None):
        from ..generation.paged import PagedCache

        dev = device or self.embed.device
        cache = PagedCache([layer.mix.cache_width() for layer in self.layers], rows, max_seq, tokens, dev, self.dtype)
        for layer in self.layers:
            self._rope(layer.mix.spec.rot, cache.max_seq, dev)
        return cache

    def _rope(self, rot, n: int, dev):
        """cos / sin tables of at least n positions. Made with the cache, before a graph captures them; outgrown
        tables stay alive for the graphs that hold them."""
        key = (rot.base, rot.dims, None if rot.scaling is None else tuple(vars(rot.scaling).values()))
        t = self._tables.get(key)
        if t is None or t[0].shape[0] < n or t[0].device != torch.device(dev):
            self._old_tables.append(t)
            t = self._tables[key] = ops.yarn_rope_tables(rot.dims, rot.base, max(n, 1), rot.scaling, dev)
        return t

    # ------------------------------------------------------------------ the step
    @torch.no_grad()
    def step(self, batch, cache, rows: Optional[torch.Tensor] = None, layer_out=None) -> torch.Tensor:
        """Run a ragged batch (``generation.ragged.RaggedBatch``) against ``cache`` and return the final hidden
        states of its tokens ``rows`` (int64 indices; all tokens by default), [R, width]. ``layer_out``: a
        list that receives the residual stream after every layer (diagnostics)."""
        eps = self.cfg.norm_eps
        dev = self.embed.device

        def tables(rot):
            return self._rope(rot, cache.max_seq, dev)
        n = len(self.layers)
        dense = {}
        x, h = ops.embed_norm(self.embed, batch.ids, self.layers[0].norm1_w, eps)
        for i, layer in enumerate(self.layers):
            nxt = self.layers[i + 1].norm1_w if i + 1 < n else self.norm_w
            a = layer.mix(h, batch, cache, tables, dense)
            if i == n - 1 and rows is not None:
                # nothing after the last layer's attention mixes tokens: go on with the wanted ones
                a, x = a.index_select(0, rows), x.index_select(0, rows)
                if rows.numel() == 0:
                    return a.new_empty(0, self.cfg.hidden_size)
            y = layer.mix.out(a)
            h = ops.branch_norm(x, y, layer.norm1b_w, layer.norm2_w if layer.mlp is not None else nxt, eps)
            if layer.mlp is not None:
                h = ops.branch_norm(x, layer.mlp(h), layer.norm2b_w, nxt, eps)
            if layer_out is not None:
                layer_out.append(x.clone())
        return h

    @torch.no_grad()
    def decode(self, tokens, pos, slot, attn_len, kv_start, cache, workspace=None) -> torch.Tensor:
        """One token per cache row of the view ``cache``: token b at position ``pos[b]``; the other arguments
        of ``CausalLM.decode`` (slots of a left-padded cache) have no part in a paged one."""
        from ..generation.ragged import RaggedBatch

        return self.step(RaggedBatch.single(tokens, cache.row_ids, pos, cache.max_seq), cache)

    def logits(self, hidden, out_f32: bool = True):
        """fp32 logits [R, vocab]"""
        return ops.project(hidden.contiguous(), self.lm_head, out_f32=True, shuf=self._head_shuf)

    def refresh_decode_weights(self, batch: Optional[int] = None):
        """Derived weight images that graph replays read, brought up to date eagerly."""
        if not self.embed.is_cuda:
            return
        for layer in self.layers:
            layer.mix.refresh()
            if layer.mlp is not None:
                layer.mlp.refresh()
        if "key" in self._head_shuf:
            self._head_shuf.get(self.lm_head)

    def add_lora(self, *a, **kw):
        raise NotImplementedError(f"{self.cfg.arch}: layered models are inference-only (no adapters, no backward)")

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, kv_start: Optional[torch.Tensor] = None) -> torch.Tensor:
        """input_ids [B, S] (left-padded; kv_start[b] = first real token) -> final hidden [B * S, width] (zeros
        at padding), through one ragged step on a temporary cache."""
        from ..generation.ragged import RaggedBatch

        B, S = input_ids.shape
        start = kv_start.tolist() if kv_start is not None else [0] * B
        cache = self.make_cache(B, S, device=input_ids.device)
        ids = input_ids.tolist()
        for b in range(B):
            cache.reserve(b, S - start[b])
        cache.sync()
        batch = RaggedBatch.build([(b, ids[b][start[b]:], 0) for b in range(B)], input_ids.device)
        h = self.step(batch, cache)
        out = h.new_zeros(B * S, h.shape[1])
        at = torch.cat([torch.arange(b * S + start[b], (b + 1) * S) for b in range(B)])
        src = torch.cat([batch.offset[b] + torch.arange(S - start[b]) for b in range(B)])
        out[at.to(h.device)] = h[src.to(h.device)]
        return out
