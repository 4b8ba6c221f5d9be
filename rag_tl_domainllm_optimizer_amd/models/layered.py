"""Layered decoders: every layer names its own mixer and feed-forward (``ModelConfig.layers``); the Vezatar and
Pafolorn designs. A norm stands before and after each sublayer, or after it only (``ModelConfig.norms``); the
residual stream is fp32.

Serving runs one step function, :meth:`LayeredLM.step`, over a ragged batch (portions of prompts beside
single decoded tokens) against a paged cache with per-row state slots (``generation.paged.PagedCache``).
``decode`` is its graph-capturable form for one token per row: no host sync, fixed launch grids. Per layer:

  input GEMM of the mixer -> mixer -> o GEMM -> [branch norm + residual + next norm] -> up GEMM with the
  activation (or the gated unit) in its epilogue (or router, sort, grouped expert GEMMs) -> down GEMM ->
  [branch norm (+ weighted expert sum) + residual + next norm]

Mixers: latent attention (:class:`LatentAttention`); windowed attention and the gated delta rule, alone or side
by side on one input GEMM and one output GEMM (:class:`BranchMixer`).

The model is inference-only (no autograd, no adapters); fp32 models run the same code on fp32 operands.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from .config import (DeltaSpec, FeedForwardSpec, LatentAttentionSpec, MixerSpec, ModelConfig, ParallelSpec,
                     WindowAttentionSpec)

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

    def state_spec(self):
        return []

    def rotations(self):
        return [self.spec.rot]

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


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def _sides(spec: MixerSpec):
    """(name, part, output multiplier) of a branch mixer"""
    if isinstance(spec, ParallelSpec):
        return [("left", spec.left, spec.left_scale), ("right", spec.right, spec.right_scale)]
    return [("mix", spec, 1.0)]


def in_layout(spec: MixerSpec):
    """Rows of a branch mixer's input matrix: ({side: {tensor: (first row, rows)}}, all rows). q | k | v of a side are
    one block; blocks start at multiples of 8 (16-B columns of the product), low-rank ones are padded to the
    product's reduction step."""
    rows, at = {}, 0
    for side, x, _ in _sides(spec):
        if isinstance(x, WindowAttentionSpec):
            blocks = [[("q", x.heads * x.dim), ("k", x.kv_heads * x.dim), ("v", x.kv_heads * x.vdim)]]
        else:
            blocks = [[("q", x.kv_heads * x.dim), ("k", x.kv_heads * x.dim), ("v", x.heads * x.vdim)]]
            blocks += [[("a1", x.a_rank)], [("g1", x.g_rank)], [("b", x.heads)]] if x.channel else \
                [[("g", x.heads * x.vdim)], [("b", x.heads)], [("a", x.heads)]]
        rows[side] = {}
        for block in blocks:
            for name, n in block:
                rows[side][name] = (at, n)
                at += n
            at = rows[side][name][0] + _up(n, 64) if name in ("a1", "g1") else _up(at, 8)
    return rows, _up(at, 64)


def out_layout(spec: MixerSpec):
    """Columns of a branch mixer's output matrix: ({side: (first column, columns)}, all columns)."""
    cols, at = {}, 0
    for side, x, _ in _sides(spec):
        cols[side] = (at, x.heads * x.vdim)
        at = _up(at + x.heads * x.vdim, 8)
    return cols, _up(at, 64)


class WindowBranch(nn.Module):
    """Norms of a windowed attention's queries and keys; the projections are the mixer's."""

    def __init__(self, spec: WindowAttentionSpec, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        self.spec = spec
        self.dims = ops.WindowDims(spec.heads, spec.kv_heads, spec.dim, spec.vdim, spec.scale, spec.softcap, spec.window,
                                   spec.keep_first)
        self.q_norm_w = nn.Parameter(torch.ones(spec.heads * spec.dim, **kw), requires_grad=False)
        self.k_norm_w = nn.Parameter(torch.ones(spec.kv_heads * spec.dim, **kw), requires_grad=False)

    def cache_width(self) -> int:
        return self.dims.cache_width

    def state_spec(self, dtype):
        return []

    def forward(self, proj, rows, eps, batch, cache, layer, tables, out, out_scale):
        cos, sin = tables(self.spec.rot)
        ops.window_attention(proj, rows["q"][0], self.dims, self.q_norm_w, self.k_norm_w, eps, cos, sin, batch,
                             cache.pool(layer), cache.table, out, out_scale)

    def refresh(self):
        pass


class DeltaBranch(nn.Module):
    """Gated delta rule: short convolutions, decays, output norm; with a decay per key channel also the outer
    halves of the low-rank decay and gate projections."""

    def __init__(self, spec: DeltaSpec, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        f32 = dict(device=device, dtype=torch.float32)
        H, D, V = spec.heads, spec.dim, spec.vdim
        self.spec = spec
        self.channels = 2 * spec.kv_heads * D + H * V
        self.conv_w = nn.Parameter(torch.empty(self.channels, spec.conv, **kw), requires_grad=False)
        self.A_log = nn.Parameter(torch.zeros(H, **f32), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(H * D if spec.channel else H, **f32), requires_grad=False)
        self.out_norm_w = nn.Parameter(torch.ones(V, **kw), requires_grad=False)
        self._shuf = {}
        if spec.channel:
            self.a2_w = nn.Parameter(torch.zeros(H * D, _up(spec.a_rank, 64), **kw), requires_grad=False)
            self.g2_w = nn.Parameter(torch.zeros(H * V, _up(spec.g_rank, 64), **kw), requires_grad=False)
            self._shuf = {"a2": ops.ShufCache(), "g2": ops.ShufCache()}

    def cache_width(self) -> int:
        return 0

    def state_spec(self, dtype):
        s = self.spec
        return [((s.heads, s.dim, s.vdim), torch.float32), ((s.conv, self.channels), dtype)]

    def forward(self, proj, rows, eps, batch, cache, layer, tables, out, out_scale):
        s = self.spec

        def cols(name, n=None):
            c0 = rows[name][0]
            return proj[:, c0:c0 + (rows[name][1] if n is None else n)]
        if s.channel:
            a = ops.project(cols("a1", self.a2_w.shape[1]), self.a2_w, shuf=self._shuf["a2"])
            z = ops.project(cols("g1", self.g2_w.shape[1]), self.g2_w, shuf=self._shuf["g2"])
        else:
            a, z = cols("a"), cols("g")
        state, ring = cache.state(layer)
        ops.delta_rule(cols("q", self.channels), cols("b"), a, z, self.conv_w, self.A_log, self.dt_bias, self.out_norm_w, eps,
                       batch, state, ring, out, out_scale, s.kv_heads, not s.channel)

    def refresh(self):
        for k, c in self._shuf.items():
            if "key" in c:
                c.get(self.a2_w if k == "a2" else self.g2_w)


class BranchMixer(nn.Module):
    """Windowed attention and / or a gated delta rule on one input: one GEMM for all their input projections, the
    branches' results (times their multipliers) side by side, one GEMM back."""

    def __init__(self, index: int, spec: MixerSpec, width: int, eps: float, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        self.index, self.spec, self.eps = index, spec, eps
        self.rows, n_in = in_layout(spec)
        self.cols, n_out = out_layout(spec)
        self.sides = _sides(spec)
        self.in_w = nn.Parameter(torch.zeros(n_in, width, **kw), requires_grad=False)
        self.o_w = nn.Parameter(torch.zeros(width, n_out, **kw), requires_grad=False)
        for side, x, _ in self.sides:
            self.add_module(side, (WindowBranch if isinstance(x, WindowAttentionSpec) else DeltaBranch)(x, device, dtype))
        self._gaps = sum(n for _, n in self.cols.values()) < n_out
        self._shuf = {"in": ops.ShufCache(), "o": ops.ShufCache()}

    def branches(self):
        return [(getattr(self, side), side, mul) for side, _, mul in self.sides]

    def cache_width(self) -> int:
        return sum(b.cache_width() for b, _, _ in self.branches())

    def state_spec(self):
        return [x for b, _, _ in self.branches() for x in b.state_spec(self.in_w.dtype)]

    def rotations(self):
        return [x.rot for _, x, _ in self.sides if isinstance(x, WindowAttentionSpec)]

    def forward(self, h, batch, cache, tables, dense):
        proj = ops.project(h, self.in_w, shuf=self._shuf["in"])
        n = (h.shape[0], self.o_w.shape[1])
        out = proj.new_zeros(n) if self._gaps else proj.new_empty(n)  # padding columns meet zero weights
        for b, side, mul in self.branches():
            c0, c = self.cols[side]
            b(proj, self.rows[side], self.eps, batch, cache, self.index, tables, out[:, c0:c0 + c], mul)
        return out

    def out(self, a):
        return ops.branch_project(a, self.o_w, self._shuf["o"])

    def refresh(self):
        for c, w in ((self._shuf["in"], self.in_w), (self._shuf["o"], self.o_w)):
            if "key" in c:
                c.get(w)
        for b, _, _ in self.branches():
            b.refresh()

    @torch.no_grad()
    def zero_padding(self):
        """Rows and columns between the blocks stay zero."""
        used = torch.zeros(self.in_w.shape[0], dtype=torch.bool)
        for side in self.rows.values():
            for r0, n in side.values():
                used[r0:r0 + n] = True
        self.in_w[(~used).to(self.in_w.device)] = 0
        used = torch.zeros(self.o_w.shape[1], dtype=torch.bool)
        for c0, n in self.cols.values():
            used[c0:c0 + n] = True
        self.o_w[:, (~used).to(self.o_w.device)] = 0
        for b, _, _ in self.branches():
            if isinstance(b, DeltaBranch) and b.spec.channel:
                b.a2_w[:, b.spec.a_rank:] = 0
                b.g2_w[:, b.spec.g_rank:] = 0


class Relu2FF(nn.Module):
    """W_down relu(W_up h)^2"""

    def __init__(self, spec: FeedForwardSpec, width: int, device, dtype):
        super().__init__()
        kw = dict(device=device, dtype=dtype)
        self.up_w = nn.Parameter(torch.empty(spec.ff, width, **kw), requires_grad=False)
        self.down_w = nn.Parameter(torch.empty(width, spec.ff, **kw), requires_grad=False)
        self._shuf = {"up": ops.ShufCache(), "down": ops.ShufCache()}

    def forward(self, h):
        return ops.branch_project(ops.act_project(h, self.up_w, ops.ACT_RELU2, self._shuf["up"]), self.down_w,
                                  self._shuf["down"])

    def refresh(self):
        for c, w in ((self._shuf["up"], self.up_w), (self._shuf["down"], self.down_w)):
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


FEED_FORWARDS = {"dense": DenseFF, "relu2": Relu2FF, "moe": MoEFF}


class LayeredLayer(nn.Module):
    def __init__(self, index, spec, cfg: ModelConfig, device, dtype):
        super().__init__()
        width = cfg.hidden_size
        kw = dict(device=device, dtype=dtype)

        def vec():
            return nn.Parameter(torch.ones(width, **kw), requires_grad=False)
        self.both = cfg.norms == "both"
        for j in "12" if spec.mlp is not None else "1":
            setattr(self, f"norm{j}_w", vec())
            if self.both:
                setattr(self, f"norm{j}b_w", vec())
            if cfg.layer_scale:
                setattr(self, f"ls{j}", vec())
        mixer = LatentAttention if isinstance(spec.mixer, LatentAttentionSpec) else BranchMixer
        self.mix = mixer(index, spec.mixer, width, cfg.norm_eps, device, dtype)
        self.mlp = None if spec.mlp is None else FEED_FORWARDS[spec.mlp.kind](spec.mlp, width, device, dtype)

    def ahead(self, j: str):
        """Weight of the norm ahead of sublayer ``j`` (None: it reads the residual stream itself)."""
        return getattr(self, f"norm{j}_w") if self.both else None

    def behind(self, j: str):
        """(weight of the norm behind sublayer ``j``, its element-wise scale or None)"""
        return getattr(self, f"norm{j}b_w" if self.both else f"norm{j}_w"), getattr(self, f"ls{j}", None)


class LayeredLM(nn.Module):
    ragged = True  # served by ragged steps over a paged cache

    def __init__(self, cfg: ModelConfig, device=None, dtype=torch.bfloat16, init: bool = True, seed: int = 0):
        super().__init__()
        assert cfg.is_layered, cfg.arch
        self.cfg, self.dtype = cfg, dtype
        kw = dict(device=device, dtype=dtype)
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size, **kw), requires_grad=False)
        self.embed_norm_w = nn.Parameter(torch.ones(cfg.hidden_size, **kw), requires_grad=False) if cfg.embed_norm else None
        self.norm_w = nn.Parameter(torch.ones(cfg.hidden_size, **kw), requires_grad=False)
        if not cfg.tie_embeddings:
            self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size, **kw), requires_grad=False)
        self.layers = nn.ModuleList([LayeredLayer(i, s, cfg, device, dtype) for i, s in enumerate(cfg.layers)])
        self._tables, self._old_tables = {}, []
        self._head_shuf = ops.ShufCache()
        if init:
            self.reset_parameters(seed)

    def head_w(self) -> torch.Tensor:
        return self.embed if self.cfg.tie_embeddings else self.lm_head

    @torch.no_grad()
    def reset_parameters(self, seed: int = 0):
        from .decoder import _normal_

        g = torch.Generator(device="cpu").manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if "norm" in leaf or leaf in ("ls1", "ls2"):
                p.fill_(1.0)
            elif leaf in ("sink", "correction", "A_log", "dt_bias"):
                p.zero_()
            else:
                _normal_(p, self.cfg.initializer_range, g)
        self._zero_padding()

    @torch.no_grad()
    def _zero_padding(self):
        """Padding stays zero: between a mixer's projections, and the unused tail of a shared expert that is no
        multiple of an expert's width."""
        for layer in self.layers:
            if isinstance(layer.mix, BranchMixer):
                layer.mix.zero_padding()
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
        cache = PagedCache([layer.mix.cache_width() for layer in self.layers], rows, max_seq, tokens, dev, self.dtype,
                           [layer.mix.state_spec() for layer in self.layers])
        for layer in self.layers:
            for rot in layer.mix.rotations():
                self._rope(rot, cache.max_seq, dev)
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
        states of its tokens ``rows`` (int64 indices; all tokens by default), [R, width], normed and times the
        logits' multiplier. ``layer_out``: a
        list that receives the residual stream after every layer (diagnostics)."""
        eps = self.cfg.norm_eps
        dev = self.embed.device

        def tables(rot):
            return self._rope(rot, cache.max_seq, dev)
        n = len(self.layers)
        dense = {}
        x, h = ops.embed_norm(self.embed, batch.ids, self.layers[0].ahead("1"), eps, self.embed_norm_w)
        for i, layer in enumerate(self.layers):
            a = layer.mix(h, batch, cache, tables, dense)
            # what comes behind the layer: the next one, or the final norm with the logits' multiplier
            nxt, mul = (self.layers[i + 1].ahead("1"), 1.0) if i + 1 < n else (self.norm_w, self.cfg.logit_scale)
            if i == n - 1 and rows is not None:
                # nothing after the last layer's mixer mixes tokens: go on with the wanted ones
                a, x = a.index_select(0, rows), x.index_select(0, rows)
                if rows.numel() == 0:
                    return a.new_empty(0, self.cfg.hidden_size)
            w, ls = layer.behind("1")
            y = layer.mix.out(a)
            if layer.mlp is None:
                h = ops.branch_norm(x, y, w, nxt, eps, ls, mul)
            else:
                h = ops.branch_norm(x, y, w, layer.ahead("2"), eps, ls)
                w, ls = layer.behind("2")
                h = ops.branch_norm(x, layer.mlp(h), w, nxt, eps, ls, mul)
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
        return ops.project(hidden.contiguous(), self.head_w(), out_f32=True, shuf=self._head_shuf)

    def refresh_decode_weights(self, batch: Optional[int] = None):
        """Derived weight images that graph replays read, brought up to date eagerly."""
        if not self.embed.is_cuda:
            return
        for layer in self.layers:
            layer.mix.refresh()
            if layer.mlp is not None:
                layer.mlp.refresh()
        if "key" in self._head_shuf:
            self._head_shuf.get(self.head_w())

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
