"""Pafolorn on the GPU: every kernel against fp32 torch arithmetic, and the model in fp32 and bf16 against the
plain implementation (pafolorn_oracle.py): whole prompts, portions, decoding, mixed batches with reused pages
and state slots, far keys and far memories, greedy generation through the captured decode step and the scheduler."""
import json
import os
import subprocess
import sys

import numpy as np
import pafolorn_common as pc
import pafolorn_oracle as oracle
import pytest
import torch

from rag_tl_domainllm_optimizer_amd import models, ops
from rag_tl_domainllm_optimizer_amd.generation import ContinuousBatcher, Generator, SamplingParams
from rag_tl_domainllm_optimizer_amd.generation.paged import PAGE, PagedCache
from rag_tl_domainllm_optimizer_amd.generation.ragged import RaggedBatch, StepEngine
from rag_tl_domainllm_optimizer_amd.ops import native

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_TOL = 2e-4   # per-position logits difference relative to their spread
BF16_TOL = 0.1   # bf16 activations and products
DTYPES = [torch.float32, torch.bfloat16]


def rel(a, b):
    a, b = a.float().cpu(), b.float().cpu()
    return float((a - b).norm() / b.norm().clamp_min(1e-30))


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, want, dtype):
    e = (got - want).pow(2).mean(-1).sqrt() / want.std()
    if dtype == torch.float32:
        assert float(e.max()) < F32_TOL, float(e.max())
    else:
        assert float(e.quantile(0.9)) < BF16_TOL and float(e.max()) < 4 * BF16_TOL, (float(e.max()), float(e.median()))


CONFIGS = {
    "odd": pc.odd,                                                                     # no MFMA kernel fits
    "even": pc.even,
    "group20_d128": lambda: pc.even(40, 2, 128, 128, 100, 3, 4, 1, 128, 64),           # two head tiles, the last half empty
    "ragged_d40_v72": lambda: pc.even(6, 3, 40, 72, 65, 64, 3, 3, 24, 40, 5, 136, 20),  # ragged sizes on the MFMA kernels
    "v256_d200": lambda: pc.even(2, 1, 200, 256, 130, 7, 2, 2, 200, 128),              # values wider than the prefill kernel's
}


@pytest.fixture(scope="module")
def model_of(tmp_path_factory):
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            cfg = CONFIGS[name]()
            w = pc.weights(cfg, 1)
            made[name, dtype] = (cfg, w, pc.load(cfg, w, tmp_path_factory.mktemp(name), DEV, dtype))
        return made[name, dtype]
    return get


# ------------------------------------------------------------------ kernels
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [4, 130, 192, 4096])
def test_output_norm_with_scale(dtype, H):
    T, eps = 5, 1e-3
    x, y = torch.randn(T, H), torch.randn(T, H).to(dtype)
    w, ls, wn = (torch.randn(H).to(dtype) for _ in range(3))
    h_tol = 1e-6 if dtype == torch.float32 else 3e-3
    want = x + oracle.rms(y.float(), eps) * w.float() * ls.float()
    for yy in (y.to(DEV), ops.SplitK(torch.stack([y.float() * 0.25, y.float() * 0.75]).to(DEV), 2, T, H, dtype)):
        xg = x.to(DEV)
        h = ops.branch_norm(xg, yy, w.to(DEV), None, eps, ls.to(DEV))
        assert rel(xg, want) < 1e-6 and torch.equal(h.float(), xg.to(dtype).float())
    xg = x.to(DEV)
    h = ops.branch_norm(xg, y.to(DEV), w.to(DEV), wn.to(DEV), eps, ls.to(DEV), 0.3)
    assert rel(h, oracle.rms(want, eps) * wn.float() * 0.3) < h_tol
    table, ids = torch.randn(9, H).to(dtype), torch.tensor([0, 8, 3, 3, 1])
    xg, h = ops.embed_norm(table.to(DEV), ids.to(DEV), None, eps, w.to(DEV))
    assert rel(xg, oracle.rms(table[ids].float(), eps) * w.float()) < 1e-6 and torch.equal(h.float(), xg.to(dtype).float())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 16, 17, 64, 65, 300, 700])
def test_squared_relu_epilogues(M, dtype):
    for K, N in ((256, 512), (128, 192), (72, 144), (44, 30), (512, 136)):
        x, w = torch.randn(M, K).to(dtype), (torch.randn(N, K) * 0.15).to(dtype)
        want = (x.float() @ w.float().T).clamp(min=0) ** 2
        assert rel(ops.act_project(x.to(DEV), w.to(DEV), ops.ACT_RELU2, ops.ShufCache()), want) < \
            (1e-6 if dtype == torch.float32 else 5e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V,rot", [(6, 3, 8, 8, 8), (16, 1, 64, 128, 32), (17, 1, 128, 64, 128), (64, 2, 192, 72, 48),
                                         (4, 4, 256, 256, 256), (5, 5, 40, 24, 6), (4, 2, 10, 7, 2)])
@pytest.mark.parametrize("size,keep,cap", [(70, 5, 4.0), (64, 64, 0.0), (1, 0, 9.0), (0, 0, 6.0), (33, 130, 5.0)])
def test_window_attention(dtype, H, G, D, V, rot, size, keep, cap):
    """one request in portions of all kinds (prompt kernel, short portions, single tokens) behind another's pages;
    per row of scores one key, at an edge of what is visible, stands out"""
    g = torch.Generator().manual_seed(H * D + size)
    T, eps = 300, 1e-3
    d = ops.WindowDims(H, G, D, V, 1.5 * D ** -0.5, cap, size, keep)
    q, k, v = (torch.randn(T, n, generator=g) for n in (H * D, G * D, G * V))
    for i in range(T):  # a query copies the key at an edge of its window or of the kept tokens
        j = (i - size + 1, i - size, keep - 1, keep, i)[i % 5]
        if 0 <= j <= i:
            q[i] = 1.5 * k[j].view(G, 1, D).expand(G, H // G, D).reshape(-1)
    qw, kw = torch.rand(H * D, generator=g) + 0.5, torch.rand(G * D, generator=g) + 0.5
    q, k, v, qw, kw = (t.to(dtype) for t in (q, k, v, qw, kw))
    mx = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": d.scale, "softcap": cap or 1e6,
          "rot": {"base": 300.0, "dims": rot}, "mask": {"size": size or 10 ** 6, "keep_first": keep}}
    w = {"q": torch.eye(H * D + G * (D + V))[:H * D], "k": torch.eye(H * D + G * (D + V))[H * D:H * D + G * D],
         "v": torch.eye(H * D + G * (D + V))[H * D + G * D:], "q.norm": qw.float(), "k.norm": kw.float()}
    want = oracle.window_attention(w, "", mx, torch.cat([q, k, v], 1).float(), eps) * 0.5
    cache = PagedCache([d.cache_width], 3, T, 2 * T + 64, DEV, dtype)
    cache.reserve(0, 100)
    cache.reserve(2, T)
    cache.sync()
    cos, sin = ops.yarn_rope_tables(rot, 300.0, cache.max_seq, None, DEV)
    proj = torch.cat([torch.zeros(T, 8), q.float(), k.float(), v.float(), torch.zeros(T, -(H * D + G * (D + V)) % 8)], 1).to(dtype).to(DEV)
    out = torch.zeros(T, (H * V + 7) // 8 * 8 + 8, dtype=dtype, device=DEV)
    at = 0
    for n in (1, 2, 130, 31, 1, 33, 64, 38):
        b = RaggedBatch.build([(2, [0] * n, at)], DEV)
        ops.window_attention(proj[at:at + n], 8, d, qw.to(DEV), kw.to(DEV), eps, cos, sin, b, cache.pool(0), cache.table,
                             out[at:at + n, :H * V], 0.5)
        at += n
    e = (out[:, :H * V].float().cpu() - want).norm(dim=1) / want.norm(dim=1)
    assert float(e.max()) < (2e-5 if dtype == torch.float32 else 4e-2), int(e.argmax())
    assert rel(out[:, :H * V], want) < (1e-5 if dtype == torch.float32 else 1.2e-2)
    assert float(out[:, H * V:].abs().max()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ch", [True, False])
@pytest.mark.parametrize("H,K,D,V,taps", [(4, 2, 32, 64, 4), (6, 3, 9, 11, 3), (3, 1, 128, 128, 2), (2, 2, 200, 72, 4), (2, 1, 64, 256, 1),
                                          (3, 3, 1, 7, 5), (2, 2, 256, 130, 4)])
def test_delta_rule(dtype, ch, H, K, D, V, taps):
    """projections in, gated read-outs and states out: single tokens beside portions, a slot that held another
    request's state, decays from none to immediate"""
    g = torch.Generator().manual_seed(H * D + V)
    T, C, eps = 150, 2 * K * D + H * V, 0.02
    x, b, z = torch.randn(T, C, generator=g), torch.randn(T, H, generator=g), torch.randn(T, H * V, generator=g)
    a = torch.randn(T, H * D if ch else H, generator=g) * 4 - 2
    x, b, z, a = (t.to(dtype) for t in (x, b, z, a))
    conv, nw = (torch.randn(C, taps, generator=g) * 0.5).to(dtype), (torch.rand(V, generator=g) + 0.5).to(dtype)
    A, dt = torch.randn(H, generator=g) * 2 - 1, torch.randn(a.shape[1], generator=g)
    y = oracle.short_conv(x.float(), conv.float())
    of = torch.tensor([h // (H // K) for h in range(H)])
    q = (oracle.unit(y[:, :K * D].view(T, K, D)) * D ** -0.5)[:, of]
    k, v = oracle.unit(y[:, K * D:2 * K * D].view(T, K, D))[:, of], y[:, 2 * K * D:].view(T, H, V)
    dec = torch.exp(-torch.exp(A)[:, None] * oracle.softplus((a.float() + dt).view(T, H, -1))).expand(T, H, D)
    o = oracle.delta_rule(q, k, v, torch.sigmoid(b.float()), dec)
    o = (oracle.rms(o, eps) * nw.float()).reshape(T, -1) * (torch.sigmoid(z.float()) if ch else oracle.silu(z.float())) * 0.7
    state, ring = torch.randn(3, H, D, V, device=DEV) * 9, torch.randn(3, taps, C, device=DEV).to(dtype) * 9
    other = state[1].clone()
    dv = [t.to(DEV) for t in (x, b, a, z, conv, A, dt, nw)]
    out, at = torch.zeros(T, H * V + 3, dtype=dtype, device=DEV), 0
    rows = {0: 0, 2: 0}  # the same sequence twice: in slot 2 as below, in slot 0 a step behind
    for n0, n2 in ((0, 1), (1, 1), (1, 2), (16, 17), (1, 1), (3, 48), (33, 80), (1, 0)):
        ent = [(r, [0] * n, rows[r]) for r, n in ((0, n0), (2, n2)) if n]
        bt = RaggedBatch.build(ent, DEV)
        src = torch.empty(sum(len(e[1]) for e in ent), dtype=torch.long)
        for e, off in zip(ent, bt.offset):
            src[off:off + len(e[1])] = e[2] + torch.arange(len(e[1]))
        part = [t[src.to(DEV)] for t in dv[:4]]
        got = torch.zeros(len(src), H * V + 3, dtype=dtype, device=DEV)
        ops.delta_rule(*part, *dv[4:], eps, bt, state, ring, got[:, :H * V], 0.7, K, not ch)
        for e, off in zip(ent, bt.offset):
            err = rel(got[off:off + len(e[1]), :H * V], o[e[2]:e[2] + len(e[1])])
            assert err < (2e-5 if dtype == torch.float32 else 8e-3), (e[0], e[2], len(e[1]), err)
            rows[e[0]] += len(e[1])
        assert float(got[:, H * V:].abs().max()) == 0
    assert rows[2] == T and torch.equal(state[1], other)


def test_parked_rows_change_nothing():
    s, r = torch.randn(2, 2, 8, 8, device=DEV), torch.randn(2, 3, 48, device=DEV)
    s0, r0 = s.clone(), r.clone()
    b = RaggedBatch.single(torch.zeros(2, dtype=torch.long, device=DEV), torch.full((2,), -1, dtype=torch.int32, device=DEV),
                           torch.full((2,), 5, dtype=torch.int32, device=DEV), 64)
    z = torch.randn(2, 16, device=DEV)
    out = torch.empty(2, 16, device=DEV)
    ops.delta_rule(torch.randn(2, 48, device=DEV), z[:, :2], z[:, :2], z, torch.randn(48, 3, device=DEV), torch.zeros(2, device=DEV),
                   torch.zeros(2, device=DEV), torch.ones(8, device=DEV), 1e-5, b, s, r, out, 1.0, 2, True)
    assert torch.equal(s, s0) and torch.equal(r, r0) and bool(torch.isfinite(out).all())


def test_wrappers_refuse_bad_shapes():
    n = native()
    i = torch.zeros(1, dtype=torch.int32, device=DEV)
    q, pool, tab = torch.randn(1, 12, device=DEV), torch.zeros(2, 64, 10, device=DEV), torch.zeros(1, 1, dtype=torch.int32, device=DEV)
    with pytest.raises(RuntimeError):  # pool of another width
        n.window_any(q, pool, tab, i, i, torch.empty(1, 12, device=DEV), 1.0, [3, 1, 4, 4, 0, 0], [1.0, 0.0])
    with pytest.raises(RuntimeError):  # heads that do not divide
        n.window_any(q, pool, tab, i, i, torch.empty(1, 12, device=DEV), 1.0, [3, 2, 4, 4, 0, 0], [1.0, 0.0])
    s, r = torch.zeros(1, 2, 8, 8, device=DEV), torch.zeros(1, 3, 48, device=DEV)
    b = RaggedBatch.single(torch.zeros(1, dtype=torch.long, device=DEV), i, i, 64)
    z = torch.randn(1, 16, device=DEV)
    with pytest.raises(RuntimeError):  # taps of another count than the ring's
        ops.delta_rule(torch.randn(1, 48, device=DEV), z[:, :2], z[:, :2], z, torch.randn(48, 4, device=DEV),
                       torch.zeros(2, device=DEV), torch.zeros(2, device=DEV), torch.ones(8, device=DEV), 1e-5, b, s, r,
                       torch.empty(1, 16, device=DEV), 1.0, 2, True)


# ------------------------------------------------------------------ model
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_portions_and_decoding(model_of, name, dtype):
    cfg, w, m = model_of(name, dtype)
    t = tokens(cfg, 260, 3)
    want = oracle.forward(cfg, w, t)
    eng = StepEngine(m, 2, 320)
    for sizes in ((260,), (129, 1), (2, 33, 64, 1, 100, 3), (2,)):
        check(pc.run(eng, t, sizes), want, dtype)


@pytest.mark.parametrize("name", ["odd", "even"])
def test_residual_after_every_layer(model_of, name):
    cfg, w, m = model_of(name, torch.float32)
    t = tokens(cfg, 70, 4)
    layers, got = [], []
    oracle.forward(cfg, w, t, layers_out=layers)
    cache = m.make_cache(1, 128)
    cache.reserve(0, len(t))
    cache.sync()
    m.step(RaggedBatch.build([(0, t, 0)], DEV), cache, layer_out=got)
    for a, b in zip(got, layers):
        torch.testing.assert_close(a.cpu(), b, rtol=5e-4, atol=5e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "even", "group20_d128"])
def test_mixed_batches_and_reused_slots(model_of, name, dtype):
    cfg, w, m = model_of(name, dtype)
    rng = np.random.default_rng(1)
    eng = StepEngine(m, 3, 8 * PAGE)
    live, nxt, done, want, got = {}, 0, 0, {}, {}
    while done < 8:
        while len(live) < 3 and nxt < 8:
            t = tokens(cfg, int(rng.integers(1, 200)), 10 + nxt)
            if sum((len(x[1]) + PAGE - 1) // PAGE for x in live.values()) + (len(t) + PAGE - 1) // PAGE > 8:
                break
            want[nxt], got[nxt] = oracle.forward(cfg, w, t), []
            live[nxt] = [eng.admit(), t, 0]
            nxt += 1
        part = [k for k in live if rng.random() < 0.7] or list(live)[:1]
        ent = [(k, live[k][1][live[k][2]:live[k][2] + int(rng.choice([1, 1, 2, 40, 90]))]) for k in part]
        lg = eng.step([(live[k][0], c, list(range(len(c)))) for k, c in ent]).cpu()
        o = 0
        for k, c in ent:
            got[k].append(lg[o:o + len(c)])
            o += len(c)
            live[k][2] += len(c)
            if live[k][2] == len(live[k][1]):
                eng.release(live.pop(k)[0])
                done += 1
    check(torch.cat([torch.cat(got[k]) for k in want]), torch.cat([want[k] for k in want]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,keep", [(70, 5), (64, 64), (128, 0), (33, 66)])
def test_needle_at_every_edge(tmp_path, dtype, size, keep):
    """one key among hundreds, just inside and just outside the window and the kept tokens, at page borders"""
    cfg, w = pc.needle_model(size, keep)
    m = pc.load(cfg, w, tmp_path, DEV, dtype)
    eng = StepEngine(m, 1, 256)
    n, hidden = 200, 0
    for at in sorted({0, keep - 1, keep, keep + 1, 63, 64, 65, n - size - 1, n - size, n - size + 1, n - 2}):
        if not 0 <= at < n - 1:
            continue
        asks = [a for a in (at + 1, at + size - 1, at + size, n - 1) if at < a < n]
        t = pc.needle_tokens(n, at, asks)
        want = oracle.forward(cfg, w, t)
        hidden += sum(not (a - at < size or at < keep) for a in asks)
        for sizes in ((n,), (n - 1, 1), (64, 40, 1), (7, 2)):
            got = pc.run(eng, t, sizes)
            for a in asks:
                assert pc.err(got[a:a + 1], want[a:a + 1]) < (F32_TOL if dtype == torch.float32 else BF16_TOL), (at, a, sizes)
    assert hidden


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ch", [True, False])
def test_far_memory(tmp_path, ch, dtype):
    """a write that only the carried state remembers, read hundreds of tokens later"""
    cfg, w = pc.memory_model(ch)
    m = pc.load(cfg, w, tmp_path, DEV, dtype)
    n = 300
    t = pc.needle_tokens(n, 3, [n - 1])
    want = oracle.forward(cfg, w, t)[-1:]
    assert pc.err(oracle.forward(cfg, w, t, fault=("state_lost",))[-1:], want) > 2 * BF16_TOL
    eng = StepEngine(m, 1, 320)
    for sizes in ((n,), (n - 1, 1), (64, 40, 1), (2,)):
        assert pc.err(pc.run(eng, t, sizes)[-1:], want) < (F32_TOL if dtype == torch.float32 else BF16_TOL), sizes


@pytest.mark.parametrize("name", ["odd", "even"])
def test_long_decoding(model_of, name):
    """several hundred tokens one by one, across page and window borders, against the whole sequence at once"""
    cfg, w, m = model_of(name, torch.float32)
    t = tokens(cfg, 400, 6)
    check(pc.run(StepEngine(m, 1, 448), t, (7, 1)), oracle.forward(cfg, w, t), torch.float32)


# ------------------------------------------------------------------ generation
@pytest.mark.parametrize("name", ["odd", "even"])
@pytest.mark.parametrize("use_graph", [True, False])
def test_greedy_generation(model_of, name, use_graph):
    cfg, w, m = model_of(name, torch.float32)
    prompts = [tokens(cfg, n, 60 + n) for n in (5, 40, 70)]
    want = [pc.greedy(cfg, w, p, 12) for p in prompts]
    gen = Generator(m, max_batch=4, max_seq=128, device=DEV, use_graph=use_graph)
    p = SamplingParams(max_new_tokens=12, do_sample=False)
    for _ in range(3):  # later calls replay the captured step on reused rows
        out = gen.generate(prompts, p, eos_ids=[-5])
        assert [r.tolist() for r in out.tokens] == want
        torch.randn(64, 64, device=DEV) @ torch.randn(64, 64, device=DEV)
        torch.cuda.synchronize()


@pytest.mark.parametrize("name", ["even", "ragged_d40_v72"])
def test_graph_replays_equal_the_eager_step(model_of, name):
    """bf16: greedy tokens and their log-probs of the captured decode step, bitwise the eager step's"""
    cfg, w, m = model_of(name, torch.bfloat16)
    prompts = [tokens(cfg, n, 70 + n) for n in (9, 130, 64, 3, 77)]
    p = SamplingParams(max_new_tokens=24, do_sample=False)
    eager = Generator(m, max_batch=8, max_seq=192, device=DEV, use_graph=False).generate(prompts, p, eos_ids=[-5])
    gen = Generator(m, max_batch=8, max_seq=192, device=DEV)
    for _ in range(4):
        out = gen.generate(prompts, p, eos_ids=[-5])
        assert torch.equal(out.tokens, eager.tokens) and torch.equal(out.logprobs, eager.logprobs)


def test_continuous_batching_in_portions(model_of):
    """waiting, half-read and finished requests beside decoding ones; new row buckets are captured on the way"""
    cfg, w, m = model_of("even", torch.float32)
    prompts = [tokens(cfg, n, 80 + n) for n in (50, 3, 170, 20, 33, 1, 90)]
    want = [pc.greedy(cfg, w, p, 6) for p in prompts]
    gen = Generator(m, max_batch=3, max_seq=192, device=DEV, cache_tokens=4 * PAGE)
    for _ in range(2):
        cb = ContinuousBatcher(gen, SamplingParams(max_new_tokens=6, do_sample=False), eos_ids=[-5], prefill_tokens=48)
        todo, got = list(enumerate(prompts)), {}
        for _ in range(300):
            while todo and cb.free_rows():
                i, pr = todo.pop(0)
                cb.admit(pr, i)
            cb.step(2)
            for r in cb.collect():
                got[r.tag] = r.tokens
            if len(got) == len(prompts):
                break
        assert [got[i] for i in range(len(prompts))] == want
        assert gen.cache.free_tokens() == 4 * PAGE


def test_preset_runs_in_serving_dtype():
    m = models.LayeredLM(models.resolve_preset("tiny-pafolorn"), device=DEV, dtype=torch.bfloat16, seed=2)
    out = Generator(m, max_batch=2, max_seq=128, device=DEV).generate([[5, 6, 7], list(range(3, 90))],
                                                                      SamplingParams(max_new_tokens=8, do_sample=False), eos_ids=[-5])
    assert out.tokens.shape == (2, 8) and bool(torch.isfinite(out.logprobs).all())


def test_trace_program(model_of, tmp_path):
    """bin/trace_run as a program of its own: answers before it asks for the next step"""
    cfg, w, m = model_of("even", torch.float32)
    pc.load(cfg, w, tmp_path / "model")
    t = tokens(cfg, 80, 5)
    p = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype",
                          "float32", "--out", str(tmp_path / "out"), "--max-tokens", "128"], stdin=subprocess.PIPE,
                         stdout=subprocess.PIPE, text=True)
    try:
        for i, (a, b) in enumerate(((0, 70), (70, 71), (71, 80))):
            p.stdin.write(json.dumps({"step": i, "entries": [{"id": "x", "tokens": t[a:b], "want": [b - a - 1]}], "end": []}) + "\n")
            p.stdin.flush()
            line = ""
            while not line.startswith("done"):
                line = p.stdout.readline()
                assert line
            assert line.split() == ["done", str(i)]
        p.stdin.close()
        assert p.wait(30) == 0
    finally:
        p.kill()
    want = oracle.forward(cfg, w, t)
    for i, k in enumerate((69, 70, 79)):
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{i}.f32", "<f4").copy())[None]
        assert pc.err(got, want[k:k + 1]) < F32_TOL
