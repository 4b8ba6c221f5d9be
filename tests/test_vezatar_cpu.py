"""Vezatar on the CPU path (fp32): reading and writing its files, every mechanism against the plain
implementation in vezatar_oracle.py, cache, ragged batches, scheduler, generation and trace replay."""
import copy
import io
import json

import numpy as np
import pytest
import torch
import vezatar_common as vc
import vezatar_oracle as oracle

from rag_tl_domainllm_optimizer_amd import models, ops
from rag_tl_domainllm_optimizer_amd.generation import ContinuousBatcher, Generator, SamplingParams
from rag_tl_domainllm_optimizer_amd.generation.paged import PAGE, PagedCache
from rag_tl_domainllm_optimizer_amd.generation.ragged import SHORT_TOKENS, RaggedBatch, StepEngine
from rag_tl_domainllm_optimizer_amd.models import io as mio
from rag_tl_domainllm_optimizer_amd.models.config import ModelConfig, config_from_hf, config_to_hf

TOL = 2e-4  # fp32 rounding reaches 4e-5 on these models


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


@pytest.fixture(scope="module")
def odd(tmp_path_factory):
    cfg = vc.odd()
    w = vc.weights(cfg, 1)
    return cfg, w, vc.load(cfg, w, tmp_path_factory.mktemp("odd"))


# ------------------------------------------------------------------ files and registry
def test_config_round_trip():
    for cfg in (vc.odd(), vc.even()):
        c = config_from_hf(cfg)
        assert c.is_layered and c.is_decoder and models.model_class(c) is models.LayeredLM
        assert config_to_hf(c) == json.loads(json.dumps(cfg))
        assert ModelConfig.from_dict(json.loads(json.dumps(c.to_dict()))) == c
    m = models.LayeredLM(models.resolve_preset("tiny-vezatar"), dtype=torch.float32)
    # parameters as the files count them: without the router's padding rows
    pad = sum(l.mlp.router_w.shape[0] - l.mlp.spec.experts - 1 for l in m.layers if isinstance(l.mlp, models.layered.MoEFF))
    n = sum(p.numel() for p in m.parameters()) - pad * m.cfg.hidden_size
    assert n == m.cfg.num_params()


def test_config_refuses_bad_sharing():
    for edit in (lambda l: l[1]["mixer"].update(kv_from=1), lambda l: l[1]["mixer"].update(kv_rank=20),
                 lambda l: l[3]["mixer"].update(kv_from=1), lambda l: l[1]["mixer"]["rot"].update(base=5.0),
                 lambda l: l[1]["mlp"]["router"].update(top=6), lambda l: l[0].update(type="other")):
        cfg = vc.odd()
        edit(cfg["layers"])
        with pytest.raises(ValueError):
            config_from_hf(cfg)
    with pytest.raises(ValueError):
        config_from_hf({"architecture": "Other"})


def test_load_is_strict(tmp_path, odd):
    cfg, w, _ = odd
    for edit in (lambda d: d.pop("l1.mlp.e2.up"), lambda d: d.update(extra=torch.zeros(2)),
                 lambda d: d.update({"l0.mix.uk": d["l0.mix.uk"][:-1].clone()}),
                 lambda d: d.update({"l1.mlp.shared.up": torch.zeros(99, 44)})):
        d = dict(w)
        edit(d)
        with pytest.raises((KeyError, ValueError)):
            vc.load(cfg, d, tmp_path / "x")


def test_save_pretrained_round_trip(tmp_path, odd):
    cfg, w, m = odd
    mio.save_pretrained(m, str(tmp_path / "s"))
    sd = mio.read_state_dict(str(tmp_path / "s"))
    assert set(sd) == set(w)
    for k in w:
        assert torch.equal(sd[k].view_as(w[k]), w[k]), k
    m2 = models.build_model(str(tmp_path / "s"), dtype=torch.float32)
    assert config_to_hf(m2.cfg) == config_to_hf(m.cfg)
    for a, b in zip(m.parameters(), m2.parameters()):
        assert torch.equal(a, b)


# ------------------------------------------------------------------ single mechanisms
@pytest.mark.parametrize("scaling", [None, (3.0, 64.0, 8.0, 0.5), (1.0, 512.0, 32.0, 1.0), (2.0, 4096.0, 4.0, 4.0)])
@pytest.mark.parametrize("dims", [2, 6, 64])
def test_rotary_tables(scaling, dims):
    m = vc.mixer(1, 4, dims, 4, 4, 1.0, base=10000.0, scaling=scaling)
    spec = models.config.layer_spec(vc.layer(m)).mixer.rot
    cos, sin = ops.yarn_rope_tables(spec.dims, spec.base, 300, spec.scaling)
    f, mult = oracle.yarn_freqs(m["rot"])
    a = torch.arange(300).double()[:, None] * f
    torch.testing.assert_close(cos, (a.cos() * mult).float(), rtol=0, atol=1e-6)
    torch.testing.assert_close(sin, (a.sin() * mult).float(), rtol=0, atol=1e-6)


def test_rotation_keeps_relative_positions():
    m = vc.mixer(1, 4, 8, 4, 4, 1.0, scaling=None)
    x = torch.randn(1, 8)
    y = torch.randn(1, 8)

    def dot(p, q):
        return float((oracle.rotate(x, torch.tensor([p]), m["rot"]) * oracle.rotate(y, torch.tensor([q]), m["rot"])).sum())
    assert abs(dot(5, 3) - dot(105, 103)) < 1e-4 and abs(dot(5, 3) - dot(5, 4)) > 1e-3


def test_gated_unit_and_router_against_oracle():
    cfg = vc.odd()
    w = {k: v.float() for k, v in vc.weights(cfg, 3).items()}
    h = torch.randn(17, cfg["width"]) * 2
    ml = cfg["layers"][0]["mlp"]
    gu = torch.cat([w["l0.mlp.gate"], w["l0.mlp.up"]])
    y = ops.branch_project(ops.glu_project(h, gu, ops.Glu(ml["limit"], 1.702, 1.0)), w["l0.mlp.down"])
    torch.testing.assert_close(y, oracle.dense_ff(w, "l0.mlp.", ml, h), rtol=1e-4, atol=1e-5)
    idx, wt = ops.moe_route(h @ w["l1.mlp.router"].T, w["l1.mlp.correction"], 2)
    oi, ow = oracle.route(w, "l1.mlp.", cfg["layers"][1]["mlp"], h)
    assert torch.equal(idx.long(), oi)
    torch.testing.assert_close(wt, ow, rtol=1e-5, atol=1e-6)


def test_branch_norm_against_oracle():
    x, y = torch.randn(5, 12), torch.randn(5, 12)
    wb, wn = torch.randn(12), torch.randn(12)
    want = x + oracle.rms(y, 0.1) * wb
    h = ops.branch_norm(x, y, wb, wn, 0.1)
    torch.testing.assert_close(x, want)
    torch.testing.assert_close(h, oracle.rms(want, 0.1) * wn)


# ------------------------------------------------------------------ the step
def test_layers_and_logits_against_oracle(odd):
    cfg, w, m = odd
    t = tokens(cfg, 90)
    layers = []
    want = oracle.forward(cfg, w, t, layers_out=layers)
    cache = m.make_cache(1, 128)
    cache.reserve(0, len(t))
    cache.sync()
    got = []
    h = m.step(RaggedBatch.build([(0, t, 0)], "cpu"), cache, layer_out=got)
    for a, b in zip(got, layers):
        torch.testing.assert_close(a, b, rtol=1e-4, atol=1e-4)
    assert vc.err(m.logits(h), want) < TOL
    assert vc.err(m.logits(m(torch.tensor([t]))), want) < TOL


def test_every_mechanism_shows_in_the_logits(odd):
    """each planted mistake moves the oracle's logits far beyond the tolerance of these tests"""
    cfg, w, _ = odd
    t = tokens(cfg, 40)
    want = oracle.forward(cfg, w, t)
    for fault in ("no_sink", "no_gate", "no_mscale", "half_layout", "no_correction", "weights_corrected", "renormalized",
                  "no_shared", "no_norm1b"):
        assert vc.err(oracle.forward(cfg, w, t, fault=(fault,)), want) > 100 * TOL, fault


@pytest.mark.parametrize("sizes", [(1,), (2,), (3, 5), (33, 2, 64), (SHORT_TOKENS, SHORT_TOKENS + 1), (63, 1, 1, 64, 65)])
def test_portions(odd, sizes):
    cfg, w, m = odd
    t = tokens(cfg, 150, 2)
    assert vc.err(vc.run(StepEngine(m, 1, 192), t, sizes), oracle.forward(cfg, w, t)) < TOL


def test_mixed_batches_and_reused_pages(odd):
    """unequal requests in one batch, left out of steps, released, their pages and rows used again in another
    order: every logit as if alone"""
    cfg, w, m = odd
    rng = np.random.default_rng(0)
    eng = StepEngine(m, 3, 5 * PAGE)
    live, done, nxt = {}, 0, 0
    want = {}
    while done < 7:
        while len(live) < 3 and nxt < 7:
            t = tokens(cfg, int(rng.integers(1, 100)), 10 + nxt)
            if sum((len(x[1]) + PAGE - 1) // PAGE for x in live.values()) + (len(t) + PAGE - 1) // PAGE > 5:
                break
            want[nxt] = oracle.forward(cfg, w, t)
            live[nxt] = [eng.admit(), t, 0]
            nxt += 1
        part = [k for k in live if rng.random() < 0.7] or list(live)[:1]
        ent = [(k, live[k][1][live[k][2]:live[k][2] + int(rng.choice([1, 1, 2, 30, 50]))]) for k in part]
        lg = eng.step([(live[k][0], c, list(range(len(c)))) for k, c in ent])
        o = 0
        for k, c in ent:
            assert vc.err(lg[o:o + len(c)], want[k][live[k][2]:live[k][2] + len(c)]) < TOL, k
            o += len(c)
            live[k][2] += len(c)
            if live[k][2] == len(live[k][1]):
                eng.release(live.pop(k)[0])
                done += 1


def test_needle_at_every_edge():
    """one far key among hundreds: page borders, the first token, the key just before"""
    cfg, w = vc.needle_model()
    m = models.LayeredLM(config_from_hf(cfg), dtype=torch.float32, init=False)
    mio.load_layered_state_dict(m, w)
    n = 200
    for at in (0, 1, 63, 64, 127, 128, 191, 192, n - 2):
        t = vc.needle_tokens(n, at)
        want = oracle.forward(cfg, w, t)[-1:]
        plain = list(t)
        plain[at] = 7
        assert vc.err(oracle.forward(cfg, w, plain)[-1:], want) > 0.2, at  # a missed needle would show
        for sizes in ((n,), (n - 1, 1), (64, 40, 1)):
            assert vc.err(vc.run(StepEngine(m, 1, 256), t, sizes)[-1:], want) < TOL, (at, sizes)


def test_first_tokens_and_single_token(odd):
    cfg, w, m = odd
    for n in (1, 2, 3):
        t = tokens(cfg, n, 40 + n)
        assert vc.err(vc.run(StepEngine(m, 1, 64), t, (n,)), oracle.forward(cfg, w, t)) < TOL


# ------------------------------------------------------------------ cache
def test_paged_cache_bookkeeping():
    c = PagedCache([8, 0, 4], rows=3, max_seq=200, tokens=256)
    assert c.n_pages == 5 and c.max_pages == 4 and c.pool(1) is None and c.pool(0).shape == (5, PAGE, 8)
    c.reserve(0, 65)
    c.reserve(1, 64)
    c.reserve(1, 64)
    assert c.free_tokens() == PAGE and not c.can_reserve(2, 65) and c.can_reserve(2, 64)
    with pytest.raises(RuntimeError):
        c.reserve(2, 65)
    with pytest.raises(ValueError):
        c.reserve(2, 300)
    c.sync()
    used = c.table[c.table > 0].tolist()
    assert len(used) == len(set(used)) == 3 and 0 not in used
    c.release(0)
    c.sync()
    assert c.table[0].tolist() == [0] * 4 and c.free_tokens() == 3 * PAGE
    c.reserve(2, 192)
    assert c.free_tokens() == 0
    c.release_all()
    assert c.free_tokens() == 256


def test_step_engine_refuses_bad_input(odd):
    cfg, w, m = odd
    eng = StepEngine(m, 2, 128)
    r = eng.admit()
    for toks, want in (([cfg["vocab"]], []), ([-1], []), ([1, 2], [2])):
        with pytest.raises(ValueError):
            eng.step([(r, toks, want)])
    eng.admit()
    with pytest.raises(RuntimeError):
        eng.admit()
    with pytest.raises(ValueError):
        StepEngine(models.build_model("tiny-llama:random"), 1, 64)


# ------------------------------------------------------------------ generation, scheduler, trace, CLI
def test_greedy_generation(odd):
    cfg, w, m = odd
    prompts = [tokens(cfg, n, 60 + n) for n in (5, 40, 1, 70)]
    want = [vc.greedy(cfg, w, p, 6) for p in prompts]
    gen = Generator(m, max_batch=4, max_seq=96, device="cpu")
    p = SamplingParams(max_new_tokens=6, do_sample=False)
    for _ in range(2):  # the second call reuses rows and pages
        out = gen.generate(prompts, p, eos_ids=[-5])
        assert [r.tolist() for r in out.tokens] == want


def test_continuous_batching_in_portions(odd):
    """more requests than rows, a pool too small for all of them, prompts entering 16 tokens at a time"""
    cfg, w, m = odd
    prompts = [tokens(cfg, n, 80 + n) for n in (50, 3, 70, 20, 33, 1)]
    want = [vc.greedy(cfg, w, p, 5) for p in prompts]
    gen = Generator(m, max_batch=3, max_seq=128, device="cpu", cache_tokens=3 * PAGE)
    cb = ContinuousBatcher(gen, SamplingParams(max_new_tokens=5, do_sample=False), eos_ids=[-5], prefill_tokens=16)
    todo, got = list(enumerate(prompts)), {}
    for _ in range(200):
        while todo and cb.free_rows():
            i, pr = todo.pop(0)
            cb.admit(pr, i)
        cb.step(1)
        for r in cb.collect():
            got[r.tag] = r.tokens
        if len(got) == len(prompts):
            break
    assert [got[i] for i in range(len(prompts))] == want
    assert gen.cache.free_tokens() == 3 * PAGE
    with pytest.raises(ValueError):
        cb.admit([1] * 124)


def test_trace_replay(tmp_path, odd):
    from rag_tl_domainllm_optimizer_amd.serve.trace import replay

    cfg, w, m = odd
    a, b = tokens(cfg, 40, 1), tokens(cfg, 9, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:39], "want": [0, 38]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 5, "entries": [{"id": "b", "tokens": b[2:], "want": [6, 0]}, {"id": "a", "tokens": a[39:], "want": [0]}],
              "end": ["a", "b"]}]
    said = []
    n = replay(m, io.StringIO("\n".join(json.dumps(s) for s in steps)), str(tmp_path), 128, said.append)
    assert n == 3 and said == ["done 0", "done 1", "done 5"]
    assert sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "5.f32"]
    wa, wb = oracle.forward(cfg, w, a), oracle.forward(cfg, w, b)
    for name, rows in (("0.f32", [wa[0], wa[38]]), ("5.f32", [wb[8], wb[2], wa[39]])):
        got = torch.from_numpy(np.fromfile(tmp_path / name, "<f4").reshape(-1, cfg["vocab"]).copy())
        assert vc.err(got, torch.stack(rows)) < TOL


def test_cli_rag_answers_with_a_layered_policy(capsys):
    from rag_tl_domainllm_optimizer_amd import cli

    cli.main(["rag", "--model.policy=tiny-vezatar:random", "--model.encoder=tiny-bert:random", "--ppo.max_new_tokens=4",
              "--ppo.max_prompt_tokens=64", "--data.synthetic_docs=24", "--retrieval.index=flat", "--query", "what is it"])
    line = [x for x in capsys.readouterr().out.splitlines() if x.startswith("{")][-1]
    assert "answer" in json.loads(line)


def test_serving_engines_with_a_layered_policy():
    """the RAG pipeline's answers, one by one, equal those of the continuous engine under load"""
    from rag_tl_domainllm_optimizer_amd.rag import RagPipeline
    from rag_tl_domainllm_optimizer_amd.retrieval import Encoder, FlatIndex
    from rag_tl_domainllm_optimizer_amd.serve import ContinuousEngine
    from rag_tl_domainllm_optimizer_amd.tokenizer import Tokenizer

    pol = models.LayeredLM(models.resolve_preset("tiny-vezatar"), dtype=torch.float32, seed=1)
    enc_m = models.build_model("tiny-bert", device="cpu", dtype=torch.float32, seed=2).eval()
    tok = Tokenizer.synthetic(pol.cfg.vocab_size, pol.cfg.arch)
    enc = Encoder(enc_m, Tokenizer.synthetic(enc_m.cfg.vocab_size, enc_m.cfg.arch), max_length=32)
    words = tok.words()
    docs = [" ".join(words[(7 * i + j) % len(words)] for j in range(12)) for i in range(30)]
    index = FlatIndex(enc.dim, "ip", "cpu")
    index.add(enc.encode(docs))
    pipe = RagPipeline(enc, index, docs, pol, tok, top_k=2, sampling=SamplingParams(max_new_tokens=4, do_sample=False),
                       max_prompt_tokens=96, max_batch=2, use_graph=False)
    qs = [f"{words[i]} {words[i + 3]}" for i in range(5)]
    direct = [pipe.answer([q])[0].answer for q in qs]
    with ContinuousEngine(pipe, chunk=2) as eng:
        assert [a.answer for a in eng.answer_many(qs, timeout=60)] == direct


def test_layered_models_refuse_adapters():
    with pytest.raises(NotImplementedError):
        models.build_model("tiny-vezatar:random").add_lora(8)


def test_wrong_config_values_are_read_not_assumed(odd):
    """every constant of config.json reaches the result: changing any of them changes the logits"""
    cfg, w, _ = odd
    t = tokens(cfg, 40, 9)
    base = None
    edits = [lambda c: None, lambda c: c["norm"].update(eps=0.5), lambda c: c["layers"][0]["mixer"].update(scale=0.7),
             lambda c: c["layers"][0]["mlp"].update(limit=0.3)]
    for k, v in (("base", 300.0),):
        edits.append(lambda c, k=k, v=v: [x["mixer"]["rot"].update({k: v}) for x in c["layers"][:2] + c["layers"][3:4]])
    for k, v in (("factor", 1.5), ("original", 16.0), ("fast", 0.9), ("slow", 0.1)):
        edits.append(lambda c, k=k, v=v: [x["mixer"]["rot"]["scaling"].update({k: v})
                                          for x in c["layers"][:2] + c["layers"][3:4]])
    for e in edits:
        c = copy.deepcopy(cfg)
        e(c)
        m = models.LayeredLM(config_from_hf(c), dtype=torch.float32, init=False)
        mio.load_layered_state_dict(m, w)
        got = vc.run(StepEngine(m, 1, 64), t, (40,))
        assert vc.err(got, oracle.forward(c, w, t)) < TOL
        if base is None:
            base = got
        else:
            assert vc.err(got, base) > 10 * TOL
