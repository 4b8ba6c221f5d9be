"""Small random Vezatar models for the tests: configurations in config.json form, weights by tensor name,
and the package's model loaded from them."""
from __future__ import annotations

import json
import os

import torch

import vezatar_oracle as oracle


def mixer(heads, dim, rot, vdim, rank, scale, base=900.0, scaling=(3.0, 64.0, 8.0, 0.5), kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale,
         "rot": {"base": base, "dims": rot}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def layer(mix, mlp=None):
    return {"type": "latent_attention", "mixer": mix, "mlp": mlp}


def dense(ff, limit=1.3):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, shared=None):
    d = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def config(vocab, width, layers, eps=3e-5):
    return {"architecture": "Vezatar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def odd():
    """sizes no MFMA kernel takes, layers of different shapes, every optional part present and absent"""
    return config(53, 44, [
        layer(mixer(3, 10, 6, 7, 22, 0.5), dense(26, 0.8)),
        layer(mixer(5, 8, 6, 9, 22, 0.45, kv_from=0), moe(5, 2, 14, 20)),
        layer(mixer(1, 4, 2, 11, 13, 0.6, base=70.0, scaling=None)),
        layer(mixer(2, 12, 6, 5, 22, 0.4, kv_from=0), moe(3, 3, 9)),
        layer(mixer(4, 6, 2, 8, 13, 0.5, base=70.0, scaling=None, kv_from=2), moe(4, 1, 16, 16)),
    ])


def even(heads=6, dim=32, rot=16, vdim=48, rank=64):
    """sizes of the MFMA kernels, two layers on one cache"""
    s = 2.0 * (dim + rot) ** -0.5
    return config(136, 192, [
        layer(mixer(heads, dim, rot, vdim, rank, s), dense(128, 2.5)),
        layer(mixer(heads, dim, rot, vdim, rank, s, kv_from=0), moe(9, 3, 128, 160)),
        layer(mixer(heads, dim, rot, vdim, rank, s, scaling=None), dense(64, 0.5)),
    ])


def weights(cfg, seed=0, dtype=torch.bfloat16, decisive=False):
    """Random tensors by name: norms around 1, sinks and corrections that matter, products of order one.
    ``decisive``: corrections far apart, so no routing call is close (bf16 comparisons: a call that falls
    the other way moves a position, and those that attend to it, by far more than rounding)."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain * k ** -0.5).to(dtype)

    def vec(name, n, mean, std):
        w[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)
    W, V = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(V, W, generator=g).to(dtype)
    lin("head", V, W)
    vec("final.norm", W, 1.0, 0.2)
    for i, s in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", s["mixer"], s["mlp"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            vec(p + n, W, 1.0, 0.2)
        H = m["heads"]
        lin(p + "mix.q", H * (m["dim"] + m["rot_dim"]), W, 2.0)
        if m.get("kv_from") is None:
            lin(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], W)
            vec(p + "mix.dkv.norm", m["kv_rank"], 1.0, 0.2)
        lin(p + "mix.uk", H * m["dim"], m["kv_rank"])
        lin(p + "mix.uv", H * m["vdim"], m["kv_rank"])
        vec(p + "mix.sink", H, 1.0, 1.0)
        lin(p + "mix.g", H * m["vdim"], W)
        lin(p + "mix.o", W, H * m["vdim"])

        def ff(q, n):
            lin(q + "gate", n, W, 2.0)
            lin(q + "up", n, W, 2.0)
            lin(q + "down", W, n)
        if f is None:
            continue
        if f["kind"] == "dense":
            ff(p + "mlp.", f["ff"])
            continue
        for e in range(f["router"]["experts"]):
            ff(f"{p}mlp.e{e}.", f["expert"]["ff"])
        lin(p + "mlp.router", f["router"]["experts"], W, 2.0)
        vec(p + "mlp.correction", f["router"]["experts"], 0.0, 0.3)
        if decisive:
            w[p + "mlp.correction"] = (2.0 * torch.randperm(f["router"]["experts"], generator=g)).to(dtype)
        if f.get("shared"):
            ff(p + "mlp.shared.", f["shared"]["ff"])
            lin(p + "mlp.shared.sg", 1, W, 2.0)
    return w


def load(cfg, w, tmp_path, device="cpu", dtype=torch.float32):
    """Through the registry: config.json + model.safetensors -> build_model."""
    from safetensors.torch import save_file

    from rag_tl_domainllm_optimizer_amd import models

    os.makedirs(tmp_path, exist_ok=True)
    with open(os.path.join(tmp_path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(tmp_path, "model.safetensors"))
    return models.build_model(str(tmp_path), device=device, dtype=dtype)


def run(eng, tokens, sizes):
    """All logits of one request fed in portions of ``sizes`` (the last one repeats)."""
    row = eng.admit()
    outs, p, i = [], 0, 0
    while p < len(tokens):
        c = tokens[p:p + sizes[min(i, len(sizes) - 1)]]
        outs.append(eng.step([(row, c, list(range(len(c))))]).cpu())
        p += len(c)
        i += 1
    eng.release(row)
    return torch.cat(outs)


def err(got, want):
    """largest per-position difference, relative to the spread of the expected logits"""
    return float(((got - want).pow(2).mean(-1).sqrt() / want.std()).max())


def greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(oracle.forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- a model in which one token asks for another: vocabulary ids 0 = asker, 1 = needle, others filler ----
ASK, NEEDLE = 0, 1


def needle_model(heads=2, dim=16, rot=8, vdim=16, rank=32, width=64, seed=5):
    """One attention layer, no feed-forward. The asker's query matches the needle's key in every head, whatever
    the distance (unrotated part only); the scores of all other pairs stay small. A needle that is seen,
    missed or counted twice shows in the asker's logits at once."""
    cfg = config(40, width, [layer(mixer(heads, dim, rot, vdim, rank, 1.0))])
    w = {k: v.float() for k, v in weights(cfg, seed).items()}
    for k in ("l0.norm1", "l0.norm1b", "final.norm", "l0.mix.dkv.norm"):
        w[k] = torch.ones_like(w[k])
    w["embed"][:, :2] = 0
    w["embed"][ASK, 0] = w["embed"][NEEDLE, 1] = 12.0
    w["l0.mix.q"] *= 0.05
    w["l0.mix.dkv"] *= 0.3
    w["l0.mix.uk"] *= 0.3
    w["l0.mix.dkv"][:rank, 1] = 0
    w["l0.mix.dkv"][0, 1] = 6.0            # needle -> latent 0
    for h in range(heads):
        w["l0.mix.uk"][h * dim, 0] = 2.0    # latent 0 -> key dimension 0
        w["l0.mix.q"][h * (dim + rot), :] = 0
        w["l0.mix.q"][h * (dim + rot), 0] = 0.4  # asker -> query dimension 0
    w["l0.mix.sink"] = torch.full((heads,), 1.0)
    return cfg, {k: v.to(torch.bfloat16) for k, v in w.items()}


def needle_tokens(n, needle_at, seed=0):
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(2, 40, (n,), generator=g).tolist()
    t[needle_at] = NEEDLE
    t[-1] = ASK
    return t
