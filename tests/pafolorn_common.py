"""Small random Pafolorn models for the tests: configurations in config.json form, weights by tensor name,
and models in which one token decides."""
from __future__ import annotations

import pafolorn_oracle as oracle
import torch
from vezatar_common import err, load, run  # noqa: F401  (they know nothing of the design)


def attn(heads, kv, dim, vdim, size, keep, rot=None, base=500.0, scale=None, softcap=12.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 1.5 * dim ** -0.5, "softcap": softcap,
            "rot": {"base": base, "dims": rot or dim}, "mask": {"size": size, "keep_first": keep}}


def delta(heads, kv, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def channel(mixer, ff=None):
    return {"type": "channel_delta", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def parallel(left, right, ls, rs, ff=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab, width, layers, eps=2e-4, logit_scale=0.6):
    return {"architecture": "Pafolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers}


def odd():
    """sizes no MFMA kernel takes; layers of different shapes, with and without feed-forward"""
    return config(59, 42, [
        parallel(attn(6, 2, 10, 7, 21, 3, rot=6), delta(6, 3, 9, 11, 3), 0.8, 1.3, 30),
        channel(delta(4, 2, 7, 5, 1), 26),
        parallel(attn(3, 3, 6, 13, 1, 0, rot=2, base=70.0, softcap=3.0), delta(2, 1, 18, 6, 5), -0.5, 0.9),
        channel(delta(3, 3, 12, 9, 4)),
        parallel(attn(5, 1, 8, 5, 300, 9, base=40.0), delta(3, 1, 5, 7, 2), 1.2, 0.4, 22),
    ])


def even(heads=8, kv=2, dim=32, vdim=64, size=80, keep=5, dheads=4, dkv=2, ddim=64, dvdim=32, taps=4, width=128, rot=None):
    """sizes of the MFMA kernels"""
    return config(136, width, [
        channel(delta(dheads, dkv, ddim, dvdim, taps)),
        parallel(attn(heads, kv, dim, vdim, size, keep, rot), delta(dheads, dheads, dvdim, ddim, taps), 0.7, 1.2, 256),
        channel(delta(dheads, dheads, ddim, dvdim, 3), 192),
        parallel(attn(heads, kv, dim, vdim, 2 * size, 0, rot), delta(dheads, dkv, ddim, ddim, 2), 0.9, 0.5, 64),
    ])


def weights(cfg, seed=0, dtype=torch.bfloat16, a_rank=10, g_rank=12):
    """Random tensors by name: norms around 1, decays from slow to fast, products of order one."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain * k ** -0.5).to(dtype)

    def vec(name, n, mean, std):
        w[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)

    def delta_w(p, m, ch):
        H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for k, n in (("q", K * D), ("k", K * D), ("v", H * V)):
            lin(p + k, n, W)
            w[p + k + ".conv"] = (torch.randn(n, m["conv"], generator=g) * 0.5 + 0.3).to(dtype)
        lin(p + "b", H, W, 1.5)
        vec(p + "A_log", H, -1.5, 1.5)
        vec(p + "norm", V, 1.0, 0.2)
        if ch:
            lin(p + "a1", a_rank, W)
            lin(p + "a2", H * D, a_rank, 1.5)
            vec(p + "dt_bias", H * D, -1.0, 1.0)
            lin(p + "g1", g_rank, W)
            lin(p + "g2", H * V, g_rank, 1.5)
        else:
            lin(p + "a", H, W)
            vec(p + "dt_bias", H, -1.0, 1.0)
            lin(p + "g", H * V, W)
        lin(p + "o", W, H * V)
    W = cfg["width"]
    w["embed"] = torch.randn(cfg["vocab"], W, generator=g).to(dtype)
    vec("embed.norm", W, 1.0, 0.2)
    vec("final.norm", W, 1.0, 0.2)
    for i, s in enumerate(cfg["layers"]):
        p, m = f"l{i}.", s["mixer"]
        for j in "12" if s["mlp"] else "1":
            vec(f"{p}norm{j}", W, 1.0, 0.2)
            vec(f"{p}ls{j}", W, 0.7, 0.2)
        if s["type"] == "channel_delta":
            delta_w(p + "mix.", m, True)
        else:
            a = m["left"]
            q = p + "mix.left."
            lin(q + "q", a["heads"] * a["dim"], W)
            lin(q + "k", a["kv_heads"] * a["dim"], W)
            lin(q + "v", a["kv_heads"] * a["vdim"], W)
            vec(q + "q.norm", a["heads"] * a["dim"], 1.0, 0.2)
            vec(q + "k.norm", a["kv_heads"] * a["dim"], 1.0, 0.2)
            lin(q + "o", W, a["heads"] * a["vdim"])
            delta_w(p + "mix.right.", m["right"], False)
        if s["mlp"]:
            lin(p + "mlp.up", s["mlp"]["ff"], W, 1.4)
            lin(p + "mlp.down", W, s["mlp"]["ff"])
    return w


def greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(oracle.forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- models in which one token asks for another: vocabulary ids 0 = asker, 1 = needle, others filler ----
ASK, NEEDLE = 0, 1


def needle_model(size, keep, heads=4, kv=2, dim=16, vdim=24, width=64, seed=5):
    """One parallel layer whose left side decides. The asker's query matches the needle's key in every head, on
    dimensions that are not rotated; all other scores stay near 0. A needle that is seen though hidden, or missed
    though visible, shows in the asker's logits at once."""
    cfg = config(40, width, [parallel(attn(heads, kv, dim, vdim, size, keep, rot=dim - 8, scale=0.8, softcap=20.0),
                                      delta(2, 2, 8, 8, 2), 1.0, 0.0)], eps=1e-5, logit_scale=1.0)
    w = {k: v.float() for k, v in weights(cfg, seed).items()}
    for k in ("embed.norm", "l0.norm1", "l0.ls1", "final.norm", "l0.mix.left.q.norm", "l0.mix.left.k.norm"):
        w[k] = torch.ones_like(w[k])
    w["embed"][:, :2] = 0
    w["embed"][ASK, 0] = w["embed"][NEEDLE, 1] = 12.0
    w["l0.mix.left.q"] *= 0.05
    for n, name, src in ((heads, "q", 0), (kv, "k", 1)):
        t = w[f"l0.mix.left.{name}"]
        for h in range(n):
            t[h * dim + dim - 1, :] = 0
            t[h * dim + dim - 1, src] = 3.0
    return cfg, {k: v.to(torch.bfloat16) for k, v in w.items()}


def memory_model(ch, heads=4, kv=2, dim=16, vdim=16, taps=3, width=64, seed=7):
    """One delta-rule layer that hardly decays and writes at the needle only; the asker's query is the needle's key.
    A state that is lost, reset late or taken from another request shows in the asker's logits."""
    m = delta(heads, kv, dim, vdim, taps)
    lay = channel(m) if ch else parallel(attn(1, 1, 8, 8, 4, 1), m, 0.0, 1.0)
    cfg = config(40, width, [lay], eps=1e-5, logit_scale=1.0)
    w = {k: v.float() for k, v in weights(cfg, seed).items()}
    p = "l0.mix." if ch else "l0.mix.right."
    for k in ("embed.norm", "l0.norm1", "l0.ls1", "final.norm", p + "norm"):
        w[k] = torch.ones_like(w[k])
    w["embed"][:, :2] = 0
    w["embed"][:, 2] = 1.0
    w["embed"][ASK, 0] = w["embed"][NEEDLE, 1] = 12.0
    for n in ("q", "k", "v"):
        w[p + n + ".conv"].zero_()
        w[p + n + ".conv"][:, -1] = 1.0
    g = torch.Generator().manual_seed(seed)
    r = 2 * torch.rand(kv * dim, generator=g)
    for n, src in (("q", 0), ("k", 1)):
        w[p + n] *= 0.2
        w[p + n][:, src] = r
    w[p + "b"].zero_()
    w[p + "b"][:, 2], w[p + "b"][:, 1] = -7.0, 5.0
    w[p + "A_log"].fill_(-9.0)
    return cfg, {k: v.to(torch.bfloat16) for k, v in w.items()}


def needle_tokens(n, needle_at, asks, seed=0):
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(2, 40, (n,), generator=g).tolist()
    t[needle_at] = NEEDLE
    for a in asks:
        t[a] = ASK
    return t
