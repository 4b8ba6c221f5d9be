"""Plain float32 restatement of the Vezatar decoder for the tests: one function per mechanism, whole
sequences at once, dense score matrices, Python loops over heads and experts. It shares no code with
the package (only torch tensor arithmetic) and reads the raw checkpoint tensors by name.

``fault`` (a set of names) plants one mistake in the oracle, so a test can show that its inputs make
that mistake visible."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def yarn_freqs(rot, fault=()):
    """(frequencies [dims/2], multiplier of cos and sin)"""
    d, base = rot["dims"], rot["base"]
    out, mult = [], 1.0
    sc = rot.get("scaling")
    if sc:
        def dim_of(turns):
            return d * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
        lo = max(math.floor(dim_of(sc["fast"])), 0)
        hi = min(math.ceil(dim_of(sc["slow"])), d - 1)
        mult = 1.0 if "no_mscale" in fault else 0.1 * math.log(sc["factor"]) + 1.0
    for i in range(d // 2):
        f = base ** (-2.0 * i / d)
        if sc:
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / sc["factor"] * ramp + f * (1.0 - ramp)
        out.append(f)
    return torch.tensor(out, dtype=torch.float64), mult


def rotate(x, pos, rot, fault=()):
    """x [T, ..., >= dims]: pairs (2i, 2i+1) of the first ``dims`` turned by pos * f_i"""
    f, mult = yarn_freqs(rot, fault)
    ang = pos.double()[:, None] * f[None, :]
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (f.numel(),)
    c, s = (ang.cos() * mult).float().view(shape), (ang.sin() * mult).float().view(shape)
    d = rot["dims"]
    u, v = x[..., 0:d:2], x[..., 1:d:2]
    y = x.clone()
    if "half_layout" in fault:
        u, v = x[..., :d // 2], x[..., d // 2:d]
        y[..., :d // 2], y[..., d // 2:d] = u * c - v * s, v * c + u * s
        return y
    y[..., 0:d:2] = u * c - v * s
    y[..., 1:d:2] = v * c + u * s
    return y


def latent_kv(w, p, mx, h, pos, eps, fault=()):
    """(latent c [T, kv_rank], rotated shared key part [T, rot_dim])"""
    y = h @ w[p + "dkv"].T
    r = mx["kv_rank"]
    c = rms(y[:, :r], eps) * w[p + "dkv.norm"]
    return c, rotate(y[:, r:], pos, mx["rot"], fault)


def latent_attention(w, p, mx, h, pos, c, kr, fault=()):
    """attention of every position over all earlier ones of the same sequence, ungated output gate on"""
    T, H, D, R, V = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D + R)
    qn, qr = q[..., :D], rotate(q[..., D:], pos, mx["rot"], fault)
    outs = []
    causal = torch.ones(T, T, dtype=torch.bool).tril()
    for i in range(H):
        k = c @ w[p + "uk"][i * D:(i + 1) * D].T
        v = c @ w[p + "uv"][i * V:(i + 1) * V].T
        s = (qn[:, i] @ k.T + qr[:, i] @ kr.T) * mx["scale"]
        s = s.masked_fill(~causal, -math.inf)
        sink = w[p + "sink"][i]
        m = torch.maximum(s.max(-1, keepdim=True).values, sink)
        e = torch.exp(s - m)
        den = e.sum(-1, keepdim=True)
        if "no_sink" not in fault:
            den = den + torch.exp(sink - m)
        outs.append((e / den) @ v)
    o = torch.cat(outs, -1)
    if "no_gate" not in fault:
        o = o * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def dense_ff(w, p, ml, h, fault=()):
    g, u = h @ w[p + "gate"].T, h @ w[p + "up"].T
    lim = ml["limit"]
    g = g.clamp(max=lim)
    u = u.clamp(-lim, lim)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def expert_ff(w, p, h):
    g = h @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(w, p, ml, h, fault=()):
    """(chosen experts [T, top], their weights [T, top])"""
    s = torch.softmax(h @ w[p + "router"].T, -1)
    choice = s if "no_correction" in fault else s + w[p + "correction"]
    idx = choice.topk(ml["router"]["top"], -1).indices
    wt = (choice if "weights_corrected" in fault else s).gather(-1, idx)
    if "renormalized" in fault:
        wt = wt / wt.sum(-1, keepdim=True)
    return idx, wt


def moe_ff(w, p, ml, h, fault=()):
    idx, wt = route(w, p, ml, h, fault)
    y = torch.zeros_like(h)
    for e in range(ml["router"]["experts"]):
        hit = idx == e
        rows = hit.any(-1)
        if rows.any():
            y[rows] += (wt * hit).sum(-1, keepdim=True)[rows] * expert_ff(w, f"{p}e{e}.", h[rows])
    if ml.get("shared") and "no_shared" not in fault:
        y = y + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert_ff(w, p + "shared.", h)
    return y


def forward(cfg, weights, tokens, fault=(), layers_out=None):
    """logits [T, vocab] of one sequence from position 0"""
    w = {k: v.float() for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = w["embed"][tokens]
    pos = torch.arange(len(tokens))
    cached = {}
    for i, spec in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", spec["mixer"], spec["mlp"]
        h = rms(x, eps) * w[p + "norm1"]
        if mx.get("kv_from") is None:
            cached[i] = latent_kv(w, p + "mix.", mx, h, pos, eps, fault)
        c, kr = cached[i if mx.get("kv_from") is None else mx["kv_from"]]
        y = latent_attention(w, p + "mix.", mx, h, pos, c, kr, fault)
        x = x + (y if "no_norm1b" in fault else rms(y, eps) * w[p + "norm1b"])
        if ml is not None:
            h = rms(x, eps) * w[p + "norm2"]
            y = (dense_ff if ml["kind"] == "dense" else moe_ff)(w, p + "mlp.", ml, h, fault)
            x = x + rms(y, eps) * w[p + "norm2b"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
