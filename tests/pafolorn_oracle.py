"""Plain float32 restatement of the Pafolorn decoder for the tests: one function per mechanism, whole
sequences at once, dense score matrices, Python loops over heads and time. It shares no code with the
package (only torch tensor arithmetic) and reads the raw checkpoint tensors by name.

``fault`` (a set of names) plants one mistake in the oracle, so a test can show that its inputs make
that mistake visible."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def silu(x):
    return x * torch.sigmoid(x)


def rotate_half(x, pos, rot, fault=()):
    """x [T, heads, dim]: dimension i of the first ``dims`` turned with dimension i + dims / 2 by
    pos * base^(-2 i / dims)"""
    d, base = rot["dims"], rot["base"]
    f = torch.tensor([base ** (-2.0 * i / d) for i in range(d // 2)], dtype=torch.float64)
    a = pos.double()[:, None] * f[None]
    c, s = a.cos().float()[:, None], a.sin().float()[:, None]
    y = x.clone()
    if "interleaved" in fault:
        u, v = x[..., 0:d:2], x[..., 1:d:2]
        y[..., 0:d:2], y[..., 1:d:2] = u * c - v * s, v * c + u * s
        return y
    u, v = x[..., :d // 2], x[..., d // 2:d]
    y[..., :d // 2], y[..., d // 2:d] = u * c - v * s, v * c + u * s
    return y


def visible(T, mask, fault=()):
    """[T, T] boolean: which keys position i sees"""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    size = mask["size"] + (1 if "window_off_by_one" in fault else 0)
    keep = 0 if "no_kept" in fault else mask["keep_first"] + (1 if "kept_off_by_one" in fault else 0)
    return (j <= i) & ((i - j < size) | (j < keep))


def window_attention(w, p, mx, h, eps, fault=()):
    """heads concatenated, before the output projection"""
    T, H, G, D, V = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    pos = torch.arange(T)
    q, k, v = h @ w[p + "q"].T, h @ w[p + "k"].T, (h @ w[p + "v"].T).view(T, G, V)
    if "head_norm" in fault:
        q = rms(q.view(T, H, D), eps).reshape(T, -1) * w[p + "q.norm"]
        k = rms(k.view(T, G, D), eps).reshape(T, -1) * w[p + "k.norm"]
    elif "no_qk_norm" not in fault:
        q, k = rms(q, eps) * w[p + "q.norm"], rms(k, eps) * w[p + "k.norm"]
    q, k = q.view(T, H, D), k.view(T, G, D)
    if "no_rotation" not in fault:
        q, k = rotate_half(q, pos, mx["rot"], fault), rotate_half(k, pos, mx["rot"], fault)
    see = visible(T, mx["mask"], fault)
    out = []
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * mx["scale"]
        if "no_softcap" not in fault:
            s = mx["softcap"] * torch.tanh(s / mx["softcap"])
        out.append(torch.softmax(s.masked_fill(~see, -math.inf), -1) @ v[:, g])
    return torch.cat(out, -1)


def short_conv(x, taps, fault=()):
    """causal convolution over time per channel, then silu; the last tap meets the current token"""
    T, n = x.shape[0], taps.shape[1]
    if "taps_reversed" in fault:
        taps = taps.flip(1)
    y = torch.zeros_like(x)
    for j in range(n):
        back = n - 1 - j
        if back < T:
            y[back:] += taps[:, j] * x[:T - back]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, decay, fault=()):
    """q, k [T, H, D] (per value head), v [T, H, V], beta [T, H], decay [T, H, D] -> o [T, H, V]"""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1])
    out = []
    for t in range(T):
        if "read_before_write" in fault:
            out.append(torch.einsum("hdv,hd->hv", S * decay[t][..., None], q[t]))
        S = S * decay[t][..., None]
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][..., None] * u[:, None]
        if "read_before_write" not in fault:
            out.append(torch.einsum("hdv,hd->hv", S, q[t]))
        if "state_lost" in fault and t % 64 == 63:
            S = torch.zeros_like(S)
    return torch.stack(out)


def delta_mixer(w, p, mx, h, eps, channel, fault=()):
    """the gated delta rule up to the output projection. ``channel``: a decay per key channel from a low-rank
    projection and a sigmoid gate from another; otherwise a decay per head and a silu gate"""
    T, H, K, D, V = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]

    def conv(name):
        x = h @ w[p + name].T
        return silu(x) if "no_conv" in fault else short_conv(x, w[p + name + ".conv"], fault)
    of = torch.tensor([n % K if "head_modulo" in fault else n // (H // K) for n in range(H)])
    q, k = conv("q").view(T, K, D), conv("k").view(T, K, D)
    if "no_unit" not in fault:
        q, k = unit(q), unit(k)
    q, k = (q * D ** -0.5)[:, of], k[:, of]
    v = conv("v").view(T, H, V)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    A = torch.exp(w[p + "A_log"])
    if channel:
        a = ((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, D)
        decay = torch.exp(-A[:, None] * softplus(a))
        z = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    else:
        a = h @ w[p + "a"].T + w[p + "dt_bias"]
        decay = torch.exp(-A * softplus(a))[..., None].expand(T, H, D)
        z = silu(h @ w[p + "g"].T)
    if "no_decay" in fault:
        decay = torch.ones_like(decay)
    o = delta_rule(q, k, v, beta, decay, fault)
    o = rms(o, eps) * w[p + "norm"]
    return o.reshape(T, -1) * (1.0 if "no_gate" in fault else z)


def mixer(w, p, spec, h, eps, fault=()):
    mx = spec["mixer"]
    if spec["type"] == "channel_delta":
        return delta_mixer(w, p, mx, h, eps, True, fault) @ w[p + "o"].T
    left = window_attention(w, p + "left.", mx["left"], h, eps, fault) @ w[p + "left.o"].T
    right = delta_mixer(w, p + "right.", mx["right"], h, eps, False, fault) @ w[p + "right.o"].T
    if "no_scales" in fault:
        return left + right
    return mx["left_scale"] * left + mx["right_scale"] * right


def dense_ff(w, p, h, fault=()):
    u = (h @ w[p + "up"].T).clamp(min=0)
    return (u if "relu_only" in fault else u * u) @ w[p + "down"].T


def forward(cfg, weights, tokens, fault=(), layers_out=None):
    """logits [T, vocab] of one sequence from position 0"""
    w = {k: v.float() for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    if "no_embed_norm" not in fault:
        x = rms(x, eps) * w["embed.norm"]

    def ls(p, n):
        return 1.0 if "no_layer_scale" in fault else w[p + n]
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms(mixer(w, p + "mix.", spec, x, eps, fault), eps) * w[p + "norm1"] * ls(p, "ls1")
        if spec["mlp"] is not None:
            x = x + rms(dense_ff(w, p + "mlp.", x, fault), eps) * w[p + "norm2"] * ls(p, "ls2")
        if layers_out is not None:
            layers_out.append(x.clone())
    y = (rms(x, eps) * w["final.norm"]) @ w["embed"].T
    return y if "no_logit_scale" in fault else y * cfg["logit_scale"]
