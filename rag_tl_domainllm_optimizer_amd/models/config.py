"""Model configurations and named presets (shapes from SURVEY Appendix E).

The presets reproduce the architectures the reference names or implies — Llama-2-7B (its
``main()`` default, reinforcement_learning_optimization_after_rag.py:469), Mistral-7B / Llama-2-13B
(north-star configs), OPT-125m (CPU plumbing) and the all-MiniLM-L6-v2 / all-mpnet-base-v2
sentence encoders (reference default reward encoder, rl.py:22,54) — with random-init weights,
since no checkpoints can be downloaded. ``"<preset>:random"`` selects a preset by name.
"""
from __future__ import annotations

import dataclasses
import json
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple, Union


# ---- layered decoders: every layer lists its own mixer and feed-forward ----
@dataclass
class YarnSpec:
    factor: float
    original: float
    fast: float
    slow: float


@dataclass
class RotarySpec:
    base: float
    dims: int
    scaling: Optional[YarnSpec] = None


@dataclass
class LatentAttentionSpec:
    """Mixer ``latent_attention``: keys and values of all heads from one cached latent per token."""
    heads: int
    dim: int                            # unrotated query / key width per head
    rot_dim: int                        # rotated query / key width (the key part is shared by the heads)
    vdim: int
    kv_rank: int
    scale: float
    rot: RotarySpec
    kv_from: Optional[int] = None       # read this layer's cache instead of an own one


@dataclass
class WindowAttentionSpec:
    """Grouped-query attention over a sliding window plus the sequence's first tokens: position i sees j <= i
    with i - j < ``window`` (0: no limit) or j < ``keep_first``. Queries and keys are normed over the whole
    projection and rotated in halves; scores pass ``softcap`` * tanh(score / softcap) (0: none)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotarySpec
    window: int = 0
    keep_first: int = 0
    softcap: float = 0.0


@dataclass
class DeltaSpec:
    """Gated delta rule: per head a [dim, vdim] state that decays, loses what it holds at the key and takes the
    new value. ``channel``: one decay per key channel and a sigmoid output gate, both from low-rank
    projections (``a_rank`` / ``g_rank``); otherwise one decay per head and a silu gate."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                           # taps of the short convolutions of q, k and v
    channel: bool = False
    a_rank: int = 0
    g_rank: int = 0


@dataclass
class ParallelSpec:
    """Two mixers side by side on one input: left_scale * left + right_scale * right."""
    left: WindowAttentionSpec
    right: DeltaSpec
    left_scale: float = 1.0
    right_scale: float = 1.0


MixerSpec = Union[LatentAttentionSpec, DeltaSpec, ParallelSpec]


@dataclass
class FeedForwardSpec:
    """``dense``: gated unit clamped at ``limit``; ``relu2``: squared relu, ungated; ``moe``: ``top`` of
    ``experts`` (+ a gated shared expert)."""
    kind: str
    ff: int
    limit: float = 0.0
    experts: int = 0
    top: int = 0
    shared_ff: int = 0


@dataclass
class LayerSpec:
    mixer: MixerSpec
    mlp: Optional[FeedForwardSpec] = None


def _window_spec(m: dict) -> WindowAttentionSpec:
    mask = m.get("mask") or {}
    return WindowAttentionSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]),
                               RotarySpec(float(m["rot"]["base"]), int(m["rot"]["dims"])), int(mask.get("size", 0)),
                               int(mask.get("keep_first", 0)), float(m.get("softcap") or 0.0))


def _delta_spec(m: dict, channel: bool) -> DeltaSpec:
    return DeltaSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], channel)


def layer_spec(d: dict, dense: str = "dense") -> LayerSpec:
    """One entry of a layered config's ``layers`` list; ``dense``: what the design's dense feed-forward is."""
    m = d["mixer"]
    if d["type"] == "latent_attention":
        r = m["rot"]
        sc = r.get("scaling")
        rot = RotarySpec(float(r["base"]), int(r["dims"]),
                         YarnSpec(*(float(sc[k]) for k in ("factor", "original", "fast", "slow"))) if sc else None)
        mixer = LatentAttentionSpec(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], float(m["scale"]), rot,
                                    m.get("kv_from"))
    elif d["type"] == "channel_delta":
        mixer = _delta_spec(m, True)
    elif d["type"] == "parallel":
        mixer = ParallelSpec(_window_spec(m["left"]), _delta_spec(m["right"], False), float(m["left_scale"]),
                             float(m["right_scale"]))
    else:
        raise ValueError(f"unknown mixer {d['type']!r}")
    ml = d.get("mlp")
    if ml is None:
        return LayerSpec(mixer)
    if ml["kind"] == "dense":
        return LayerSpec(mixer, FeedForwardSpec(dense, ml["ff"], limit=float(ml["limit"]) if dense == "dense" else 0.0))
    if ml["kind"] != "moe":
        raise ValueError(f"unknown feed-forward {ml['kind']!r}")
    shared = ml.get("shared")
    return LayerSpec(mixer, FeedForwardSpec("moe", ml["expert"]["ff"], experts=ml["router"]["experts"],
                                            top=ml["router"]["top"], shared_ff=shared["ff"] if shared else 0))


def _mixer_dict(m: MixerSpec) -> Tuple[str, dict]:
    def delta(x):
        return {"heads": x.heads, "kv_heads": x.kv_heads, "dim": x.dim, "vdim": x.vdim, "conv": x.conv}
    if isinstance(m, DeltaSpec):
        return "channel_delta", delta(m)
    if isinstance(m, ParallelSpec):
        a = m.left
        left = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                "softcap": a.softcap, "rot": {"base": a.rot.base, "dims": a.rot.dims},
                "mask": {"size": a.window, "keep_first": a.keep_first}}
        return "parallel", {"left": left, "right": delta(m.right), "left_scale": m.left_scale, "right_scale": m.right_scale}
    rot = {"base": m.rot.base, "dims": m.rot.dims}
    if m.rot.scaling is not None:
        rot["scaling"] = dataclasses.asdict(m.rot.scaling)
    d = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank, "scale": m.scale,
         "rot": rot}
    if m.kv_from is not None:
        d["kv_from"] = m.kv_from
    return "latent_attention", d


def layer_spec_dict(s: LayerSpec) -> dict:
    """Inverse of :func:`layer_spec`."""
    kind, mixer = _mixer_dict(s.mixer)
    ml = None
    if s.mlp is not None and s.mlp.kind == "dense":
        ml = {"kind": "dense", "ff": s.mlp.ff, "limit": s.mlp.limit}
    elif s.mlp is not None and s.mlp.kind == "relu2":
        ml = {"kind": "dense", "ff": s.mlp.ff}
    elif s.mlp is not None:
        ml = {"kind": "moe", "expert": {"ff": s.mlp.ff}, "router": {"experts": s.mlp.experts, "top": s.mlp.top}}
        if s.mlp.shared_ff:
            ml["shared"] = {"ff": s.mlp.shared_ff}
    return {"type": kind, "mixer": mixer, "mlp": ml}


def _mixer_from_fields(m: dict) -> MixerSpec:
    """A mixer spec from its ``dataclasses.asdict`` form."""
    def rot(r):
        return RotarySpec(r["base"], r["dims"], YarnSpec(**r["scaling"]) if r["scaling"] else None)
    if "left" in m:
        return ParallelSpec(WindowAttentionSpec(**{**m["left"], "rot": rot(m["left"]["rot"])}), DeltaSpec(**m["right"]),
                            m["left_scale"], m["right_scale"])
    return DeltaSpec(**m) if "conv" in m else LatentAttentionSpec(**{**m, "rot": rot(m["rot"])})


def with_ranks(cfg: "ModelConfig", shapes: Dict[str, Tuple[int, ...]]) -> "ModelConfig":
    """The low ranks of channel-decay mixers, which only the checkpoint's tensor shapes give."""
    for i, s in enumerate(cfg.layers or ()):
        if isinstance(s.mixer, DeltaSpec) and s.mixer.channel:
            for field_, name in (("a_rank", "a1"), ("g_rank", "g1")):
                shape = shapes.get(f"l{i}.mix.{name}")
                if shape is None:
                    raise KeyError(f"checkpoint tensors do not fit the config: missing l{i}.mix.{name}")
                setattr(s.mixer, field_, int(shape[0]))
    return cfg


def _check_delta(i: int, m: DeltaSpec):
    if min(m.heads, m.kv_heads, m.dim, m.vdim, m.conv) < 1 or m.heads % m.kv_heads:
        raise ValueError(f"layer {i}: delta rule of {m.heads} heads on {m.kv_heads} key heads, {m.dim} x {m.vdim}")


def _check_window(i: int, m: WindowAttentionSpec):
    if min(m.heads, m.kv_heads, m.dim, m.vdim) < 1 or m.heads % m.kv_heads:
        raise ValueError(f"layer {i}: {m.heads} query heads on {m.kv_heads} key heads")
    if m.rot.dims % 2 or m.rot.dims > m.dim:
        raise ValueError(f"layer {i}: rotation of {m.rot.dims} of {m.dim} dimensions")
    if m.window < 0 or m.keep_first < 0 or m.softcap < 0:
        raise ValueError(f"layer {i}: negative window, kept tokens or softcap")


def _check_layers(layers: List[LayerSpec]):
    for i, s in enumerate(layers):
        m = s.mixer
        if isinstance(m, DeltaSpec):
            _check_delta(i, m)
            continue
        if isinstance(m, ParallelSpec):
            _check_window(i, m.left)
            _check_delta(i, m.right)
            continue
        if m.rot_dim % 2 or m.rot.dims % 2 or m.rot.dims > m.rot_dim:
            raise ValueError(f"layer {i}: rotation of {m.rot.dims} of {m.rot_dim} dimensions")
        if m.kv_from is not None:
            src = layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
            if not isinstance(src, LatentAttentionSpec) or src.kv_from is not None or \
                    (src.kv_rank, src.rot_dim, src.rot) != (m.kv_rank, m.rot_dim, m.rot):
                raise ValueError(f"layer {i}: kv_from {m.kv_from} must be an earlier layer with its own latent of "
                                 "equal rank and rotation")
    for i, s in enumerate(layers):
        if s.mlp is not None and s.mlp.kind == "moe" and not 1 <= s.mlp.top <= s.mlp.experts:
            raise ValueError(f"layer {i}: top {s.mlp.top} of {s.mlp.experts} experts")


@dataclass
class ModelConfig:
    arch: str = "llama"                 # llama | mistral | opt | bert | mpnet | vezatar | pafolorn
    vocab_size: int = 32000
    hidden_size: int = 4096
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 32
    head_dim: int = 128
    intermediate_size: int = 11008
    max_position: int = 4096
    norm_eps: float = 1e-5
    rope_theta: float = 10000.0
    sliding_window: int = 0             # 0 = full attention
    hidden_act: str = "silu"
    tie_embeddings: bool = False
    bias: bool = False                  # linear biases (OPT/BERT/MPNet)
    # token ids
    bos_token_id: int = 1
    eos_token_id: int = 2
    pad_token_id: int = 0
    # encoder specifics
    type_vocab_size: int = 0
    relative_buckets: int = 0
    relative_max_distance: int = 128
    position_offset: int = 0            # OPT learned positions start at index 2; MPNet at pad+1
    # misc
    name: str = "custom"
    initializer_range: float = 0.02
    # layered decoders (arch "vezatar", "pafolorn"): one spec per layer; the per-layer sizes above do not apply
    layers: Optional[List[LayerSpec]] = None
    norms: str = "both"                 # a norm before and after every sublayer ("both"), or after it only ("out")
    layer_scale: bool = False           # an element-wise scale on every sublayer's normed output
    embed_norm: bool = False            # a norm on the embedding
    logit_scale: float = 1.0

    @property
    def is_layered(self) -> bool:
        return self.layers is not None

    @property
    def is_decoder(self) -> bool:
        return self.is_layered or self.arch in ("llama", "mistral", "opt")

    @property
    def qkv_dim(self) -> int:
        return (self.num_heads + 2 * self.num_kv_heads) * self.head_dim

    def to_dict(self):
        return dataclasses.asdict(self)

    @classmethod
    def from_dict(cls, d):
        names = {f.name for f in dataclasses.fields(cls)}
        cfg = cls(**{k: v for k, v in d.items() if k in names})
        if cfg.layers is not None and isinstance(cfg.layers[0], dict):
            cfg.layers = [LayerSpec(_mixer_from_fields(x["mixer"]), FeedForwardSpec(**x["mlp"]) if x["mlp"] else None)
                          for x in cfg.layers]
        return cfg

    def num_params(self) -> int:
        H, F, V, L = self.hidden_size, self.intermediate_size, self.vocab_size, self.num_layers
        if self.is_layered:
            per_norms = (2 if self.norms == "both" else 1) + (1 if self.layer_scale else 0)
            n = (1 if self.tie_embeddings else 2) * V * H + H + (H if self.embed_norm else 0)
            for s in self.layers:
                n += per_norms * H + _mixer_params(s.mixer, H)
                f = s.mlp
                if f is None:
                    continue
                n += per_norms * H
                if f.kind == "relu2":
                    n += 2 * H * f.ff
                    continue
                n += 3 * H * f.ff * max(f.experts, 1) + 3 * H * f.shared_ff
                if f.kind == "moe":
                    n += f.experts * (H + 1) + (H if f.shared_ff else 0)
            return n
        attn = H * self.qkv_dim + self.num_heads * self.head_dim * H
        if self.arch in ("llama", "mistral"):
            mlp = 3 * H * F
            per = attn + mlp + 2 * H
            emb = V * H * (1 if self.tie_embeddings else 2)
            return L * per + emb + H
        mlp = 2 * H * F
        return L * (attn + mlp) + V * H


def _mixer_params(m: MixerSpec, H: int) -> int:
    if isinstance(m, ParallelSpec):
        a = m.left
        q, k, v = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
        return (q + k + v) * H + q + k + H * a.heads * a.vdim + _mixer_params(m.right, H)
    if isinstance(m, DeltaSpec):
        c, v = 2 * m.kv_heads * m.dim + m.heads * m.vdim, m.heads * m.vdim
        n = c * (H + m.conv) + m.heads * (H + 1) + m.vdim + H * v  # projections, taps, beta, A_log, norm, output
        if not m.channel:
            return n + m.heads * (H + 1) + v * H
        d = m.heads * m.dim
        return n + m.a_rank * (H + d) + d + m.g_rank * (H + v)
    n = m.heads * ((m.dim + m.rot_dim) * H + (m.dim + m.vdim) * m.kv_rank + 2 * m.vdim * H + 1)
    return n if m.kv_from is not None else n + (m.kv_rank + m.rot_dim) * H + m.kv_rank


def layered_config(arch: str, vocab_size: int, hidden_size: int, layers: List[LayerSpec], norm_eps: float,
                   name: str = "custom", **kw) -> ModelConfig:
    """ModelConfig of a layered decoder. Its files name no special tokens: generation stops at the ids the
    caller gives (the tokenizer's)."""
    _check_layers(layers)
    kw = {"bos_token_id": -1, "eos_token_id": -1, "pad_token_id": 0, **kw}
    m = layers[0].mixer if layers else None
    if isinstance(m, LatentAttentionSpec):
        kw.update(num_heads=m.heads, num_kv_heads=1, head_dim=m.kv_rank + m.rot_dim, rope_theta=m.rot.base)
    elif m is not None:
        m = m.left if isinstance(m, ParallelSpec) else m
        kw.update(num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim)
    return ModelConfig(arch=arch, vocab_size=vocab_size, hidden_size=hidden_size, num_layers=len(layers),
                       intermediate_size=0, max_position=1 << 20, norm_eps=norm_eps, name=name, layers=layers, **kw)


def pafolorn_config(vocab_size: int, hidden_size: int, layers: List[LayerSpec], norm_eps: float, logit_scale: float,
                    name: str = "pafolorn", **kw) -> ModelConfig:
    """Output norms with a layer scale, a normed embedding that is also the (scaled) head."""
    return layered_config("pafolorn", vocab_size, hidden_size, layers, norm_eps, name, norms="out", layer_scale=True,
                          embed_norm=True, tie_embeddings=True, logit_scale=logit_scale, **kw)


def _vezatar_preset(name, vocab, width, n, heads, dim, rot, vdim, rank, ff, moe, shared_ff, factor=4.0):
    """Layers in pairs: own latent + dense feed-forward, shared latent + experts (``moe`` = (experts, top, ff))."""
    layers = []
    for i in range(n):
        r = RotarySpec(10000.0, rot, YarnSpec(factor, 4096.0, 32.0, 1.0))
        m = LatentAttentionSpec(heads, dim, rot, vdim, rank, (dim + rot) ** -0.5, r, i - 1 if i % 2 else None)
        f = FeedForwardSpec("moe", moe[2], experts=moe[0], top=moe[1], shared_ff=shared_ff) if i % 2 and moe else \
            FeedForwardSpec("dense", ff, limit=7.0)
        layers.append(LayerSpec(m, f))
    return layered_config("vezatar", vocab, width, layers, 1e-6, name, bos_token_id=1, eos_token_id=2)


def _pafolorn_preset(name, vocab, width, n, heads, kv, dim, vdim, ff, window, keep, taps, rank):
    """A channel-decay layer without feed-forward, then three parallel layers, again and again."""
    layers = []
    for i in range(n):
        if i % 4 == 0:
            layers.append(LayerSpec(DeltaSpec(heads, heads, dim, vdim, taps, True, rank, rank)))
            continue
        left = WindowAttentionSpec(heads, kv, dim, vdim, dim ** -0.5, RotarySpec(10000.0, dim), window, keep, 50.0)
        layers.append(LayerSpec(ParallelSpec(left, DeltaSpec(heads // 2, heads // 2, dim, vdim, taps), 0.7, 0.7),
                                FeedForwardSpec("relu2", ff)))
    return pafolorn_config(vocab, width, layers, 1e-6, 0.5, name, bos_token_id=1, eos_token_id=2)


PRESETS = {
    "pafolorn-7b": _pafolorn_preset("pafolorn-7b", 32000, 4096, 32, 32, 8, 128, 128, 14336, 4096, 4, 4, 128),
    "pafolorn-2k": _pafolorn_preset("pafolorn-2k", 32000, 2048, 24, 16, 4, 128, 128, 7168, 4096, 4, 4, 128),
    "tiny-pafolorn": _pafolorn_preset("tiny-pafolorn", 512, 128, 4, 4, 2, 32, 32, 256, 48, 3, 4, 16),
    # real models' layer sizes (Mistral-7B's width and head count, and half of both; 64 experts), a comparison
    # decoder of the half width, and a test size
    "vezatar-7b": _vezatar_preset("vezatar-7b", 32000, 4096, 32, 32, 128, 64, 128, 512, 14336, (64, 8, 1408), 2816),
    "vezatar-2k": _vezatar_preset("vezatar-2k", 32000, 2048, 24, 16, 128, 64, 128, 512, 7168, (64, 6, 896), 1792),
    "mistral-2k": ModelConfig(arch="mistral", vocab_size=32000, hidden_size=2048, num_layers=24, num_heads=16,
                              num_kv_heads=4, head_dim=128, intermediate_size=7168, max_position=32768,
                              norm_eps=1e-5, rope_theta=10000.0, sliding_window=4096, name="mistral-2k"),
    "tiny-vezatar": _vezatar_preset("tiny-vezatar", 512, 192, 4, 6, 32, 16, 48, 64, 256, (10, 3, 64), 128),
    "mistral-7b": ModelConfig(arch="mistral", vocab_size=32000, hidden_size=4096, num_layers=32, num_heads=32,
                              num_kv_heads=8, head_dim=128, intermediate_size=14336, max_position=32768,
                              norm_eps=1e-5, rope_theta=10000.0, sliding_window=4096, name="mistral-7b"),
    # OpenChat-3.5 (README.md:25 lists OpenChat): the Mistral-7B architecture with two added
    # chat tokens (vocab 32002), rope theta 1e4, 8k context
    "openchat-3.5": ModelConfig(arch="mistral", vocab_size=32002, hidden_size=4096, num_layers=32, num_heads=32,
                                num_kv_heads=8, head_dim=128, intermediate_size=14336, max_position=8192,
                                norm_eps=1e-5, rope_theta=10000.0, sliding_window=4096, name="openchat-3.5"),
    "llama2-7b": ModelConfig(arch="llama", vocab_size=32000, hidden_size=4096, num_layers=32, num_heads=32,
                             num_kv_heads=32, head_dim=128, intermediate_size=11008, max_position=4096,
                             norm_eps=1e-5, name="llama2-7b"),
    "llama2-13b": ModelConfig(arch="llama", vocab_size=32000, hidden_size=5120, num_layers=40, num_heads=40,
                              num_kv_heads=40, head_dim=128, intermediate_size=13824, max_position=4096,
                              norm_eps=1e-5, name="llama2-13b"),
    "opt-125m": ModelConfig(arch="opt", vocab_size=50272, hidden_size=768, num_layers=12, num_heads=12,
                            num_kv_heads=12, head_dim=64, intermediate_size=3072, max_position=2048,
                            norm_eps=1e-5, hidden_act="relu", tie_embeddings=True, bias=True, bos_token_id=2,
                            eos_token_id=2, pad_token_id=1, position_offset=2, name="opt-125m"),
    "minilm-l6": ModelConfig(arch="bert", vocab_size=30522, hidden_size=384, num_layers=6, num_heads=12,
                             num_kv_heads=12, head_dim=32, intermediate_size=1536, max_position=512,
                             norm_eps=1e-12, hidden_act="gelu", bias=True, type_vocab_size=2, pad_token_id=0,
                             bos_token_id=101, eos_token_id=102, name="all-MiniLM-L6-v2"),
    "mpnet-base": ModelConfig(arch="mpnet", vocab_size=30527, hidden_size=768, num_layers=12, num_heads=12,
                              num_kv_heads=12, head_dim=64, intermediate_size=3072, max_position=514,
                              norm_eps=1e-5, hidden_act="gelu", bias=True, relative_buckets=32,
                              pad_token_id=1, bos_token_id=0, eos_token_id=2, position_offset=2,
                              name="all-mpnet-base-v2"),
    # small shapes for tests and smoke runs (GPU-kernel compatible head dims)
    "tiny-llama": ModelConfig(arch="llama", vocab_size=512, hidden_size=256, num_layers=2, num_heads=4,
                              num_kv_heads=2, head_dim=64, intermediate_size=512, max_position=512,
                              norm_eps=1e-5, name="tiny-llama"),
    "tiny-mistral": ModelConfig(arch="mistral", vocab_size=512, hidden_size=256, num_layers=2, num_heads=4,
                                num_kv_heads=2, head_dim=64, intermediate_size=512, max_position=512,
                                norm_eps=1e-5, sliding_window=64, name="tiny-mistral"),
    "tiny-opt": ModelConfig(arch="opt", vocab_size=512, hidden_size=256, num_layers=2, num_heads=4,
                            num_kv_heads=4, head_dim=64, intermediate_size=512, max_position=512, norm_eps=1e-5,
                            hidden_act="relu", tie_embeddings=True, bias=True, bos_token_id=2, eos_token_id=2,
                            pad_token_id=1, position_offset=2, name="tiny-opt"),
    "tiny-bert": ModelConfig(arch="bert", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                             num_kv_heads=4, head_dim=32, intermediate_size=256, max_position=128, norm_eps=1e-12,
                             hidden_act="gelu", bias=True, type_vocab_size=2, name="tiny-bert"),
    "tiny-mpnet": ModelConfig(arch="mpnet", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                              num_kv_heads=4, head_dim=32, intermediate_size=256, max_position=130,
                              norm_eps=1e-5, hidden_act="gelu", bias=True, relative_buckets=32, pad_token_id=1,
                              bos_token_id=0, eos_token_id=2, position_offset=2, name="tiny-mpnet"),
}

ALIASES = {
    "mistralai/mistral-7b-v0.1": "mistral-7b",
    "mistral": "mistral-7b",
    "openchat/openchat_3.5": "openchat-3.5",
    "openchat": "openchat-3.5",
    "meta-llama/llama-2-7b-hf": "llama2-7b",
    "meta-llama/llama-2-13b-hf": "llama2-13b",
    "facebook/opt-125m": "opt-125m",
    "sentence-transformers/all-minilm-l6-v2": "minilm-l6",
    "all-minilm-l6-v2": "minilm-l6",
    "sentence-transformers/all-mpnet-base-v2": "mpnet-base",
    "all-mpnet-base-v2": "mpnet-base",
}


def resolve_preset(name: str) -> Optional[ModelConfig]:
    """Map ``"mistral-7b:random"``, an HF hub id, or a preset name to a config (or None)."""
    key = name.split(":")[0].strip().lower()
    key = ALIASES.get(key, key)
    cfg = PRESETS.get(key)
    return dataclasses.replace(cfg) if cfg is not None else None


def config_from_hf(d: dict) -> ModelConfig:
    """Build a ModelConfig from a config.json dict: HF model types (llama / mistral / opt / bert / mpnet) or
    a layered architecture (``"architecture"``: ``"Vezatar"`` or ``"Pafolorn"``)."""
    if "architecture" in d:
        arch = d["architecture"]
        if arch not in ("Vezatar", "Pafolorn"):
            raise ValueError(f"unsupported architecture {arch!r}")
        eps, name = float(d["norm"]["eps"]), d.get("_ragtl_preset", arch.lower())
        if arch == "Vezatar":
            return layered_config("vezatar", d["vocab"], d["width"], [layer_spec(x) for x in d["layers"]], eps, name)
        return pafolorn_config(d["vocab"], d["width"], [layer_spec(x, "relu2") for x in d["layers"]], eps,
                               float(d.get("logit_scale", 1.0)), name)
    mt = d.get("model_type", "llama")
    if mt in ("llama", "mistral"):
        H = d["hidden_size"]
        nh = d["num_attention_heads"]
        return ModelConfig(arch=mt, vocab_size=d["vocab_size"], hidden_size=H, num_layers=d["num_hidden_layers"],
                           num_heads=nh, num_kv_heads=d.get("num_key_value_heads", nh),
                           head_dim=d.get("head_dim") or H // nh, intermediate_size=d["intermediate_size"],
                           max_position=d.get("max_position_embeddings", 4096), norm_eps=d.get("rms_norm_eps", 1e-6),
                           rope_theta=d.get("rope_theta", 10000.0), sliding_window=d.get("sliding_window") or 0,
                           tie_embeddings=d.get("tie_word_embeddings", False), bos_token_id=d.get("bos_token_id", 1),
                           eos_token_id=d.get("eos_token_id", 2), pad_token_id=d.get("pad_token_id") or 0,
                           name=d.get("_name_or_path", mt))
    if mt == "opt":
        H = d["hidden_size"]
        nh = d["num_attention_heads"]
        return ModelConfig(arch="opt", vocab_size=d["vocab_size"], hidden_size=H, num_layers=d["num_hidden_layers"],
                           num_heads=nh, num_kv_heads=nh, head_dim=H // nh, intermediate_size=d["ffn_dim"],
                           max_position=d.get("max_position_embeddings", 2048), norm_eps=1e-5,
                           hidden_act=d.get("activation_function", "relu"), tie_embeddings=True, bias=True,
                           bos_token_id=d.get("bos_token_id", 2), eos_token_id=d.get("eos_token_id", 2),
                           pad_token_id=d.get("pad_token_id", 1), position_offset=2, name=d.get("_name_or_path", mt))
    if mt in ("bert", "mpnet"):
        H = d["hidden_size"]
        nh = d["num_attention_heads"]
        return ModelConfig(arch=mt, vocab_size=d["vocab_size"], hidden_size=H, num_layers=d["num_hidden_layers"],
                           num_heads=nh, num_kv_heads=nh, head_dim=H // nh, intermediate_size=d["intermediate_size"],
                           max_position=d.get("max_position_embeddings", 512),
                           norm_eps=d.get("layer_norm_eps", 1e-12), hidden_act=d.get("hidden_act", "gelu"),
                           bias=True, type_vocab_size=d.get("type_vocab_size", 0) if mt == "bert" else 0,
                           relative_buckets=d.get("relative_attention_num_buckets", 32) if mt == "mpnet" else 0,
                           pad_token_id=d.get("pad_token_id", 0), bos_token_id=d.get("bos_token_id", 0),
                           eos_token_id=d.get("eos_token_id", 2), position_offset=2 if mt == "mpnet" else 0,
                           name=d.get("_name_or_path", mt))
    raise ValueError(f"unsupported model_type {mt!r}")


def config_to_hf(cfg: ModelConfig) -> dict:
    """config.json dict of the checkpoints ``save_pretrained`` writes."""
    if cfg.is_layered:
        d = {"architecture": {"vezatar": "Vezatar", "pafolorn": "Pafolorn"}[cfg.arch], "vocab": cfg.vocab_size,
             "width": cfg.hidden_size, "norm": {"eps": cfg.norm_eps}, "layers": [layer_spec_dict(s) for s in cfg.layers]}
        if cfg.arch == "pafolorn":
            d["logit_scale"] = cfg.logit_scale
        return d
    if cfg.arch in ("llama", "mistral"):
        d = {
            "architectures": ["MistralForCausalLM" if cfg.arch == "mistral" else "LlamaForCausalLM"],
            "model_type": cfg.arch, "vocab_size": cfg.vocab_size, "hidden_size": cfg.hidden_size,
            "num_hidden_layers": cfg.num_layers, "num_attention_heads": cfg.num_heads,
            "num_key_value_heads": cfg.num_kv_heads, "head_dim": cfg.head_dim,
            "intermediate_size": cfg.intermediate_size, "max_position_embeddings": cfg.max_position,
            "rms_norm_eps": cfg.norm_eps, "rope_theta": cfg.rope_theta, "hidden_act": "silu",
            "tie_word_embeddings": cfg.tie_embeddings, "bos_token_id": cfg.bos_token_id,
            "eos_token_id": cfg.eos_token_id, "pad_token_id": cfg.pad_token_id, "torch_dtype": "bfloat16",
            "attention_bias": False, "initializer_range": cfg.initializer_range,
        }
        if cfg.arch == "mistral":
            d["sliding_window"] = cfg.sliding_window or None
        return d
    if cfg.arch == "opt":
        return {"architectures": ["OPTForCausalLM"], "model_type": "opt", "vocab_size": cfg.vocab_size,
                "hidden_size": cfg.hidden_size, "num_hidden_layers": cfg.num_layers,
                "num_attention_heads": cfg.num_heads, "ffn_dim": cfg.intermediate_size,
                "max_position_embeddings": cfg.max_position, "activation_function": cfg.hidden_act,
                "do_layer_norm_before": True, "word_embed_proj_dim": cfg.hidden_size,
                "bos_token_id": cfg.bos_token_id, "eos_token_id": cfg.eos_token_id, "pad_token_id": cfg.pad_token_id,
                "enable_bias": True, "layer_norm_elementwise_affine": True, "torch_dtype": "bfloat16",
                "tie_word_embeddings": True}
    if cfg.arch == "bert":
        return {"architectures": ["BertModel"], "model_type": "bert", "vocab_size": cfg.vocab_size,
                "hidden_size": cfg.hidden_size, "num_hidden_layers": cfg.num_layers,
                "num_attention_heads": cfg.num_heads, "intermediate_size": cfg.intermediate_size,
                "max_position_embeddings": cfg.max_position, "hidden_act": cfg.hidden_act,
                "layer_norm_eps": cfg.norm_eps, "type_vocab_size": cfg.type_vocab_size,
                "pad_token_id": cfg.pad_token_id}
    if cfg.arch == "mpnet":
        return {"architectures": ["MPNetModel"], "model_type": "mpnet", "vocab_size": cfg.vocab_size,
                "hidden_size": cfg.hidden_size, "num_hidden_layers": cfg.num_layers,
                "num_attention_heads": cfg.num_heads, "intermediate_size": cfg.intermediate_size,
                "max_position_embeddings": cfg.max_position, "hidden_act": cfg.hidden_act,
                "layer_norm_eps": cfg.norm_eps, "relative_attention_num_buckets": cfg.relative_buckets,
                "pad_token_id": cfg.pad_token_id, "bos_token_id": cfg.bos_token_id,
                "eos_token_id": cfg.eos_token_id}
    raise ValueError(cfg.arch)


def dump(cfg: ModelConfig) -> str:
    return json.dumps(cfg.to_dict(), indent=1)
