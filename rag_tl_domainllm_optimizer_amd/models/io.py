"""HF-layout checkpoint IO (safetensors) for the native fused-parameter models.

``save_pretrained`` writes config.json + generation_config.json + model.safetensors (sharded with
model.safetensors.index.json above ``max_shard_bytes``) using HF tensor names, so the output loads
with ``transformers.AutoModelForCausalLM.from_pretrained`` and vice versa — the ``{tag}_policy/``
artifact of the reference's save_checkpoint (reinforcement_learning_optimization_after_rag.py:365-370).
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict, List, Tuple

import torch

from .config import (LatentAttentionSpec, ModelConfig, ParallelSpec, WindowAttentionSpec, config_from_hf, config_to_hf,
                     with_ranks)

# (hf_name, native_param_name, row_start, row_count) ; row_count None = whole tensor
Mapping = List[Tuple[str, str, int, int]]


def decoder_mapping(cfg: ModelConfig) -> Mapping:
    m: Mapping = []
    Hq, Hkv, D, F = cfg.num_heads, cfg.num_kv_heads, cfg.head_dim, cfg.intermediate_size
    if cfg.arch == "opt":
        p = "model.decoder"
        m += [(f"{p}.embed_tokens.weight", "embed", 0, None), (f"{p}.embed_positions.weight", "pos_embed", 0, None),
              (f"{p}.final_layer_norm.weight", "norm_w", 0, None), (f"{p}.final_layer_norm.bias", "norm_b", 0, None)]
        for i in range(cfg.num_layers):
            L, n = f"{p}.layers.{i}", f"layers.{i}"
            m += [(f"{L}.self_attn_layer_norm.weight", f"{n}.ln1_w", 0, None),
                  (f"{L}.self_attn_layer_norm.bias", f"{n}.ln1_b", 0, None),
                  (f"{L}.final_layer_norm.weight", f"{n}.ln2_w", 0, None),
                  (f"{L}.final_layer_norm.bias", f"{n}.ln2_b", 0, None),
                  (f"{L}.self_attn.out_proj.weight", f"{n}.o_w", 0, None),
                  (f"{L}.self_attn.out_proj.bias", f"{n}.o_b", 0, None),
                  (f"{L}.fc1.weight", f"{n}.fc1_w", 0, None), (f"{L}.fc1.bias", f"{n}.fc1_b", 0, None),
                  (f"{L}.fc2.weight", f"{n}.fc2_w", 0, None), (f"{L}.fc2.bias", f"{n}.fc2_b", 0, None)]
            for proj, r0, rn in (("q_proj", 0, Hq * D), ("k_proj", Hq * D, Hkv * D), ("v_proj", (Hq + Hkv) * D, Hkv * D)):
                m += [(f"{L}.self_attn.{proj}.weight", f"{n}.qkv_w", r0, rn),
                      (f"{L}.self_attn.{proj}.bias", f"{n}.qkv_b", r0, rn)]
        return m
    m += [("model.embed_tokens.weight", "embed", 0, None), ("model.norm.weight", "norm_w", 0, None)]
    if not cfg.tie_embeddings:
        m.append(("lm_head.weight", "lm_head", 0, None))
    for i in range(cfg.num_layers):
        L, n = f"model.layers.{i}", f"layers.{i}"
        m += [(f"{L}.input_layernorm.weight", f"{n}.ln1_w", 0, None),
              (f"{L}.post_attention_layernorm.weight", f"{n}.ln2_w", 0, None),
              (f"{L}.self_attn.q_proj.weight", f"{n}.qkv_w", 0, Hq * D),
              (f"{L}.self_attn.k_proj.weight", f"{n}.qkv_w", Hq * D, Hkv * D),
              (f"{L}.self_attn.v_proj.weight", f"{n}.qkv_w", (Hq + Hkv) * D, Hkv * D),
              (f"{L}.self_attn.o_proj.weight", f"{n}.o_w", 0, None),
              (f"{L}.mlp.gate_proj.weight", f"{n}.gate_up_w", 0, F),
              (f"{L}.mlp.up_proj.weight", f"{n}.gate_up_w", F, F),
              (f"{L}.mlp.down_proj.weight", f"{n}.down_w", 0, None)]
    return m


def encoder_mapping(cfg: ModelConfig) -> Mapping:
    H = cfg.hidden_size
    m: Mapping = [("embeddings.word_embeddings.weight", "word_embed", 0, None),
                  ("embeddings.position_embeddings.weight", "pos_embed", 0, None),
                  ("embeddings.LayerNorm.weight", "emb_ln_w", 0, None),
                  ("embeddings.LayerNorm.bias", "emb_ln_b", 0, None)]
    if cfg.type_vocab_size:
        m.append(("embeddings.token_type_embeddings.weight", "type_embed", 0, None))
    if cfg.arch == "mpnet":
        m.append(("encoder.relative_attention_bias.weight", "rel_bias", 0, None))
    for i in range(cfg.num_layers):
        L, n = f"encoder.layer.{i}", f"layers.{i}"
        if cfg.arch == "bert":
            qkv = [(f"{L}.attention.self.query", 0), (f"{L}.attention.self.key", H), (f"{L}.attention.self.value", 2 * H)]
            o, ln1 = f"{L}.attention.output.dense", f"{L}.attention.output.LayerNorm"
        else:
            qkv = [(f"{L}.attention.attn.q", 0), (f"{L}.attention.attn.k", H), (f"{L}.attention.attn.v", 2 * H)]
            o, ln1 = f"{L}.attention.attn.o", f"{L}.attention.LayerNorm"
        for base, r0 in qkv:
            m += [(f"{base}.weight", f"{n}.qkv_w", r0, H), (f"{base}.bias", f"{n}.qkv_b", r0, H)]
        m += [(f"{o}.weight", f"{n}.o_w", 0, None), (f"{o}.bias", f"{n}.o_b", 0, None),
              (f"{ln1}.weight", f"{n}.ln1_w", 0, None), (f"{ln1}.bias", f"{n}.ln1_b", 0, None),
              (f"{L}.intermediate.dense.weight", f"{n}.fc1_w", 0, None),
              (f"{L}.intermediate.dense.bias", f"{n}.fc1_b", 0, None),
              (f"{L}.output.dense.weight", f"{n}.fc2_w", 0, None), (f"{L}.output.dense.bias", f"{n}.fc2_b", 0, None),
              (f"{L}.output.LayerNorm.weight", f"{n}.ln2_w", 0, None),
              (f"{L}.output.LayerNorm.bias", f"{n}.ln2_b", 0, None)]
    return m


class Part:
    """A piece of a checkpoint tensor that a native parameter holds: rows [row0, row0 + rows) and columns
    [col0, col0 + cols) of the (2-D or 1-D) parameter; ``dim`` / ``start`` / ``size`` select the tensor's
    slice."""

    __slots__ = ("name", "param", "row0", "rows", "dim", "start", "size", "col0", "cols")

    def __init__(self, name, param, row0=0, rows=None, dim=None, start=0, size=None, col0=0, cols=None):
        self.name, self.param, self.row0, self.rows = name, param, row0, rows
        self.dim, self.start, self.size = dim, start, size
        self.col0, self.cols = col0, size if dim == 1 and cols is None else cols

    def of(self, t: torch.Tensor) -> torch.Tensor:
        """The part's place in the native parameter ``t``."""
        if self.rows is not None:
            t = t[self.row0:self.row0 + self.rows]
        return t if self.cols is None else t[:, self.col0:self.col0 + self.cols]


def _latent_parts(L: str, n: str, x: LatentAttentionSpec) -> List[Part]:
    nq, nk, ng = x.heads * (x.dim + x.rot_dim), x.kv_rank + x.rot_dim, x.heads * x.vdim
    own = x.kv_from is None
    m = [Part(f"{L}.q", f"{n}.in_w", 0, nq), Part(f"{L}.g", f"{n}.in_w", nq + (nk if own else 0), ng),
         Part(f"{L}.uk", f"{n}.kv_up_w", 0, x.heads * x.dim), Part(f"{L}.uv", f"{n}.kv_up_w", x.heads * x.dim, ng),
         Part(f"{L}.sink", f"{n}.sink"), Part(f"{L}.o", f"{n}.o_w")]
    if own:
        m += [Part(f"{L}.dkv", f"{n}.in_w", nq, nk), Part(f"{L}.dkv.norm", f"{n}.latent_norm_w")]
    return m


def _branch_parts(L: str, n: str, spec) -> List[Part]:
    """One mixer, or two side by side: input projections stacked, output projections side by side."""
    from .layered import in_layout, out_layout

    m = []
    pair = isinstance(spec, ParallelSpec)
    rows, _ = in_layout(spec)
    cols, _ = out_layout(spec)
    for side, x in ((("left", spec.left), ("right", spec.right)) if pair else (("mix", spec),)):
        t = f"{L}.{side}" if pair else L
        m += [Part(f"{t}.{k}", f"{n}.in_w", r0, rn) for k, (r0, rn) in rows[side].items()]
        m.append(Part(f"{t}.o", f"{n}.o_w", col0=cols[side][0], cols=cols[side][1]))
        q = f"{n}.{side}"
        if isinstance(x, WindowAttentionSpec):
            m += [Part(f"{t}.q.norm", f"{q}.q_norm_w"), Part(f"{t}.k.norm", f"{q}.k_norm_w")]
            continue
        c0 = 0
        for k, c in (("q", x.kv_heads * x.dim), ("k", x.kv_heads * x.dim), ("v", x.heads * x.vdim)):
            m.append(Part(f"{t}.{k}.conv", f"{q}.conv_w", c0, c))
            c0 += c
        m += [Part(f"{t}.A_log", f"{q}.A_log"), Part(f"{t}.dt_bias", f"{q}.dt_bias"), Part(f"{t}.norm", f"{q}.out_norm_w")]
        if x.channel:
            m += [Part(f"{t}.a2", f"{q}.a2_w", cols=x.a_rank), Part(f"{t}.g2", f"{q}.g2_w", cols=x.g_rank)]
    return m


def layered_mapping(cfg: ModelConfig) -> List[Part]:
    """Tensor names of a layered decoder -> its fused parameters: the projections of a mixer's input as one
    matrix, [uk; uv] and the taps of q, k and v as one each, experts stacked, the shared expert cut into
    parts of an expert's width behind them."""
    m = [Part("embed", "embed"), Part("final.norm", "norm_w")]
    if not cfg.tie_embeddings:
        m.append(Part("head", "lm_head"))
    if cfg.embed_norm:
        m.append(Part("embed.norm", "embed_norm_w"))
    for i, s in enumerate(cfg.layers):
        L, n = f"l{i}", f"layers.{i}"
        latent = isinstance(s.mixer, LatentAttentionSpec)
        m += (_latent_parts if latent else _branch_parts)(f"{L}.mix", f"{n}.mix", s.mixer)
        f = s.mlp
        for j in "12" if f is not None else "1":
            m.append(Part(f"{L}.norm{j}", f"{n}.norm{j}_w"))
            if cfg.norms == "both":
                m.append(Part(f"{L}.norm{j}b", f"{n}.norm{j}b_w"))
            if cfg.layer_scale:
                m.append(Part(f"{L}.ls{j}", f"{n}.ls{j}"))
        if f is None:
            continue
        p = f"{L}.mlp"
        W = cfg.hidden_size
        if f.kind == "relu2":
            m += [Part(f"{p}.up", f"{n}.mlp.up_w"), Part(f"{p}.down", f"{n}.mlp.down_w")]
            continue
        if f.kind == "dense":
            m += [Part(f"{p}.gate", f"{n}.mlp.gate_up_w", 0, f.ff), Part(f"{p}.up", f"{n}.mlp.gate_up_w", f.ff, f.ff),
                  Part(f"{p}.down", f"{n}.mlp.down_w")]
            continue
        m += [Part(f"{p}.router", f"{n}.mlp.router_w", 0, f.experts), Part(f"{p}.correction", f"{n}.mlp.correction")]
        for e in range(f.experts):
            m += [Part(f"{p}.e{e}.gate", f"{n}.mlp.gate_up_w", 2 * e * f.ff, f.ff),
                  Part(f"{p}.e{e}.up", f"{n}.mlp.gate_up_w", (2 * e + 1) * f.ff, f.ff),
                  Part(f"{p}.e{e}.down", f"{n}.mlp.down_w", e * W, W)]
        if f.shared_ff:
            m.append(Part(f"{p}.shared.sg", f"{n}.mlp.router_w", f.experts, 1))
            for j, c0 in enumerate(range(0, f.shared_ff, f.ff)):
                e, c = f.experts + j, min(f.ff, f.shared_ff - c0)
                m += [Part(f"{p}.shared.gate", f"{n}.mlp.gate_up_w", 2 * e * f.ff, c, 0, c0, c),
                      Part(f"{p}.shared.up", f"{n}.mlp.gate_up_w", (2 * e + 1) * f.ff, c, 0, c0, c),
                      Part(f"{p}.shared.down", f"{n}.mlp.down_w", e * W, W, 1, c0, c)]
    return m


@torch.no_grad()
def load_layered_state_dict(model, sd: Dict[str, torch.Tensor]):
    """Strict load: every expected tensor present with the shape the config gives, and no other."""
    params = dict(model.named_parameters())
    parts = layered_mapping(model.cfg)
    missing = sorted({p.name for p in parts} - set(sd))
    extra = sorted(set(sd) - {p.name for p in parts})
    if missing or extra:
        raise KeyError(f"checkpoint tensors do not fit the config: missing {missing[:6]}, unexpected {extra[:6]}")
    left = {}
    for p in parts:
        src, dst = sd[p.name], p.of(params[p.param])
        left[p.name] = left.get(p.name, src.numel())
        if p.dim is not None:
            src = src.narrow(p.dim, p.start, p.size)
        if tuple(src.shape) != tuple(dst.shape):
            raise ValueError(f"{p.name}: shape {tuple(sd[p.name].shape)} does not fit the config")
        left[p.name] -= src.numel()
        dst.copy_(src.to(dst.device, dst.dtype))
    if any(left.values()):
        raise ValueError(f"checkpoint tensors larger than the config: {[k for k, v in left.items() if v][:6]}")


def layered_state_dict(model, dtype=None) -> Dict[str, torch.Tensor]:
    params = dict(model.named_parameters())
    pieces: Dict[str, list] = {}
    for p in layered_mapping(model.cfg):
        t = p.of(params[p.param].detach())
        pieces.setdefault(p.name, []).append((p.dim or 0, t.to("cpu")))
    out = {k: (torch.cat([t for _, t in v], v[0][0]) if len(v) > 1 else v[0][1]) for k, v in pieces.items()}
    return {k: (t.to(dtype) if dtype is not None else t).contiguous() for k, t in out.items()}


def mapping_for(model) -> Mapping:
    return decoder_mapping(model.cfg) if model.cfg.is_decoder else encoder_mapping(model.cfg)


def to_hf_state_dict(model, dtype=None) -> Dict[str, torch.Tensor]:
    if model.cfg.is_layered:
        return layered_state_dict(model, dtype)
    params = dict(model.named_parameters())
    out = {}
    for hf, nat, r0, rn in mapping_for(model):
        t = params[nat].detach()
        if rn is not None:
            t = t[r0:r0 + rn]
        t = t.to("cpu")
        out[hf] = (t.to(dtype) if dtype is not None else t).contiguous()
    return out


@torch.no_grad()
def load_hf_state_dict(model, sd: Dict[str, torch.Tensor], strict: bool = True, prefix_strip: str = ""):
    if model.cfg.is_layered:
        load_layered_state_dict(model, sd)
        return []
    params = dict(model.named_parameters())
    missing = []
    for hf, nat, r0, rn in mapping_for(model):
        key = hf
        if key not in sd:
            alt = [k for k in sd if k.endswith(hf)]
            key = alt[0] if alt else None
        if key is None:
            missing.append(hf)
            continue
        src = sd[key]
        dst = params[nat]
        if rn is not None:
            dst = dst[r0:r0 + rn]
        dst.copy_(src.to(dst.device, dst.dtype).view_as(dst))
    if strict and missing:
        raise KeyError(f"missing tensors in checkpoint: {missing[:8]}{'...' if len(missing) > 8 else ''}")
    return missing


def save_pretrained(model, path: str, max_shard_bytes: int = 5 * 1024 ** 3, dtype=torch.bfloat16,
                    generation_config: dict = None, write_weights: bool = True):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        d = config_to_hf(model.cfg)
        d["_ragtl_preset"] = model.cfg.name
        json.dump(d, f, indent=2)
    if model.cfg.is_decoder:
        gc = {"bos_token_id": model.cfg.bos_token_id, "eos_token_id": model.cfg.eos_token_id,
              "pad_token_id": model.cfg.pad_token_id, "do_sample": True, "temperature": 0.7, "max_length": 512}
        gc.update(generation_config or {})
        with open(os.path.join(path, "generation_config.json"), "w") as f:
            json.dump(gc, f, indent=2)
    if not write_weights:
        return
    sd = to_hf_state_dict(model, dtype)
    total = sum(t.numel() * t.element_size() for t in sd.values())
    if total <= max_shard_bytes:
        save_file(sd, os.path.join(path, "model.safetensors"), metadata={"format": "pt"})
        return
    shards, cur, cur_b = [], {}, 0
    for k, t in sd.items():
        b = t.numel() * t.element_size()
        if cur and cur_b + b > max_shard_bytes:
            shards.append(cur)
            cur, cur_b = {}, 0
        cur[k] = t
        cur_b += b
    if cur:
        shards.append(cur)
    wm = {}
    for i, sh in enumerate(shards):
        name = f"model-{i + 1:05d}-of-{len(shards):05d}.safetensors"
        save_file(sh, os.path.join(path, name), metadata={"format": "pt"})
        for k in sh:
            wm[k] = name
    with open(os.path.join(path, "model.safetensors.index.json"), "w") as f:
        json.dump({"metadata": {"total_size": total}, "weight_map": wm}, f, indent=2)


def read_state_dict(path: str) -> Dict[str, torch.Tensor]:
    from safetensors.torch import load_file

    idx = os.path.join(path, "model.safetensors.index.json")
    if os.path.exists(idx):
        with open(idx) as f:
            wm = json.load(f)["weight_map"]
        sd = {}
        for name in sorted(set(wm.values())):
            sd.update(load_file(os.path.join(path, name)))
        return sd
    st = os.path.join(path, "model.safetensors")
    if os.path.exists(st):
        return load_file(st)
    pt = os.path.join(path, "pytorch_model.bin")
    if os.path.exists(pt):
        return torch.load(pt, map_location="cpu", weights_only=True)
    raise FileNotFoundError(f"no weights found in {path}")


def load_config(path: str) -> ModelConfig:
    with open(os.path.join(path, "config.json")) as f:
        return config_from_hf(json.load(f))


def from_pretrained(path: str, device="cpu", dtype=torch.bfloat16):
    from . import model_class

    cfg = load_config(path)
    sd = read_state_dict(path)
    if cfg.is_layered:
        with_ranks(cfg, {k: tuple(t.shape) for k, t in sd.items()})
    model = model_class(cfg)(cfg, device=device, dtype=dtype, init=False)
    load_hf_state_dict(model, sd)
    return model
