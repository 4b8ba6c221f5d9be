"""Trace replay: given token ids through a model step by step, logits out, nothing sampled.

Steps come as JSON lines on standard input::

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

All entries of a step are one batch of ``generation.ragged.StepEngine`` — portions of prompts beside single
decoded tokens — on the cache that earlier steps left. A request is admitted at its first entry and gives
its pages and row back when a step's ``end`` names it. The logits of the wanted places go to
``<out>/<step>.f32`` (little-endian fp32 [wanted, vocab], in the order of the entries); a line ``done <step>``
on standard output follows every step."""
from __future__ import annotations

import json
import os
import sys

import torch

MAX_LIVE = 4  # requests alive at a time


def replay(model, lines, out_dir: str, max_tokens: int, emit=None, max_live: int = MAX_LIVE) -> int:
    """Run the steps in ``lines``; returns their number."""
    from ..generation.ragged import StepEngine

    emit = emit or (lambda s: print(s, flush=True))
    os.makedirs(out_dir, exist_ok=True)
    eng = StepEngine(model, max_live, max_tokens)
    rows, n = {}, 0
    for line in lines:
        if not line.strip():
            continue
        st = json.loads(line)
        entries = []
        for e in st.get("entries", []):
            if e["id"] not in rows:
                rows[e["id"]] = eng.admit()
            entries.append((rows[e["id"]], e["tokens"], e.get("want", [])))
        logits = eng.step(entries)
        if logits.shape[0]:
            logits.float().cpu().numpy().astype("<f4").tofile(os.path.join(out_dir, f"{st['step']}.f32"))
        for rid in st.get("end", []):
            if rid in rows:
                eng.release(rows.pop(rid))
        emit(f"done {st['step']}")
        n += 1
    return n


def run(args) -> int:
    from .. import ops
    from ..models import build_model

    if not torch.cuda.is_available():
        print("trace: no GPU", file=sys.stderr)
        return 1
    ops.native()  # built on the first call of a fresh checkout
    model = build_model(args.model, device=torch.device("cuda", torch.cuda.current_device()), dtype=getattr(torch, args.dtype)).eval()
    replay(model, sys.stdin, args.out, args.max_tokens)
    return 0
