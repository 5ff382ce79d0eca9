"""Trace replay: given token ids through a served model, step by step, logits out.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Reads one JSON object a line from standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Every step is one batch of the engine's own prefill or decode step over its caches (LLMEngine.feed); nothing
is sampled. A step in which something is wanted writes OUT/<step>.f32: the logits at the wanted places, in
the order of the entries and of "want", little-endian fp32 [wanted, vocab]. After every step a line
"done <step>" is printed. "end" lists requests whose cache blocks and state slot are given back.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

EXIT_DTYPE = 3  # the model does not run in the asked number format


def parse(argv):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=8192, help="most tokens that live requests hold at any time")
    ap.add_argument("--max-batch", type=int, default=256, help="most live requests")
    ap.add_argument("--device", default="cuda", help="cuda (default), or cpu for the plain CPU backend")
    return ap.parse_args(argv)


def make_engine(a, raw, family):
    from .engine.llm_engine import LLMEngine
    from .models.registry import build_model

    if a.device != "cpu":
        import torch

        from .ops import _lib

        if not torch.cuda.is_available():
            raise RuntimeError("no GPU visible (--device cpu runs the CPU backend)")
        _lib.ensure_kernels(family)
    model = build_model(a.model, a.device, a.dtype, raw)
    live = max(1, min(a.max_batch, a.max_tokens))
    blocks = -(-a.max_tokens // 64) + live + 2  # every live request may hold one partly filled block
    return LLMEngine(model, num_blocks=blocks, max_batch=live, max_model_len=max(64, a.max_tokens))


def main(argv=None):
    a = parse(argv)
    from .models.registry import family_of, norm_dtype, read_config

    raw = read_config(a.model)
    family = family_of(raw)
    if norm_dtype(a.dtype) not in family.dtypes:
        print("trace_run: %s has no %s path" % (family.name, a.dtype), file=sys.stderr)
        return EXIT_DTYPE
    engine = make_engine(a, raw, family)
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = engine.open_sequence()
            entries.append((live[e["id"]], e["tokens"], e.get("want") or []))
        logits = engine.feed(entries)
        if logits.shape[0]:
            path = os.path.join(a.out, "%d.f32" % step["step"])
            with open(path + ".part", "wb") as f:
                f.write(logits.numpy().astype("<f4").tobytes())
            os.replace(path + ".part", path)
        for i in step.get("end") or []:
            engine.close_sequence(live.pop(i))
        print("done %d" % step["step"], flush=True)
    return 0
