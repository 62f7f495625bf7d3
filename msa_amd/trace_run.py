"""Replays a trace of given token ids through a model, step by step, and writes the logits it asks for.

A step is one JSON line on standard input: ``{"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [0]}],
"end": ["b"]}``.  Each entry appends ``tokens`` to a sequence (opening it if the id is new); ``want`` indexes into ``tokens`` and
selects the rows of ``OUT/<step>.f32`` (little-endian fp32, ``[rows, vocab]``); ``end`` closes sequences behind the step.
``done <step>`` on standard output acknowledges it.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, default=0, help="initial cache capacity in tokens (it grows)")
    args = ap.parse_args(argv)

    from . import build
    build.ensure_seq()
    import torch
    from .registry import load_model
    if not torch.cuda.is_available():
        sys.exit("trace_run: no GPU visible; the HIP path has no CPU fallback")
    model = load_model(args.model, getattr(torch, args.dtype), "cuda:0")
    if not hasattr(model, "step"):
        sys.exit(f"trace_run: {type(model).__name__} does not run token traces")
    cache = model.create_cache(capacity=args.max_tokens or 256)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = model.step(cache, [(e["id"], e["tokens"], e.get("want", [])) for e in step["entries"]])
        if logits is not None:
            logits.cpu().numpy().astype("<f4", copy=False).tofile(os.path.join(args.out, f"{step['step']}.f32"))
        else:
            torch.cuda.synchronize()
        for key in step.get("end", []):
            cache.close(key)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
