"""Trace replay: given token ids go through a model step by step and the logits asked for are written to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps

A step is one JSON line {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}: each entry brings a request's
next tokens, `want` the places among them whose logits are written to OUT/<n>.f32 (little-endian float32, in the order of
the entries and of `want`); the requests in `end` give their caches back.  'done <n>' is printed after each step.
"""

import argparse
import json
import os
import sys

EXIT_DTYPE = 3


def replay(model, lines, out_dir, max_tokens, emit):
    """Run the steps in `lines`; emit(text) after each."""
    import numpy as np

    from . import generation

    pool = generation.CachePool(model, max_tokens)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for e in step.get("entries", []):
            want = [int(w) for w in e.get("want", [])]
            logits = model.step(pool.get(e["id"]), e["tokens"], want)
            if want:
                rows.append(logits.float().cpu().numpy())
        model.check_health()
        for request in step.get("end", []):
            pool.end(request)
        if rows:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(np.ascontiguousarray(np.concatenate(rows), dtype="<f4").tobytes())
        emit(f"done {step['step']}")


def main(argv=None, ensure=None):
    """`ensure(library)` makes sure that a shared library is built (bin/trace_run passes the builder)."""
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids through a model.")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, *.safetensors)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="directory for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens that the live requests hold at any time")
    a = ap.parse_args(argv)

    import torch

    from . import generation, models

    if ensure is not None:
        ensure(models.entry_for(models.read_config(a.model)).library)
    try:
        model = models.load_model(a.model, dtype=getattr(torch, a.dtype))
    except generation.UnsupportedDtype as e:
        print(f"trace_run: {e}", file=sys.stderr)
        return EXIT_DTYPE
    os.makedirs(a.out, exist_ok=True)
    replay(model, sys.stdin, a.out, a.max_tokens, lambda text: print(text, flush=True))
    return 0
