"""Command line of the token loop.

    python -m air_hip.generate --model DIR --prompt 12,7,99 -n 32 [--dtype bfloat16|float32] [--eos 2] [--stream]

Prompt and output are token ids (there is no tokenizer here); the model class is chosen by DIR/config.json.
"""

import argparse


def main(argv=None):
    ap = argparse.ArgumentParser(prog="air_hip.generate", description="Greedy generation from token ids.")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, *.safetensors)")
    ap.add_argument("--prompt", required=True, help="comma-separated token ids")
    ap.add_argument("-n", "--n-tokens", type=int, default=10, help="tokens decoded after the first")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--eos", default="", help="comma-separated end-of-sequence ids")
    ap.add_argument("--stream", action="store_true", help="print every token as it is produced")
    a = ap.parse_args(argv)

    import torch

    from . import generation, models

    ids = lambda text: [int(t) for t in text.split(",") if t.strip()]
    model = models.load_model(a.model, dtype=getattr(torch, a.dtype))
    on_token = (lambda t: print(t, flush=True)) if a.stream else None
    out = generation.generate(model, ids(a.prompt), a.n_tokens, ids(a.eos), on_token)
    if not a.stream:
        print(",".join(str(t) for t in out))
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
