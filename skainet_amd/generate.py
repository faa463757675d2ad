"""Greedy generation from the command line, for every registered architecture:

    python -m skainet_amd.generate --model PATH --prompt 17,4,99 --tokens 32

Token ids in, token ids out (the library has no tokenizer).
"""
from __future__ import annotations

import argparse
import sys

from . import models, runtime


def main(argv=None):
    ap = argparse.ArgumentParser(prog="python -m skainet_amd.generate", description="greedy generation, token ids in and out")
    ap.add_argument("--model", required=True, help="a .gguf file, or a folder with config.json and model.safetensors")
    ap.add_argument("--prompt", required=True, help="token ids with commas between them")
    ap.add_argument("--tokens", type=int, default=32, help="tokens to generate")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16", help="compute path of models that have the choice")
    a = ap.parse_args(argv)
    prompt = [int(t) for t in a.prompt.split(",") if t.strip()]
    if not prompt or a.tokens < 1:
        ap.error("the prompt and the number of tokens must not be empty")
    with runtime.Context(0) as ctx:
        model = models.load_model(ctx, a.model, dtype=a.dtype, max_tokens=len(prompt) + a.tokens)
        print(",".join(str(t) for t in model.generate(prompt, a.tokens)))
        model.free()
    return 0


if __name__ == "__main__":
    sys.exit(main())
