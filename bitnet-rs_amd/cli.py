"""Greedy generation from a shell, token ids in and out:

    bin/generate --model PATH --tokens 1,2,3 --new 16 [--dtype bfloat16|float32] [--max-pos N]

PATH: a folder with config.json + model.safetensors of a registered architecture, or a .gguf file.
"""
from __future__ import annotations

import argparse
import importlib
import os
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def parse(argv) -> argparse.Namespace:
    ap = argparse.ArgumentParser(prog="generate", description="greedy generation, token ids in and out")
    ap.add_argument("--model", required=True, help="folder with config.json + model.safetensors, or a .gguf file")
    ap.add_argument("--tokens", required=True, help="the prompt: token ids, with commas between them")
    ap.add_argument("--new", type=int, default=16, help="tokens to generate")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--max-pos", type=int, default=None, help="positions to reserve (default: what this call needs)")
    a = ap.parse_args(argv)
    try:
        a.tokens = [int(t) for t in a.tokens.split(",")]
    except ValueError:
        ap.error("--tokens: integers with commas between them")
    if a.new < 1:
        ap.error("--new: at least 1")
    if a.max_pos is None:
        a.max_pos = len(a.tokens) + a.new + 2
    return a


def main(argv=None) -> int:
    a = parse(argv)
    if ROOT not in sys.path:
        sys.path.insert(0, ROOT)
    pkg = importlib.import_module("bitnet-rs_amd")
    if not os.path.exists(pkg.LIB_PATH) or not os.path.exists(pkg.HOST_LIB_PATH):
        pkg._load_build_module().build()
    try:
        model = pkg.open_model(a.model, a.dtype, a.max_pos)
        print(",".join(str(t) for t in model.generate(a.tokens, a.new)))
        model.close()
    except pkg.BitNetHipError as e:
        print(f"generate: {e}", file=sys.stderr)
        return 1
    return 0


if __name__ == "__main__":
    sys.exit(main())
