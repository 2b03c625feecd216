"""Command line.

    python -m clusterfusionplus_amd generate --model DIR --tokens 5,17,3 [--tokens 9,4] --max-new 32
    python -m clusterfusionplus_amd models

Prompts and results are token ids: tokenisation stays with the caller."""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="clusterfusionplus_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="greedy continuation of token-id prompts")
    g.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    g.add_argument("--tokens", action="append", required=True, metavar="ID,ID,...", help="a prompt; may be given several times")
    g.add_argument("--max-new", type=int, default=32)
    g.add_argument("--stop", type=int, action="append", default=[], help="a token id that ends a sequence")
    g.add_argument("--dtype", default="", choices=["", "bfloat16", "float32", "float16"], help="element type (default: the model's own)")
    g.add_argument("--portion", type=int, default=2048, help="prompt tokens per turn")
    g.add_argument("--slots", type=int, default=1, help="sequences that are live at a time")
    sub.add_parser("models", help="the architectures that can be loaded")
    a = ap.parse_args(argv)
    from .registry import architectures, load_model
    if a.command == "models":
        print("\n".join(architectures()))
        return 0
    from .engine import Engine
    prompts = [[int(t) for t in p.split(",")] for p in a.tokens]
    model = load_model(a.model, a.dtype, capacity=max(len(p) for p in prompts) + a.max_new, slots=a.slots, max_portion=a.portion)
    for tokens in Engine(model, portion=a.portion).generate(prompts, a.max_new, a.stop):
        print(json.dumps(tokens))
    return 0


if __name__ == "__main__":
    sys.exit(main())
