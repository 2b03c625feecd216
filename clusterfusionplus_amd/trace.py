"""Trace replay: given token ids through a model, step by step, logits to files (bin/trace_run).

    python -m clusterfusionplus_amd.trace --model DIR --dtype bfloat16 --out DIR --max-tokens N

Standard input: one JSON object a line, {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [0, 1]}], "end": []}.
For a step in which something is wanted DIR/<step>.f32 receives the logits (little-endian 32-bit floats, [wanted, vocab]);
after every step `done <step>` is printed.  `end` lists the sequences that are over after the step.  The tokens go through
the engine's own state manager and the model's own step function; nothing is sampled."""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    ap.add_argument("--dtype", default="", choices=["", "bfloat16", "float32", "float16"], help="element type (default: the model's own)")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens that live sequences hold at any time")
    ap.add_argument("--slots", type=int, default=1, help="sequences that may be live at a time")
    a = ap.parse_args(argv)

    from .registry import dtypes_of, load_model
    from .weights import read_config
    types = dtypes_of(read_config(a.model))
    if a.dtype and a.dtype not in types:
        print(f"trace_run: this model does not run in {a.dtype}; it runs in {', '.join(types)}", file=sys.stderr)
        return 3

    from .engine import Engine
    model = load_model(a.model, a.dtype, capacity=a.max_tokens, slots=a.slots)
    engine = Engine(model)
    os.makedirs(a.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for e in step["entries"]:
            logits = engine.feed(e["id"], e["tokens"], e.get("want", []))
            if logits.shape[0]:
                rows.append(logits.cpu())
        if rows:
            with open(os.path.join(a.out, f"{step['step']}.f32"), "wb") as f:
                for r in rows:
                    f.write(r.numpy().astype("<f4").tobytes())
        for key in step.get("end", []):
            if key in engine.states:
                engine.finish(key)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
