"""Replay of a trace: given tokens through a model step by step, logits to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Reads one JSON object a line from standard input:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
and drives the engine: each entry's tokens continue the sequence of its id, "want" names places among
them.  For a step in which something is wanted DIR/<step>.f32 receives the logits, little-endian 32-bit
floats, in the order of the entries and of "want"; then "done <step>" is printed.  The sequences in
"end" are given back afterwards.  Nothing is sampled.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from pathlib import Path

import numpy as np


def parse(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="feed token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live sequences hold at any time")
    ap.add_argument("--slots", type=int, default=8, help="most sequences that live at any time")
    return ap.parse_args(argv)


def replay(engine, lines, out: Path, report=print):
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        number = int(step["step"])
        entries = [(e["id"], [int(t) for t in e["tokens"]], [int(k) for k in e["want"]]) for e in step["entries"]]
        got = engine.feed(entries)
        rows = [row for rows in got for row in rows]
        if rows:
            part = out / f".{number}.f32.part"
            np.stack(rows).astype("<f4", copy=False).tofile(part)
            os.replace(part, out / f"{number}.f32")
        for name in step.get("end", []):
            if name in engine.sequences:
                engine.release(name)
        report(f"done {number}")


def main(argv=None) -> int:
    args = parse(argv)
    from . import build, models
    from .engine import Engine

    if models.needs_sequence_library(models.read_config(args.model)):
        build.build_seq(force=False, verbose=False)
    out = Path(args.out)
    out.mkdir(parents=True, exist_ok=True)
    cap = max(1, args.max_tokens)
    runner = models.load_model(args.model, slots=args.slots, cap=cap, max_rows=min(2048, cap), dtype=args.dtype)
    try:
        replay(Engine(runner), iter(sys.stdin.readline, ""), out, lambda text: print(text, flush=True))
    finally:
        runner.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
