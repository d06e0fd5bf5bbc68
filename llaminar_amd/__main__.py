"""Command line: python -m llaminar_amd generate|trace|models ...

  generate --model DIR --prompt 5,17,3 [--prompt ...] --max-new N   greedy continuations, one line per prompt
  trace    --model DIR --dtype ... --out DIR --max-tokens N          replay of a trace (llaminar_amd.trace)
  models                                                             the registered architectures
"""
from __future__ import annotations

import argparse
import sys


def _ids(text: str) -> list[int]:
    return [int(t) for t in text.replace(",", " ").split()]


def _generate(argv) -> int:
    ap = argparse.ArgumentParser(prog="llaminar_amd generate")
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--prompt", action="append", required=True, type=_ids, help="token ids with commas between them; may be repeated")
    ap.add_argument("--max-new", type=int, default=16)
    ap.add_argument("--stop", type=_ids, default=[], help="token ids that end a continuation")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--slots", type=int, default=8)
    ap.add_argument("--portion", type=int, default=512, help="most tokens of a prompt in one step")
    args = ap.parse_args(argv)
    from . import models
    from .engine import Engine

    cap = max(len(p) for p in args.prompt) + args.max_new
    runner = models.load_model(args.model, slots=args.slots, cap=cap, dtype=args.dtype)
    try:
        for output in Engine(runner, portion=args.portion).generate(args.prompt, args.max_new, args.stop):
            print(",".join(str(t) for t in output))
    finally:
        runner.close()
    return 0


def main(argv=None) -> int:
    argv = sys.argv[1:] if argv is None else argv
    if argv[:1] == ["generate"]:
        return _generate(argv[1:])
    if argv[:1] == ["trace"]:
        from . import trace

        return trace.main(argv[1:])
    if argv == ["models"]:
        from . import models

        print("\n".join(models.families()))
        return 0
    print(__doc__.strip(), file=sys.stderr)
    return 2


if __name__ == "__main__":
    sys.exit(main())
