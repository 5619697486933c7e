"""Replays given token ids through a model, step by step, and writes the logits that are asked for (``bin/trace_run``; ``python -m
aria_amd.trace_run``).  It samples nothing: the scheduler, the caches and the step function are the ones generation uses.

    trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

A step is one JSON object a line: {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}.  ``want``: places among
the step's tokens whose logits go to OUT/<step>.f32 (little-endian float32 [wanted, vocab], entries in order); ``end``: requests finished after the
step.  Each finished step prints ``done <step>``.  Exit code 3: the model does not compute in that dtype."""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None, stdin=None, stdout=None, device=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json + model.safetensors)")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    stdin, stdout = stdin or sys.stdin, stdout or sys.stdout

    import torch

    from . import registry
    from .serving import Scheduler

    try:
        model = registry.serving_model(registry.load_model(args.model, device or "cuda", getattr(torch, args.dtype)))
    except TypeError as e:
        print(f"trace_run: {e}", file=sys.stderr)
        return 3
    sched = Scheduler(model, args.max_tokens)
    for line in stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = step["entries"]
        if entries:
            wanted = [e.get("want") or [] for e in entries]
            logits = sched.step([e["id"] for e in entries], [e["tokens"] for e in entries], wanted)
            if logits is not None:
                path = os.path.join(args.out, f"{step['step']}.f32")
                with open(path + ".part", "wb") as f:
                    f.write(logits.float().cpu().contiguous().numpy().astype("<f4").tobytes())
                os.replace(path + ".part", path)
        for r in step.get("end") or []:
            sched.finish(r)
        print(f"done {step['step']}", file=stdout, flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
