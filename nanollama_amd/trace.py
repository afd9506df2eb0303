"""Replays a trace of token runs through a model, step by step, and writes the logits that are asked for (bin/trace_run).

Standard input, one JSON object a line:  {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}.  A step is one batch
through the scheduler; the logits at the wanted places go to OUT/<step>.f32 ([wanted, vocab], little-endian float32, in the order
of the entries and their places); requests in "end" give their streams back.  "done <step>" is printed after every step.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

MAX_STREAMS = 128


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token runs and store logits")
    ap.add_argument("--model", required=True, help="model folder (config.json, model.safetensors) or GGUF file")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="upper bound of the tokens held by live requests together: positions per stream")
    ap.add_argument("--device", type=int, default=0)
    args = ap.parse_args(argv)

    from .registry import load_model
    from .scheduler import Scheduler
    n = max(1, args.max_tokens)
    model = load_model(args.model, device=args.device, max_streams=min(MAX_STREAMS, n), dtype=args.dtype, seq_len=n, build=True)
    sched = Scheduler(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [(e["id"], e["tokens"], e.get("want", [])) for e in step["entries"]]
        if entries:
            rows = [r for r in sched.step(entries) if len(r)]
            if rows:
                np.concatenate(rows).astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
        sched.finish(step.get("end", []))
        print(f"done {step['step']}", flush=True)
    model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
