"""Trace replay: feed given token ids through a model step by step and write
the logits asked for.

    replay --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come as JSON lines on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

An entry brings the next tokens of a request and the places among them whose
logits are wanted; a request is admitted with its first entry and may pause
between steps.  `end` lists the requests to be released after the step.  All
entries of a step run as one batch through Engine.step_entries, on a cache
pool of N tokens.  Wanted logits go to DIR/<step>.f32 as little-endian f32
[wanted, vocab]; 'done <step>' is printed after every step.  Nothing is
sampled.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

LIVE_REQUESTS = 4


def main(argv=None) -> int:
    p = argparse.ArgumentParser(prog="replay", description=__doc__,
                                formatter_class=argparse.
                                RawDescriptionHelpFormatter)
    p.add_argument("--model", required=True,
                   help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=("bfloat16", "float32"),
                   default="bfloat16")
    p.add_argument("--out", required=True)
    p.add_argument("--max-tokens", type=int, required=True,
                   help="most tokens live requests hold at any time")
    p.add_argument("--device", default=None)
    args = p.parse_args(argv)

    import torch

    from . import load_model
    from .serve import Engine, StepEntry

    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    device = args.device or ("cuda:0" if torch.cuda.is_available() else None)
    if device is None:
        print("replay: no GPU (use --device cpu for the reference "
              "semantics)", file=sys.stderr)
        return 2
    model = load_model(args.model, device=device,
                       dtype=getattr(torch, args.dtype))
    pages = -(-args.max_tokens // 64)
    engine = Engine(model, kv_pages=pages, max_batch=LIVE_REQUESTS,
                    max_seq_len=pages * 64, state_slots=LIVE_REQUESTS)
    live: dict[str, list[int]] = {}          # id -> [seq_id, tokens so far]
    next_id = 0
    for line in sys.stdin:
        if not line.strip():
            continue
        msg = json.loads(line)
        entries = []
        for e in msg["entries"]:
            if e["id"] not in live:
                live[e["id"]] = [next_id, 0]
                next_id += 1
            seq = live[e["id"]]
            entries.append(StepEntry(seq[0], e["tokens"], seq[1], e["want"]))
            seq[1] += len(e["tokens"])
        logits = engine.step_entries(entries) if entries else None
        if any(e.want for e in entries):
            path = os.path.join(args.out, f"{msg['step']}.f32")
            with open(path, "wb") as fh:
                fh.write(logits.float().cpu().numpy().astype("<f4").tobytes())
        elif entries and device != "cpu":
            torch.cuda.synchronize()
        for rid in msg["end"]:
            engine.kv.free(live.pop(rid)[0])
        print(f"done {msg['step']}", flush=True)
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
