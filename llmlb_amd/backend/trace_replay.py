"""Feeds given token ids through the serving engine, step by step, and
writes the logits that are asked for (nothing is sampled).

  bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR
                --max-tokens N [--device cuda:0] [--max-live 4]

Standard input brings one JSON object a line:

  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
   "end": []}

All entries of a step are one batch of ``Engine.run_batch``.  For a step
in which something is wanted, OUT/<step>.f32 gets the logits as
little-endian floats [wanted, vocab]; after every step the line
``done <step>`` is printed.  ``end`` lists the requests whose pages and
state slots are given back after the step.  The cache pool holds
``--max-tokens`` tokens and ``--max-live`` state slots.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def parse_args(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and weights, or a preset")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens held by live requests at a time")
    ap.add_argument("--max-live", type=int, default=4,
                    help="most live requests at a time")
    ap.add_argument("--device", default="cuda:0")
    return ap.parse_args(argv)


def open_engine(args):
    from ..models.registry import resolve
    from .engine import Engine, EngineConfig
    from .kv_cache import BLOCK_SIZE

    if args.device.startswith("cuda"):
        import torch
        from ..ops.build import ensure_library
        ensure_library("hybrid")
        torch.set_float32_matmul_precision("highest")
        torch.cuda.set_device(args.device)
    cfg, folder = resolve(args.model)
    cfg.max_pos = max(args.max_tokens, BLOCK_SIZE)
    blocks = -(-args.max_tokens // BLOCK_SIZE) + 1   # block 0 is reserved
    return Engine(EngineConfig(
        model=cfg, device=args.device, dtype=args.dtype,
        kv_cache_blocks=blocks, max_batch=args.max_live,
        weights_path=folder))


def replay(engine, lines, out_dir: str, say=print) -> None:
    live: dict = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        work = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = engine.open_sequence()
            work.append((live[e["id"]], e["tokens"], e["want"]))
        logits = engine.run_batch(work)
        if logits.shape[0]:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(logits.cpu().numpy().astype("<f4").tobytes())
        for rid in step["end"]:
            engine.close_sequence(live.pop(rid))
        say(f"done {step['step']}")
        sys.stdout.flush()


def main(argv=None) -> int:
    args = parse_args(argv)
    os.makedirs(args.out, exist_ok=True)
    replay(open_engine(args), sys.stdin, args.out)
    return 0


if __name__ == "__main__":
    sys.exit(main())
