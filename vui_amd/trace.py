"""Trace replay: known token ids are run as recorded steps and the logits of chosen places are kept.  No sampling.

    bin/trace_run --model FOLDER --dtype float32 --out LOGITS --max-tokens 4096 < steps.jsonl

Every input line is one step in JSON:

    {"step": 12, "entries": [{"id": "r7", "tokens": [41, 8], "want": [1]}], "end": ["r7"]}

An entry continues (or starts) the request named by its id with these tokens; `want` picks places among them by index.  Requests
named in `end` give their slot back once the step is through.  LOGITS/12.f32 then holds the picked rows one after the other as
little-endian fp32 (no file for a step that picks none), and `done 12` on standard output says that it does."""
from __future__ import annotations

import argparse
import json
import os
import sys


def ensure_library() -> None:
    """A fresh checkout has no built library: compile the part the token models need."""
    from . import _lib

    if not os.path.exists(_lib.LIB_PATH) and not os.path.exists(_lib.LM_LIB_PATH):
        from .build import build_lm

        build_lm(verbose=False)


def replay(engine, lines, out_dir: str, emit) -> None:
    """lines: an iterable of JSON texts; emit(text): one line of output."""
    rows: dict = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        parts = []
        for e in step["entries"]:
            row = rows.get(e["id"])
            if row is None:
                row = rows[e["id"]] = engine.new_row()
            got = row.extend(e["tokens"], e["want"])
            if e["want"]:
                parts.append(got.cpu().numpy().astype("<f4"))
        if parts:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            with open(path, "wb") as f:
                for p in parts:
                    f.write(p.tobytes())
        for rid in step["end"]:
            row = rows.pop(rid, None)
            if row is not None:
                row.close()
        emit(f"done {step['step']}")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token steps and write logits.")
    ap.add_argument("--model", required=True, help="checkpoint folder (config.json, model.safetensors)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="positions to size a slot for")
    ap.add_argument("--max-rows", type=int, default=4, help="most requests alive at a time")
    args = ap.parse_args(argv)
    ensure_library()

    import torch

    from .lm_engine import TokenEngine

    with torch.inference_mode():
        engine = TokenEngine(args.model, max_rows=args.max_rows, max_seq=max(1, args.max_tokens),
                             dtype=torch.float32 if args.dtype == "float32" else torch.bfloat16)
        replay(engine, iter(sys.stdin.readline, ""), args.out, lambda s: print(s, flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
