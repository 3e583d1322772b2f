"""Replays a trace: given token ids go through a model step by step, logits are written, nothing is sampled.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries`: for each request its next tokens and the places among them whose logits are wanted; `end`: requests that
are finished after the step.  A step in which something is wanted writes OUT/<step>.f32, the logits in the order of the
entries and of `want` (little-endian fp32, [wanted, vocab]).  After every step `done <step>` is printed."""
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
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens live requests hold at any time")
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
