"""Command line: `python -m vui_amd <command>`.

    models                     the registered designs
    info PATH                  what a local checkpoint holds
    generate --model DIR ...   tokens of a token model, one JSON line per prompt
    trace ...                  replay a trace of token steps (as bin/trace_run)

Vui checkpoints speak through vui_amd.engine.Engine / vui_amd.inference, whose inputs are embeddings and codes."""
from __future__ import annotations

import argparse
import json
import os
import sys


def _ids(text: str) -> "list[int]":
    return [int(t) for t in text.replace(",", " ").split()]


def cmd_models(args) -> int:
    from .registry import model_class, registered

    for name in registered():
        doc = (model_class(name).__doc__ or sys.modules[model_class(name).__module__].__doc__ or "").strip().split("\n")[0]
        print(f"{name}\t{doc}")
    return 0


def cmd_info(args) -> int:
    from .config import Config, GatedLinearAttentionConfig, LatentAttentionConfig, LMConfig, SigmoidAttentionConfig
    from .registry import DEFAULT, read_architecture

    arch = read_architecture(args.path)
    out: dict = {"architecture": arch}
    if arch == DEFAULT:
        if args.path.endswith(".safetensors"):
            from safetensors import safe_open

            with safe_open(args.path, framework="pt") as f:
                m = Config.from_dict(json.loads((f.metadata() or {}).get("config", "{}"))).model
            out.update(width=m.d_model, layers=m.n_layers, heads=m.n_heads, ff=m.ffn, codebooks=m.n_quantizers)
    else:
        with open(os.path.join(args.path, "config.json")) as f:
            c = LMConfig.from_dict(json.load(f))
        per_token = per_row = 0
        kinds = []
        for i, _ in c.runs():
            mx = c.layers[i].mixer
            if isinstance(mx, LatentAttentionConfig):
                kinds.append("latent_attention" if mx.kv_from is None else f"latent_attention<-{mx.kv_from}")
                per_token += mx.kv_rank + mx.rot_dim if mx.kv_from is None else 0
            elif isinstance(mx, SigmoidAttentionConfig):
                kinds.append("sigmoid_attention")
                per_token += mx.kv_heads * (mx.dim + mx.vdim)
            elif isinstance(mx, GatedLinearAttentionConfig):
                kinds.append("gla")
                per_row += 4 * mx.heads * mx.dim * mx.vdim
            else:
                kinds.append("mingru")
                per_row += 4 * mx.width
        out.update(width=c.width, vocab=c.vocab, layers=kinds, cached_values_per_token=per_token, state_bytes_per_row=per_row)
    print(json.dumps(out))
    return 0


def cmd_generate(args) -> int:
    prompts = [_ids(t) for t in args.tokens]
    if args.tokens_file:
        with open(args.tokens_file) as f:
            prompts += [_ids(ln) for ln in f if ln.strip()]
    if not prompts or any(not p for p in prompts):
        print("generate: no prompt (--tokens or --tokens-file)", file=sys.stderr)
        return 2
    from .trace import ensure_library

    ensure_library()
    import torch

    from .engine import GenConfig
    from .lm_engine import TokenEngine, TokenRequest

    max_seq = args.max_seq or max(len(p) for p in prompts) + args.max_new
    eng = TokenEngine(args.model, max_rows=min(args.max_rows, len(prompts)), max_seq=max_seq,
                      dtype=torch.float32 if args.dtype == "float32" else torch.bfloat16)
    greedy = args.temperature <= 0
    cfg = GenConfig(temperature=1.0 if greedy else args.temperature, top_k=1 if greedy else args.top_k, top_p=args.top_p or None,
                    rep_penalty=args.rep_penalty, rep_window=args.rep_window, seed=args.seed)
    stop = frozenset(_ids(args.stop)) if args.stop else frozenset()
    for p, o in zip(prompts, eng.generate([TokenRequest(p, args.max_new, stop) for p in prompts], cfg)):
        print(json.dumps({"prompt": p, "tokens": o}))
    return 0


def main(argv=None) -> int:
    argv = sys.argv[1:] if argv is None else argv
    if argv[:1] == ["trace"]:
        from .trace import main as trace_main

        return trace_main(argv[1:])
    ap = argparse.ArgumentParser(prog="vui_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    sub.add_parser("models").set_defaults(run=cmd_models)
    p = sub.add_parser("info")
    p.add_argument("path")
    p.set_defaults(run=cmd_info)
    p = sub.add_parser("generate")
    p.add_argument("--model", required=True, help="checkpoint folder (config.json, model.safetensors)")
    p.add_argument("--tokens", action="append", default=[], help="prompt as token ids, e.g. 1,2,3 (may be given several times)")
    p.add_argument("--tokens-file", help="one prompt of token ids a line")
    p.add_argument("--max-new", type=int, default=64)
    p.add_argument("--stop", default="", help="token ids that end an answer")
    p.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    p.add_argument("--top-k", type=int, default=0)
    p.add_argument("--top-p", type=float, default=0.0)
    p.add_argument("--rep-penalty", type=float, default=1.0)
    p.add_argument("--rep-window", type=int, default=0)
    p.add_argument("--seed", type=int, default=0)
    p.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    p.add_argument("--max-rows", type=int, default=16, help="prompts decoded together")
    p.add_argument("--max-seq", type=int, default=0, help="positions per slot (default: the longest prompt and its answer)")
    p.set_defaults(run=cmd_generate)
    sub.add_parser("trace", help="replay a trace of token steps", add_help=False)
    args = ap.parse_args(argv)
    return args.run(args)


if __name__ == "__main__":
    sys.exit(main())
