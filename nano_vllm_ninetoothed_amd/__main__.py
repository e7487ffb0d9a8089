"""Command line: generate from token ids, replay a trace, list the registered models, build the kernels.

    python -m nano_vllm_ninetoothed_amd generate --model DIR --prompt 5,17,3 --prompt 8,1 --max-tokens 16
    python -m nano_vllm_ninetoothed_amd trace --model DIR --out DIR --max-tokens 4096 < steps.jsonl
    python -m nano_vllm_ninetoothed_amd models
"""
from __future__ import annotations

import argparse
import json
import sys


def _generate(args) -> int:
    import torch
    from .engine import Engine
    prompts = [[int(t) for t in p.split(",")] for p in args.prompt]
    need = sum((len(p) + args.max_tokens + args.block_size - 1) // args.block_size for p in prompts)
    longest = max(len(p) for p in prompts) + args.max_tokens
    eng = Engine.from_pretrained(args.model, dtype=getattr(torch, args.dtype), num_blocks=max(1, need), block_size=args.block_size,
                                 max_num_seqs=max(1, len(prompts)), max_model_len=longest, chunked_prefill=args.chunked_prefill,
                                 max_num_batched_tokens=args.max_num_batched_tokens)
    if any(not 0 <= t < eng.model.vocab for p in prompts for t in p):
        print("a prompt holds a token id outside the vocabulary", file=sys.stderr)
        return 2
    if args.graphs:
        eng.capture_decode_graphs(max_bs=min(256, max(1, len(prompts))), max_model_len=longest)
    outs, stats = eng.generate(prompts, args.max_tokens, args.temperature)
    for o in outs:
        print(json.dumps(o))
    print(json.dumps({k: round(v, 4) for k, v in stats.items()}), file=sys.stderr)
    return 0


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="nano_vllm_ninetoothed_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="generate from prompts of token ids (greedy)")
    g.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    g.add_argument("--prompt", action="append", required=True, help="comma-separated token ids; may be given several times")
    g.add_argument("--max-tokens", type=int, default=32)
    g.add_argument("--temperature", type=float, default=0.6)
    g.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    g.add_argument("--block-size", type=int, default=256)
    g.add_argument("--max-num-batched-tokens", type=int, default=16384)
    g.add_argument("--chunked-prefill", action="store_true", help="portions of prompts beside decoded tokens in one step")
    g.add_argument("--graphs", action="store_true", help="replay the decode step from HIP graphs")
    t = sub.add_parser("trace", help="replay a trace of steps (JSON lines on standard input)")
    from . import trace
    trace.add_arguments(t)
    sub.add_parser("models", help="list the registered architectures")
    sub.add_parser("build", help="compile the HIP library")
    args = ap.parse_args(argv)
    if args.command == "generate":
        return _generate(args)
    if args.command == "trace":
        return trace.run(args)
    if args.command == "build":
        from . import build
        print(build.build(force=True))
        return 0
    from .models import architectures
    print("\n".join(architectures()))
    return 0


if __name__ == "__main__":
    sys.exit(main())
