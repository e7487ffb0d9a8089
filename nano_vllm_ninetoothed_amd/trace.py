"""Replays a trace of steps on a model: JSON lines on standard input, logits in files.

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [0, 1]}], "end": ["a"]}

Every line is one step of the engine: its entries form one batch, each with the next tokens of a request (admitted at its
first entry) and the places among them whose logits are wanted; the requests under "end" give back what they hold.  Wanted
logits go to OUT/<step>.f32 as little-endian float32 [wanted, vocab]; "done <step>" is printed after every step.
Exit code 3: the model does not run in the given dtype.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

PAGE = 64     # tokens per cache page of a replay


def add_arguments(ap: argparse.ArgumentParser) -> None:
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help=f"tokens the cache holds: the sum over live requests, each rounded up to a multiple of {PAGE}")
    ap.add_argument("--max-requests", type=int, default=4, help="state slots: requests that are live at any time")


def run(args) -> int:
    import torch
    from .engine import Engine
    from .models import load_config, model_class
    dtype = getattr(torch, args.dtype)
    if dtype not in model_class(load_config(args.model)).dtypes:
        print(f"this model does not run in {args.dtype}", file=sys.stderr)
        return 3
    torch.backends.cuda.matmul.allow_tf32 = False
    blocks = max(1, (args.max_tokens + PAGE - 1) // PAGE)
    eng = Engine.from_pretrained(args.model, dtype=dtype, num_blocks=blocks, block_size=PAGE, max_num_seqs=args.max_requests,
                                 max_model_len=blocks * PAGE)
    vocab = eng.model.vocab
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        rec = json.loads(line)
        portions = []
        for e in rec["entries"]:
            if any(not 0 <= t < vocab for t in e["tokens"]):
                raise ValueError(f"request {e['id']}: token id outside the vocabulary")
            if e["id"] not in live:
                live[e["id"]] = eng.open_sequence()
            if e["tokens"]:
                portions.append((live[e["id"]], e["tokens"], e["want"]))
        logits = eng.run_portions(portions) if portions else None
        if logits is not None:
            data = logits.float().cpu().numpy().astype("<f4", copy=False).tobytes()
            with open(os.path.join(args.out, f"{rec['step']}.f32"), "wb") as f:
                f.write(data)
        for name in rec["end"]:
            eng.close_sequence(live.pop(name))
        torch.cuda.synchronize()
        print(f"done {rec['step']}", flush=True)
    return 0


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    add_arguments(ap)
    return run(ap.parse_args(argv))
