"""Replays a recorded trace of steps through the engine and writes the logits it asks for.

One JSON object a line on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries`: per request its next tokens and the places among them whose logits are wanted; `end`: requests that are
finished after this step.  For a step that wants something OUT/<step>.f32 receives the logits as little-endian fp32
[wanted, vocab] in the order of the entries; after every step a line 'done <step>' is printed.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_REQUESTS = 4
TOKEN_ROUND = 64


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", required=True, type=int,
                    help=f"tokens live requests hold at most, each request's count rounded up to a multiple of {TOKEN_ROUND}")
    ap.add_argument("--max-requests", type=int, default=MAX_REQUESTS, help="live requests at most")
    args = ap.parse_args(argv)

    import torch

    from . import build
    from .engine import Engine, Entry
    from .model_loader import load_config
    from .models import kernel_sources, load_model

    if not torch.cuda.is_available():
        raise RuntimeError("no GPU (there is no CPU fallback)")
    build.ensure(kernel_sources(load_config(args.model)))
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.backends.cuda.matmul.allow_bf16_reduced_precision_reduction = False
    dev = torch.device("cuda", 0)
    model = load_model(args.model, getattr(torch, args.dtype), dev, args.max_tokens)
    engine = Engine(model, args.max_tokens, args.max_requests)
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = engine.open()
            entries.append(Entry(live[e["id"]], e["tokens"], e.get("want") or []))
        logits = engine.step(entries)
        if logits is not None:
            logits.cpu().numpy().astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
        else:
            torch.cuda.synchronize(dev)
        for name in step.get("end") or []:
            engine.close(live.pop(name))
        print(f"done {step['step']}", flush=True)
    return 0
