"""Trace replay: token ids in, logits out, through the engine's own prefill and decode steps.

    bin/trace_run --model DIR --dtype bfloat16 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries` of a step are one batch: the next ids of each request and the places among them whose logits are asked for.  The logits of a step
are written to OUT/<step>.f32 (little-endian fp32 [wanted, vocab], in the order of the entries); after every step a line "done <step>" is
printed.  Requests named in `end` give their slot back.  The engine computes in bf16 (fp32 accumulation, residual, norms and softmax): a
request for float32 ends with exit code 3.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def parse_args(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids through a model and write logits.")
    ap.add_argument("--model", required=True, help="checkpoint directory: config.json and *.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="directory of the logits files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens the live requests hold at any time (sizes the cache)")
    ap.add_argument("--device", default="cuda:0")
    return ap.parse_args(argv)


def replay(model, lines, out_dir: str, say=print) -> None:
    """Run the steps of `lines` (JSON texts) on `model` (an EngineModel with `forward_step`)."""
    import torch
    live = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = step.get("entries", [])
        for e in entries:
            if e["id"] not in live:
                live[e["id"]] = model.new_stream()
        logits = model.forward_step([(live[e["id"]], e["tokens"], e.get("want", [])) for e in entries]) if entries else []
        wanted = [x for x in logits if x.shape[0]]
        if wanted:
            data = torch.cat(wanted).cpu().numpy().astype("<f4", copy=False)
            part = os.path.join(out_dir, f".{step['step']}.part")
            data.tofile(part)
            os.replace(part, os.path.join(out_dir, f"{step['step']}.f32"))
        else:
            torch.cuda.synchronize(model.device)
        for name in step.get("end", []):
            live.pop(name).release()
        say(f"done {step['step']}", flush=True)


def main(argv=None) -> int:
    args = parse_args(argv)
    if args.dtype == "float32":
        print("trace_run: the engine has no fp32 mode (bf16 operands, fp32 accumulation)", file=sys.stderr)
        return 3
    from . import _lib
    if not _lib.lib_available():
        from . import build
        build.build_engine(verbose=False)
    from .modeling import load_model
    history = 16                                        # the runner samples nothing: the shortest generation headroom will do
    n = max(1, args.max_tokens)
    model = load_model(args.model, device_map=args.device, max_streams=min(n, 256), max_kv_len=n + history, max_new_rows=max(64, min(n, 4096)),
                       max_history=history)
    replay(model, sys.stdin, args.out)
    return 0
