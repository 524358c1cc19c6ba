"""Command line: `python -m livecc_amd generate --model DIR --ids 5,17,3 [--ids ...]` -- ids in, ids out, one batched generate call.

The model class follows the checkpoint's config.json.  (`bin/trace_run` replays given ids and writes logits.)"""
import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m livecc_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="generate token ids from prompts of token ids (text prompts only)")
    g.add_argument("--model", required=True, help="checkpoint directory")
    g.add_argument("--ids", action="append", required=True, help="comma-separated prompt ids; repeat for a batch")
    g.add_argument("--max-new-tokens", type=int, default=16)
    g.add_argument("--repetition-penalty", type=float, default=1.0)
    g.add_argument("--do-sample", action="store_true")
    g.add_argument("--temperature", type=float, default=1.0)
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--top-p", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=None)
    g.add_argument("--device", default="cuda:0")
    a = ap.parse_args(argv)
    import numpy as np
    from .modeling import load_model
    prompts = [np.asarray([int(t) for t in p.split(",")], dtype=np.int64) for p in a.ids]
    model = load_model(a.model, device_map=a.device, max_streams=len(prompts), max_history=max(a.max_new_tokens, 1),
                       max_kv_len=max(len(p) for p in prompts) + 2 * a.max_new_tokens)
    outs = model.generate_batch([dict(input_ids=p) for p in prompts], max_new_tokens=a.max_new_tokens, repetition_penalty=a.repetition_penalty,
                                do_sample=a.do_sample, temperature=a.temperature, top_k=a.top_k, top_p=a.top_p, seed=a.seed)
    for p, o in zip(prompts, outs):
        print(json.dumps({"prompt": p.tolist(), "generated": o.sequences[0, len(p):].tolist()}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
