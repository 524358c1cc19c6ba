"""Prefill and decode throughput of a layer-list decoder beside the Qwen2-VL language model at equal size (random weights, token ids only):
`python bench.py --workload decoder [--decoder-model bemuzen] [--decoder-size 7b] [--decoder-layers 28]`.  One JSON line per model and size.

Same width, feed-forward, query heads, head size, depth and vocabulary; the other model has grouped-query attention.  debunex: latent attention
(query rank 0.43 width, latent rank 512, one latent per two layers).  bemuzen: grouped-query attention with a distance bias beside linear
attention of the same heads, every fourth layer a state-space layer instead.  `decoder_layer_flops` / `step_bytes` are what the model's own
equations need, so tokens/s of both are also given as a fraction of the dense bf16 peak (prefill) and of the HBM rate (decode)."""
import dataclasses
import json
import time

import numpy as np
import torch

PEAK_FLOPS, PEAK_BYTES = 2.5e15, 8.0e12
LIKE = {"2b": "qwen2vl-2b", "7b": "livecc-7b"}
CHUNK = 64          # tokens the linear-attention products of a prefill are formed over (scores inside a chunk, states between chunks)


def cut(cfg, layers: int):
    c = dataclasses.replace(cfg)
    if hasattr(cfg, "layers"):
        c.layers = cfg.layers[:layers]
    else:
        c.num_hidden_layers, c.vit_depth = layers, 1
    return c


def decoder_layer_flops(l, width: int, S: int, past: int) -> float:
    """Multiply-adds x 2 of one layer over S new rows behind `past` cached ones (prefill form, real sizes)."""
    m = l.mixer
    keys = past + (S + 1) / 2
    if hasattr(m, "recurrent"):
        r = m.recurrent
        k = r.state if hasattr(r, "state") else r.dim
        # chunked recurrence per head: half a chunk of scores and values, the state read and updated
        n = S * r.heads * ((k + r.vdim) * CHUNK / 2 + 2 * k * r.vdim) + S * width * (r.heads * r.vdim + 3 * l.ff)
        if hasattr(m, "left"):
            a = m.left
            n += S * width * (a.heads * a.dim + a.kv_heads * (a.dim + a.vdim) + a.heads * a.vdim + 2 * r.heads * (r.dim + r.vdim))
            n += S * keys * a.heads * (a.dim + a.vdim)
        else:
            n += S * (width * (2 * r.heads * r.vdim + 2 * r.groups * r.state + r.heads) + r.conv_taps * (r.heads * r.vdim + 2 * r.groups * r.state))
        return 2.0 * n
    lin = width * (m.q_rank + m.heads + (m.kv_rank if m.kv_from is None else 0)) + m.q_rank * m.heads * m.dim + width * (m.heads * m.vdim + 3 * l.ff)
    lin_keys = m.kv_rank * m.heads * (m.dim + m.vdim)
    return 2.0 * (S * lin + (past + S) * lin_keys + S * keys * m.heads * (m.dim + m.vdim))


def gqa_layer_flops(cfg, S: int, past: int) -> float:
    keys = past + (S + 1) / 2
    h, i = cfg.hidden_size, cfg.intermediate_size
    return 2.0 * (S * (h * cfg.qkv_dim + cfg.q_dim * h + 3 * h * i) + S * keys * cfg.num_attention_heads * 2 * 128)


def flops_of(cfg, S: int, past: int = 0) -> float:
    if hasattr(cfg, "layers"):
        n = sum(decoder_layer_flops(l, cfg.hidden_size, S, past) for l in cfg.layers)
    else:
        n = cfg.num_hidden_layers * gqa_layer_flops(cfg, S, past)
    return n + 2.0 * cfg.hidden_size * cfg.vocab_size          # logits of the last row


def step_bytes(cfg, B: int, L: int) -> float:
    return cfg.decode_weight_bytes() + B * (L * cfg.kv_bytes_per_token + 2 * getattr(cfg, "state_bytes", 0))          # a state is read and written


def build(name: str, layers: int, rows: int, kv: int, streams: int):
    from livecc_amd.config import get_config
    from livecc_amd.engine import Engine
    from livecc_amd.weights import make_arena
    cfg = cut(get_config(name), layers)
    arena = make_arena(cfg, "cuda").fill_random(0)
    return cfg, Engine(cfg, arena, "cuda", max_slots=streams, max_kv_len=kv, max_new_rows=rows, max_patches=1024, max_history=256)


def timed(fn, reps: int, warm: int = 1) -> float:
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / reps


def run_model(name: str, layers: int, prefills, decodes, reps: int, say):
    from livecc_amd.engine import Sampling
    rows, streams = max(prefills + [2048]), max([b for b, _ in decodes] + [1])
    cfg, eng = build(name, layers, rows, max(prefills + [l for _, l in decodes]) + 512, streams)
    rng, sp = np.random.default_rng(0), Sampling(suppress_eos=True, eos_token=0)
    V = min(cfg.vocab_size, 150000)
    out = dict(model=name, layers=layers, prefill=[], decode=[])
    for S in prefills:
        ids = rng.integers(0, V, S).astype(np.int32)
        pos = np.tile(np.arange(S), (3, 1))

        def one():
            eng.reset_slot(0)
            eng.prefill([0], [ids], [pos], None, sp)
        t = timed(one, reps)
        f = flops_of(cfg, S)
        out["prefill"].append(dict(tokens=S, ms=round(t * 1e3, 3), tokens_per_s=round(S / t, 1), fraction_of_peak=round(f / t / PEAK_FLOPS, 4)))
        say(f"{name} prefill {S}: {t * 1e3:.2f} ms")
    for B, L in decodes:
        ids = rng.integers(0, V, 64).astype(np.int32)
        for s in range(B):           # L cached keys per stream: a short prefill, then the length is set (the rows are zeros: the work is the same)
            eng.reset_slot(s)
            eng.prefill([s], [ids], [np.tile(np.arange(64), (3, 1))], None, sp)
        n = 16

        def steps():
            for s in range(B):
                eng.set_slot_length(s, L, L, keep_state=True)
            eng.decode(list(range(B)), n, 1, sp)
        t = timed(steps, reps, warm=2) / n
        out["decode"].append(dict(streams=B, keys=L, ms_per_step=round(t * 1e3, 4), tokens_per_s=round(B / t, 1),
                                  fraction_of_hbm=round(step_bytes(cfg, B, L) / t / PEAK_BYTES, 4)))
        say(f"{name} decode {B} x {L} keys: {t * 1e3:.3f} ms per step")
    del eng
    torch.cuda.empty_cache()
    return out


def main(args) -> None:
    sizes = [args.decoder_size] if args.decoder_size else list(LIKE)
    prefills = [int(x) for x in args.decoder_prefill.split(",") if x]
    decodes = [tuple(int(y) for y in x.split("x")) for x in args.decoder_decode.split(",") if x]
    for size in sizes:
        for name in [f"{args.decoder_model}-{size}"] + ([] if args.decoder_only else [LIKE[size]]):
            r = run_model(name, args.decoder_layers, prefills, decodes, max(1, args.steps), lambda m: print(m, flush=True))
            print(json.dumps(dict(metric="decoder_vs_gqa", size=size, dtype="bf16", data="synthetic", **r)), flush=True)
