"""Plain, slow implementation of the Bemuzen decoder from its equations: one function per mechanism, whole sequences, token-by-token
recurrences, no cache, no batching.  It shares no code with `livecc_amd`; the tests compare the HIP engine with it.

Notation: x_t is the residual of token t (32-bit); every weight is [out, in] and applied as W x; rms(x) = sqrt(mean(x^2) + eps).
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch
import torch.nn.functional as F


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_around_one(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The model's norm: the weight is stored as its distance from one."""
    return over_rms(x, eps) * (1.0 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gated_mlp(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def bigram_rows(tokens: List[int], buckets: int, mul_prev: int, mul_cur: int) -> List[int]:
    """Row of the bigram table for every token: a hash of (previous, current); the row behind the buckets for a first token."""
    return [buckets if t == 0 else (tokens[t - 1] * mul_prev + tokens[t] * mul_cur) % buckets for t in range(len(tokens))]


def query_temperature(positions: torch.Tensor, coef: float, every: int) -> torch.Tensor:
    """Grows with the logarithm of the position, in steps of `every`."""
    return 1.0 + coef * torch.log(torch.floor((positions + 1) / every) + 1.0)


def head_slopes(heads: int) -> torch.Tensor:
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float64)


def biased_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, slopes: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, e]: causal softmax attention with slope_h (i - j) taken off every score -> [T, H, e]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    dist = torch.arange(T, dtype=q.dtype)[:, None] - torch.arange(T, dtype=q.dtype)[None, :]
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale - slopes[h].to(q.dtype) * dist
        out[:, h] = torch.softmax(s.masked_fill(dist < 0, float("-inf")), dim=-1) @ v[:, g]
    return out


def softmax_mixer(h: torch.Tensor, W: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """GQA with per-head query / key norms, a query temperature and a distance bias; no rotation."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = over_rms((h @ W["q"].T).view(T, H, m["dim"]), eps) * W["q.norm"]
    k = over_rms((h @ W["k"].T).view(T, G, m["dim"]), eps) * W["k.norm"]
    v = (h @ W["v"].T).view(T, G, m["vdim"])
    q = q * query_temperature(torch.arange(T, dtype=h.dtype), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    return biased_attention(q, k, v, m["scale"], head_slopes(H)).reshape(T, -1) @ W["o"].T


def decayed_outer_products(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, weight: torch.Tensor,
                           state: Optional[torch.Tensor] = None):
    """q, k [T, H, n], v [T, H, e], decay, weight [T, H]: S_t = decay_t S_{t-1} + weight_t k_t v_t^T, o_t = S_t^T q_t.
    Returns (o [T, H, e], the last S [H, n, e])."""
    T, H, n = k.shape
    S = torch.zeros(H, n, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = S * decay[t][:, None, None] + weight[t][:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out, S


def lightning_mixer(h: torch.Tensor, W: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Linear attention with a fixed decay per head, a norm over all heads together and a sigmoid output gate."""
    T, H = h.shape[0], m["heads"]
    q, k, v = silu(h @ W["q"].T).view(T, H, -1), silu(h @ W["k"].T).view(T, H, -1), silu(h @ W["v"].T).view(T, H, -1)
    decay = torch.tensor(m["decay"], dtype=h.dtype).expand(T, H)
    o, _ = decayed_outer_products(q, k, v, decay, torch.ones(T, H, dtype=h.dtype))
    o = over_rms(o.reshape(T, -1), eps) * W["norm"]
    return (o * torch.sigmoid(h @ W["g"].T)) @ W["o"].T


def parallel_mixer(h: torch.Tensor, W: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Mean of the two outputs, each brought to unit rms over the width and weighted."""
    sub = lambda side: {n[len(side) + 1:]: w for n, w in W.items() if n.startswith(side + ".")}
    left, right = softmax_mixer(h, sub("left"), m["left"], eps), lightning_mixer(h, sub("right"), m["right"], eps)
    return 0.5 * (over_rms(left, eps) * W["left.out"] + over_rms(right, eps) * W["right.out"])


def causal_conv(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """u [T, channels], w [channels, taps]: out_t = b + sum_j w_j u_(t - taps + 1 + j), terms with a negative index left out."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u) + b
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * u[s]
    return out


def mamba2_mixer(h: torch.Tensor, W: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """State-space duality: heads of vdim values over a shared state input B and output C per group, decay and step size from dt."""
    T, H, G, N, e = h.shape[0], m["heads"], m["groups"], m["state"], m["vdim"]
    inner = H * e
    z, xbc, dt = torch.split(h @ W["in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, W["conv"], W["conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    x = x.reshape(T, H, e)
    group = torch.arange(H) // (H // G)
    B, C = B.reshape(T, G, N)[:, group], C.reshape(T, G, N)[:, group]
    dt = F.softplus(dt + W["dt_bias"], threshold=1e9)
    decay = torch.exp(-torch.exp(W["A_log"]) * dt)
    y, _ = decayed_outer_products(C, B, x, decay, dt)
    y = (y + W["D"][:, None] * x).reshape(T, inner) * silu(z)
    y = over_rms(y.view(T, m["norm_groups"], -1), eps).reshape(T, inner) * W["norm"]
    return y @ W["o"].T


MIXERS = {"parallel": parallel_mixer, "mamba2": mamba2_mixer}


def run(cfg: dict, T: Dict[str, torch.Tensor], tokens: List[int], taps: Optional[list] = None, dtype=torch.float64) -> torch.Tensor:
    """Logits [len(tokens), vocab] of one sequence.  `T`: tensors by checkpoint name; `taps` receives the residual after every layer."""
    g = lambda n: T[n].to(dtype)
    eps = cfg["norm"]["eps"]
    b = cfg["embedding"]["bigram"]
    tokens = [int(t) for t in tokens]
    x = g("embed")[tokens] + g("bigram")[bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        W = {n[len(p + "mix."):]: g(n) for n in T if n.startswith(p + "mix.")}
        y = MIXERS[layer["type"]](norm_around_one(x, g(p + "norm1"), eps), W, layer["mixer"], eps)
        x = x + norm_around_one(y, g(p + "norm1b"), eps)
        if layer.get("mlp") is not None:
            assert layer["mlp"]["kind"] == "dense", layer["mlp"]
            y = gated_mlp(norm_around_one(x, g(p + "norm2"), eps), g(p + "mlp.gate"), g(p + "mlp.up"), g(p + "mlp.down"))
            x = x + norm_around_one(y, g(p + "norm2b"), eps)
        if taps is not None:
            taps.append(x)
    return (norm_around_one(x, g("final.norm"), eps) @ g("head").T) * cfg["logit_scale"]


def load(path: str):
    from safetensors.torch import load_file
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return cfg, load_file(os.path.join(path, "model.safetensors"))
