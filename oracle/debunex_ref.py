"""Plain, slow implementation of the Debunex decoder from its equations: one function per mechanism, whole sequences, no cache, no batching.
It shares no code with `livecc_amd`; the tests compare the HIP engine with it.

Notation: x_t is the residual of token t (32-bit); N the layer's norm; every weight is [out, in] and applied as W x.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def dynamic_tanh(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """Elementwise norm without statistics: tanh(alpha x) w + b."""
    return torch.tanh(alpha * x) * w + b


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gated_mlp(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def latent_of(h: torch.Tensor, dkv: torch.Tensor, norm: torch.Tensor, eps: float) -> torch.Tensor:
    """What the cache holds for a token: the normed down-projection c."""
    return rms_unit(h @ dkv.T, eps) * norm


def queries_of(h: torch.Tensor, dq: torch.Tensor, norm: torch.Tensor, uq: torch.Tensor, heads: int, eps: float) -> torch.Tensor:
    """[T, heads, dim]: queries through their own normed latent."""
    q = (rms_unit(h @ dq.T, eps) * norm) @ uq.T
    return q.view(h.shape[0], heads, -1)


def causal_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, first: int = 0) -> torch.Tensor:
    """q [T, H, d] for the positions first .. first + T - 1 over keys k [L, H, d], values v [L, H, e] -> [T, H, e]."""
    T, L = q.shape[0], k.shape[0]
    s = torch.einsum("thd,lhd->htl", q, k) * scale
    hidden = torch.arange(L)[None, :] > (first + torch.arange(T))[:, None]
    s = s.masked_fill(hidden[None].to(s.device), float("-inf"))
    return torch.einsum("htl,lhe->the", torch.softmax(s, dim=-1), v)


def latent_attention(h: torch.Tensor, c: torch.Tensor, W: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """h [T, width] of all tokens of a sequence, c [T, rank] the latent of the layer that owns the cache."""
    H = m["heads"]
    q = queries_of(h, W["dq"], W["dq.norm"], W["uq"], H, eps)
    k = (c @ W["uk"].T).view(c.shape[0], H, -1)
    v = (c @ W["uv"].T).view(c.shape[0], H, -1)
    o = causal_softmax_attention(q, k, v, m["scale"])
    o = o * torch.sigmoid(h @ W["g"].T)[:, :, None]
    return o.reshape(h.shape[0], -1) @ W["o"].T


def soft_cap(z: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return z if not cap else cap * torch.tanh(z / cap)


def run(cfg: dict, T: Dict[str, torch.Tensor], tokens: List[int], taps: Optional[list] = None, dtype=torch.float64) -> torch.Tensor:
    """Logits [len(tokens), vocab] of one sequence.  `T`: tensors by checkpoint name; `taps` receives the residual after every layer."""
    g = lambda n: T[n].to(dtype)
    eps = cfg["norm"]["eps"]
    dyt = lambda x, n: dynamic_tanh(x, g(n + ".alpha"), g(n), g(n + ".b"))
    x = g("embed")[torch.as_tensor(tokens)]
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        assert layer["type"] == "latent_attention", layer["type"]
        p, m = f"l{i}.", layer["mixer"]
        h = dyt(x, p + "norm1")
        W = {n[len(p + "mix."):]: g(n) for n in T if n.startswith(p + "mix.")}
        j = m.get("kv_from")
        if j is None:
            latents[i] = latent_of(h, W["dkv"], W["dkv.norm"], eps)
            j = i
        y = latent_attention(h, latents[j], W, m, eps)
        if layer.get("mlp") is not None:
            assert layer["mlp"]["kind"] == "dense", layer["mlp"]
            y = y + gated_mlp(h, g(p + "mlp.gate"), g(p + "mlp.up"), g(p + "mlp.down"))
        x = x + y
        if taps is not None:
            taps.append(x)
    return soft_cap(dyt(x, "final.norm") @ g("head").T, cfg.get("logit_softcap"))


def load(path: str):
    from safetensors.torch import load_file
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return cfg, load_file(os.path.join(path, "model.safetensors"))
