"""Small Debunex models for the tests: configurations, random weights whose attention is sharp (a far key decides a token), the oracle's logits."""
import numpy as np
import torch

from livecc_amd.config import DebunexConfig, DecoderLayerSpec as L, LatentMixerSpec as M
from livecc_amd.weights import DecoderArena, decoder_param_shapes
from oracle import debunex_ref as R

LIMIT = 0.025         # worst row: rms of the logit difference over the rms of the logits; bf16 operands measure 0.008-0.015 at these sizes


def configs():
    """name -> configuration.  Sizes off every padding multiple, per-layer sizes, shared latents of several patterns, layers without a
    feed-forward, single heads, more heads than one 16-head tile, head sizes above the MFMA kernels', no cap."""
    return {
        "mixed": DebunexConfig(331, 200, [L(M(5, 24, 40, 72, 56, 0.31), 150), L(M(3, 40, 16, 48, 100, 0.2), 0), L(M(2, 72, 88, 30, 56, 0.17, 0), 90),
                                          L(M(18, 16, 24, 96, 100, 0.4, 1), 128)], 1e-5, 20.0, name="mixed"),
        "even": DebunexConfig(256, 128, [L(M(4, 64, 64, 64, 64, 0.2), 256), L(M(4, 64, 64, 64, 64, 0.2), 256)], 1e-6, None, name="even"),
        "wide-heads": DebunexConfig(100, 96, [L(M(2, 136, 200, 130, 150, 0.1), 64), L(M(1, 8, 8, 8, 150, 0.5, 0), 40)], 1e-3, 5.0, name="wide-heads"),
        "full-heads": DebunexConfig(513, 320, [L(M(33, 128, 128, 192, 200, 0.12), 100), L(M(3, 100, 128, 64, 300, 0.1), 320), L(M(7, 128, 33, 65, 300, 0.1, 1), 0),
                                               L(M(2, 48, 48, 64, 300, 0.15, 1), 64)], 1e-5, 30.0, name="full-heads"),
    }


def make_weights(cfg: DebunexConfig, seed: int = 0, sharp: float = 2.5) -> dict:
    """bf16 tensors by checkpoint name.  Scores have a standard deviation of about `sharp` whatever the configured scale is."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shp in decoder_param_shapes(cfg).items():
        if name.endswith(".alpha"):
            t = torch.tensor(0.6 + 0.3 * torch.rand((), generator=g).item())
        else:
            t = torch.randn(shp, generator=g)
            if name == "embed":
                t = t * 1.2
            elif len(shp) == 2:
                t = t * shp[1] ** -0.5
                if name.endswith(".uq"):
                    m = cfg.layers[int(name[1:name.index(".")])].mixer
                    t = t * (sharp / (m.scale * m.dim ** 0.5))
                if name.endswith(".o"):
                    t = t * 2.0
                if name == "head":
                    t = t * 4.0
            elif name.endswith(".b"):
                t = t * 0.2
            else:
                t = 1.0 + 0.2 * t
        out[name] = t.to(torch.bfloat16)
    return out


def ids_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg.vocab_size, n).tolist()


def oracle_logits(cfg, T, ids, **kw) -> torch.Tensor:
    return R.run(cfg.to_dict(), T, list(ids), **kw)


def error(got: torch.Tensor, want: torch.Tensor) -> float:
    """Worst row: rms difference (mean taken off) over the rms of all wanted logits."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(dim=-1, keepdim=True)
    return (d.pow(2).mean(dim=-1).sqrt().max() / want.double().pow(2).mean().sqrt()).item()


def arena(cfg, T, device):
    return DecoderArena(cfg, device).load_state_dict(lambda n: T[n])
