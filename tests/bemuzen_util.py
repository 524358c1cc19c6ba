"""Small Bemuzen models for the tests: configurations, random weights under which far tokens matter (sharp scores, slow decays), the oracle's logits."""
import numpy as np
import torch

from livecc_amd.config import BemuzenConfig, DecoderLayerSpec as L, LightningMixerSpec as Lin, ParallelMixerSpec as P, SoftmaxMixerSpec as A, SsdMixerSpec as S
from livecc_amd.weights import BemuzenArena, bemuzen_param_shapes
from oracle import bemuzen_ref as R

# of the logits' rms; bf16 operands measure 0.01-0.03 at these sizes (median row 0.006), planted faults 0.1-6
LIMIT = 0.045


def configs():
    """name -> configuration.  Sizes off every padding multiple, per-layer sizes, shared and own keys, layers without a feed-forward, heads and groups
    that norm groups cut through, one to seven convolution taps, head sizes above the MFMA prefill kernel's, more heads per key than one tile."""
    return {
        "mixed": BemuzenConfig(331, 200, [L(P(A(6, 2, 24, 40, 0.31, 0.4, 37), Lin(3, 40, 24, [0.5, 0.97, 1.0])), 150), L(S(6, 20, 24, 3, 4, 4), 0),
                                          L(P(A(4, 4, 72, 88, 0.17, 0.2, 64), Lin(2, 72, 100, [0.9, 0.0])), 0), L(S(5, 24, 40, 1, 2, 1), 90)],
                               97, 31, 5, 1e-5, 1.7, name="mixed"),
        "even": BemuzenConfig(256, 128, [L(P(A(4, 1, 64, 64, 0.2, 0.3, 100), Lin(2, 64, 64, [0.8, 0.995])), 256), L(S(2, 64, 64, 2, 4, 2), 256)], 769, 17, 3, 1e-6, 1.0,
                              name="even"),
        "wide-heads": BemuzenConfig(100, 96, [L(P(A(2, 1, 136, 200, 0.1, 0.1, 16), Lin(2, 200, 130, [0.99, 0.6])), 64), L(S(3, 70, 150, 1, 1, 5), 40),
                                              L(P(A(1, 1, 8, 8, 0.5, 0.0, 1), Lin(3, 8, 24, [0.93, 0.5, 0.99])), 24)], 1, 3, 2, 1e-3, 0.6, name="wide-heads"),
        "many-heads": BemuzenConfig(513, 320, [L(S(9, 128, 128, 3, 7, 9), 100), L(P(A(34, 2, 128, 33, 0.12, 0.4, 90), Lin(7, 128, 128, [0.9 + 0.014 * h for h in range(7)])), 320),
                                               L(P(A(3, 3, 100, 128, 0.1, 0.2, 50), Lin(5, 16, 40, [0.75, 0.99, 0.999, 0.3, 0.95])), 64)], 4099, 211, 13, 1e-5, 2.5,
                                    name="many-heads"),
    }


def make_weights(cfg: BemuzenConfig, seed: int = 0, sharp: float = 2.0) -> dict:
    """bf16 tensors by checkpoint name.  Scores have a standard deviation of about `sharp` whatever the configured scale is; state-space heads
    forget over a few to a few hundred tokens."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shp in bemuzen_param_shapes(cfg).items():
        t = torch.randn(shp, generator=g)
        mixer = cfg.layers[int(name[1:name.index(".")])].mixer if name.startswith("l") else None
        if name.endswith(("norm1", "norm1b", "norm2", "norm2b", "final.norm")):
            t = t * 0.2                                    # stored around zero
        elif name.endswith("left.q.norm"):
            t = (1.0 + 0.2 * t) * (sharp / (mixer.left.scale * mixer.left.dim ** 0.5))
        elif name.endswith("conv"):
            t = t * shp[1] ** -0.5
        elif name.endswith("conv.b"):
            t = t * 0.1
        elif name.endswith("A_log"):
            t = t - 2.5
        elif name.endswith("dt_bias"):
            t = t - 1.0
        elif name in ("embed", "bigram"):
            t = t * (1.0 if name == "embed" else 0.5)
        elif len(shp) == 2:
            t = t * shp[1] ** -0.5 * (3.0 if name == "head" else 1.0)
        else:
            t = 1.0 + 0.2 * t
        out[name] = t.to(torch.bfloat16)
    return out


def ids_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg.vocab_size, n).tolist()


def oracle_logits(cfg, T, ids, **kw) -> torch.Tensor:
    return R.run(cfg.to_dict(), T, list(ids), **kw)


def error(got: torch.Tensor, want: torch.Tensor) -> float:
    """Rms difference of a row (mean taken off) over the rms of all wanted logits: the worst of 99 rows in 100, or half the worst of all -- a
    group norm whose group happens to cancel (a twentieth of its usual size) multiplies that row's rounding."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(dim=-1, keepdim=True)
    e = (d.pow(2).mean(dim=-1).sqrt() / want.double().pow(2).mean().sqrt()).sort().values
    return max(e[int(0.99 * (len(e) - 1))], e[-1] / 2).item()


def arena(cfg, T, device):
    return BemuzenArena(cfg, device).load_state_dict(lambda n: T[n])
