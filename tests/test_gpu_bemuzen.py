"""-m gpu: Bemuzen on the engine against the plain implementation of its equations (oracle/bemuzen_ref.py), mechanism by mechanism, then the
whole model: prompts, decoding, portions, batches, slots that are used again, and greedy generation through the model's entry points."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import bemuzen_ref as R
from tests import bemuzen_util as U

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


def _p(t):
    return None if t is None else t.data_ptr()


@pytest.fixture(scope="module")
def lib(dev):
    from livecc_amd import _lib
    torch.cuda.set_device(dev)
    return _lib.load()


def _ok(rc):
    from livecc_amd import _lib
    _lib.check(rc, "operator")
    torch.cuda.synchronize()


def _st():
    return torch.cuda.current_stream().cuda_stream


def _up(n):
    return -(-n // 64) * 64


def _near(got, want, rel=2.0 ** -8, absolute=1e-6):
    return bool(((got.double().cpu() - want.double()).abs() <= want.double().abs() * rel + absolute).all())


def _heads(t, pad):
    """[.., heads, d] -> [.., heads * pad] with zeros behind every head."""
    out = torch.zeros(*t.shape[:-1], pad, dtype=t.dtype)
    out[..., :t.shape[-1]] = t
    return out.reshape(*t.shape[:-2], -1)


def _model(cfg, T, dev, **kw):
    from livecc_amd.modeling import BemuzenForCausalLM
    a = dict(max_streams=6, max_kv_len=900, max_new_rows=700, max_history=48)
    a.update(kw)
    return BemuzenForCausalLM(cfg, U.arena(cfg, T, dev), dev, **a)


def _arenas(n, size, dev, fill=None):
    a = [torch.zeros(size, dtype=torch.bfloat16, device=dev) if fill is None else torch.full((size,), fill, dtype=torch.bfloat16, device=dev) for _ in range(n)]
    return a, torch.tensor([x.data_ptr() for x in a], dtype=torch.int64, device=dev)


# --------------------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# --------------------------------------------------------------------------------------------------------------------------------
def test_bigram_embedding_of_portions_and_decoded_tokens(dev, lib):
    W, D, V, eps = 128, 100, 60, 1e-3
    buckets, mp, mc = 37, 2000003, 1000033                              # products beyond 32 bits
    emb, big = torch.zeros(V, W).bfloat16(), torch.zeros(buckets + 1, W).bfloat16()
    emb[:, :D], big[:, :D] = torch.randn(V, D), torch.randn(buckets + 1, D)
    w = torch.zeros(W).bfloat16()
    w[:D] = 0.3 * torch.randn(D)
    # three streams in one call: a fresh one, one that goes on after token 11, one row alone that goes on after token 59
    ids, slot, pos, row0 = [7, 59, 7, 12, 13, 5], [1, 1, 1, 0, 0, 2], [0, 1, 2, 40, 41, 9], [0, 0, 0, 3, 3, 5]
    prev = [11, 22, 59]
    before = [None, 7, 59, 11, 12, 59]
    dv = [t.to(dev) for t in (emb, big, w)]
    x, h = torch.empty(6, W, device=dev), torch.empty(6, W, dtype=torch.bfloat16, device=dev)
    a, b, c, d, p = (_i32(v, dev) for v in (ids, slot, pos, row0, prev))
    _ok(lib.lcc_embed_bigram_rms(_p(a), _p(b), _p(c), _p(d), None, _p(p), _p(dv[0]), _p(dv[1]), buckets, mp, mc, _p(dv[2]), eps, _p(x), _p(h), 6, D, W, _st()))
    rows = [buckets if q is None else (q * mp + t * mc) % buckets for q, t in zip(before, ids)]
    want = emb[ids].double() + big[rows].double()
    assert torch.equal(x.cpu().double(), want.float().double())
    assert _near(h[:, :D], R.norm_around_one(want[:, :D], w[:D].double(), eps), absolute=1e-5) and h[:, D:].abs().sum() == 0
    # decode: current tokens and positions per slot; slot 1 is empty
    cur, kv = _i32([4, 5, 6], dev), _i32([3, 0, 8], dev)
    st = _i32([2, 1, 0], dev)
    _ok(lib.lcc_embed_bigram_rms(_p(cur), _p(st), None, None, _p(kv), _p(p), _p(dv[0]), _p(dv[1]), buckets, mp, mc, _p(dv[2]), eps, _p(x), _p(h), 3, D, W, _st()))
    rows = [(59 * mp + 6 * mc) % buckets, buckets, (11 * mp + 4 * mc) % buckets]
    assert torch.equal(x[:3].cpu().double(), (emb[[6, 5, 4]].double() + big[rows].double()).float().double())


@pytest.mark.parametrize("pair", [False, True])
@pytest.mark.parametrize("rows,width,ns,nb", [(1, 64, 1, 2), (3, 200, 4, 1), (9, 2100, 2, 3), (2, 5000, 1, 1)])
def test_norms_around_the_residual(dev, lib, rows, width, ns, nb, pair):
    W, eps = _up(width), 1e-2
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], W - width)], -1)
    x, a, b = pad(torch.randn(rows, width) * 2), pad(torch.randn(ns, rows, width)), pad(torch.randn(nb, rows, width) * 5)
    wa, wb, wp, wn = (pad(torch.randn(width)).bfloat16() for _ in range(4))
    xd, h = x.to(dev), torch.empty(rows, W, dtype=torch.bfloat16, device=dev)
    d = [t.to(dev) for t in (a, b, wa, wb, wp, wn)]
    _ok(lib.lcc_post_norm_resid(_p(d[0]), ns, _p(d[1]) if pair else None, nb, _p(d[2]), _p(d[3]), _p(d[4]), _p(d[5]), _p(xd), _p(h), rows, width, W, eps, _st()))
    cut = lambda t: t.double()[..., :width]
    y = cut(a).sum(0)
    if pair:
        y = 0.5 * (R.over_rms(y, eps) * cut(wa) + R.over_rms(cut(b).sum(0), eps) * cut(wb))
    want = cut(x) + R.norm_around_one(y, cut(wp), eps)
    assert (xd.cpu().double()[:, :width] - want).abs().max() < 2e-5 and xd[:, width:].abs().sum() == 0          # the residual stays fp32
    assert _near(h[:, :width], R.norm_around_one(want, cut(wn), eps), absolute=2e-5) and h[:, width:].abs().sum() == 0


def test_attention_inputs_norms_temperature_and_cache(dev, lib):
    from livecc_amd import _lib
    H, G, d, e, S, ns, L, eps, coef, every = 3, 2, 40, 72, 6, 2, 96, 3e-2, 0.7, 16
    dp, ep = 64, 128
    q, k, v = torch.randn(ns, S, H, d), torch.randn(ns, S, G, d), torch.randn(ns, S, G, e)
    part = torch.cat([_heads(q, dp), _heads(k, dp), _heads(v, ep), torch.randn(ns, S, 64)], -1)
    wq, wk = torch.zeros(dp).bfloat16(), torch.zeros(dp).bfloat16()
    wq[:d], wk[:d] = 1 + 0.2 * torch.randn(d), 1 + 0.2 * torch.randn(d)
    slot, pos = [1, 1, 0, 0, 2, 2], [14, 15, 0, 31, 32, 95]               # the temperature steps at p + 1 = 16, 32, ..
    k_off, v_off = 128, 128 + G * L * dp
    arenas, base = _arenas(3, v_off + G * L * ep, dev, 9.0)
    dv = [t.to(dev) for t in (part, wq, wk)]
    sd, pd = _i32(slot, dev), _i32(pos, dev)
    qo = torch.empty(S, H * dp, dtype=torch.bfloat16, device=dev)
    a = _lib.GqaInput(partial=_p(dv[0]), nsplit=ns, rows=S, ldn=part.shape[-1], heads=H, kv_heads=G, dim=d, dim_pad=dp, vdim_pad=ep, eps=eps, q_norm=_p(dv[1]),
                      k_norm=_p(dv[2]), temp_coef=coef, temp_every=every, q=_p(qo), tok_stream=_p(sd), tok_pos=_p(pd), kv_base=_p(base), k_off=k_off, v_off=v_off, lmax=L)
    _ok(lib.lcc_mixer_prep(C.byref(a), None, _st()))
    qs, ks, vs = q.double().sum(0), k.double().sum(0), v.double().sum(0)
    temp = R.query_temperature(torch.tensor(pos, dtype=torch.float64), coef, every)
    assert temp[0] == 1 and temp[1] > 1.4
    assert _near(qo.view(S, H, dp)[:, :, :d], R.over_rms(qs, eps) * wq[:d].double() * temp[:, None, None], absolute=1e-5) and qo.view(S, H, dp)[:, :, d:].abs().sum() == 0
    K = [t[k_off:k_off + G * L * dp].view(G, L, dp).cpu() for t in arenas]
    V = [t[v_off:].view(G, L // 32, ep, 32).permute(0, 1, 3, 2).reshape(G, L, ep).cpu() for t in arenas]
    kw = R.over_rms(ks, eps) * wk[:d].double()
    for i, (s, p) in enumerate(zip(slot, pos)):
        assert _near(K[s][:, p, :d], kw[i], absolute=1e-5) and K[s][:, p, d:].abs().sum() == 0
        assert _near(V[s][:, p, :e], vs[i]) and V[s][:, p, e:].abs().sum() == 0
    for s in range(3):
        keep = [p for p in range(L) if (s, p) not in set(zip(slot, pos))]
        assert (K[s][:, keep] == 9).all() and (V[s][:, keep] == 9).all() and (arenas[s][:k_off] == 9).all()


def _kv_slots(lens, G, d, e, L, dev, g):
    """Random keys and values of every slot, in the arena's layout; returns (k [G, L, d], v [G, L, e]) per slot, arenas, base, offsets."""
    k_off, v_off = 64, 64 + G * L * d
    kv, arenas = [], []
    for _ in lens:
        k, v = torch.randn(G, L, d, generator=g).bfloat16(), torch.randn(G, L, e, generator=g).bfloat16()
        kv.append((k, v))
        vt = v.view(G, L // 32, 32, e).permute(0, 1, 3, 2).reshape(-1)
        arenas.append(torch.cat([torch.zeros(64).bfloat16(), k.reshape(-1), vt]).to(dev))
    base = torch.tensor([a.data_ptr() for a in arenas], dtype=torch.int64, device=dev)
    return kv, arenas, base, k_off, v_off


SLOPES_LOG2 = 1.4426950408889634


@pytest.mark.parametrize("dim,vdim,heads,kv,new,past", [(64, 64, 4, 2, [1, 31, 32, 33], [0, 0, 0, 0]), (128, 128, 6, 1, [257, 40], [0, 70]), (64, 128, 2, 2, [513], [5]),
                                                        (128, 64, 3, 1, [64, 2, 255], [256, 31, 0]), (192, 64, 4, 2, [40, 3], [0, 300]), (64, 256, 2, 1, [300], [1])])
def test_biased_attention_of_packed_streams(dev, lib, dim, vdim, heads, kv, new, past):
    g = torch.Generator().manual_seed(dim + vdim)
    S, L = sum(new), -(-max(n + p for n, p in zip(new, past)) // 64) * 64
    kvs, arenas, base, k_off, v_off = _kv_slots(new, kv, dim, vdim, L, dev, g)
    q = torch.randn(S, heads, dim, generator=g).bfloat16()
    row, grp = 0, []
    for s, (n, p) in enumerate(zip(new, past)):
        grp += [(row + i, min(256, n - i), p + i, s) for i in range(0, n, 256)]
        # single keys that decide a row in spite of the distance: the first, one at a tile border, its own
        for i, j in ((n - 1, 0), (n // 2, min(31, p + n // 2)), (max(0, n - 2), p + max(0, n - 2))):
            for h in range(heads):
                q[row + i, h] = (kvs[s][0][h // (heads // kv), j].float() * 12).bfloat16()
        row += n
    slope = R.head_slopes(heads)
    qd, sl = q.to(dev), (slope * SLOPES_LOG2).float().to(dev)
    out = torch.full((S, heads * vdim), 7.0, dtype=torch.bfloat16, device=dev)
    tabs = [_i32([x[i] for x in grp], dev) for i in range(4)]
    scale = 4.0 / dim
    _ok(lib.lcc_gqa_attn_prefill(_p(qd), _p(out), *[_p(t) for t in tabs], len(grp), S, heads, kv, dim, vdim, scale, _p(sl), _p(base), k_off, v_off, L, _st()))
    got, row = out.view(S, heads, vdim).double().cpu(), 0
    for s, (n, p) in enumerate(zip(new, past)):
        full = torch.cat([torch.zeros(p, heads, dim).double(), q[row:row + n].double()])
        k, v = (t[:, :p + n].permute(1, 0, 2).double() for t in kvs[s])
        want = R.biased_attention(full, k, v, scale, slope)[p:]
        assert (got[row:row + n] - want).abs().max() < 0.03, (s, n, p)
        row += n


@pytest.mark.parametrize("dim,vdim,heads,kv,lens,ns", [(64, 64, 6, 1, [1, 2, 31, 32, 33, 64, 65], 2), (128, 128, 12, 2, [700], 11), (128, 64, 34, 2, [64] * 18, 1),
                                                       (192, 256, 3, 3, [200, 10], 4), (256, 128, 2, 1, [65], 64), (256, 256, 4, 2, [500, 1, 63], 3), (64, 192, 5, 5, [97], 3)])
def test_biased_decode_attention(dev, lib, dim, vdim, heads, kv, lens, ns):
    g = torch.Generator().manual_seed(dim * 3 + vdim)
    B, L = len(lens), -(-max(lens) // 64) * 64
    kvs, arenas, base, k_off, v_off = _kv_slots(lens, kv, dim, vdim, L, dev, g)
    order = list(range(B))[::-1]                                        # row b uses slot B - 1 - b
    q = torch.randn(B, heads, dim, generator=g).bfloat16()
    for b, s in enumerate(order):
        for h, j in zip(range(min(3, heads)), (0, min(31, lens[s] - 1), lens[s] - 1)):
            q[b, h] = (kvs[s][0][h // (heads // kv), j].float() * 12).bfloat16()
    slope = R.head_slopes(heads)
    n1, qd, sd, sl = _i32([n - 1 for n in lens], dev), q.to(dev), _i32(order, dev), (slope * SLOPES_LOG2).float().to(dev)
    wo, wm = torch.full((B * heads * ns * vdim,), float("nan"), device=dev), torch.full((B * heads * ns * 2,), float("nan"), device=dev)
    out = torch.zeros(B, heads * vdim, dtype=torch.bfloat16, device=dev)
    scale = 4.0 / dim
    _ok(lib.lcc_gqa_attn_decode(_p(qd), _p(sd), _p(n1), B, heads, kv, dim, vdim, scale, _p(sl), _p(base), k_off, v_off, L, ns, _p(wo), _p(wm), _p(out), _st()))
    for b, s in enumerate(order):
        n = lens[s]
        full = torch.cat([torch.zeros(n - 1, heads, dim).double(), q[b:b + 1].double()])
        k, v = (t[:, :n].permute(1, 0, 2).double() for t in kvs[s])
        want = R.biased_attention(full, k, v, scale, slope)[-1]
        assert (out[b].view(heads, vdim).double().cpu() - want).abs().max() < 0.03, (b, n)


# ---- recurrence ----
def _rec_tables(lens, seg, fresh, slots, dev):
    r, n, s, f, s0, ns, row = [], [], [], [], [], [], 0
    for b, L in enumerate(lens):
        s0.append(len(r))
        for i in range(0, L, seg):
            r.append(row + i), n.append(min(seg, L - i)), s.append(slots[b]), f.append(int(fresh[b] and i == 0))
        ns.append(len(r) - s0[-1])
        row += L
    return [_i32(x, dev) for x in (r, n, s, f)], len(r), [_i32(x, dev) for x in (s0, ns)]


@pytest.mark.parametrize("n,e,heads,groups,lens,seg", [(24, 40, 3, 3, [1, 2, 63, 64, 65, 130], 1000), (64, 64, 4, 1, [300], 128), (100, 130, 2, 2, [200, 5, 129], 64),
                                                       (130, 64, 6, 3, [70, 64], 1000), (256, 20, 2, 1, [190], 64), (128, 128, 2, 2, [700], 256)])
def test_chunked_recurrence(dev, lib, n, e, heads, groups, lens, seg):
    """Against the token-by-token recurrence: unequal streams, fresh and carried states, segments; head 0 hardly decays and the first key of every
    stream stands out, so a state that is lost or scaled anywhere shows in the last rows."""
    g = torch.Generator().manual_seed(n + e)
    np_, ep, S = _up(n), _up(e), sum(lens)
    q, k, v = (torch.randn(S, h, d, generator=g).bfloat16() for h, d in ((groups, n), (groups, n), (heads, e)))
    dt = torch.rand(S, heads, generator=g) * 0.5 + 0.05
    rate = -torch.rand(heads, generator=g) * 3
    rate[0] = -1e-4
    skip = torch.randn(heads, generator=g)
    row = 0
    for L in lens:
        v[row] = v[row] * 8
        row += L
    slots, fresh = list(range(len(lens)))[::-1], [b % 2 == 0 for b in range(len(lens))]
    off = 128
    arenas, base = _arenas(len(lens), off + 2 * heads * np_ * ep, dev, 3.0)
    state = [torch.randn(heads, n, e, generator=g) for _ in lens]
    for b, s in enumerate(slots):
        if not fresh[b]:
            t = torch.zeros(heads, np_, ep)
            t[:, :n, :e] = state[b]
            arenas[s][off:] = t.reshape(-1).view(torch.bfloat16).to(dev)
    dv = [_heads(q, np_).to(dev), _heads(k, np_).to(dev), _heads(v, ep).to(dev), dt.to(dev), rate.to(dev), skip.to(dev)]
    y = torch.full((S, heads * ep), float("nan"), device=dev)
    (tabs, n_seg, strs) = _rec_tables(lens, seg, fresh, slots, dev)
    ss, sd = torch.full((n_seg * heads * np_ * ep,), float("nan"), device=dev), torch.full((n_seg * heads,), float("nan"), device=dev)
    _ok(lib.lcc_rec_scan(*[_p(t) for t in dv], _p(y), heads, groups, np_, ep, *[_p(t) for t in tabs], n_seg, *[_p(t) for t in strs], len(lens), _p(ss), _p(sd),
                         _p(base), off, _st()))
    row, share = 0, torch.arange(heads) // (heads // groups)
    for b, L in enumerate(lens):
        sl = slice(row, row + L)
        decay = torch.exp2(rate.double() * dt[sl].double())
        want, S1 = R.decayed_outer_products(q[sl].double()[:, share], k[sl].double()[:, share], v[sl].double(), decay, dt[sl].double(),
                                            None if fresh[b] else state[b].double())
        want = want + skip.double()[:, None] * v[sl].double()
        got = y[sl].view(L, heads, ep).cpu().double()
        # probabilities go through bf16 inside a chunk, nothing else does
        assert (got[:, :, :e] - want).abs().max() < 4e-3 * want.abs().max() and (got[:, :, e:] == 0).all(), (b, L)
        end = arenas[slots[b]][off:].cpu().view(torch.float32).view(heads, np_, ep).double()
        assert (end[:, :n, :e] - S1).abs().max() < 2e-5 * S1.abs().max() + 1e-6, (b, L)      # the state itself is 32-bit
        row += L


def _rec_input(part, S, ldn, cfg, dv, **kw):
    from livecc_amd import _lib
    return _lib.RecInput(partial=_p(part), nsplit=part.shape[0], rows=S, ldn=ldn, **cfg, **{k: _p(t) for k, t in dv.items()}, **kw)


@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_short_convolution_across_portions_and_decoded_tokens(dev, lib, taps):
    """One stream in portions of 1, 2, 9, 3 rows, then token by token; the inputs of earlier calls come out of the slot."""
    H, G, n, e, ns = 2, 1, 24, 40, 2
    np_, ep = 64, 64
    hv, gk = H * ep, G * np_
    ch, ldn = hv + 2 * gk, hv + hv + 2 * gk + 64
    total = 22
    u = torch.randn(ns, total, ch)
    mask = torch.cat([_heads(torch.ones(H, e), ep), _heads(torch.ones(G, n), np_), _heads(torch.ones(G, n), np_)])
    u = u * mask
    dtc = torch.randn(ns, total, H)
    part = torch.cat([torch.randn(ns, total, hv), u, dtc, torch.zeros(ns, total, 64 - H)], -1)
    w, b = (torch.randn(taps, ch) * mask).bfloat16(), (torch.randn(ch) * mask).bfloat16()
    dtb, rate, skip = torch.tensor([-0.5, 30.0]), torch.tensor([-0.2, -0.01]), torch.randn(H)
    conv_off = 128
    state_off = conv_off + 2 * taps * ch
    arenas, base = _arenas(1, state_off + 2 * H * np_ * ep, dev, 5.0)         # garbage: positions before the start must not be read
    want = R.silu(R.causal_conv(u.double().sum(0), w.double().T, b.double()))
    dts = torch.nn.functional.softplus(dtc.double().sum(0) + dtb.double(), threshold=1e9)
    cfg = dict(q_col=2 * hv + gk, k_col=2 * hv, v_col=hv, dt_col=2 * hv + 2 * gk, heads=H, groups=G, key_pad=np_, vdim_pad=ep, taps=taps, conv_col=hv, conv_ch=ch,
               state_off=state_off, conv_off=conv_off)
    const = {k: t.to(dev) for k, t in dict(conv_w=w, conv_b=b, rate=rate, dt_bias=dtb, skip=skip).items()}
    S_ref = torch.zeros(H, n, e, dtype=torch.float64)
    at = 0
    for L in (1, 2, 9, 3):
        p = part[:, at:at + L].contiguous().to(dev)
        t = dict(tok_stream=_i32([0] * L, dev), tok_pos=_i32(range(at, at + L), dev), tok_row0=_i32([0] * L, dev), tok_last=_i32([L - 1] * L, dev), kv_base=base,
                 q=torch.empty(L, gk, dtype=torch.bfloat16, device=dev), k=torch.empty(L, gk, dtype=torch.bfloat16, device=dev),
                 v=torch.empty(L, hv, dtype=torch.bfloat16, device=dev), dt=torch.empty(L, H, device=dev))
        a = _rec_input(p, L, ldn, cfg, {**const, **t})
        _ok(lib.lcc_mixer_prep(None, C.byref(a), _st()))
        x = want[at:at + L]
        assert _near(t["v"], x[:, :hv]) and _near(t["k"], x[:, hv:hv + gk]) and _near(t["q"], x[:, hv + gk:]), (at, L)
        assert (t["dt"].cpu().double() - dts[at:at + L]).abs().max() < 1e-5
        (tabs, n_seg, strs) = _rec_tables([L], 1000, [at == 0], [0], dev)
        y = torch.empty(L, hv, device=dev)
        _ok(lib.lcc_rec_scan(_p(t["q"]), _p(t["k"]), _p(t["v"]), _p(t["dt"]), _p(const["rate"]), _p(const["skip"]), _p(y), H, G, np_, ep, *[_p(z) for z in tabs], n_seg,
                             *[_p(z) for z in strs], 1, None, None, _p(base), state_off, _st()))
        out = torch.empty(L, _up(H * e), dtype=torch.bfloat16, device=dev)
        wn = torch.ones(H * e).bfloat16().to(dev)
        _ok(lib.lcc_rec_norm(_p(y), _p(p), ns, L, ldn, 0, 1, H, e, ep, 1, 1e-5, _p(wn), _p(out), out.shape[1], C.byref(a), _st()))
        at += L
    ref = lambda lo, hi, S0: R.decayed_outer_products(want[lo:hi, hv + gk:hv + gk + n][:, None].expand(-1, H, -1), want[lo:hi, hv:hv + n][:, None].expand(-1, H, -1),
                                                      want[lo:hi, :hv].view(-1, H, ep)[:, :, :e], torch.exp2(rate.double() * dts[lo:hi]), dts[lo:hi], S0)
    _, S_ref = ref(0, at, None)
    kv, done = _i32([at], dev), _i32([0], dev)
    slot0 = _i32([0], dev)
    for t in range(at, total):
        for frozen in (1, 0):                        # a frozen slot's step leaves its state as it is
            done.fill_(frozen)
            kv.fill_(t)
            p = part[:, t:t + 1].contiguous().to(dev)
            a = _rec_input(p, 1, ldn, cfg, dict(const, tok_stream=slot0, kv_len=kv, done=done, kv_base=base))
            y = torch.empty(1, hv, device=dev)
            _ok(lib.lcc_rec_decode(C.byref(a), None, _p(y), _st()))
        o, S_ref = ref(t, t + 1, S_ref)
        o = o + skip.double()[:, None] * want[t:t + 1, :hv].view(-1, H, ep)[:, :, :e]
        assert (y.cpu().double().view(1, H, ep)[:, :, :e] - o).abs().max() < 0.01 * o.abs().max() + 1e-3, t


@pytest.mark.parametrize("n,e,heads,rows", [(24, 40, 3, 1), (64, 64, 2, 19), (130, 100, 2, 3), (256, 130, 1, 2)])
def test_state_step_of_linear_attention(dev, lib, n, e, heads, rows):
    """Fixed decays (also 0 and 1), rows in other slots' order, an empty slot whose arena still holds another stream's state."""
    np_, ep, ns = _up(n), _up(e), 2
    q, k, v = (torch.randn(ns, rows, heads, d) for d in (n, n, e))
    part = torch.cat([torch.randn(ns, rows, 64), _heads(q, np_), _heads(k, np_), _heads(v, ep)], -1)
    decay = torch.tensor([1.0, 0.0, 0.7][:heads], dtype=torch.float64)
    rate = torch.log2(decay.clamp_min(2.0 ** -1000)).float().to(dev)
    arenas, base = _arenas(rows, 128 + 2 * heads * np_ * ep, dev, 2.0)
    order = list(range(rows))[::-1]
    kv = [0 if s == rows - 1 else 5 + s for s in range(rows)]
    state = [torch.randn(heads, n, e) for _ in range(rows)]
    for s in range(rows):
        t = torch.zeros(heads, np_, ep)
        t[:, :n, :e] = state[s]
        arenas[s][128:] = t.reshape(-1).view(torch.bfloat16).to(dev)
    pd = part.to(dev)
    y = torch.empty(rows, heads * ep, device=dev)
    sd, kd = _i32(order, dev), _i32(kv, dev)
    a = _rec_input(pd, rows, part.shape[-1], dict(q_col=64, k_col=64 + heads * np_, v_col=64 + 2 * heads * np_, dt_col=-1, heads=heads, groups=heads, key_pad=np_,
                                                  vdim_pad=ep, taps=0, conv_col=0, conv_ch=0, state_off=128, conv_off=0),
                   dict(rate=rate, tok_stream=sd, kv_len=kd, kv_base=base))
    _ok(lib.lcc_rec_decode(C.byref(a), None, _p(y), _st()))
    qs, ks, vs = (R.silu(t.double().sum(0)) for t in (q, k, v))
    for b, s in enumerate(order):
        S0 = torch.zeros(heads, n, e, dtype=torch.float64) if kv[s] == 0 else state[s].double()
        o, S1 = R.decayed_outer_products(qs[b:b + 1], ks[b:b + 1], vs[b:b + 1], decay[None], torch.ones(1, heads, dtype=torch.float64), S0)
        assert (y[b].view(heads, ep)[:, :e].cpu().double() - o[0]).abs().max() < 1e-5 * o.abs().max() + 1e-5
        end = arenas[s][128:].cpu().view(torch.float32).view(heads, np_, ep).double()
        assert (end[:, :n, :e] - S1).abs().max() < 1e-5 * S1.abs().max() + 1e-6


@pytest.mark.parametrize("gate_first", [0, 1])
@pytest.mark.parametrize("heads,vdim,groups,rows", [(4, 64, 2, 3), (6, 20, 4, 5), (5, 13, 1, 2), (9, 128, 9, 1), (3, 24, 3, 70)])
def test_gated_group_norm(dev, lib, heads, vdim, groups, rows, gate_first):
    ep, ns, eps, inner = _up(vdim), 2, 2e-2, heads * vdim
    y, gate = torch.randn(rows, heads, vdim) * 3, torch.randn(ns, rows, heads, vdim) * 2
    part = torch.cat([torch.randn(ns, rows, 64), _heads(gate, ep)], -1).to(dev)
    w = torch.randn(inner).bfloat16()
    yd, wd, ld = _heads(y, ep).to(dev), w.to(dev), _up(inner) + 64
    out = torch.full((rows, ld), 7.0, dtype=torch.bfloat16, device=dev)
    _ok(lib.lcc_rec_norm(_p(yd), _p(part), ns, rows, part.shape[-1], 64, gate_first, heads, vdim, ep, groups, eps, _p(wd), _p(out), ld, None, _st()))
    z = gate.double().sum(0).reshape(rows, inner)
    x = y.double().reshape(rows, inner) * (R.silu(z) if gate_first else 1.0)
    want = R.over_rms(x.view(rows, groups, -1), eps).reshape(rows, inner) * w.double() * (1.0 if gate_first else torch.sigmoid(z))
    assert _near(out[:, :inner], want, absolute=1e-5) and out[:, inner:].abs().sum() == 0


# --------------------------------------------------------------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------------------------------------------------------------
N_LONG = 330


@pytest.fixture(scope="module", params=sorted(U.configs()))
def case(request, dev):
    cfg = U.configs()[request.param]
    T = U.make_weights(cfg, 3)
    ids = U.ids_of(cfg, N_LONG, 11)
    taps = []
    want = U.oracle_logits(cfg, T, ids, taps=taps)
    return dict(cfg=cfg, T=T, ids=ids, want=want, taps=taps, model=_model(cfg, T, dev))


def _run(model, ids, portions, want=None):
    """Logits of every position (or of the wanted ones) of one stream fed in portions of the given sizes."""
    st, at, out = model.new_stream(), 0, []
    for n in portions:
        places = [i for i in range(n) if want is None or at + i in want]
        out.append(model.forward_step([(st, ids[at:at + n], places)])[0])
        at += n
    assert at == len(ids) and st.get_seq_length() == at
    st.release()
    return torch.cat(out).cpu()


def test_every_position_of_a_prompt(case):
    e = U.error(_run(case["model"], case["ids"], [N_LONG]), case["want"])
    print(f"{case['cfg'].name}: worst row {e:.4f} of the logits' rms")
    assert e < U.LIMIT


def test_residual_after_every_layer(case):
    m, n = case["model"], 37
    taps = m.engine.set_llm_taps(64)
    try:
        st = m.new_stream()
        m.forward_step([(st, case["ids"][:n - 1], [])])
        torch.cuda.synchronize()
        pre = taps[1:, :n - 1, :case["cfg"].hidden_size].clone()
        m.forward_step([(st, case["ids"][n - 1:n], [])])
        torch.cuda.synchronize()
        dec = taps[1:, 0, :case["cfg"].hidden_size].clone()
        st.release()
    finally:
        m.engine.set_llm_taps(0)
    for i, x in enumerate(case["taps"]):
        scale = x[:n].pow(2).mean().sqrt()
        assert (pre[i].double().cpu() - x[:n - 1]).pow(2).mean().sqrt() < 0.015 * scale, i
        assert (dec[i].double().cpu() - x[n - 1]).pow(2).mean().sqrt() < 0.02 * scale, i


def test_token_by_token_from_the_first_one(case):
    n = 150          # over the 64- and 128-token borders
    got = _run(case["model"], case["ids"][:n], [1] * n)
    assert U.error(got, case["want"][:n]) < U.LIMIT


@pytest.mark.parametrize("portions", [[2] * 20 + [290], [31, 33, 64, 2, 200], [300, 1, 2, 1, 26], [1, 255, 2, 72], [7] * 47 + [1]])
def test_portions_of_several_sizes(case, portions):
    got = _run(case["model"], case["ids"], portions)
    assert U.error(got, case["want"]) < U.LIMIT


def test_a_prompt_longer_than_one_launch_sequence(case, dev):
    m = _model(case["cfg"], case["T"], dev, max_new_rows=100, max_streams=2)
    want = {0, 1, 98, 99, 100, 101, 199, 200, 329}
    got = _run(m, case["ids"], [N_LONG], want)
    assert U.error(got, case["want"][sorted(want)]) < U.LIMIT
    a, b = m.new_stream(), m.new_stream()
    la, lb = m.forward_step([(a, case["ids"][:90], [0, 89]), (b, case["ids"][:230], [229, 3])])
    assert U.error(la, case["want"][[0, 89]]) < U.LIMIT and U.error(lb, case["want"][[229, 3]]) < U.LIMIT


def test_unequal_requests_in_one_batch_equal_each_alone(case):
    m, ids, want = case["model"], case["ids"], case["want"]
    lens = [1, 97, 260, 32, 2]
    streams = [m.new_stream() for _ in lens]
    got = m.forward_step([(s, ids[:n], [n - 1, 0]) for s, n in zip(streams, lens)])
    for n, lg in zip(lens, got):
        assert U.error(lg, want[[n - 1, 0]]) < U.LIMIT, n
    live = list(range(len(lens)))
    for step in range(40):                       # decoded together; the shorter requests end earlier
        if step in (3, 20, 35):
            streams[live.pop()].release()
        got = m.forward_step([(streams[i], [ids[lens[i] + step]], [0]) for i in live])
        for i, lg in zip(live, got):
            assert U.error(lg, want[[lens[i] + step]]) < U.LIMIT, (i, step)
    for i in live:
        streams[i].release()


def test_slots_are_clean_when_they_are_used_again(case):
    m, ids = case["model"], case["ids"]
    first = m.new_stream()
    slot = first.slot
    m.forward_step([(first, ids, [])])                    # fills the arena, the states and the previous token
    first.release()
    for cut in (40, 1, 2):
        st = m.new_stream()
        assert st.slot == slot
        other = U.ids_of(case["cfg"], cut + 30, 5 + cut)
        want = U.oracle_logits(case["cfg"], case["T"], other)
        got = m.forward_step([(st, other[:cut], list(range(cut)))])[0]
        assert U.error(got, want[:cut]) < U.LIMIT
        for j in range(cut, cut + 30):
            got = m.forward_step([(st, [other[j]], [0])])[0]
            assert U.error(got, want[[j]]) < U.LIMIT, j
        st.release()


def test_mixed_steps_of_prompts_and_decoded_tokens(case):
    m, ids, want = case["model"], case["ids"], case["want"]
    a, b, c = m.new_stream(), m.new_stream(), m.new_stream()
    m.forward_step([(a, ids[:50], [])])
    la, lb, lc = m.forward_step([(a, [ids[50]], [0]), (b, ids[:65], [64]), (c, [ids[0]], [0])])
    assert U.error(la, want[[50]]) < U.LIMIT and U.error(lb, want[[64]]) < U.LIMIT and U.error(lc, want[[0]]) < U.LIMIT
    la, lb, lc = m.forward_step([(a, ids[51:53], [1]), (b, [ids[65]], [0]), (c, [ids[1]], [0])])
    assert U.error(la, want[[52]]) < U.LIMIT and U.error(lb, want[[65]]) < U.LIMIT and U.error(lc, want[[1]]) < U.LIMIT
    for s in (a, b, c):
        s.release()


def test_the_comparison_would_show_a_fault_of_any_mechanism(case):
    """Mistakes planted in the oracle: the engine's logits are far from each of them."""
    from livecc_amd.config import ParallelMixerSpec
    cfg, T, n = case["cfg"], case["T"], 200
    got = _run(case["model"], case["ids"][:n], [n])
    raw = cfg.to_dict()

    def faulty(patch=None, scale=None, config=None):
        saved = {k: getattr(R, k) for k in (patch or {})}
        tensors = {k: (v * scale[1] if k.endswith(scale[0]) else v) for k, v in T.items()} if scale else T
        try:
            for k, f in (patch or {}).items():
                setattr(R, k, f)
            return R.run(config or raw, tensors, case["ids"][:n])
        finally:
            for k, f in saved.items():
                setattr(R, k, f)

    rec, conv = R.decayed_outer_products, R.causal_conv

    def state_lost(q, k, v, decay, weight, state=None):
        decay = decay.clone()
        decay[64] = 0
        return rec(q, k, v, decay, weight, state)
    big = json.loads(json.dumps(raw))
    big["embedding"]["bigram"]["mul_prev"] += 1
    faults = {"state lost at a chunk border": faulty({"decayed_outer_products": state_lost}),
              "no step sizes": faulty({"decayed_outer_products": lambda q, k, v, d, w, s=None: rec(q, k, v, d, torch.ones_like(w), s)}),
              "no distance bias": faulty({"head_slopes": lambda h: torch.zeros(h, dtype=torch.float64)}),
              "slopes of the next head": faulty({"head_slopes": lambda h: torch.tensor([2.0 ** (-8.0 * (i + 2) / h) for i in range(h)], dtype=torch.float64)}),
              "no query norm weight": faulty(scale=("left.q.norm", 0.6)), "no output gate": faulty(scale=("right.g", 0.0)),
              "other bigram rows": faulty(config=big), "no bigram rows": faulty(scale=("bigram", 0.0)),
              "no feed-forward": faulty({"silu": R.silu, "gated_mlp": lambda h, g, u, d: (h * 0) @ torch.zeros(h.shape[1], h.shape[1], dtype=h.dtype)}),
              "plain weights": faulty({"norm_around_one": lambda x, w, eps: R.over_rms(x, eps) * w}),
              "left output alone": faulty(scale=("right.out", 0.0)), "scale": faulty(config={**raw, "logit_scale": raw["logit_scale"] * 1.1})}
    if any(not isinstance(l.mixer, ParallelMixerSpec) and l.mixer.conv_taps > 1 for l in cfg.layers):
        faults["convolution one token late"] = faulty({"causal_conv": lambda u, w, b: torch.cat([conv(u, w, b)[:1], conv(u, w, b)[:-1]])})
        faults["no skip"] = faulty(scale=("mix.D", 0.0))
    if cfg.name != "wide-heads":                       # (one layer of it has a coefficient of 0, the other a small one)
        faults["no query temperature"] = faulty({"query_temperature": lambda p, c, e: torch.ones_like(p)})
    seen = {name: U.error(got, want) for name, want in faults.items()}
    if cfg.bigram_buckets == 1:
        seen.pop("other bigram rows")                  # one row for every pair
    print({k: round(v, 3) for k, v in seen.items()})
    for name, e in seen.items():
        assert e > 2.0 * U.LIMIT, (name, e)      # the smallest: a scale that is 10 % off


def test_far_tokens_reach_the_last_row(dev):
    """A changed first token shows in the last logits of the engine as in the oracle's, in prompts and in decoding."""
    cfg = U.configs()["even"]
    T = U.make_weights(cfg, 9)
    # slow decays, and step sizes that are large for a first token (which alone has the last bigram row) and small for all others
    T["bigram"][-1] *= 2
    u = T["bigram"][-1].float()
    for i, l in enumerate(cfg.layers):
        p = f"l{i}.mix."
        if p + "A_log" in T:
            T[p + "A_log"][:], T[p + "dt_bias"][:] = -9.0, -12.0
            T[p + "in"][-l.mixer.heads:] = (3.0 * u / u.norm()).bfloat16()
    m = _model(cfg, T, dev)
    a = U.ids_of(cfg, 200, 4)
    b = [(a[0] + 1) % cfg.vocab_size] + a[1:]
    la, lb = U.oracle_logits(cfg, T, a)[-1:], U.oracle_logits(cfg, T, b)[-1:]
    away = U.error(lb, la)
    assert away > 2 * U.LIMIT, away
    for portions in ([200], [64, 64, 72], [100] + [1] * 100):
        ga, gb = (_run(m, x, portions, {199}) for x in (a, b))
        assert U.error(ga, la) < U.LIMIT and U.error(gb, lb) < U.LIMIT and abs(U.error(gb, ga.double()) - away) < U.LIMIT


# ---- generation through the model's entry points ----
def _greedy(cfg, T, prompt, steps):
    """(ids, smallest lead of the chosen id) of greedy decoding with the oracle."""
    ids, lead = list(prompt), 1e9
    for _ in range(steps):
        z = U.oracle_logits(cfg, T, ids)[-1]
        top = z.topk(2)
        lead = min(lead, ((top.values[0] - top.values[1]) / z.pow(2).mean().sqrt()).item())
        ids.append(int(top.indices[0]))
    return ids[len(prompt):], lead


def _clear_prompts(cfg, T, sizes, steps):
    """Prompts whose greedy continuation is decided by more than rounding."""
    out, seed = [], 100
    for n in sizes:
        while True:
            p = U.ids_of(cfg, n, seed)
            seed += 1
            toks, lead = _greedy(cfg, T, p, steps)
            if lead > 3 * U.LIMIT:
                out.append((p, toks))
                break
            assert seed < 400
    return out


@pytest.mark.parametrize("name", ["mixed", "wide-heads"])
def test_greedy_generation_alone_in_a_batch_and_continued(dev, name):
    cfg = U.configs()[name]
    T = U.make_weights(cfg, 8)
    m = _model(cfg, T, dev)
    steps = 6
    cases = _clear_prompts(cfg, T, [3, 40, 33, 1], steps)
    for p, toks in cases:
        r = m.generate(torch.tensor([p]), max_new_tokens=steps)
        assert r.sequences[0, len(p):].tolist() == toks
        r.past_key_values.release()
    outs = m.generate_batch([dict(input_ids=np.asarray(p)) for p, _ in cases], max_new_tokens=steps, output_logits=True)
    for (p, toks), r in zip(cases, outs):
        assert r.sequences[0, len(p):].tolist() == toks and r.logits.dtype == torch.float32 and r.logits.shape == (steps, cfg.vocab_size)
        want = U.oracle_logits(cfg, T, p + toks)[len(p) - 1:-1]
        assert U.error(r.logits, want) < U.LIMIT
        r.past_key_values.release()
    # a second call goes on from the cached sequence
    p, toks = cases[1]
    r = m.generate(torch.tensor([p]), max_new_tokens=3)
    r2 = m.generate(r.sequences.cpu(), past_key_values=r.past_key_values, max_new_tokens=3)
    assert r2.sequences[0, len(p):].tolist() == toks
    r2.past_key_values.release()
    # an EOS id ends a request early and freezes its state on the device; the others go on.  A later call goes on behind the EOS
    eos = cases[1][1][2]
    r = m.generate_batch([dict(input_ids=np.asarray(p)) for p, _ in cases], max_new_tokens=steps, eos_token_id=eos)
    for (p, toks), x in zip(cases, r):
        cut = toks.index(eos) + 1 if eos in toks else steps
        assert x.sequences[0, len(p):].tolist() == toks[:cut]
    p, toks = cases[1]
    seq = p + toks[:toks.index(eos) + 1]
    st = r[1].past_key_values
    got = m.forward_step([(st, seq[st.get_seq_length():] + [5, 6], [-1 + len(seq) - st.get_seq_length() + 2])])[0]
    assert U.error(got, U.oracle_logits(cfg, T, seq + [5, 6])[-1:]) < U.LIMIT


def test_sampling_arguments_reach_the_sampler(dev):
    cfg = U.configs()["mixed"]
    T = U.make_weights(cfg, 8)
    m = _model(cfg, T, dev)
    p = U.ids_of(cfg, 20, 1)
    z = U.oracle_logits(cfg, T, p)[-1]
    one = lambda **kw: m.generate(torch.tensor([p]), max_new_tokens=1, output_scores=True, **kw)
    r = one(do_sample=True, top_k=5, temperature=2.0, seed=3)
    assert r.sequences[0, -1].item() in set(z.topk(6).indices.tolist())
    assert int(torch.isfinite(r.scores).sum()) == 5 and r.scores.shape == (cfg.vocab_size,)
    picks = {one(do_sample=True, top_k=0, temperature=50.0, seed=k).sequences[0, -1].item() for k in range(12)}
    assert len(picks) > 6 and all(0 <= t < cfg.vocab_size for t in picks)          # ids of the padded vocabulary are never drawn


def test_many_streams_decode_in_groups(dev):
    """70 streams: one packed prefill, decode groups of 64 + 6, rows beyond the fused launches."""
    cfg = U.configs()["even"]
    T = U.make_weights(cfg, 2)
    m = _model(cfg, T, dev, max_streams=70, max_kv_len=160, max_new_rows=2048)
    seqs = [U.ids_of(cfg, 1 + (7 * i) % 40, 1000 + i) + U.ids_of(cfg, 3, i) for i in range(70)]
    wants = [U.oracle_logits(cfg, T, s) for s in seqs]
    st = [m.new_stream() for _ in seqs]
    got = m.forward_step([(s, x[:-3], [len(x) - 4]) for s, x in zip(st, seqs)])
    for g, w in zip(got, wants):
        assert U.error(g, w[[-4]]) < U.LIMIT
    for j in (3, 2, 1):
        got = m.forward_step([(s, [x[-j]], [0]) for s, x in zip(st, seqs)])
        for g, w in zip(got, wants):
            assert U.error(g, w[[-j]]) < U.LIMIT
    for n in (17, 33, 48):                       # other batch sizes of the unfused decode step, from the middle of the streams
        st2 = st[:n]
        got = m.forward_step([(s, [5], [0]) for s in st2])
        for k in range(n):
            seqs[k] = seqs[k] + [5]
        for k in (0, n - 1):
            assert U.error(got[k], U.oracle_logits(cfg, T, seqs[k])[[-1]]) < U.LIMIT


def test_fused_and_separate_decode_launches_agree(dev, lib):
    cfg = U.configs()["many-heads"]
    T = U.make_weights(cfg, 4)
    m = _model(cfg, T, dev)
    seqs = [U.ids_of(cfg, n, n) for n in (40, 90, 64)]
    res = []
    for fused in (1, 0):
        old = lib.lcc_debug_set_decoder_fused(fused)
        try:
            st = [m.new_stream() for _ in seqs]
            m.forward_step([(s, x[:-2], []) for s, x in zip(st, seqs)])
            m.forward_step([(s, [x[-2]], [0]) for s, x in zip(st, seqs)])
            res.append([g.clone() for g in m.forward_step([(s, [x[-1]], [0]) for s, x in zip(st, seqs)])])
            for s in st:
                s.release()
        finally:
            lib.lcc_debug_set_decoder_fused(old)
    for a, b, x in zip(*res, seqs):
        want = U.oracle_logits(cfg, T, x)[[-1]]
        assert U.error(a, want) < U.LIMIT and U.error(b, want) < U.LIMIT


def test_long_prompts_in_segments_and_long_decoding(dev):
    cfg = U.configs()["even"]
    T = U.make_weights(cfg, 6)
    m = _model(cfg, T, dev, max_kv_len=1500, max_new_rows=1300)
    ids = U.ids_of(cfg, 1050, 77)
    ref = U.oracle_logits(cfg, T, ids)
    at = sorted({40, 63, 64, 127, 128, 255, 256, 257, 511, 512, 700, 1023, 1024, 1049})
    assert U.error(_run(m, ids, [1050], set(at)), ref[at]) < U.LIMIT            # segments of the recurrence
    st, other = m.new_stream(), m.new_stream()                                  # a long and a short stream in one launch sequence
    a, b = m.forward_step([(st, ids[:1000], [999, 512]), (other, ids[:90], [89])])
    assert U.error(a, ref[[999, 512]]) < U.LIMIT and U.error(b, ref[[89]]) < U.LIMIT
    a, b = m.forward_step([(st, ids[1000:1030], [29]), (other, ids[90:900], [809, 0])])      # both carry a state in
    assert U.error(a, ref[[1029]]) < U.LIMIT and U.error(b, ref[[899, 90]]) < U.LIMIT
    st.release(), other.release()
    st = m.new_stream()
    m.forward_step([(st, ids[:30], [])])
    got = []
    for j in range(30, 1050):
        r = m.forward_step([(st, [ids[j]], [0] if j in at else [])])[0]
        if j in at:
            got.append(r.cpu())
    assert U.error(torch.cat(got), ref[at]) < U.LIMIT


def test_calls_the_engine_cannot_serve_are_errors(dev):
    from livecc_amd import _lib
    cfg = U.configs()["even"]
    m = _model(cfg, U.make_weights(cfg), dev, max_kv_len=128, max_new_rows=64, max_history=16, max_streams=2)
    st = m.new_stream()
    with pytest.raises(_lib.LccError, match="out of range"):
        m.forward_step([(st, [0, cfg.vocab_size], [])])
    with pytest.raises(_lib.LccError, match="capacity"):
        m.forward_step([(st, [1] * 120, [])])
    m.forward_step([(st, [1] * 9, [])])
    with pytest.raises(_lib.LccError, match="rolled back"):
        m.engine.set_slot_length(st.slot, 4, 4)


def test_command_line_and_trace_runner_from_a_checkpoint_directory(dev, tmp_path):
    from safetensors.torch import save_file
    cfg = U.configs()["mixed"]
    T = U.make_weights(cfg, 12)
    save_file({k: v.contiguous() for k, v in T.items()}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg.to_dict()))
    out = tmp_path / "out"
    out.mkdir()
    a, b = U.ids_of(cfg, 80, 1), U.ids_of(cfg, 33, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:78], "want": [77, 5]}, {"id": "y", "tokens": b[:32], "want": [31]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": [a[78]], "want": []}, {"id": "y", "tokens": [b[32]], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": [a[79]], "want": [0]}], "end": ["x"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(out), "--max-tokens", "113"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = U.oracle_logits(cfg, T, a), U.oracle_logits(cfg, T, b)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg.vocab_size))
    assert U.error(read(0), torch.stack([wa[77], wa[5], wb[31]])) < U.LIMIT
    assert U.error(read(1), wb[[32]]) < U.LIMIT and U.error(read(2), wa[[79]]) < U.LIMIT
    [(p, toks)] = _clear_prompts(cfg, T, [12], 4)
    r = subprocess.run([sys.executable, "-m", "livecc_amd", "generate", "--model", str(tmp_path), "--ids", ",".join(map(str, p)), "--max-new-tokens", "4"],
                       cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert json.loads(r.stdout.strip().splitlines()[-1])["generated"] == toks
