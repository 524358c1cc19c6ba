"""-m gpu: Debunex on the engine against the plain implementation of its equations (oracle/debunex_ref.py), mechanism by mechanism, then the
whole model: prompts, decoding, portions, batches, slots that are used again, and greedy generation through the model's entry points."""
import numpy as np
import pytest
import torch

from oracle import debunex_ref as R
from tests import debunex_util as U

pytestmark = pytest.mark.gpu


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


def _model(cfg, T, dev, **kw):
    from livecc_amd.modeling import DebunexForCausalLM
    a = dict(max_streams=6, max_kv_len=900, max_new_rows=700, max_history=48)
    a.update(kw)
    return DebunexForCausalLM(cfg, U.arena(cfg, T, dev), dev, **a)


# --------------------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# --------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("rows,dim,ns", [(1, 64, 1), (3, 192, 4), (70, 1024, 2)])
def test_residual_add_and_dynamic_tanh(dev, lib, rows, dim, ns):
    g = torch.Generator().manual_seed(rows)
    x, part = torch.randn(rows, dim, generator=g) * 3, torch.randn(ns, rows, dim, generator=g)
    w, b, al = (torch.randn(dim, generator=g).bfloat16(), torch.randn(dim, generator=g).bfloat16(), torch.tensor([0.37]).bfloat16())
    xd, pd, wd, bd, ad = x.to(dev), part.to(dev), w.to(dev), b.to(dev), al.to(dev)
    h = torch.empty(rows, dim, dtype=torch.bfloat16, device=dev)
    _ok(lib.lcc_resid_dyt(_p(xd), _p(pd), ns, _p(wd), _p(bd), _p(ad), _p(h), rows, dim, _st()))
    want = x.double() + part.double().sum(0)
    assert (xd.cpu().double() - want).abs().max() < 1e-5          # the residual stays fp32
    y = R.dynamic_tanh(want, al.double(), w.double(), b.double())
    assert ((h.cpu().double() - y).abs() <= y.abs() * 2 ** -8 + 1e-5).all()


def test_embedding_and_first_norm_by_row_and_by_slot(dev, lib):
    table = torch.randn(50, 128).bfloat16()
    w, b, al = torch.randn(128).bfloat16(), torch.randn(128).bfloat16(), torch.tensor([-0.8]).bfloat16()
    td, wd, bd, ad = table.to(dev), w.to(dev), b.to(dev), al.to(dev)
    x, h = torch.empty(3, 128, device=dev), torch.empty(3, 128, dtype=torch.bfloat16, device=dev)
    ids, ind = _i32([7, 49, 0, 12], dev), _i32([3, 1, 2], dev)
    for indirect, want in ((None, [7, 49, 0]), (ind, [12, 49, 0])):
        _ok(lib.lcc_embed_dyt(_p(ids), _p(indirect), _p(td), _p(wd), _p(bd), _p(ad), _p(x), _p(h), 3, 128, _st()))
        e = table[want].double()
        assert torch.equal(x.cpu().double(), e)
        y = R.dynamic_tanh(e, al.double(), w.double(), b.double())
        assert ((h.cpu().double() - y).abs() <= y.abs() * 2 ** -8 + 1e-5).all()


@pytest.mark.parametrize("cap", [0.0, 4.0])
def test_logit_cap_and_the_padded_ids(dev, lib, cap):
    part = torch.randn(3, 5, 128) * 4
    pd = part.to(dev)
    out, dense = torch.empty(5, 128, device=dev), torch.empty(5, 101, device=dev)
    _ok(lib.lcc_logits_cap(_p(pd), 3, 5, 128, 101, cap, _p(out), _p(dense), _st()))
    want = R.soft_cap(part.double().sum(0), cap)[:, :101]
    assert (dense.cpu().double() - want).abs().max() < 2e-5 and torch.equal(out.cpu()[:, :101], dense.cpu())
    assert torch.isinf(out.cpu()[:, 101:]).all() and (out.cpu()[:, 101:] < 0).all()


@pytest.mark.parametrize("q_rank,kv_rank,heads,own,ns", [(64, 64, 4, True, 1), (50, 100, 19, True, 3), (129, 300, 3, False, 2), (600, 513, 1, True, 1)])
def test_input_norms_cache_append_and_gates(dev, lib, q_rank, kv_rank, heads, own, ns):
    from livecc_amd.config import pad_kv_rank
    qp, rp, S, eps, off, L = -(-q_rank // 64) * 64, pad_kv_rank(kv_rank), 5, 2e-2, 128, 70
    ldn = qp + (rp if own else 0) + -(-heads // 16) * 16
    part = torch.randn(ns, S, ldn) * 0.3
    part[:, :, q_rank:qp] = 0
    if own:
        part[:, :, qp + kv_rank:qp + rp] = 0
    wq, wk = torch.zeros(qp).bfloat16(), torch.zeros(rp).bfloat16()
    wq[:q_rank], wk[:kv_rank] = 1 + 0.3 * torch.randn(q_rank), 1 + 0.3 * torch.randn(kv_rank)
    arenas = [torch.full((off + L * rp,), 9.0, dtype=torch.bfloat16, device=dev) for _ in range(3)]
    base = torch.tensor([a.data_ptr() for a in arenas], dtype=torch.int64, device=dev)
    slot, pos = [2, 0, 0, 1, 2], [69, 0, 1, 33, 5]
    pd, wqd, wkd, sd, td = part.to(dev), wq.to(dev), wk.to(dev), _i32(slot, dev), _i32(pos, dev)
    cq, gate = torch.empty(S, qp, dtype=torch.bfloat16, device=dev), torch.empty(S, heads, device=dev)
    _ok(lib.lcc_latent_norm_append(_p(pd), ns, S, ldn, q_rank, qp, _p(wqd), kv_rank, rp if own else 0, _p(wkd), heads, eps, _p(sd), _p(td), None, _p(base), off,
                                   _p(cq), _p(gate), _st()))
    z = part.double().sum(0)
    near = lambda got, want: ((got.double().cpu() - want).abs() <= want.abs() * 2 ** -8 + 1e-6).all()
    assert near(cq[:, :q_rank], R.rms_unit(z[:, :q_rank], eps) * wq[:q_rank].double()) and cq[:, q_rank:].abs().sum() == 0
    g0 = qp + (rp if own else 0)
    assert (gate.cpu().double() - torch.sigmoid(z[:, g0:g0 + heads])).abs().max() < 1e-6
    rows = [a[off:].view(L, rp) for a in arenas]
    if own:
        want = R.rms_unit(z[:, qp:qp + kv_rank], eps) * wk[:kv_rank].double()
        for i, (s, p) in enumerate(zip(slot, pos)):
            assert near(rows[s][p, :kv_rank], want[i]) and rows[s][p, kv_rank:].abs().sum() == 0
    touched = {(s, p) for s, p in zip(slot, pos)} if own else set()
    for s in range(3):
        keep = [p for p in range(L) if (s, p) not in touched]
        assert (rows[s][keep] == 9).all() and (arenas[s][:off] == 9).all()


def test_gathered_latents_are_zero_past_a_streams_keys(dev, lib):
    from livecc_amd.weights import pack_weight
    rp, lens = 128, [5, 33]
    arenas = [torch.randn(64 + 64 * rp, device=dev).bfloat16() for _ in lens]
    base = torch.tensor([a.data_ptr() for a in arenas], dtype=torch.int64, device=dev)
    ts, tk, tn, want = [], [], [], []
    for s, n in enumerate(lens):
        T = -(-n // 32) * 32
        w = arenas[s][64:].view(64, rp)[:T].clone()
        w[n:] = 0
        want.append(w)
        for k in range(0, T, 16):
            ts.append(s), tk.append(k), tn.append(n)
    rows, frag = (torch.empty(len(ts) * 16, rp, dtype=torch.bfloat16, device=dev) for _ in range(2))
    a, b, c = _i32(ts, dev), _i32(tk, dev), _i32(tn, dev)
    _ok(lib.lcc_latent_gather(_p(base), 64, rp, _p(a), _p(b), _p(c), len(ts), _p(rows), _p(frag), _st()))
    assert torch.equal(rows, torch.cat(want)) and torch.equal(frag, pack_weight(torch.cat(want)))


@pytest.mark.parametrize("dim,vdim,heads,new,past", [(64, 64, 2, [1, 31, 32, 33], [0, 0, 0, 0]), (128, 128, 3, [257, 40], [0, 70]), (64, 128, 1, [513], [5]),
                                                     (128, 64, 5, [64, 2, 255], [256, 31, 0]), (192, 64, 2, [40, 3], [0, 300]), (24, 200, 1, [300], [1])])
def test_multi_head_attention_of_packed_streams(dev, lib, dim, vdim, heads, new, past):
    g = torch.Generator().manual_seed(dim + vdim)
    S, T, row, grp, segs = sum(new), 0, 0, [], []
    for n, p in zip(new, past):
        grp += [(row + q, min(256, n - q), p + q, T) for q in range(0, n, 256)]
        segs.append((row, n, p, T))
        T, row = T + -(-(n + p) // 32) * 32, row + n
    q, k, v = (torch.randn(r, heads, d, generator=g).bfloat16() for r, d in ((S, dim), (T, dim), (T, vdim)))
    for r, n, p, t in segs:          # one query and one far key of every stream stand out: the first, the last before a border, its own
        for i, j in ((n - 1, 0), (n - 1 if n < 3 else n // 2, min(31, p)), (max(0, n - 2), p + max(0, n - 2))):
            q[r + i] = (k[t + j].float() * 3).bfloat16() if dim >= 64 else q[r + i]
    gate = torch.rand(S, heads, generator=g)
    qd, kd, vtd, gd = q.to(dev), k.to(dev), v.permute(1, 2, 0).reshape(heads * vdim, T).contiguous().to(dev), gate.to(dev)
    ldo = heads * vdim + 8
    out = torch.full((S, ldo), 7.0, dtype=torch.bfloat16, device=dev)
    tabs = [_i32([x[i] for x in grp], dev) for i in range(4)]
    _ok(lib.lcc_attn_mha(_p(qd), _p(kd), _p(vtd), T, _p(gd), _p(out), ldo, *[_p(t) for t in tabs], len(grp), S, heads, dim, vdim, 0.2, _st()))
    assert (out[:, heads * vdim:] == 7).all()
    got = out[:, :heads * vdim].view(S, heads, vdim).double().cpu()
    for r, n, p, t in segs:
        want = R.causal_softmax_attention(q[r:r + n].double(), k[t:t + p + n].double(), v[t:t + p + n].double(), 0.2, first=p) * gate[r:r + n, :, None].double()
        assert (got[r:r + n] - want).abs().max() < 0.03, (r, n, p)


@pytest.mark.parametrize("rank,heads,vdim,lens,ns", [(64, 3, 64, [1, 2, 63, 64, 65, 128, 129], 2), (128, 16, 64, [700], 11), (192, 17, 128, [64] * 18, 1),
                                                     (256, 70, 64, [200, 10], 4), (384, 5, 192, [65], 128), (512, 28, 128, [500, 1, 64], 3),
                                                     (768, 33, 64, [129], 2), (1024, 16, 64, [130, 3], 5)])
def test_latent_decode_attention(dev, lib, rank, heads, vdim, lens, ns):
    g = torch.Generator().manual_seed(rank)
    B, off = len(lens), 256
    L = -(-max(lens) // 64) * 64
    arenas = [torch.randn(off + L * rank, generator=g).bfloat16().to(dev) for _ in lens]
    order = list(range(B))[::-1]                                     # row b uses slot B - 1 - b
    base = torch.tensor([arenas[s].data_ptr() for s in range(B)], dtype=torch.int64, device=dev)
    q = torch.randn(B, heads, rank, generator=g).bfloat16()
    for b, s in enumerate(order):                                    # heads 0, 1, 2: the first key, the last of a 64-key tile, the newest
        c = arenas[s][off:].view(L, rank).cpu()
        for h, j in zip(range(min(3, heads)), (0, min(63, lens[s] - 1), lens[s] - 1)):
            q[b, h] = (c[j].float() * 2).bfloat16()
    kv = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=dev)
    uv, gate = (torch.randn(heads * vdim, rank, generator=g) * 0.1).bfloat16(), torch.rand(B, heads, generator=g)
    qd, uvd, gd, sd = q.to(dev), uv.to(dev), gate.to(dev), _i32(order, dev)
    wo, wm = torch.full((B * heads * ns * rank,), float("nan"), device=dev), torch.full((B * heads * ns * 2,), float("nan"), device=dev)
    out = torch.zeros(B, heads * vdim, dtype=torch.bfloat16, device=dev)
    scale = rank ** -0.5
    _ok(lib.lcc_latent_attn_decode(_p(qd), _p(sd), _p(kv), _p(base), off, B, heads, rank, scale, ns, _p(wo), _p(wm), _p(uvd), vdim, _p(gd), _p(out), heads * vdim,
                                   _st()))
    for b, s in enumerate(order):
        c = arenas[s][off:].view(L, rank)[:lens[s]].double().cpu()
        o = torch.softmax(q[b].double() @ c.T * scale, -1) @ c
        want = (o[:, None, :] * uv.double().view(heads, vdim, rank)).sum(-1) * gate[b].double()[:, None]
        assert (out[b].view(heads, vdim).double().cpu() - want).abs().max() < 0.012 * want.abs().max() + 1e-3, (b, lens[s])


@pytest.mark.parametrize("rows,heads,dim,rank,ns", [(1, 1, 64, 64, 1), (16, 3, 128, 192, 2), (33, 2, 192, 512, 5)])
def test_absorbed_queries(dev, lib, rows, heads, dim, rank, ns):
    from livecc_amd.weights import pack_weight
    part, uk = torch.randn(ns, rows, heads * dim), torch.randn(heads, dim, rank).bfloat16()
    pd, ukt = part.to(dev), pack_weight(uk.transpose(1, 2).reshape(heads * rank, dim).contiguous()).to(dev)
    out = torch.empty(rows, heads, rank, dtype=torch.bfloat16, device=dev)
    _ok(lib.lcc_latent_absorb(_p(pd), ns, rows, heads, dim, _p(ukt), rank, _p(out), _st()))
    q = part.sum(0).bfloat16().double().view(rows, heads, dim)
    want = torch.stack([q[:, h] @ uk[h].double() for h in range(heads)], 1)
    assert (out.double().cpu() - want).abs().max() < 0.008 * want.abs().max()


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
        assert (pre[i].double().cpu() - x[:n - 1]).pow(2).mean().sqrt() < 0.01 * scale, i
        assert (dec[i].double().cpu() - x[n - 1]).pow(2).mean().sqrt() < 0.015 * scale, i


def test_token_by_token_from_the_first_one(case):
    n = 150          # over two 64-key tiles and the 128 border
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
    # and together with another stream: packed groups, each with its own wanted rows
    a, b = m.new_stream(), m.new_stream()
    la, lb = m.forward_step([(a, case["ids"][:90], [0, 89]), (b, case["ids"][:230], [229, 3])])
    assert U.error(la, case["want"][[0, 89]]) < U.LIMIT and U.error(lb, case["want"][[229, 3]]) < U.LIMIT


def test_unequal_requests_in_one_batch_equal_each_alone(case):
    m, ids, want = case["model"], case["ids"], case["want"]
    lens = [1, 97, 260, 32, 2]
    streams = [m.new_stream() for _ in lens]
    seqs = [ids[:n] for n in lens]
    got = m.forward_step([(s, x, [len(x) - 1, 0]) for s, x in zip(streams, seqs)])
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
    m.forward_step([(first, ids, [])])                    # fills the arena far beyond what the next request uses
    first.release()
    st = m.new_stream()
    assert st.slot == slot
    other = U.ids_of(case["cfg"], 70, 5)
    want = U.oracle_logits(case["cfg"], case["T"], other)
    got = m.forward_step([(st, other[:40], [0, 39])])[0]
    assert U.error(got, want[[0, 39]]) < U.LIMIT
    for j in range(40, 70):
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
    cfg, T, n = case["cfg"], case["T"], 200
    got = _run(case["model"], case["ids"][:n], [n])
    raw = cfg.to_dict()

    def faulty(patch=None, tensors=None, config=None):
        saved = {k: getattr(R, k) for k in (patch or {})}
        try:
            for k, f in (patch or {}).items():
                setattr(R, k, f)
            return R.run(config or raw, tensors or T, case["ids"][:n])
        finally:
            for k, f in saved.items():
                setattr(R, k, f)

    attn = R.causal_softmax_attention

    def without_key(j):
        def f(q, k, v, scale, first=0):
            o = attn(q, k, v, scale, first)
            o[j + 1:] = attn(q, torch.cat([k[:j], k[j + 1:]]), torch.cat([v[:j], v[j + 1:]]), scale, -1)[j + 1:]
            return o
        return f

    def window(q, k, v, scale, first=0):
        o = attn(q, k, v, scale, first)
        o[150:] = torch.cat([attn(q[i:i + 1], k[i - 127:i + 1], v[i - 127:i + 1], scale, 127) for i in range(150, len(q))])
        return o
    faults = {"first key lost": faulty({"causal_softmax_attention": without_key(0)}), "key at a tile border lost": faulty({"causal_softmax_attention": without_key(63)}),
              "a window of 128": faulty({"causal_softmax_attention": window}),
              "no query norm": faulty(tensors={k: (v * 1.3 if k.endswith("dq.norm") else v) for k, v in T.items()}),
              "no gate": faulty(tensors={k: (v * 0 + 0 if k.endswith("mix.g") else v) for k, v in T.items()}),
              "no feed-forward": faulty(tensors={k: (v * 0 if k.endswith("mlp.down") else v) for k, v in T.items()}),
              "no norm bias": faulty(tensors={k: (v * 0 if k.endswith("norm1.b") else v) for k, v in T.items()}),
              "alpha of another layer": faulty(tensors={k: (v * 0.8 if k.endswith("norm1.alpha") else v) for k, v in T.items()})}
    for name, want in faults.items():
        assert U.error(got, want) > 2.5 * U.LIMIT, name


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
    cases = _clear_prompts(cfg, T, [3, 70, 33, 1], steps)
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
    # an EOS id ends a request early; the others go on
    r = m.generate_batch([dict(input_ids=np.asarray(p)) for p, _ in cases], max_new_tokens=steps, eos_token_id=cases[1][1][2])
    for (p, toks), x in zip(cases, r):
        cut = toks.index(cases[1][1][2]) + 1 if cases[1][1][2] in toks else steps
        assert x.sequences[0, len(p):].tolist() == toks[:cut]


def test_sampling_arguments_reach_the_sampler(dev):
    cfg = U.configs()["mixed"]
    T = U.make_weights(cfg, 8)
    m = _model(cfg, T, dev)
    p = U.ids_of(cfg, 20, 1)
    z = U.oracle_logits(cfg, T, p)[-1]
    greedy = int(z.argmax())
    one = lambda **kw: m.generate(torch.tensor([p]), max_new_tokens=1, output_scores=True, **kw)
    assert one(do_sample=True, top_k=1).sequences[0, -1].item() == greedy
    r = one(do_sample=True, top_k=5, temperature=2.0, seed=3)
    assert r.sequences[0, -1].item() in set(z.topk(6).indices.tolist())
    assert int(torch.isfinite(r.scores).sum()) == 5 and r.scores.shape == (cfg.vocab_size,)
    assert (r.scores.max().item() - z.max().item() / 2.0) < 0.1
    s = one(repetition_penalty=3.0).scores.double().cpu()
    seen = sorted(set(p))
    want = z.clone()
    want[seen] = torch.where(want[seen] < 0, want[seen] * 3.0, want[seen] / 3.0)
    assert (s - want).abs().max() < 0.1 * z.abs().max()
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
        lens = [s.get_seq_length() for s in st2]
        ids = [5] * n
        got = m.forward_step([(s, [i], [0]) for s, i in zip(st2, ids)])
        assert [s.get_seq_length() for s in st2] == [x + 1 for x in lens]
        for k, g in enumerate(got[:3]):
            seqs[k] = seqs[k] + [5]
            assert U.error(g, U.oracle_logits(cfg, T, seqs[k])[[-1]]) < U.LIMIT


def test_fused_and_separate_decode_launches_agree(dev, lib):
    cfg = U.configs()["full-heads"]
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


def test_long_decoding_stays_with_the_prompt_form(dev):
    cfg = U.configs()["even"]
    T = U.make_weights(cfg, 6)
    m = _model(cfg, T, dev, max_kv_len=1500, max_new_rows=1100)
    ids = U.ids_of(cfg, 1050, 77)
    at = sorted({40, 63, 64, 127, 128, 255, 256, 511, 512, 700, 1023, 1024, 1049})
    want = _run(m, ids, [1050], set(at))
    st = m.new_stream()
    m.forward_step([(st, ids[:30], [])])
    got = []
    for j in range(30, 1050):
        r = m.forward_step([(st, [ids[j]], [0] if j in at else [])])[0]
        if j in at:
            got.append(r.cpu())
    assert U.error(torch.cat(got), want) < U.LIMIT
    assert U.error(want[:4], U.oracle_logits(cfg, T, ids[:128])[[40, 63, 64, 127]]) < U.LIMIT


def test_calls_the_engine_cannot_serve_are_errors(dev):
    from livecc_amd import _lib
    cfg = U.configs()["even"]
    m = _model(cfg, U.make_weights(cfg), dev, max_kv_len=128, max_new_rows=64, max_history=16, max_streams=2)
    st = m.new_stream()
    with pytest.raises(_lib.LccError, match="out of range"):
        m.forward_step([(st, [0, cfg.vocab_size], [])])
    with pytest.raises(_lib.LccError, match="capacity"):
        m.forward_step([(st, [1] * 120, [])])
    with pytest.raises(ValueError):
        m.forward_step([(st, [1, 2], [2])])
    with pytest.raises(ValueError):
        m.forward_step([(st, [1], []), (st, [2], [])])
    st.release()
    with pytest.raises(ValueError):
        m.forward_step([(st, [1], [])])
    with pytest.raises(_lib.LccError, match="vision"):
        m.engine.vit_encode([dict(frames=torch.zeros(2, 28, 28, 3, dtype=torch.uint8, device=dev))])


def test_trace_runner_from_a_checkpoint_directory(dev, tmp_path):
    """bin/trace_run end to end: a child process, its files and its lines."""
    import json
    import os
    import subprocess
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
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
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(out), "--max-tokens", "113"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = U.oracle_logits(cfg, T, a), U.oracle_logits(cfg, T, b)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg.vocab_size))
    assert U.error(read(0), torch.stack([wa[77], wa[5], wb[31]])) < U.LIMIT
    assert U.error(read(1), wb[[32]]) < U.LIMIT and U.error(read(2), wa[[79]]) < U.LIMIT
