"""CPU: the Bemuzen family's configuration and registry, weight layout, engine sizing, and the oracle itself."""
import ctypes as C
import json
import os
import sys

import pytest
import torch

from livecc_amd import _lib, config as CFG
from livecc_amd.engine import Engine
from livecc_amd.weights import BemuzenArena, bemuzen_param_shapes, bemuzen_weight_shapes, make_arena
from oracle import bemuzen_ref as R
from tests import bemuzen_util as U

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- configuration ----
def test_config_round_trips_through_the_checkpoint_form(tmp_path):
    for name, cfg in U.configs().items():
        d = tmp_path / name
        d.mkdir()
        (d / "config.json").write_text(json.dumps(cfg.to_dict()))
        assert CFG.get_config(str(d)) == cfg
        assert CFG.architecture_of(str(d)) == "Bemuzen"


def test_every_size_and_constant_comes_from_the_config():
    raw = U.configs()["mixed"].to_dict()
    raw.update(width=72, vocab=99, logit_scale=0.25)
    raw["norm"]["eps"] = 3e-4
    raw["embedding"]["bigram"] = {"buckets": 11, "mul_prev": 70001, "mul_cur": 9}
    raw["layers"][0]["mixer"]["left"].update(scale=0.77, vdim=19, q_temp={"coef": 0.9, "every": 5})
    raw["layers"][0]["mixer"]["right"].update(decay=[0.1, 0.2, 0.3])
    raw["layers"][1]["mixer"].update(conv=9, norm_groups=2)
    c = CFG.BemuzenConfig.from_dict(raw)
    assert (c.norm_eps, c.logit_scale, c.hidden_size, c.vocab_size, c.bigram_buckets, c.bigram_mul_prev, c.bigram_mul_cur) == (3e-4, 0.25, 72, 99, 11, 70001, 9)
    a, r, s = c.layers[0].mixer.left, c.layers[0].mixer.right, c.layers[1].mixer
    assert (a.scale, a.vdim, a.q_temp_coef, a.q_temp_every, r.decay, s.conv_taps, s.norm_groups) == (0.77, 19, 0.9, 5, [0.1, 0.2, 0.3], 9, 2)
    assert [l.ff for l in c.layers] == [150, 0, 0, 90]


@pytest.mark.parametrize("change, message", [
    (lambda r: r["layers"][0].update(type="sliding"), "unknown layer type"),
    (lambda r: r["layers"][0]["mlp"].update(kind="experts"), "unknown feed-forward"),
    (lambda r: r["layers"][0]["mixer"]["left"].update(kv_heads=4), "key/value heads"),
    (lambda r: r["layers"][0]["mixer"]["left"].update(dim=257), "head sizes"),
    (lambda r: r["layers"][0]["mixer"]["right"].update(decay=[0.5]), "one decay"),
    (lambda r: r["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5, 1.5]), "one decay"),
    (lambda r: r["layers"][1]["mixer"].update(groups=4), "groups"),
    (lambda r: r["layers"][1]["mixer"].update(norm_groups=7), "norm groups"),
    (lambda r: r["layers"][1]["mixer"].update(state=300), "recurrent key sizes"),
    (lambda r: r["layers"][1]["mixer"].update(conv=17), "taps"),
    (lambda r: r["layers"][1]["mixer"].update(heads=0), "positive"),
    (lambda r: r.update(width=9000), "widths above"),
])
def test_configs_the_family_does_not_have_are_refused(change, message):
    raw = U.configs()["mixed"].to_dict()
    change(raw)
    with pytest.raises(ValueError, match=message):
        CFG.BemuzenConfig.from_dict(raw)


def test_registry_picks_the_model_class_by_config(tmp_path):
    from livecc_amd import modeling as MD
    assert MD.MODEL_CLASSES["Bemuzen"] is MD.BemuzenForCausalLM and MD.BemuzenForCausalLM.config_class is CFG.BemuzenConfig
    (tmp_path / "config.json").write_text(json.dumps(U.configs()["even"].to_dict()))
    with pytest.raises(ValueError, match="not a Debunex checkpoint"):
        MD.DebunexForCausalLM.from_pretrained(str(tmp_path), device_map="cuda:0")
    with pytest.raises(ValueError, match="fp8"):
        make_arena(U.configs()["even"], "cpu", llm_fp8=True)


# ---- weights ----
@pytest.mark.parametrize("name", sorted(U.configs()))
def test_arena_holds_every_tensor_in_the_engines_order(name):
    cfg = U.configs()[name]
    T = U.make_weights(cfg, 1)
    a = U.arena(cfg, T, "cpu")
    D = cfg.hidden_size
    assert torch.equal(a.view("bigram")[:, :D], T["bigram"]) and a.view("bigram")[:, D:].abs().sum() == 0
    assert torch.equal(a.logical("lm_head")[:cfg.vocab_size, :D], T["head"]) and a.logical("lm_head")[cfg.vocab_size:].abs().sum() == 0
    f32 = lambda n: a.view(n).view(torch.float32)
    for i, l in enumerate(cfg.layers):
        m, r, p, s = l.mixer, l.mixer.recurrent, f"dec.{i}.", f"l{i}.mix."
        rows = a.logical(p + "in_w")
        assert rows.shape == (m.in_rows, cfg.width_pad) and rows[:, D:].abs().sum() == 0
        at = 0

        def block(heads, d, pad):
            nonlocal at
            x = rows[at:at + heads * pad].view(heads, pad, -1)
            at += heads * pad
            assert x[:, d:].abs().sum() == 0
            return x[:, :d, :D].reshape(heads * d, D)
        if isinstance(m, CFG.ParallelMixerSpec):
            q = m.left
            for n, h, d, pad in (("left.q", q.heads, q.dim, q.dim_pad), ("left.k", q.kv_heads, q.dim, q.dim_pad), ("left.v", q.kv_heads, q.vdim, q.vdim_pad),
                                 ("right.q", r.heads, r.dim, r.key_pad), ("right.k", r.heads, r.dim, r.key_pad), ("right.v", r.heads, r.vdim, r.vdim_pad),
                                 ("right.g", r.heads, r.vdim, r.vdim_pad)):
                assert torch.equal(block(h, d, pad), T[s + n]), n
            assert torch.allclose(f32(p + "slope"), R.head_slopes(q.heads).float() / torch.log(torch.tensor(2.0)), rtol=1e-6)
            want = torch.tensor(r.decay, dtype=torch.float64)
            assert (torch.exp2(f32(p + "rec_rate").double()) - want).abs().max() < 1e-6
            o = a.logical(p + "lo_w")[:D].view(D, q.heads, q.vdim_pad)
            assert torch.equal(o[:, :, :q.vdim].reshape(D, -1), T[s + "left.o"]) and o[:, :, q.vdim:].abs().sum() == 0
            assert torch.equal(a.logical(p + "ro_w")[:D, :r.heads * r.vdim], T[s + "right.o"])
        else:
            got = torch.cat([block(m.heads, m.vdim, m.vdim_pad), block(m.heads, m.vdim, m.vdim_pad), block(m.groups, m.state, m.key_pad),
                             block(m.groups, m.state, m.key_pad), rows[at:at + m.heads, :D]])
            assert torch.equal(got, T[s + "in"]) and rows[at + m.heads:].abs().sum() == 0
            w = a.view(p + "conv_w")
            assert w.shape == (m.conv_taps, m.conv_channels)
            assert torch.equal(w[:, :m.heads * m.vdim_pad].view(m.conv_taps, m.heads, m.vdim_pad)[:, :, :m.vdim].reshape(m.conv_taps, -1).T,
                               T[s + "conv"][:m.heads * m.vdim])
            last = w[:, -m.groups * m.key_pad:].view(m.conv_taps, m.groups, m.key_pad)
            assert torch.equal(last[:, :, :m.state].reshape(m.conv_taps, -1).T, T[s + "conv"][-m.groups * m.state:]) and last[:, :, m.state:].abs().sum() == 0
            assert torch.equal(f32(p + "rec_dt_bias"), T[s + "dt_bias"].float()) and torch.equal(f32(p + "rec_skip"), T[s + "D"].float())
            assert torch.allclose(torch.exp2(f32(p + "rec_rate")), torch.exp(-torch.exp(T[s + "A_log"].float())), rtol=1e-5)
        if l.ff:
            assert torch.equal(a.logical(p + "down_w")[:D, :l.ff], T[f"l{i}.mlp.down"])


def test_wrong_shapes_are_refused():
    cfg = U.configs()["even"]
    T = U.make_weights(cfg)
    T["l1.mix.conv"] = T["l1.mix.conv"][:, 1:]
    with pytest.raises(ValueError, match="l1.mix.conv"):
        U.arena(cfg, T, "cpu")


def test_random_fill_has_the_checkpoints_tensors():
    a = BemuzenArena(CFG.bemuzen_tiny(), "cpu").fill_random(3)
    assert torch.isfinite(a.view("dec.0.in_w").float()).all() and (a.view("dec.2.rec_rate").view(torch.float32) < 0).all()
    assert set(bemuzen_param_shapes(CFG.bemuzen_tiny())) >= {"bigram", "l2.mix.A_log", "l0.mix.right.out", "l0.norm2b"}


# ---- engine sizing and argument checks (host logic of the library) ----
def _create(lib, cfg, slots=4, kv=640, rows=700, mutate=None):
    layers = (_lib.DecoderLayer * cfg.num_hidden_layers)(*[Engine._sandwich_layer(l) for l in cfg.layers])
    dc = _lib.DecoderConfigC(cfg.vocab_size, cfg.vocab_pad, cfg.width_pad, cfg.num_hidden_layers, cfg.norm_eps, 0.0, _lib.BLOCK_SANDWICH, cfg.hidden_size, cfg.logit_scale,
                             cfg.bigram_buckets, cfg.bigram_mul_prev, cfg.bigram_mul_cur)
    lim = _lib.EngineLimits(slots, kv, rows, 0, 16)
    if mutate:
        mutate(dc, layers, lim)
    return lib.lcc_engine_create_decoder(C.byref(dc), layers, C.byref(lim))


def test_engine_sizes_follow_the_config(built_lib):
    for cfg in U.configs().values():
        e = _create(built_lib, cfg)
        assert e, built_lib.lcc_last_error()
        need = 640 * cfg.kv_bytes_per_token + cfg.state_bytes
        assert need <= built_lib.lcc_engine_kv_bytes_per_slot(e) < need + 256 * 4 * len(cfg.layers)
        assert built_lib.lcc_engine_workspace_bytes(e) > 0 and built_lib.lcc_engine_meta_bytes(e) > 0
        miss = C.create_string_buffer(4096)
        assert built_lib.lcc_engine_weights_ready(e, miss, 4096) == 0
        assert set(n for n, _ in bemuzen_weight_shapes(cfg)) == set(miss.value.decode().split())
        built_lib.lcc_engine_destroy(e)


@pytest.mark.parametrize("mutate", [
    lambda dc, L, lim: setattr(L[0], "mixer", 1), lambda dc, L, lim: setattr(dc, "block", 7), lambda dc, L, lim: setattr(dc, "block", 0),
    lambda dc, L, lim: setattr(L[0], "kv_heads", 5), lambda dc, L, lim: setattr(L[0], "dim_pad", 320), lambda dc, L, lim: setattr(L[0], "q_temp_every", 0),
    lambda dc, L, lim: setattr(L[0], "rec_conv_taps", 2), lambda dc, L, lim: setattr(L[1], "rec_conv_taps", 0), lambda dc, L, lim: setattr(L[1], "rec_key_pad", 320),
    lambda dc, L, lim: setattr(L[1], "rec_groups", 4), lambda dc, L, lim: setattr(L[1], "rec_norm_groups", 7), lambda dc, L, lim: setattr(dc, "width", 300),
    lambda dc, L, lim: setattr(dc, "bigram_buckets", 0), lambda dc, L, lim: setattr(lim, "max_kv_len", 100)])
def test_engine_refuses_what_its_kernels_do_not_serve(built_lib, mutate):
    assert not _create(built_lib, U.configs()["mixed"], mutate=mutate)
    assert built_lib.lcc_last_error()


def test_operators_check_their_arguments_before_any_launch(built_lib):
    one, l = C.c_void_p(16), built_lib
    assert l.lcc_post_norm_resid(one, 1, None, 1, None, None, one, one, one, one, 1, 80, 64, 1e-5, None) != 0                       # width > stored
    assert l.lcc_post_norm_resid(one, 1, one, 1, None, one, one, one, one, one, 1, 64, 64, 1e-5, None) != 0                         # a pair without its norms
    assert l.lcc_gqa_attn_prefill(one, one, one, one, one, one, 1, 1, 3, 2, 64, 64, 1.0, None, one, 0, 0, 64, None) != 0             # 3 heads over 2
    assert l.lcc_gqa_attn_decode(one, one, one, 1, 2, 1, 96, 64, 1.0, None, one, 0, 0, 64, 1, one, one, one, None) != 0              # no kernel for 96
    assert l.lcc_gqa_attn_decode(one, one, one, 1, 2, 1, 64, 64, 1.0, None, one, 0, 0, 64, 65, one, one, one, None) != 0             # too many splits
    assert l.lcc_rec_scan(one, one, one, None, one, None, one, 2, 2, 320, 64, one, one, one, one, 1, one, one, 1, None, None, one, 0, None) != 0
    assert l.lcc_rec_scan(one, one, one, None, one, None, one, 2, 2, 64, 64, one, one, one, one, 2, one, one, 1, None, None, one, 0, None) != 0      # no scratch
    assert l.lcc_rec_norm(one, one, 1, 1, 64, 64, 0, 1, 64, 64, 1, 1e-5, one, one, 64, None, None) != 0                              # gate columns missing
    assert l.lcc_rec_decode(None, None, one, None) != 0
    r = _lib.RecInput(partial=16, nsplit=1, rows=1, ldn=192, q_col=0, k_col=64, v_col=128, dt_col=-1, heads=1, groups=1, key_pad=64, vdim_pad=64, rate=16,
                      tok_stream=16, kv_base=16)
    assert l.lcc_mixer_prep(None, C.byref(r), None) != 0                                                                           # no positions
    r.v_col = 160
    assert l.lcc_rec_decode(C.byref(r), None, one, None) != 0                                                                      # columns past the row


def test_a_recurrent_state_is_not_rolled_back():
    e = Engine.__new__(Engine)
    e.has_recurrent_state, e.slot_length = True, lambda s: (9, 9)
    with pytest.raises(_lib.LccError, match="rolled back"):
        e.set_slot_length(0, 5, 5)


def test_decoder_bench_counts_both_models_alike():
    sys.path.insert(0, os.path.join(ROOT, "tools"))
    import bench_decoder as B
    for size, gqa in B.LIKE.items():
        a, b = CFG.get_config(f"bemuzen-{size}"), CFG.get_config(gqa)
        m = a.layers[0].mixer.left
        assert (a.hidden_size, a.vocab_size, a.num_hidden_layers, a.layers[0].ff, m.heads, m.kv_heads, m.dim) == \
               (b.hidden_size, b.vocab_size, b.num_hidden_layers, b.intermediate_size, b.num_attention_heads, b.num_key_value_heads, b.head_dim)
        assert 1.0 < B.flops_of(a, 2048) / B.flops_of(b, 2048) < 1.5
        assert 1.0 < B.step_bytes(a, 1, 1024) / B.step_bytes(b, 1, 1024) < 1.5


# ---- the oracle ----
def test_oracle_bigram_rows_and_query_temperature():
    assert R.bigram_rows([5, 7, 7], 10, 3, 4) == [10, (15 + 28) % 10, (21 + 28) % 10]
    t = R.query_temperature(torch.arange(8, dtype=torch.float64), 0.5, 4)
    assert torch.equal(t[:3], torch.ones(3, dtype=torch.float64))          # steps at p + 1 = 4, 8, ..
    assert torch.allclose(t[3:7], 1 + 0.5 * torch.log(torch.tensor(2.0, dtype=torch.float64)).expand(4)) and t[7] > t[6]


def test_oracle_attention_bias_and_causality():
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(9, h, 4, generator=g, dtype=torch.float64) for h in (4, 2, 2))
    o = R.biased_attention(q, k, v, 0.5, R.head_slopes(4))
    assert torch.allclose(o[0, 3], v[0, 1])
    k2, v2 = k.clone(), v.clone()
    k2[6], v2[6] = 9, 9
    o2 = R.biased_attention(q, k2, v2, 0.5, R.head_slopes(4))
    assert torch.equal(o[:6], o2[:6]) and not torch.equal(o[6:], o2[6:])
    s = (q[8, 2] * k[:, 1]).sum(-1) * 0.5 + 2.0 ** -6 * torch.arange(9, dtype=torch.float64)      # the bias up to a constant of the row
    assert torch.allclose(o[8, 2], torch.softmax(s, -1) @ v[:, 1])


def test_oracle_recurrence_is_the_decayed_sum():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(7, 2, n, generator=g, dtype=torch.float64) for n in (3, 3, 5))
    a, w = torch.rand(7, 2, generator=g, dtype=torch.float64), torch.rand(7, 2, generator=g, dtype=torch.float64)
    o, S = R.decayed_outer_products(q, k, v, a, w)
    want = sum(a[s + 1:7, 1].prod() * w[s, 1] * (q[6, 1] @ k[s, 1]) * v[s, 1] for s in range(7))
    assert torch.allclose(o[6, 1], want)
    o1, S1 = R.decayed_outer_products(q[:4], k[:4], v[:4], a[:4], w[:4])
    o2, S2 = R.decayed_outer_products(q[4:], k[4:], v[4:], a[4:], w[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_oracle_convolution_and_norm():
    u = torch.arange(1.0, 6.0, dtype=torch.float64)[:, None]
    assert R.causal_conv(u, torch.tensor([[0.0, 10.0, 1.0]], dtype=torch.float64), torch.tensor([0.5], dtype=torch.float64)).flatten().tolist() == [1.5, 12.5, 23.5, 34.5, 45.5]
    x = torch.tensor([3.0, 4.0], dtype=torch.float64)
    assert torch.allclose(R.norm_around_one(x, torch.tensor([0.0, 1.0], dtype=torch.float64), 0.0), x / 12.5 ** 0.5 * torch.tensor([1.0, 2.0], dtype=torch.float64))
