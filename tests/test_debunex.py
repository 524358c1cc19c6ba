"""CPU: the Debunex family's configuration and registry, weight layout, engine sizing, trace replay and the oracle itself."""
import ctypes as C
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from livecc_amd import _lib, config as CFG, trace
from livecc_amd.weights import DecoderArena, decoder_param_shapes, fp8_weight_names, interleave_gate_up, make_arena
from oracle import debunex_ref as R
from tests import debunex_util as U

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- configuration ----
def test_config_round_trips_through_the_checkpoint_form(tmp_path):
    for name, cfg in U.configs().items():
        d = tmp_path / name
        d.mkdir()
        (d / "config.json").write_text(json.dumps(cfg.to_dict()))
        assert CFG.get_config(str(d)) == cfg
        assert CFG.architecture_of(str(d)) == "Debunex"


def test_every_size_and_constant_comes_from_the_config():
    raw = U.configs()["mixed"].to_dict()
    raw["norm"]["eps"], raw["logit_softcap"], raw["width"], raw["vocab"] = 3e-4, 7.5, 72, 99
    raw["layers"][1]["mixer"].update(scale=0.77, vdim=19)
    c = CFG.DebunexConfig.from_dict(raw)
    assert (c.norm_eps, c.logit_softcap, c.hidden_size, c.vocab_size) == (3e-4, 7.5, 72, 99)
    assert (c.layers[1].mixer.scale, c.layers[1].mixer.vdim, c.layers[1].ff) == (0.77, 19, 0)
    assert [l.mixer.kv_from for l in c.layers] == [None, None, 0, 1]


@pytest.mark.parametrize("change, message", [
    (lambda r: r["layers"][0].update(type="sliding"), "unknown layer type"),
    (lambda r: r["layers"][0]["mlp"].update(kind="experts"), "unknown feed-forward"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=3), "not an earlier layer"),
    (lambda r: r["layers"][3]["mixer"].update(kv_from=2), "of its own"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=1), "no latent of rank"),
    (lambda r: r["layers"][0]["mixer"].update(kv_rank=1025), "latent rank"),
    (lambda r: r["layers"][0]["mixer"].update(heads=0), "positive"),
])
def test_configs_the_family_does_not_have_are_refused(change, message):
    raw = U.configs()["mixed"].to_dict()
    change(raw)
    with pytest.raises(ValueError, match=message):
        CFG.DebunexConfig.from_dict(raw)


def test_registry_picks_the_model_class_by_config(tmp_path):
    from livecc_amd import modeling as MD
    assert set(MD.MODEL_CLASSES) == set(CFG.ARCHITECTURES) | {None}
    assert MD.MODEL_CLASSES["Debunex"] is MD.DebunexForCausalLM
    assert issubclass(MD.DebunexForCausalLM, MD.EngineModel) and issubclass(MD.LiveCCForConditionalGeneration, MD.EngineModel)
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(KeyError, match="unknown architecture"):
        CFG.architecture_of(str(tmp_path))
    with pytest.raises(ValueError, match="bf16"):
        MD.DebunexForCausalLM.from_pretrained(str(tmp_path), torch_dtype="float32")
    with pytest.raises(RuntimeError, match="no CPU path"):
        MD.DebunexForCausalLM.from_pretrained(str(tmp_path), device_map="cpu")


def test_padded_sizes():
    assert [CFG.pad_kv_rank(r) for r in (1, 64, 65, 193, 257, 385, 512, 513, 1024)] == [64, 64, 128, 256, 384, 512, 512, 768, 1024]
    assert [CFG.pad_head_dim(d) for d in (1, 64, 65, 128, 129)] == [64, 64, 128, 128, 192]
    c = U.configs()["mixed"]
    assert (c.width_pad, c.vocab_pad) == (256, 384)
    assert c.kv_bytes_per_token == 2 * (64 + 128)          # two latents, padded ranks
    assert c.layers[0].mixer.in_rows == 128 + 64 + 16 and c.layers[2].mixer.in_rows == 64 + 16


# ---- weights ----
@pytest.mark.parametrize("name", sorted(U.configs()))
def test_arena_holds_every_tensor_in_the_engines_order(name):
    cfg = U.configs()[name]
    T = U.make_weights(cfg, 1)
    a = U.arena(cfg, T, "cpu")
    W = cfg.width_pad
    assert torch.equal(a.logical("embed")[:, :cfg.hidden_size], T["embed"]) and a.logical("embed")[:, cfg.hidden_size:].abs().sum() == 0
    assert torch.equal(a.logical("lm_head")[:cfg.vocab_size, :cfg.hidden_size], T["head"]) and a.logical("lm_head")[cfg.vocab_size:].abs().sum() == 0
    for i, l in enumerate(cfg.layers):
        m, p, s = l.mixer, f"dec.{i}.", f"l{i}."
        H, Q, Rp = m.heads, m.q_rank_pad, m.kv_rank_pad
        inw = a.logical(p + "in_w")
        assert torch.equal(inw[:m.q_rank, :cfg.hidden_size], T[s + "mix.dq"]) and inw[m.q_rank:Q].abs().sum() == 0
        g0 = Q
        if m.kv_from is None:
            assert torch.equal(inw[Q:Q + m.kv_rank, :cfg.hidden_size], T[s + "mix.dkv"])
            g0 += Rp
        assert torch.equal(inw[g0:g0 + H, :cfg.hidden_size], T[s + "mix.g"]) and inw.shape == (m.in_rows, W)
        uk = a.logical(p + "uk_w").view(H, m.dim_pad, Rp)
        assert torch.equal(uk[:, :m.dim, :m.kv_rank].reshape(H * m.dim, m.kv_rank), T[s + "mix.uk"])
        assert torch.equal(a.logical(p + "ukt_w").view(H, Rp, m.dim_pad).transpose(1, 2), uk)
        uv = a.view(p + "uv_w").view(H, m.vdim_pad, Rp)          # row-major
        assert torch.equal(uv[:, :m.vdim, :m.kv_rank].reshape(H * m.vdim, m.kv_rank), T[s + "mix.uv"])
        out = a.logical(p + "out_w")
        assert torch.equal(out[:cfg.hidden_size, :H * m.vdim_pad].view(cfg.hidden_size, H, m.vdim_pad)[:, :, :m.vdim].reshape(cfg.hidden_size, -1), T[s + "mix.o"])
        if l.ff:
            assert torch.equal(out[:cfg.hidden_size, H * m.vdim_pad:H * m.vdim_pad + l.ff], T[s + "mlp.down"])
            gu = a.logical(p + "gate_up_w").view(l.ff_pad // 16, 2, 16, W)
            assert torch.equal(gu[:, 0].reshape(l.ff_pad, W)[:l.ff, :cfg.hidden_size], T[s + "mlp.gate"])
            assert torch.equal(gu[:, 1].reshape(l.ff_pad, W)[:l.ff, :cfg.hidden_size], T[s + "mlp.up"])
        assert a.view(p + "norm_alpha").item() == T[s + "norm1.alpha"].item()


def test_wrong_shapes_missing_tensors_and_fp8_are_refused(tmp_path):
    cfg = U.configs()["even"]
    T = U.make_weights(cfg)
    T["l1.mix.uq"] = T["l1.mix.uq"][:-1]
    with pytest.raises(ValueError, match="l1.mix.uq"):
        U.arena(cfg, T, "cpu")
    with pytest.raises(ValueError, match="fp8"):
        make_arena(cfg, "cpu", llm_fp8=True)
    from safetensors.torch import save_file
    from livecc_amd.weights import from_pretrained
    T = U.make_weights(cfg)
    save_file({k: v.contiguous() for k, v in T.items() if k != "final.norm.b"}, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError, match="final.norm.b"):
        from_pretrained(str(tmp_path), cfg, "cpu")
    save_file({k: v.contiguous() for k, v in T.items()}, str(tmp_path / "model.safetensors"))
    a, b = from_pretrained(str(tmp_path), cfg, "cpu"), U.arena(cfg, T, "cpu")
    assert all(torch.equal(a.view(n), b.view(n)) for n in a.names())


# ---- engine sizing and argument checks (host logic of the library) ----
def _create(lib, cfg, slots=4, kv=640, rows=128, mutate=None):
    layers = (_lib.DecoderLayer * cfg.num_hidden_layers)()
    for i, l in enumerate(cfg.layers):
        m = l.mixer
        layers[i] = _lib.DecoderLayer(_lib.MIXER_LATENT, m.heads, m.q_rank, m.kv_rank, m.dim_pad, m.vdim_pad, m.q_rank_pad, m.kv_rank_pad,
                                      -1 if m.kv_from is None else m.kv_from, m.scale, l.ff_pad)
    dc = _lib.DecoderConfigC(cfg.vocab_size, cfg.vocab_pad, cfg.width_pad, cfg.num_hidden_layers, cfg.norm_eps, cfg.logit_softcap or 0.0)
    lim = _lib.EngineLimits(slots, kv, rows, 0, 16)
    if mutate:
        mutate(dc, layers, lim)
    return lib.lcc_engine_create_decoder(C.byref(dc), layers, C.byref(lim))


def test_engine_sizes_follow_the_config(built_lib):
    for cfg in U.configs().values():
        e = _create(built_lib, cfg)
        assert e, built_lib.lcc_last_error()
        owners = [l.mixer.kv_rank_pad for l in cfg.layers if l.mixer.kv_from is None]
        assert built_lib.lcc_engine_kv_bytes_per_slot(e) == 640 * cfg.kv_bytes_per_token == 640 * 2 * sum(owners)
        assert built_lib.lcc_engine_workspace_bytes(e) > 0 and built_lib.lcc_engine_meta_bytes(e) > 0 and built_lib.lcc_engine_state_bytes(e) > 0
        miss = C.create_string_buffer(4096)
        assert built_lib.lcc_engine_weights_ready(e, miss, 4096) == 0
        assert set(n for n, _ in DecoderArena(cfg, "cpu").shapes) == set(miss.value.decode().split())
        built_lib.lcc_engine_destroy(e)


@pytest.mark.parametrize("mutate", [
    lambda dc, L, lim: setattr(L[0], "mixer", 9), lambda dc, L, lim: setattr(L[0], "kv_rank_pad", 320), lambda dc, L, lim: setattr(L[0], "dim_pad", 40),
    lambda dc, L, lim: setattr(L[2], "kv_from", 2), lambda dc, L, lim: setattr(L[2], "kv_from", 1), lambda dc, L, lim: setattr(lim, "max_kv_len", 100),
    lambda dc, L, lim: setattr(dc, "width_pad", 200), lambda dc, L, lim: setattr(dc, "vocab_pad", 320), lambda dc, L, lim: setattr(L[1], "ff_pad", 10),
    lambda dc, L, lim: setattr(lim, "max_new_rows", 0)])
def test_engine_refuses_what_its_kernels_do_not_serve(built_lib, mutate):
    assert not _create(built_lib, U.configs()["mixed"], mutate=mutate)
    assert built_lib.lcc_last_error()


def test_operators_check_their_arguments_before_any_launch(built_lib):
    one = C.c_void_p(16)
    assert built_lib.lcc_latent_attn_decode(one, one, one, one, 0, 1, 1, 320, 1.0, 1, one, one, one, 64, None, one, 64, None) != 0      # no kernel for rank 320
    assert built_lib.lcc_latent_attn_decode(one, one, one, one, 0, 1, 1, 64, 1.0, 129, one, one, one, 64, None, one, 64, None) != 0     # too many splits
    assert built_lib.lcc_attn_mha(one, one, one, 30, None, one, 64, one, one, one, one, 1, 1, 1, 64, 64, 1.0, None) != 0                 # ldv % 32
    assert built_lib.lcc_latent_absorb(one, 1, 1, 1, 96, one, 64, one, None) != 0
    assert built_lib.lcc_resid_dyt(None, one, 1, one, one, one, one, 1, 64, None) != 0
    assert built_lib.lcc_latent_norm_append(one, 1, 1, 100, 64, 64, one, 64, 64, one, 4, 1e-5, one, one, one, one, 0, one, one, None) != 0      # columns missing


# ---- trace replay ----
class FakeStream:
    def __init__(self, log):
        self.log, self.n = log, 0

    def release(self):
        self.log.append("release")


class FakeModel:
    device = "cpu"

    def __init__(self):
        self.log = []

    def new_stream(self):
        return FakeStream(self.log)

    def forward_step(self, entries):
        out = []
        for st, ids, want in entries:
            out.append(torch.tensor([[float(st.n + w), float(ids[w])] for w in want]).reshape(len(want), 2))
            st.n += len(ids)
        self.log.append([len(e[1]) for e in entries])
        return out


def test_trace_replay_writes_the_wanted_rows_in_order_and_gives_slots_back(tmp_path, monkeypatch):
    monkeypatch.setattr(torch.cuda, "synchronize", lambda *a: None)
    m, said = FakeModel(), io.StringIO()
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [2, 0]}, {"id": "b", "tokens": [9], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [4], "want": []}, {"id": "b", "tokens": [8], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": [6], "want": [0]}], "end": ["a"]}]
    trace.replay(m, [json.dumps(x) + "\n" for x in lines], str(tmp_path), say=lambda t, flush: said.write(t + "\n"))
    assert said.getvalue() == "done 0\ndone 1\ndone 2\n"
    assert np.fromfile(tmp_path / "0.f32", dtype="<f4").tolist() == [2.0, 3.0, 0.0, 5.0]
    assert not (tmp_path / "1.f32").exists()
    assert np.fromfile(tmp_path / "2.f32", dtype="<f4").tolist() == [4.0, 6.0]
    assert m.log == [[3, 1], [1, 1], "release", [1], "release"]


def test_trace_runner_refuses_fp32_at_the_start(tmp_path):
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "8"],
                       stdin=subprocess.DEVNULL, capture_output=True, text=True)
    assert r.returncode == 3 and "no fp32 mode" in r.stderr


def test_generate_command_needs_a_model():
    r = subprocess.run([sys.executable, "-m", "livecc_amd", "generate", "--ids", "1,2"], cwd=ROOT, capture_output=True, text=True)
    assert r.returncode == 2 and "--model" in r.stderr


# ---- the oracle ----
def test_oracle_attention_sees_every_earlier_key_and_none_later():
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(6, 2, 8, generator=g, dtype=torch.float64) for _ in range(3))
    o = R.causal_softmax_attention(q, k, v, 0.5)
    assert torch.allclose(o[0], v[0])
    for t in range(6):
        s = torch.stack([(q[t] * k[j]).sum(-1) * 0.5 for j in range(t + 1)])
        w = torch.softmax(s, 0)
        assert torch.allclose(o[t], (w[:, :, None] * v[:t + 1]).sum(0))
    assert torch.allclose(R.causal_softmax_attention(q[4:], k, v, 0.5, first=4), o[4:])


def test_oracle_score_and_value_maps_commute_with_the_latent():
    """(q . Uk c) = (Uk^T q . c) and sum_j p_j Uv c_j = Uv sum_j p_j c_j: what the decode kernels use."""
    g = torch.Generator().manual_seed(1)
    q, c, uk, uv = (torch.randn(*s, generator=g, dtype=torch.float64) for s in ((5,), (7, 3), (5, 3), (4, 3)))
    s = (c @ uk.T) @ q
    assert torch.allclose(s, c @ (uk.T @ q))
    p = torch.softmax(s, 0)
    assert torch.allclose(p @ (c @ uv.T), uv @ (p @ c))


def test_oracle_norms_cap_and_gate():
    x = torch.tensor([[3.0, -4.0]], dtype=torch.float64)
    assert torch.allclose(R.rms_unit(x, 0.5), x / (12.5 + 0.5) ** 0.5)
    one = torch.ones(2, dtype=torch.float64)
    assert torch.allclose(R.dynamic_tanh(x, torch.tensor(0.5, dtype=torch.float64), 2 * one, 3 * one), 2 * torch.tanh(0.5 * x) + 3)
    assert torch.allclose(R.soft_cap(x, 2.0), 2 * torch.tanh(x / 2)) and torch.equal(R.soft_cap(x, None), x)
    cfg = U.configs()["even"]
    T = U.make_weights(cfg)
    base = U.oracle_logits(cfg, T, [1, 2, 3])
    T["l0.mix.g"] = T["l0.mix.g"] * 0          # every gate of the layer is 1/2
    assert U.error(U.oracle_logits(cfg, T, [1, 2, 3]), base) > 0.05


def test_oracle_shared_latents_are_the_owners():
    """Changing the owner's down-projection changes its reader; a reader has no down-projection."""
    cfg = U.configs()["full-heads"]
    T = U.make_weights(cfg)
    assert "l2.mix.dkv" not in T and "l1.mix.dkv" in T
    base = U.oracle_logits(cfg, T, U.ids_of(cfg, 9, 0))
    T2 = dict(T)
    T2["l1.mix.dkv.norm"] = T["l1.mix.dkv.norm"] * 1.5
    taps, taps2 = [], []
    U.oracle_logits(cfg, T, U.ids_of(cfg, 9, 0), taps=taps)
    assert U.error(U.oracle_logits(cfg, T2, U.ids_of(cfg, 9, 0), taps=taps2), base) > 0.02
    assert torch.equal(taps[0], taps2[0]) and not torch.equal(taps[2], taps2[2])


def test_decoder_bench_counts_both_models_alike():
    sys.path.insert(0, os.path.join(ROOT, "tools"))
    import bench_decoder as B
    for size, gqa in B.LIKE.items():
        a, b = CFG.get_config(f"debunex-{size}"), CFG.get_config(gqa)
        assert (a.hidden_size, a.vocab_size, a.num_hidden_layers, a.layers[0].ff, a.layers[0].mixer.heads) == \
               (b.hidden_size, b.vocab_size, b.num_hidden_layers, b.intermediate_size, b.num_attention_heads)
        assert 0.8 < B.flops_of(a, 2048) / B.flops_of(b, 2048) < 1.25
        assert 0.8 < B.step_bytes(a, 1, 1024) / B.step_bytes(b, 1, 1024) < 1.25


def test_qwen2vl_weight_layout_is_untouched():
    c = CFG.tiny()
    a = make_arena(c, "cpu")
    assert type(a).__name__ == "WeightArena" and a.is_packed("llm.0.qkv_w") and not a.is_packed("embed") and len(fp8_weight_names(c)) > 0
    w = torch.arange(32 * 32, dtype=torch.float32).view(32, 32)
    assert torch.equal(interleave_gate_up(w, -w)[16:32], -w[:16])
    assert set(decoder_param_shapes(CFG.debunex_tiny())) >= {"embed", "head", "final.norm.alpha", "l2.mix.g"}
