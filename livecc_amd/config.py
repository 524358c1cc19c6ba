"""Model-shape descriptions: the LiveCC / Qwen2-VL hot path, and decoders given as a list of layers (`DebunexConfig`).

The reference never defines shapes itself: `demo/infer.py:43-47` calls
`Qwen2VLForConditionalGeneration.from_pretrained(model_path, ...)` and the shapes come
from the checkpoint's `config.json` (HF `configuration_qwen2_vl.py`, classes
`Qwen2VLVisionConfig` / `Qwen2VLTextConfig` / `Qwen2VLConfig`).  This dataclass is the
single description both the native engine and the HF oracle are built from.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Any, List, Optional


@dataclasses.dataclass
class LiveCCConfig:
    # ---- language model (Qwen2VLTextConfig) ----
    vocab_size: int = 152064
    hidden_size: int = 3584
    intermediate_size: int = 18944
    num_hidden_layers: int = 28
    num_attention_heads: int = 28
    num_key_value_heads: int = 4
    head_dim: int = 128
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1e6
    mrope_section: List[int] = dataclasses.field(default_factory=lambda: [16, 24, 24])
    max_position_embeddings: int = 32768
    tie_word_embeddings: bool = False
    # ---- vision tower (Qwen2VLVisionConfig) ----
    vit_depth: int = 32
    vit_embed_dim: int = 1280
    vit_num_heads: int = 16
    vit_mlp_ratio: int = 4
    patch_size: int = 14
    temporal_patch_size: int = 2
    spatial_merge_size: int = 2
    in_channels: int = 3
    # ---- special ids (Qwen2VLConfig) ----
    image_token_id: int = 151655
    video_token_id: int = 151656
    vision_start_token_id: int = 151652
    vision_end_token_id: int = 151653
    eos_token_id: int = 151645      # <|im_end|>
    bos_token_id: int = 151643      # <|endoftext|>
    name: str = "livecc-7b"

    # ---- derived ----
    @property
    def vit_head_dim(self) -> int:
        return self.vit_embed_dim // self.vit_num_heads

    @property
    def vit_mlp_dim(self) -> int:
        return self.vit_embed_dim * self.vit_mlp_ratio

    @property
    def patch_dim(self) -> int:  # 3*2*14*14 = 1176
        return self.in_channels * self.temporal_patch_size * self.patch_size * self.patch_size

    @property
    def merge_dim(self) -> int:  # 1280*4 = 5120
        return self.vit_embed_dim * self.spatial_merge_size ** 2

    @property
    def q_dim(self) -> int:
        return self.num_attention_heads * self.head_dim

    @property
    def kv_dim(self) -> int:
        return self.num_key_value_heads * self.head_dim

    @property
    def qkv_dim(self) -> int:
        return self.q_dim + 2 * self.kv_dim

    @property
    def kv_bytes_per_token(self) -> int:  # bf16 K+V over all layers
        return 2 * self.num_hidden_layers * self.kv_dim * 2

    def validate(self) -> None:
        assert self.head_dim == 128, "LLM attention kernels are built for head_dim 128 (all Qwen2-VL sizes)"
        assert self.vit_head_dim == 80, "ViT attention kernel is built for head_dim 80 (all Qwen2-VL sizes)"
        assert sum(self.mrope_section) * 2 == self.head_dim
        assert self.num_attention_heads % self.num_key_value_heads == 0
        assert self.num_attention_heads // self.num_key_value_heads <= 16
        for d in (self.hidden_size, self.intermediate_size, self.vit_embed_dim, self.vit_mlp_dim):
            assert d % 16 == 0, f"dimension {d} must be a multiple of 16"
        assert self.vocab_size % 16 == 0

    # ---- llm / vit parameter and byte counts ----
    def llm_layer_params(self) -> int:
        h, i = self.hidden_size, self.intermediate_size
        return h * self.qkv_dim + self.qkv_dim + self.q_dim * h + 3 * h * i + 2 * h

    def decode_weight_bytes(self) -> int:
        """bf16 weight bytes streamed by one decode step (layers + final norm + lm_head)."""
        return 2 * (self.num_hidden_layers * self.llm_layer_params() + self.hidden_size
                    + self.vocab_size * self.hidden_size)

    # ---- conversions ----
    def to_hf(self, dtype=None, attn_implementation: str = "sdpa"):
        """Build the HF `Qwen2VLConfig` with the same shapes (oracle side)."""
        from transformers import Qwen2VLConfig
        text = dict(
            vocab_size=self.vocab_size, hidden_size=self.hidden_size,
            intermediate_size=self.intermediate_size, num_hidden_layers=self.num_hidden_layers,
            num_attention_heads=self.num_attention_heads, num_key_value_heads=self.num_key_value_heads,
            max_position_embeddings=self.max_position_embeddings, rms_norm_eps=self.rms_norm_eps,
            rope_parameters={"rope_type": "default", "rope_theta": self.rope_theta,
                             "mrope_section": list(self.mrope_section)},
            bos_token_id=self.bos_token_id, eos_token_id=self.eos_token_id,
        )
        vision = dict(
            depth=self.vit_depth, embed_dim=self.vit_embed_dim, hidden_size=self.hidden_size,
            mlp_ratio=self.vit_mlp_ratio, num_heads=self.vit_num_heads, in_channels=self.in_channels,
            patch_size=self.patch_size, spatial_merge_size=self.spatial_merge_size,
            temporal_patch_size=self.temporal_patch_size,
        )
        cfg = Qwen2VLConfig(
            text_config=text, vision_config=vision,
            image_token_id=self.image_token_id, video_token_id=self.video_token_id,
            vision_start_token_id=self.vision_start_token_id, vision_end_token_id=self.vision_end_token_id,
            tie_word_embeddings=self.tie_word_embeddings,
        )
        cfg._attn_implementation = attn_implementation
        if dtype is not None:
            cfg.dtype = dtype
        return cfg

    @classmethod
    def from_hf(cls, hf_cfg, name: str = "from-hf") -> "LiveCCConfig":
        t, v = hf_cfg.text_config, hf_cfg.vision_config
        rp = t.rope_parameters
        eos = t.eos_token_id if not isinstance(t.eos_token_id, (list, tuple)) else t.eos_token_id[0]
        return cls(
            vocab_size=t.vocab_size, hidden_size=t.hidden_size, intermediate_size=t.intermediate_size,
            num_hidden_layers=t.num_hidden_layers, num_attention_heads=t.num_attention_heads,
            num_key_value_heads=t.num_key_value_heads,
            head_dim=getattr(t, "head_dim", None) or t.hidden_size // t.num_attention_heads,
            rms_norm_eps=t.rms_norm_eps, rope_theta=float(rp["rope_theta"]),
            mrope_section=list(rp["mrope_section"]), max_position_embeddings=t.max_position_embeddings,
            tie_word_embeddings=bool(getattr(hf_cfg, "tie_word_embeddings", False)),
            vit_depth=v.depth, vit_embed_dim=v.embed_dim, vit_num_heads=v.num_heads,
            vit_mlp_ratio=v.mlp_ratio, patch_size=v.patch_size, temporal_patch_size=v.temporal_patch_size,
            spatial_merge_size=v.spatial_merge_size, in_channels=v.in_channels,
            image_token_id=hf_cfg.image_token_id, video_token_id=hf_cfg.video_token_id,
            vision_start_token_id=hf_cfg.vision_start_token_id, vision_end_token_id=hf_cfg.vision_end_token_id,
            eos_token_id=eos, bos_token_id=t.bos_token_id if t.bos_token_id is not None else 151643,
            name=name,
        )

    @classmethod
    def from_pretrained(cls, path: str) -> "LiveCCConfig":
        """Read a checkpoint directory's config.json (what `from_pretrained` does in demo/infer.py:43)."""
        with open(os.path.join(path, "config.json")) as f:
            raw = json.load(f)
        from transformers import Qwen2VLConfig
        return cls.from_hf(Qwen2VLConfig(**raw), name=os.path.basename(os.path.normpath(path)))


# Public checkpoint shapes (re-verified at load when a checkpoint is given).
def livecc_7b() -> LiveCCConfig:
    return LiveCCConfig(name="livecc-7b")


def qwen2vl_2b() -> LiveCCConfig:
    return LiveCCConfig(vocab_size=151936, hidden_size=1536, intermediate_size=8960, num_hidden_layers=28,
                        num_attention_heads=12, num_key_value_heads=2, tie_word_embeddings=True,
                        name="qwen2vl-2b")


def qwen2vl_2b_untied() -> LiveCCConfig:
    """Qwen2-VL-2B shapes with a separate lm_head (parity tests with the `decisive` synthetic weights, whose lm_head is a row
    permutation of the embedding table)."""
    c = qwen2vl_2b()
    c.tie_word_embeddings, c.name = False, "qwen2vl-2b-untied"
    return c


def qwen2vl_72b() -> LiveCCConfig:
    return LiveCCConfig(hidden_size=8192, intermediate_size=29568, num_hidden_layers=80,
                        num_attention_heads=64, num_key_value_heads=8, name="qwen2vl-72b")


def tiny(vocab_size: int = 2048) -> LiveCCConfig:
    """Small shapes with the true head dims (128 / 80) for fast CPU-oracle parity tests."""
    return LiveCCConfig(
        vocab_size=vocab_size, hidden_size=256, intermediate_size=512, num_hidden_layers=2,
        num_attention_heads=2, num_key_value_heads=1, vit_depth=2, vit_embed_dim=160, vit_num_heads=2,
        image_token_id=vocab_size - 9, video_token_id=vocab_size - 8, vision_start_token_id=vocab_size - 12,
        vision_end_token_id=vocab_size - 11, eos_token_id=vocab_size - 3, bos_token_id=vocab_size - 5,
        name="tiny",
    )


def small() -> LiveCCConfig:
    """Mid-size shapes (GQA group 7 like the 7B, 4 layers) for GPU parity runs that finish in seconds."""
    return LiveCCConfig(
        vocab_size=8192, hidden_size=896, intermediate_size=2432, num_hidden_layers=4,
        num_attention_heads=7, num_key_value_heads=1, vit_depth=4, vit_embed_dim=320, vit_num_heads=4,
        image_token_id=8183, video_token_id=8184, vision_start_token_id=8180, vision_end_token_id=8181,
        eos_token_id=8189, bos_token_id=8187, name="small",
    )


# ---- layer-list decoders ----
def _up(n: int, m: int = 64) -> int:
    return (n + m - 1) // m * m


def pad_head_dim(d: int) -> int:
    """Stored channels per head: 64 or 128 (the MFMA attention kernels), else the next multiple of 64."""
    return _up(d)


KV_RANK_TILES = (1, 2, 3, 4, 6, 8, 12, 16)       # 64-channel tiles the latent decode attention is built for


def pad_kv_rank(r: int) -> int:
    for t in KV_RANK_TILES:
        if r <= 64 * t:
            return 64 * t
    raise ValueError(f"latent rank {r} exceeds {64 * KV_RANK_TILES[-1]}, the largest the latent attention kernels are built for")


@dataclasses.dataclass
class LatentMixerSpec:
    """Latent attention without positions: queries and keys / values through normed low-rank vectors, a sigmoid gate per head."""
    heads: int
    dim: int                      # query / key channels per head
    vdim: int                     # value channels per head
    q_rank: int
    kv_rank: int
    scale: float
    kv_from: Optional[int] = None  # the layer whose cached latent this one reads (None: its own)

    @property
    def dim_pad(self) -> int:
        return pad_head_dim(self.dim)

    @property
    def vdim_pad(self) -> int:
        return pad_head_dim(self.vdim)

    @property
    def q_rank_pad(self) -> int:
        return _up(self.q_rank)

    @property
    def kv_rank_pad(self) -> int:
        return pad_kv_rank(self.kv_rank)

    @property
    def in_rows(self) -> int:
        """Rows of the fused input projection: query latent | own cache latent | gates."""
        return self.q_rank_pad + (self.kv_rank_pad if self.kv_from is None else 0) + _up(self.heads, 16)


@dataclasses.dataclass
class DecoderLayerSpec:
    mixer: Any                    # LatentMixerSpec, ParallelMixerSpec or SsdMixerSpec
    ff: int = 0                   # width of the gated feed-forward; 0: none

    @property
    def ff_pad(self) -> int:
        return _up(self.ff)


@dataclasses.dataclass
class DebunexConfig:
    """A decoder-only language model given as a list of layers; both sublayers of a layer run in parallel behind one Dynamic-Tanh norm."""
    vocab_size: int
    hidden_size: int
    layers: List[DecoderLayerSpec]
    norm_eps: float = 1e-5
    logit_softcap: Optional[float] = None
    max_position_embeddings: int = 32768          # default KV capacity of a stream; the model itself has no positions
    eos_token_id: Optional[int] = None
    name: str = "debunex"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def width_pad(self) -> int:
        return _up(self.hidden_size)

    @property
    def vocab_pad(self) -> int:
        return _up(self.vocab_size)

    @property
    def kv_bytes_per_token(self) -> int:
        return sum(2 * l.mixer.kv_rank_pad for l in self.layers if l.mixer.kv_from is None)

    def decode_weight_bytes(self) -> int:
        """bf16 weight bytes one decode step reads (stored sizes)."""
        n = self.vocab_pad * self.width_pad
        for l in self.layers:
            m = l.mixer
            n += m.in_rows * self.width_pad + m.heads * m.dim_pad * (m.q_rank_pad + m.kv_rank_pad) + m.heads * m.vdim_pad * m.kv_rank_pad
            n += self.width_pad * (m.heads * m.vdim_pad + 3 * l.ff_pad)
        return 2 * n

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a decoder needs at least one layer")
        for i, l in enumerate(self.layers):
            m = l.mixer
            if min(m.heads, m.dim, m.vdim, m.q_rank, m.kv_rank) < 1 or l.ff < 0:
                raise ValueError(f"layer {i}: sizes must be positive")
            if max(m.dim_pad, m.vdim_pad) > 1024:
                raise ValueError(f"layer {i}: head sizes above 1024 are not supported")
            pad_kv_rank(m.kv_rank)
            if m.kv_from is not None:
                if not 0 <= m.kv_from < i:
                    raise ValueError(f"layer {i}: kv_from {m.kv_from} is not an earlier layer")
                o = self.layers[m.kv_from].mixer
                if o.kv_from is not None or o.kv_rank != m.kv_rank:
                    raise ValueError(f"layer {i}: layer {m.kv_from} has no latent of rank {m.kv_rank} of its own")

    @classmethod
    def from_dict(cls, raw: dict, name: str = "debunex") -> "DebunexConfig":
        layers = []
        for i, e in enumerate(raw["layers"]):
            if e["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown layer type {e['type']!r}")
            m = e["mixer"]
            mlp = e.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            kf = m.get("kv_from")
            layers.append(DecoderLayerSpec(
                LatentMixerSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]),
                                scale=float(m["scale"]), kv_from=None if kf is None else int(kf)), 0 if mlp is None else int(mlp["ff"])))
        cap, eos = raw.get("logit_softcap"), raw.get("eos_token_id")
        cfg = cls(vocab_size=int(raw["vocab"]), hidden_size=int(raw["width"]), layers=layers, norm_eps=float(raw["norm"]["eps"]),
                  logit_softcap=None if cap is None else float(cap), eos_token_id=None if eos is None else int(eos), name=name)
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        """The config.json form."""
        out = {"architecture": "Debunex", "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps}, "layers": []}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        for l in self.layers:
            m = {k: v for k, v in dataclasses.asdict(l.mixer).items() if v is not None}
            out["layers"].append({"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None})
        return out

    @classmethod
    def from_pretrained(cls, path: str) -> "DebunexConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), name=os.path.basename(os.path.normpath(path)))


def _debunex(width, vocab, n_layers, ff, heads, dim, vdim, q_rank, kv_rank, share, name, cap=30.0, eps=1e-5) -> DebunexConfig:
    """`share`: layers per cached latent (1: every layer its own)."""
    layers = [DecoderLayerSpec(LatentMixerSpec(heads, dim, vdim, q_rank, kv_rank, dim ** -0.5, None if i % share == 0 else i - i % share), ff)
              for i in range(n_layers)]
    return DebunexConfig(vocab, width, layers, eps, cap, name=name)


def debunex_tiny() -> DebunexConfig:
    return _debunex(192, 320, 3, 256, 3, 24, 40, 48, 56, 2, "debunex-tiny")


def debunex_2b() -> DebunexConfig:
    """Qwen2-VL-2B's width, feed-forward, heads, depth and vocabulary with latent attention."""
    return _debunex(1536, 151936, 28, 8960, 12, 128, 128, 768, 512, 2, "debunex-2b")


def debunex_7b() -> DebunexConfig:
    """LiveCC-7B's width, feed-forward, heads, depth and vocabulary with latent attention."""
    return _debunex(3584, 152064, 28, 18944, 28, 128, 128, 1536, 512, 2, "debunex-7b")


# ---- layer-list decoders with pre- and post-norms around every sublayer: attention beside linear attention, state-space layers ----
MAX_REC_KEY = 256             # channels of a recurrent state's key side the scan kernels are built for (after padding)
MAX_SOFTMAX_HEAD = 256        # head sizes of the grouped-query decode attention with a distance bias (after padding)
MAX_CONV_TAPS = 16
MAX_ROW_WIDTH = 8192          # widest row of the row-norm kernels


@dataclasses.dataclass
class SoftmaxMixerSpec:
    """Grouped-query softmax attention: per-head query / key norms, a query temperature, a linear distance bias per head, no rotation."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp_coef: float
    q_temp_every: int

    @property
    def dim_pad(self) -> int:
        return pad_head_dim(self.dim)

    @property
    def vdim_pad(self) -> int:
        return pad_head_dim(self.vdim)

    def slopes(self) -> List[float]:
        """Score taken off per token of distance."""
        return [2.0 ** (-8.0 * (h + 1) / self.heads) for h in range(self.heads)]


@dataclasses.dataclass
class LightningMixerSpec:
    """Linear attention with a fixed decay per head."""
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    groups = property(lambda self: self.heads)        # every head has keys and queries of its own
    norm_groups = 1
    conv_taps = 0

    @property
    def key_pad(self) -> int:
        return _up(self.dim)

    @property
    def vdim_pad(self) -> int:
        return _up(self.vdim)


@dataclasses.dataclass
class ParallelMixerSpec:
    """Softmax attention and linear attention over one input; their normed outputs are averaged."""
    left: SoftmaxMixerSpec
    right: LightningMixerSpec

    @property
    def recurrent(self) -> LightningMixerSpec:
        return self.right

    @property
    def in_rows(self) -> int:
        """Rows of the fused input projection: left q | k | v | right q | k | v | gate."""
        l, r = self.left, self.right
        return (l.heads + l.kv_heads) * l.dim_pad + l.kv_heads * l.vdim_pad + 2 * r.heads * (r.key_pad + r.vdim_pad)

    @property
    def kv_bytes_per_token(self) -> int:
        return 2 * self.left.kv_heads * (self.left.dim_pad + self.left.vdim_pad)


@dataclasses.dataclass
class SsdMixerSpec:
    """State-space duality (Mamba-2): a short causal convolution, decays and step sizes from the input, a gated group norm."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv_taps: int
    norm_groups: int

    @property
    def recurrent(self) -> "SsdMixerSpec":
        return self

    @property
    def key_pad(self) -> int:
        return _up(self.state)

    @property
    def vdim_pad(self) -> int:
        return _up(self.vdim)

    @property
    def conv_channels(self) -> int:
        """Stored channels of the convolution: x | B | C."""
        return self.heads * self.vdim_pad + 2 * self.groups * self.key_pad

    @property
    def in_rows(self) -> int:
        """Rows of the input projection: z | x | B | C | dt."""
        return self.heads * self.vdim_pad + self.conv_channels + _up(self.heads)

    kv_bytes_per_token = 0


@dataclasses.dataclass
class BemuzenConfig:
    """A decoder-only language model given as a list of layers: mixer and feed-forward one after the other, a norm before and after each; a hashed
    bigram embedding beside the token's own."""
    vocab_size: int
    hidden_size: int
    layers: List[DecoderLayerSpec]
    bigram_buckets: int
    bigram_mul_prev: int
    bigram_mul_cur: int
    norm_eps: float = 1e-5
    logit_scale: float = 1.0
    max_position_embeddings: int = 32768          # default KV capacity of a stream
    eos_token_id: Optional[int] = None
    name: str = "bemuzen"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def width_pad(self) -> int:
        return _up(self.hidden_size)

    @property
    def vocab_pad(self) -> int:
        return _up(self.vocab_size)

    @property
    def kv_bytes_per_token(self) -> int:
        return sum(l.mixer.kv_bytes_per_token for l in self.layers)

    @property
    def state_bytes(self) -> int:
        """Recurrent state of one stream (fp32)."""
        n = 0
        for l in self.layers:
            r = l.mixer.recurrent
            n += 4 * r.heads * r.key_pad * r.vdim_pad + (4 * r.conv_taps * r.conv_channels if r.conv_taps else 0)
        return n

    def decode_weight_bytes(self) -> int:
        """bf16 weight bytes one decode step reads (stored sizes)."""
        n = self.vocab_pad * self.width_pad
        for l in self.layers:
            m, r = l.mixer, l.mixer.recurrent
            n += self.width_pad * (m.in_rows + _up(r.heads * r.vdim) + 3 * l.ff_pad)
            if isinstance(m, ParallelMixerSpec):
                n += self.width_pad * m.left.heads * m.left.vdim_pad
        return 2 * n

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a decoder needs at least one layer")
        if min(self.vocab_size, self.hidden_size, self.bigram_buckets) < 1:
            raise ValueError("vocabulary, width and bigram buckets must be positive")
        if self.width_pad > MAX_ROW_WIDTH:
            raise ValueError(f"widths above {MAX_ROW_WIDTH} are not supported")
        if min(self.bigram_mul_prev, self.bigram_mul_cur) < 0:
            raise ValueError("bigram multipliers must not be negative")
        for i, l in enumerate(self.layers):
            m, r = l.mixer, l.mixer.recurrent
            if l.ff < 0 or min(r.heads, r.vdim, r.groups, r.norm_groups) < 1:
                raise ValueError(f"layer {i}: sizes must be positive")
            if isinstance(m, ParallelMixerSpec):
                a = m.left
                if min(a.heads, a.kv_heads, a.dim, a.vdim, a.q_temp_every, r.dim) < 1:
                    raise ValueError(f"layer {i}: sizes must be positive")
                if a.heads % a.kv_heads:
                    raise ValueError(f"layer {i}: {a.heads} heads over {a.kv_heads} key/value heads")
                if max(a.dim_pad, a.vdim_pad) > MAX_SOFTMAX_HEAD:
                    raise ValueError(f"layer {i}: head sizes above {MAX_SOFTMAX_HEAD} are not supported")
                if len(r.decay) != r.heads or min(r.decay) < 0.0 or max(r.decay) > 1.0:
                    raise ValueError(f"layer {i}: one decay in [0, 1] per head")
            else:
                if min(m.state, m.conv_taps) < 1 or m.conv_taps > MAX_CONV_TAPS:
                    raise ValueError(f"layer {i}: state must be positive, convolution taps in 1..{MAX_CONV_TAPS}")
                if m.heads % m.groups or (m.heads * m.vdim) % m.norm_groups:
                    raise ValueError(f"layer {i}: {m.heads} heads in {m.groups} groups, {m.heads * m.vdim} channels in {m.norm_groups} norm groups")
            if r.key_pad > MAX_REC_KEY:
                raise ValueError(f"layer {i}: recurrent key sizes above {MAX_REC_KEY} are not supported")

    @classmethod
    def from_dict(cls, raw: dict, name: str = "bemuzen") -> "BemuzenConfig":
        layers = []
        for i, e in enumerate(raw["layers"]):
            m, mlp = e["mixer"], e.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            if e["type"] == "parallel":
                l, r = m["left"], m["right"]
                spec = ParallelMixerSpec(
                    SoftmaxMixerSpec(int(l["heads"]), int(l["kv_heads"]), int(l["dim"]), int(l["vdim"]), float(l["scale"]), float(l["q_temp"]["coef"]),
                                     int(l["q_temp"]["every"])),
                    LightningMixerSpec(int(r["heads"]), int(r["dim"]), int(r["vdim"]), [float(x) for x in r["decay"]]))
            elif e["type"] == "mamba2":
                spec = SsdMixerSpec(int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["conv"]), int(m["norm_groups"]))
            else:
                raise ValueError(f"layer {i}: unknown layer type {e['type']!r}")
            layers.append(DecoderLayerSpec(spec, 0 if mlp is None else int(mlp["ff"])))
        b, eos = raw["embedding"]["bigram"], raw.get("eos_token_id")
        cfg = cls(vocab_size=int(raw["vocab"]), hidden_size=int(raw["width"]), layers=layers, bigram_buckets=int(b["buckets"]),
                  bigram_mul_prev=int(b["mul_prev"]), bigram_mul_cur=int(b["mul_cur"]), norm_eps=float(raw["norm"]["eps"]),
                  logit_scale=float(raw["logit_scale"]), eos_token_id=None if eos is None else int(eos), name=name)
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        """The config.json form."""
        out = {"architecture": "Bemuzen", "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps},
               "logit_scale": self.logit_scale, "layers": [],
               "embedding": {"bigram": {"buckets": self.bigram_buckets, "mul_prev": self.bigram_mul_prev, "mul_cur": self.bigram_mul_cur}}}
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        for l in self.layers:
            m = l.mixer
            if isinstance(m, ParallelMixerSpec):
                a, r = m.left, m.right
                kind, mix = "parallel", {
                    "left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                             "q_temp": {"coef": a.q_temp_coef, "every": a.q_temp_every}},
                    "right": {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "decay": list(r.decay)}}
            else:
                kind, mix = "mamba2", {"heads": m.heads, "vdim": m.vdim, "state": m.state, "groups": m.groups, "conv": m.conv_taps, "norm_groups": m.norm_groups}
            out["layers"].append({"type": kind, "mixer": mix, "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None})
        return out

    @classmethod
    def from_pretrained(cls, path: str) -> "BemuzenConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), name=os.path.basename(os.path.normpath(path)))


def _bemuzen(width, vocab, n_layers, ff, left, right, ssd, every, name) -> BemuzenConfig:
    """Every `every`-th layer is a state-space layer, the others run attention beside linear attention."""
    layers = [DecoderLayerSpec(dataclasses.replace(ssd) if i % every == every - 1 else ParallelMixerSpec(dataclasses.replace(left), dataclasses.replace(right)), ff)
              for i in range(n_layers)]
    return BemuzenConfig(vocab, width, layers, 65521, 8191, 131, name=name)


def _decays(heads: int) -> List[float]:
    return [1.0 - 2.0 ** (-2.0 - 6.0 * h / max(heads - 1, 1)) for h in range(heads)]


def bemuzen_tiny() -> BemuzenConfig:
    return _bemuzen(192, 320, 3, 224, SoftmaxMixerSpec(6, 2, 24, 40, 0.2, 0.25, 48), LightningMixerSpec(3, 40, 24, _decays(3)), SsdMixerSpec(6, 24, 40, 2, 3, 3),
                    3, "bemuzen-tiny")


def bemuzen_2b() -> BemuzenConfig:
    """Qwen2-VL-2B's width, feed-forward, attention heads, depth and vocabulary."""
    return _bemuzen(1536, 151936, 28, 8960, SoftmaxMixerSpec(12, 2, 128, 128, 128 ** -0.5, 0.1, 4096), LightningMixerSpec(12, 128, 128, _decays(12)),
                    SsdMixerSpec(48, 64, 128, 1, 4, 1), 4, "bemuzen-2b")


def bemuzen_7b() -> BemuzenConfig:
    """LiveCC-7B's width, feed-forward, attention heads, depth and vocabulary."""
    return _bemuzen(3584, 152064, 28, 18944, SoftmaxMixerSpec(28, 4, 128, 128, 128 ** -0.5, 0.1, 4096), LightningMixerSpec(28, 128, 128, _decays(28)),
                    SsdMixerSpec(112, 64, 128, 1, 4, 1), 4, "bemuzen-7b")


# config.json "architecture" -> configuration class; checkpoints without the key are Qwen2-VL ones
ARCHITECTURES = {"Debunex": DebunexConfig, "Bemuzen": BemuzenConfig}
DECODER_CONFIGS = tuple(ARCHITECTURES.values())          # layer lists: served by the engine's decoder family


PRESETS = {"livecc-7b": livecc_7b, "qwen2vl-2b": qwen2vl_2b, "qwen2vl-2b-untied": qwen2vl_2b_untied, "qwen2vl-72b": qwen2vl_72b,
           "tiny": tiny, "small": small, "debunex-tiny": debunex_tiny, "debunex-2b": debunex_2b, "debunex-7b": debunex_7b,
           "bemuzen-tiny": bemuzen_tiny, "bemuzen-2b": bemuzen_2b, "bemuzen-7b": bemuzen_7b}


def architecture_of(path: str) -> Optional[str]:
    """The "architecture" of a checkpoint directory's config.json, None for a Qwen2-VL one."""
    with open(os.path.join(path, "config.json")) as f:
        arch = json.load(f).get("architecture")
    if arch is not None and arch not in ARCHITECTURES:
        raise KeyError(f"unknown architecture {arch!r} in {path}; known: {sorted(ARCHITECTURES)}")
    return arch


def get_config(name: str):
    if name in PRESETS:
        return PRESETS[name]()
    if os.path.isdir(name):
        arch = architecture_of(name)
        return (LiveCCConfig if arch is None else ARCHITECTURES[arch]).from_pretrained(name)
    raise KeyError(f"unknown config {name!r}; presets: {sorted(PRESETS)}")
