"""Model configurations (public architecture hyper-parameters; random-init weights).

The four families BASELINE.json names for the LLM service:
  * Llama-3-8B  (smart reply / summarize, TP=1)        - flagship bench model
  * Llama-3-70B (ask-AI, TP=8 over xGMI)
  * Gemma-2B    (smart reply, TP=1; MQA, head_dim 256, GELU-tanh, (1+w) norm)
  * Mixtral-8x7B (context suggestions; top-2 of 8 experts, EP)
plus tiny variants of each for CPU tests.

:class:`HybridConfig` describes models whose layers differ (mixer kind, sizes, window, with or
without a feed-forward): the Ralesun design, latent attention and channel-wise gated delta-rule
mixers one after the other with their feed-forward; the Mebalorn design, talking-heads attention
and minGRU mixers beside it; the Nurilorn design, attention with convolved projections and
capped scores, followed by a clamped feed-forward or routed experts; and the Garesun design,
retention, matrix memory and latent attention with shared latents beside squared-relu experts.
Their checkpoints carry a config.json, parsed by :func:`config_from_dict`.
"""
from __future__ import annotations

import dataclasses
import json
import os
from dataclasses import dataclass, field


@dataclass(frozen=True)
class ModelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    intermediate_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    head_dim: int
    rope_theta: float = 500000.0
    rope_scaling: dict | None = field(default=None, hash=False, compare=False)
    rms_eps: float = 1e-5
    max_position: int = 8192
    act: str = "silu"                # silu | gelu_tanh
    gemma_norm: bool = False         # weight convention (1 + w)
    embed_scale: bool = False        # Gemma multiplies embeddings by sqrt(H)
    tie_embeddings: bool = False
    num_experts: int = 0             # 0 = dense MLP
    experts_per_token: int = 2
    bos_token_id: int = 1
    eos_token_id: int = 2
    init_std: float = 0.02
    query_pre_attn_scalar: float | None = None
    prefill_chunk: int = 16384       # engine prefill step, tokens (LLMEngine.prefill_chunk_tokens)

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    @property
    def attn_scale(self) -> float:
        s = self.query_pre_attn_scalar or self.head_dim
        return float(s) ** -0.5

    @property
    def is_moe(self) -> bool:
        return self.num_experts > 0

    def num_params(self) -> int:
        H, I, L, V = self.hidden_size, self.intermediate_size, self.num_layers, self.vocab_size
        attn = H * (self.q_size + 2 * self.kv_size) + self.q_size * H
        mlp = 3 * H * I * (self.num_experts if self.is_moe else 1) + (H * self.num_experts)
        emb = V * H * (1 if self.tie_embeddings else 2)
        return L * (attn + mlp + 2 * H) + emb + H

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return 2 * self.num_layers * self.kv_size * dtype_bytes

    def replace(self, **kw) -> "ModelConfig":
        return dataclasses.replace(self, **kw)


LLAMA3_8B = ModelConfig(
    name="llama-3-8b", vocab_size=128256, hidden_size=4096, intermediate_size=14336,
    num_layers=32, num_heads=32, num_kv_heads=8, head_dim=128, rope_theta=500000.0,
    rms_eps=1e-5, max_position=8192, bos_token_id=128000, eos_token_id=128001)

LLAMA3_70B = ModelConfig(
    name="llama-3-70b", vocab_size=128256, hidden_size=8192, intermediate_size=28672,
    num_layers=80, num_heads=64, num_kv_heads=8, head_dim=128, rope_theta=500000.0,
    rms_eps=1e-5, max_position=8192, bos_token_id=128000, eos_token_id=128001,
    prefill_chunk=36864)  # a whole ask wave (256 x ~136 tokens) in one step, profiles/r6t

GEMMA_2B = ModelConfig(
    name="gemma-2b", vocab_size=256000, hidden_size=2048, intermediate_size=16384,
    num_layers=18, num_heads=8, num_kv_heads=1, head_dim=256, rope_theta=10000.0,
    rms_eps=1e-6, max_position=8192, act="gelu_tanh", gemma_norm=True, embed_scale=True,
    tie_embeddings=True, bos_token_id=2, eos_token_id=1)

MIXTRAL_8X7B = ModelConfig(
    name="mixtral-8x7b", vocab_size=32000, hidden_size=4096, intermediate_size=14336,
    num_layers=32, num_heads=32, num_kv_heads=8, head_dim=128, rope_theta=1e6,
    rms_eps=1e-5, max_position=32768, num_experts=8, experts_per_token=2,
    bos_token_id=1, eos_token_id=2,
    prefill_chunk=32768)  # 8k rows per expert in the prefill MoE GEMMs, profiles/r6t

# Tiny shapes with the same structural features, for CPU tests and smoke runs.
TINY_LLAMA = ModelConfig(
    name="tiny-llama", vocab_size=512, hidden_size=256, intermediate_size=512,
    num_layers=2, num_heads=4, num_kv_heads=2, head_dim=64, rope_theta=10000.0,
    max_position=1024, bos_token_id=1, eos_token_id=2)

TINY_GEMMA = ModelConfig(
    name="tiny-gemma", vocab_size=512, hidden_size=256, intermediate_size=512,
    num_layers=2, num_heads=2, num_kv_heads=1, head_dim=128, rope_theta=10000.0,
    rms_eps=1e-6, max_position=1024, act="gelu_tanh", gemma_norm=True, embed_scale=True,
    tie_embeddings=True, bos_token_id=2, eos_token_id=1)

TINY_MIXTRAL = ModelConfig(
    name="tiny-mixtral", vocab_size=512, hidden_size=256, intermediate_size=256,
    num_layers=2, num_heads=4, num_kv_heads=2, head_dim=64, rope_theta=1e6,
    max_position=1024, num_experts=4, experts_per_token=2, bos_token_id=1, eos_token_id=2)


# ------------------------------------------------------------------ layers of mixed kinds
@dataclass(frozen=True)
class LatentAttention:
    """Attention over per-token latents: heads of ``dim`` unrotated + ``rot_dim`` rotated query
    dims, values of ``vdim``, latents of ``kv_rank``; ``window`` tokens visible (None: all);
    the first ``rot_dims`` rotated dims turned in interleaved pairs; a softmax sink and a sigmoid
    gate per head.  ``kv_from``: attends to that layer's cached latents instead of its own."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int | None
    rot_base: float
    rot_dims: int
    sink: bool = True
    gate: bool = False
    kv_from: int | None = None

    def __post_init__(self):
        if self.rot_dims % 2 or self.rot_dims > self.rot_dim:
            raise ValueError(f"rotated dims {self.rot_dims} of a {self.rot_dim}-wide part")
        if self.kv_rank % 2 or self.rot_dim % 2:
            raise ValueError("latent attention kernels take even latents and rotated parts")
        if not self.scale > 0:
            raise ValueError("scores need a positive scale")
        if self.window is not None and self.window < 1:
            raise ValueError("a window holds at least the token itself")
        if self.kv_rank > 1024 or self.vdim > 1024:
            raise ValueError("latent attention kernels take latents and values up to 1024")


@dataclass(frozen=True)
class ChannelDelta:
    """Gated delta rule with one decay per head and key channel; ``conv`` taps of the short
    convolutions; ``decay_rank`` / ``gate_rank``: inner sizes of the decay and gate projections
    (a checkpoint's tensors set them)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int | None = None
    gate_rank: int | None = None

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("heads must divide by kv_heads")
        if self.dim > 256 or self.vdim > 512:
            raise ValueError("delta-rule kernels take dim <= 256 and vdim <= 512")

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclass(frozen=True)
class TalkingAttention:
    """Grouped-query attention without rotation: biased projections, unit-rms queries and keys of
    ``dim``, values of ``vdim``, a softmax sink per head, normalised weights mixed across the
    query heads."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    sink: bool = True

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("heads must divide by kv_heads")
        if not self.scale > 0:
            raise ValueError("scores need a positive scale")
        if max(self.dim, self.vdim) > 256:
            raise ValueError("talking-heads kernels take head sizes up to 256")
        if self.heads * (self.dim + self.vdim + 144) > 40000:
            raise ValueError("talking-heads kernels hold a query of all heads in LDS: too many heads")

    @property
    def params(self) -> int:
        """Parameters besides the input and output projections."""
        return self.heads * (self.dim + 1 + self.heads) + \
            self.kv_heads * (self.dim + self.vdim) + 2 * self.dim


@dataclass(frozen=True)
class GatedAverage:
    """minGRU: ``width`` channels, each a gated average of projected candidates."""
    width: int

    def __post_init__(self):
        if self.width < 1:
            raise ValueError("a recurrence needs channels")


def _check_memory(m) -> None:
    if m.heads < 1 or not 1 <= m.dim <= 256 or not 1 <= m.vdim <= 1024:
        raise ValueError("matrix memories take keys up to 256 and values up to 1024 wide")


@dataclass(frozen=True)
class Retention:
    """Linear attention with a fixed ``decay`` per head; the first ``rot_dims`` dims of queries and
    keys turned in pairs half of them apart."""
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]
    rot_base: float = 10000.0
    rot_dims: int = 0

    def __post_init__(self):
        _check_memory(self)
        if len(self.decay) != self.heads or not all(0 < x <= 1 for x in self.decay):
            raise ValueError("retention takes a decay above 0 and up to 1 for each head")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"rotated dims {self.rot_dims} of a {self.dim}-wide head")


@dataclass(frozen=True)
class MatrixMemory:
    """mLSTM: linear attention with exponential input and sigmoid forget gates per head and token,
    both capped at +-``gate_cap`` in the logarithm, read out against a normaliser."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def __post_init__(self):
        _check_memory(self)
        if not self.gate_cap > 0:
            raise ValueError("gates are capped at a positive number")


@dataclass(frozen=True)
class RotaryScaling:
    """Rotation for contexts ``factor`` times the ``original`` one (ops.build_interleaved_rope):
    pairs that turn more than ``fast`` times within it keep their speed, those below ``slow`` turns
    are slowed down by the factor."""
    factor: float
    original: float
    fast: float
    slow: float

    def __post_init__(self):
        if min(self.factor, self.original, self.fast, self.slow) <= 0:
            raise ValueError("rotation scaling takes positive numbers")


@dataclass(frozen=True)
class GroupedAttention:
    """Grouped-query attention whose projected queries, keys and values pass a causal convolution
    of ``conv`` taps (0: none); the first ``rot_dims`` dims of queries and keys turned in interleaved pairs;
    scores capped at +-``softcap`` (0: not); a softmax sink of score 0; values mixed with those of
    the first mixing layer (``v_mix``); a sigmoid gate per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    rot_scaling: RotaryScaling | None = None
    conv: int = 0
    softcap: float = 0.0
    v_mix: bool = False
    sink: bool = True
    gate: bool = True

    def __post_init__(self):
        if self.heads < 1 or self.kv_heads < 1 or self.heads % self.kv_heads:
            raise ValueError("heads must divide by kv_heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"rotated dims {self.rot_dims} of a {self.dim}-wide head")
        if not self.scale > 0 or self.softcap < 0:
            raise ValueError("scores need a positive scale and cap")
        if max(self.dim, self.vdim) > 1024:
            raise ValueError("grouped attention kernels take head sizes up to 1024")
        if not 0 <= self.conv <= 64:
            raise ValueError("projection convolutions take up to 64 taps")

    @property
    def channels(self) -> int:
        return (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim


@dataclass(frozen=True)
class Experts:
    """A mixture of ``count`` small feed-forwards, ``top`` of them per token, chosen by softmax
    scores within the ``keep`` best of ``groups`` equal groups of neighbours."""
    count: int
    top: int
    groups: int = 1
    keep: int = 1

    def __post_init__(self):
        if not 1 <= self.keep <= self.groups <= 64 or self.count % self.groups:
            raise ValueError("experts form up to 64 equal groups")
        if not 1 <= self.top <= min(16, self.keep * (self.count // self.groups)) or self.count > 256:
            raise ValueError("routing takes up to 256 experts, 16 of them per token, and as many as "
                             "the kept groups hold")


@dataclass(frozen=True)
class Layer:
    mixer: LatentAttention | ChannelDelta | TalkingAttention | GatedAverage | GroupedAttention | \
        Retention | MatrixMemory
    ff: int | None = None  # feed-forward size; None: the layer is its mixer alone
    limit: float = 0.0     # bound of the clamped activation
    experts: Experts | None = None  # the feed-forward is this mixture, ``ff`` each expert's size
    shared: int | None = None  # size of the expert that every token uses beside them


@dataclass(frozen=True)
class HybridConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: tuple[Layer, ...]
    norm_eps: float = 1e-6
    act: str = "gelu_tanh"
    max_position: int = 8192
    bos_token_id: int = 1
    eos_token_id: int = 2
    init_std: float = 0.02
    prefill_chunk: int = 16384
    # the layers' structure: "serial" (norm, mixer, norm, gated feed-forward), "parallel" (mixer
    # and squared-relu feed-forward on two layer norms of the same stream) or "joint" (both on one
    # layer norm)
    block: str = "serial"
    # serial: "dyt" (Dynamic Tanh) or "group_rms" (RMS norms of norm_groups parts of a row, factors
    # per column on what a sublayer adds); joint: "layer" (layer norms without bias)
    norm: str = "dyt"
    norm_groups: int = 1
    embed_scale: float = 1.0
    residual_mult: float = 1.0            # on everything a sublayer adds
    logit_scale: float = 1.0
    conv_taps: int = 1                    # parallel: causal convolution added to sublayer inputs
    sinusoids: bool = False               # sinusoidal positions added to the embedding
    logit_softcap: float | None = None
    side_dim: int = 0                     # joint: size of a token's own input to each layer

    def __post_init__(self):
        if self.block not in ("serial", "parallel", "joint"):
            raise ValueError(f"unknown layer structure {self.block!r}")
        if self.block != "parallel" and (self.conv_taps != 1 or self.sinusoids or self.logit_softcap):
            raise ValueError("convolved inputs, sinusoids and a logit cap come with parallel layers")
        if self.norm not in ("dyt", "group_rms", "layer"):
            raise ValueError(f"unknown norm {self.norm!r}")
        if (self.norm == "layer") != (self.block == "joint"):
            raise ValueError("joint layers, and only they, have layer norms without bias")
        if self.norm != "group_rms" and (self.norm_groups, self.residual_mult,
                                         self.logit_scale) != (1, 1.0, 1.0):
            raise ValueError("groups and scales come with norms in groups")
        if self.norm == "dyt" and self.embed_scale != 1.0:
            raise ValueError("an embedding scale comes with norms in groups and layer norms")
        self._check_joint()
        if self.norm == "group_rms":
            if self.block != "serial" or self.norm_groups < 1 or \
                    self.hidden_size % self.norm_groups or self.hidden_size + self.norm_groups > 16384:
                raise ValueError("norms in groups take equal parts of serial rows up to 16K columns")
        if self.act == "clamped" and any(l.ff and not l.limit > 0 for l in self.layers):
            raise ValueError("the clamped activation needs a positive limit")
        if any(l.experts and not (l.ff and self.norm != "dyt" and self.block != "parallel")
               for l in self.layers):
            raise ValueError("experts are feed-forwards of layers with norms in groups, or joint ones")
        if len({l.mixer.kv_heads * l.mixer.vdim for l in self.layers
                if isinstance(l.mixer, GroupedAttention) and l.mixer.v_mix}) > 1:
            raise ValueError("layers that mix values need values of one size")
        if not 1 <= self.conv_taps <= 12:
            raise ValueError("input convolutions take 1 to 12 taps")
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ValueError("a logit cap is positive")
        if self.block == "parallel" and \
                self.hidden_size > (8192 if self.hidden_size % 8 == 0 else 4096):
            raise ValueError("convolved layer norms take up to 8192 columns (4096 unless a "
                             "multiple of 8)")

    is_moe = False
    tie_embeddings = False

    def _check_joint(self) -> None:
        joint = self.block == "joint"
        if not joint and (self.side_dim or any(l.shared for l in self.layers)):
            raise ValueError("side inputs and shared experts come with joint layers")
        if joint and (self.act != "relu2" or self.hidden_size > 16384 or self.side_dim < 0):
            raise ValueError("joint layers take squared-relu feed-forwards and rows up to 16K columns")
        if any(l.shared and not l.experts for l in self.layers):
            raise ValueError("a shared expert stands beside others")
        for i, m in enumerate(l.mixer for l in self.layers):
            if not joint and (isinstance(m, (Retention, MatrixMemory))
                              or isinstance(m, LatentAttention) and (m.gate or m.kv_from is not None)):
                raise ValueError("matrix memories, head gates and shared latents come with joint layers")
            if isinstance(m, LatentAttention) and m.kv_from is not None:
                s = self.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
                if not isinstance(s, LatentAttention) or s.kv_from is not None or \
                        (s.kv_rank, s.rot_dim, s.rot_dims, s.rot_base) != \
                        (m.kv_rank, m.rot_dim, m.rot_dims, m.rot_base):
                    raise ValueError(f"layer {i} cannot read the latents of layer {m.kv_from}")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def windows(self) -> tuple:
        """Distinct windows of the attention layers (None: unlimited)."""
        return tuple(dict.fromkeys(l.mixer.window for l in self.layers
                                   if isinstance(l.mixer, LatentAttention)))

    @property
    def taps(self) -> int:
        """The longest causal convolution whose portions are walked in tiles."""
        return max([self.conv_taps] + [l.mixer.conv for l in self.layers
                                       if isinstance(l.mixer, GroupedAttention)])

    def num_params(self) -> int:
        if self.norm == "group_rms":
            return self._num_params_scaled()
        if self.block == "joint":
            return self._num_params_joint()
        W, n = self.hidden_size, 2 * self.vocab_size * self.hidden_size + 2 * self.hidden_size
        serial = self.block == "serial"
        for l in self.layers:
            m = l.mixer
            if isinstance(m, LatentAttention):
                n += W * (m.heads * (m.dim + m.rot_dim + m.vdim) + m.kv_rank + m.rot_dim)
                n += m.kv_rank * (m.heads * (m.dim + m.vdim) + 1) + (m.heads if m.sink else 0)
            elif isinstance(m, TalkingAttention):
                n += W * (m.heads + m.kv_heads) * (m.dim + m.vdim) + m.params
            elif isinstance(m, GatedAverage):
                n += 4 * W * m.width + 2 * m.width
            else:
                ra, rg = m.decay_rank or m.dim, m.gate_rank or m.vdim
                n += W * (m.channels + m.heads * (1 + m.vdim) + ra + rg)
                n += m.channels * m.conv + m.heads * (m.dim * (ra + 1) + m.vdim * rg + 1) + m.vdim
            per = 2 * W + (1 if serial else self.conv_taps * W)  # a sublayer's norm
            n += per
            if l.ff:
                n += (3 if serial else 2) * W * l.ff + per
        return n

    def _num_params_scaled(self) -> int:
        W = self.hidden_size
        n = 2 * self.vocab_size * W + W
        for l in self.layers:
            m = l.mixer
            n += W * (m.channels + m.heads * (m.vdim + m.gate)) + 2 * W + int(m.v_mix)
            n += m.channels * m.conv
            if l.ff:
                n += 3 * W * l.ff * (l.experts.count if l.experts else 1) + 2 * W
                n += W * l.experts.count if l.experts else 0
        return n

    def _num_params_joint(self) -> int:
        W, side = self.hidden_size, self.side_dim
        n = W + self.vocab_size * (2 * W + self.num_layers * side)
        for l in self.layers:
            m = l.mixer
            if isinstance(m, LatentAttention):
                n += W * m.heads * (m.dim + m.rot_dim + m.vdim + m.gate) + m.kv_rank * m.heads * (m.dim + m.vdim)
                n += (m.heads if m.sink else 0)
                n += 0 if m.kv_from is not None else W * (m.kv_rank + m.rot_dim) + m.kv_rank
            else:
                n += W * m.heads * (2 * m.dim + 3 * m.vdim)
                n += m.heads * (2 * W + 2 + m.vdim) if isinstance(m, MatrixMemory) else 0
            n += W + (W * (2 * side + 1) if side else 0)
            if l.ff:
                n += 2 * W * (l.ff * (l.experts.count if l.experts else 1) + (l.shared or 0))
                n += W * l.experts.count if l.experts else 0
        return n

    def replace(self, **kw) -> "HybridConfig":
        return dataclasses.replace(self, **kw)


def _ralesun(d: dict, name: str) -> HybridConfig:
    layers = []
    for e in d["layers"]:
        m = e["mixer"]
        if e["type"] == "latent_attention":
            mixer = LatentAttention(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"],
                                    float(m["scale"]), (m.get("mask") or {}).get("size"),
                                    float(m["rot"]["base"]), m["rot"]["dims"])
        elif e["type"] == "channel_delta":
            mixer = ChannelDelta(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"])
        else:
            raise ValueError(f"unknown layer type {e['type']!r}")
        mlp = e["mlp"]
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        layers.append(Layer(mixer, mlp["ff"] if mlp else None))
    # the format names no special tokens: generation ends by length or by stop tokens
    return HybridConfig(name, d["vocab"], d["width"], tuple(layers), float(d["norm"]["eps"]),
                        max_position=d.get("max_position", 32768), bos_token_id=0, eos_token_id=-1)


def _mebalorn(d: dict, name: str) -> HybridConfig:
    layers = []
    for e in d["layers"]:
        m = e["mixer"]
        if e["type"] == "attention":
            mixer = TalkingAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]))
        elif e["type"] == "mingru":
            mixer = GatedAverage(m["width"])
        else:
            raise ValueError(f"unknown layer type {e['type']!r}")
        mlp = e["mlp"]
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        layers.append(Layer(mixer, mlp["ff"] if mlp else None))
    return HybridConfig(name, d["vocab"], d["width"], tuple(layers), float(d["norm"]["eps"]),
                        act="relu2", max_position=d.get("max_position", 32768), bos_token_id=0,
                        eos_token_id=-1, block="parallel", conv_taps=d["canon"]["taps"],
                        sinusoids=True, logit_softcap=float(d["logit_softcap"]))


def _nurilorn(d: dict, name: str) -> HybridConfig:
    layers = []
    for e in d["layers"]:
        m = e["mixer"]
        if e["type"] != "attention":
            raise ValueError(f"unknown layer type {e['type']!r}")
        rot = m.get("rot") or {"base": 10000.0, "dims": 0}
        s = rot.get("scaling")
        scaling = RotaryScaling(float(s["factor"]), float(s["original"]), float(s["fast"]),
                                float(s["slow"])) if s else None
        mixer = GroupedAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]),
                                 float(rot["base"]), rot["dims"], scaling, m.get("conv") or 0,
                                 float(m.get("softcap") or 0.0), bool(m.get("v_mix")))
        mlp = e["mlp"]
        if mlp is None:
            layers.append(Layer(mixer))
        elif mlp["kind"] == "dense":
            layers.append(Layer(mixer, mlp["ff"], float(mlp["limit"])))
        elif mlp["kind"] == "moe":
            r, g = mlp["router"], mlp["router"].get("groups") or {"count": 1, "keep": 1}
            layers.append(Layer(mixer, mlp["expert"]["ff"], float(mlp["expert"]["limit"]),
                                Experts(r["experts"], r["top"], g["count"], g["keep"])))
        else:
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return HybridConfig(name, d["vocab"], d["width"], tuple(layers), float(d["norm"]["eps"]),
                        act="clamped", max_position=d.get("max_position", 32768), bos_token_id=0,
                        eos_token_id=-1, norm="group_rms", norm_groups=d["norm"]["groups"],
                        embed_scale=float(d["embedding"]["scale"]),
                        residual_mult=float(d["residual_mult"]),
                        logit_scale=float(d["logit_scale"]))


def _garesun(d: dict, name: str) -> HybridConfig:
    layers = []
    for e in d["layers"]:
        m = e["mixer"]
        rot = m.get("rot") or {"base": 10000.0, "dims": 0}
        if e["type"] == "latent_attention":
            mixer = LatentAttention(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"],
                                    float(m["scale"]), None, float(rot["base"]), rot["dims"],
                                    sink=False, gate=True, kv_from=m.get("kv_from"))
        elif e["type"] == "retention":
            mixer = Retention(m["heads"], m["dim"], m["vdim"], tuple(map(float, m["decay"])),
                              float(rot["base"]), rot["dims"])
        elif e["type"] == "mlstm":
            mixer = MatrixMemory(m["heads"], m["dim"], m["vdim"], float(m["gate_cap"]))
        else:
            raise ValueError(f"unknown layer type {e['type']!r}")
        mlp = e["mlp"]
        if mlp is None:
            layers.append(Layer(mixer))
        elif mlp["kind"] == "moe":
            r, shared = mlp["router"], mlp.get("shared")
            layers.append(Layer(mixer, mlp["expert"]["ff"], experts=Experts(r["experts"], r["top"]),
                                shared=shared["ff"] if shared else None))
        else:
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return HybridConfig(name, d["vocab"], d["width"], tuple(layers), float(d["norm"]["eps"]),
                        act="relu2", max_position=d.get("max_position", 32768), bos_token_id=0,
                        eos_token_id=-1, block="joint", norm="layer",
                        embed_scale=float(d["embedding"]["scale"]), side_dim=d["token_side"]["dim"])


# checkpoint configuration ("architecture" key) -> parser
ARCHITECTURES = {"Ralesun": _ralesun, "Mebalorn": _mebalorn, "Nurilorn": _nurilorn,
                 "Garesun": _garesun}


def config_from_dict(d: dict, name: str = "") -> HybridConfig:
    arch = d.get("architecture")
    if arch not in ARCHITECTURES:
        raise KeyError(f"unknown architecture {arch!r}; known: {sorted(ARCHITECTURES)}")
    return ARCHITECTURES[arch](d, name or arch.lower())


def load_config(path: str) -> HybridConfig:
    """Configuration of a checkpoint folder."""
    with open(os.path.join(path, "config.json")) as f:
        return config_from_dict(json.load(f), os.path.basename(os.path.abspath(path)))


def _stack(blocks: int, latent: LatentAttention, delta: ChannelDelta, ff: int) -> tuple:
    """Latent-attention layers with a feed-forward, each followed by a bare delta-rule layer."""
    return (Layer(latent, ff), Layer(delta)) * blocks


# Random-init presets of the design at the layer sizes of Llama-3-8B and of half its width.
RALESUN_8B = HybridConfig(
    name="ralesun-8b", vocab_size=128256, hidden_size=4096, layers=_stack(
        32, LatentAttention(32, 128, 64, 128, 512, 192 ** -0.5, 1024, 500000.0, 64),
        ChannelDelta(32, 32, 128, 128, 4, 128, 128), 14336),
    bos_token_id=128000, eos_token_id=128001)

RALESUN_2B = HybridConfig(
    name="ralesun-2b", vocab_size=128256, hidden_size=2048, layers=_stack(
        24, LatentAttention(16, 128, 64, 128, 512, 192 ** -0.5, 1024, 500000.0, 64),
        ChannelDelta(16, 16, 128, 128, 4, 128, 128), 7168),
    bos_token_id=128000, eos_token_id=128001)

TINY_RALESUN = HybridConfig(
    name="tiny-ralesun", vocab_size=512, hidden_size=192, layers=(
        Layer(ChannelDelta(4, 2, 16, 24, 3, 16, 24), 320),
        Layer(LatentAttention(3, 24, 8, 40, 64, 0.2, 37, 10000.0, 8)),
        Layer(ChannelDelta(2, 2, 40, 32, 4, 24, 16)),
        Layer(LatentAttention(5, 16, 16, 32, 48, 0.15, 70, 50000.0, 16), 256)),
    max_position=1024, init_std=0.06)

def _alternating(blocks: int, average: GatedAverage, attention: TalkingAttention, ff: int) -> tuple:
    return (Layer(average, ff), Layer(attention, ff)) * blocks


def _parallel(name: str, width: int, layers: tuple, vocab: int = 128256, **kw) -> HybridConfig:
    return HybridConfig(name, vocab, width, layers, act="relu2", block="parallel", conv_taps=4,
                        sinusoids=True, logit_softcap=30.0, **kw)


# Two matrices to a feed-forward of 1.5 times Llama's size, a recurrence as large as an attention.
MEBALORN_8B = _parallel("mebalorn-8b", 4096, _alternating(
    16, GatedAverage(2560), TalkingAttention(32, 8, 128, 128, 128 ** -0.5), 21504),
    bos_token_id=128000, eos_token_id=128001)

MEBALORN_2B = _parallel("mebalorn-2b", 2048, _alternating(
    12, GatedAverage(1280), TalkingAttention(16, 4, 128, 128, 128 ** -0.5), 10752),
    bos_token_id=128000, eos_token_id=128001)

TINY_MEBALORN = _parallel("tiny-mebalorn", 160, (
    Layer(TalkingAttention(6, 3, 24, 40, 0.2), 200), Layer(GatedAverage(72)),
    Layer(TalkingAttention(2, 2, 32, 16, 0.3)), Layer(GatedAverage(136), 320)), vocab=384,
    max_position=1024, init_std=0.06)


def _scaled(name: str, width: int, layers: tuple, vocab: int = 128256, **kw) -> HybridConfig:
    kw = {"norm_groups": 8, "embed_scale": 16.0, "residual_mult": 0.5, **kw}
    return HybridConfig(name, vocab, width, layers, act="clamped", norm="group_rms", **kw)


def _routed(heads: int, kv_heads: int, dense: int, ff: int, layers: int) -> tuple:
    """A dense layer, then layers of 16 experts, 4 of them per token out of 2 of 4 groups."""
    m = GroupedAttention(heads, kv_heads, 128, 128, 128 ** -0.5, 500000.0, 64,
                         RotaryScaling(4.0, 8192, 32.0, 1.0), 4, 30.0, True)
    return (Layer(m, dense, 7.0),) + (Layer(m, ff, 7.0, Experts(16, 4, 4, 2)),) * (layers - 1)


# Llama's attention sizes; four experts of a token together as wide as its feed-forward.
NURILORN_24B = _scaled("nurilorn-24b", 4096, _routed(32, 8, 14336, 3584, 32),
                       bos_token_id=128000, eos_token_id=128001)

NURILORN_5B = _scaled("nurilorn-5b", 2048, _routed(16, 4, 7168, 1792, 24),
                      bos_token_id=128000, eos_token_id=128001)

TINY_NURILORN = _scaled("tiny-nurilorn", 160, (
    Layer(GroupedAttention(6, 2, 24, 16, 0.2, 10000.0, 12, RotaryScaling(2.0, 128, 8.0, 1.0), 3,
                           15.0, True), 200, 2.0),
    Layer(GroupedAttention(2, 2, 32, 24, 0.2, 10000.0, 32, None, 2, 15.0)),
    Layer(GroupedAttention(4, 1, 16, 32, 0.25, 5000.0, 8, None, 4, 15.0, True), 72, 2.0,
          Experts(6, 2, 3, 2))), vocab=384, norm_groups=4, embed_scale=4.0, max_position=1024,
    init_std=0.06)

def _joint(name: str, width: int, layers: tuple, side: int, vocab: int = 128256, **kw) -> HybridConfig:
    return HybridConfig(name, vocab, width, layers, act="relu2", block="joint", norm="layer",
                        embed_scale=4.0, side_dim=side, **kw)


def retention_decays(heads: int) -> tuple[float, ...]:
    """Spans from 32 tokens to thousands, one per head."""
    return tuple(1 - 2.0 ** (-5 - 7 * h / max(heads - 1, 1)) for h in range(heads))


def _memories(blocks: int, heads: int, ff: int, experts: Experts) -> tuple:
    """Blocks of matrix memory, latent attention, retention, and an attention that reads the same
    latents; a shared expert twice as wide as the others."""
    out = []
    for b in range(blocks):
        att = LatentAttention(heads, 128, 64, 128, 512, 192 ** -0.5, None, 500000.0, 64, False, True)
        for m in (MatrixMemory(heads, 128, 128, 15.0), att,
                  Retention(heads, 128, 128, retention_decays(heads), 500000.0, 128),
                  dataclasses.replace(att, kv_from=4 * b + 1)):
            out.append(Layer(m, ff, experts=experts, shared=2 * ff))
    return tuple(out)


# Llama's head sizes; a token's four routed experts and its shared one together as many parameters
# as its feed-forward.
GARESUN_24B = _joint("garesun-24b", 4096, _memories(8, 32, 3584, Experts(20, 4)), 256,
                     bos_token_id=128000, eos_token_id=128001)

GARESUN_5B = _joint("garesun-5b", 2048, _memories(6, 16, 1792, Experts(20, 4)), 128,
                    bos_token_id=128000, eos_token_id=128001)

TINY_GARESUN = _joint("tiny-garesun", 160, (
    Layer(LatentAttention(3, 24, 8, 40, 48, 0.2, None, 10000.0, 8, False, True), 72,
          experts=Experts(6, 2), shared=104),
    Layer(Retention(2, 48, 32, (0.9, 0.99), 5000.0, 32)),
    Layer(MatrixMemory(3, 16, 40, 10.0), 40, experts=Experts(5, 3)),
    Layer(LatentAttention(5, 16, 8, 24, 48, 0.25, None, 10000.0, 8, False, True, kv_from=0), 56,
          experts=Experts(8, 1), shared=48)), 24, vocab=384, max_position=1024, init_std=0.06)

REGISTRY = {c.name: c for c in (LLAMA3_8B, LLAMA3_70B, GEMMA_2B, MIXTRAL_8X7B,
                                TINY_LLAMA, TINY_GEMMA, TINY_MIXTRAL, RALESUN_8B, RALESUN_2B,
                                TINY_RALESUN, MEBALORN_8B, MEBALORN_2B, TINY_MEBALORN,
                                NURILORN_24B, NURILORN_5B, TINY_NURILORN,
                                GARESUN_24B, GARESUN_5B, TINY_GARESUN)}


def get_config(name: str) -> ModelConfig | HybridConfig:
    """Configuration of a registered model, or of a checkpoint folder."""
    try:
        return REGISTRY[name]
    except KeyError:
        if os.path.isfile(os.path.join(name, "config.json")):
            return load_config(name)
        raise KeyError(f"unknown model {name!r}; known: {sorted(REGISTRY)}") from None
