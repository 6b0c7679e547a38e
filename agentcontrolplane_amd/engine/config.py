"""Model + engine configuration.

Model presets are the architectures BASELINE.json names (Llama-3 8B/70B,
Mixtral 8x7B) plus tiny test configs; weights are random-init (no network),
shapes and dtypes are the real ones.  A checkpoint directory whose
config.json names a registered architecture needs no preset: model="auto"
reads it (models/configs.py).
"""
from __future__ import annotations

import dataclasses
import math
from typing import Optional, Tuple, Union


@dataclasses.dataclass(frozen=True)
class WavelengthScaling:
    """Rotation slowed by ``factor`` at wavelengths beyond original / low, unchanged
    below original / high, blended in between (models/rotary.py)."""

    factor: float
    low: float
    high: float
    original: float


@dataclasses.dataclass(frozen=True)
class YarnScaling:
    """Rotation slowed by ``factor`` along a ramp over the dimensions, from the one that
    makes ``fast`` turns over the original length to the one that makes ``slow``; cos
    and sin grow by 0.1 ln(factor) + 1 (models/rotary.py)."""

    factor: float
    original: float
    fast: float
    slow: float


RotaryScaling = Union[None, WavelengthScaling, YarnScaling]


@dataclasses.dataclass(frozen=True)
class RotarySpec:
    """Rotation of a head's first ``dims`` dimensions, i with i + dims/2."""

    base: float
    dims: int
    scaling: RotaryScaling = None


@dataclasses.dataclass(frozen=True)
class QueryTemperature:
    """Queries at position p times 1 + coef ln(floor((p + 1) / every) + 1)."""

    coef: float
    every: float


@dataclasses.dataclass(frozen=True)
class DistanceBias:
    """Learned score bias per head and bucket of the distance: half of the buckets
    hold one distance each, the others widen geometrically up to ``reach``."""

    buckets: int
    reach: float


@dataclasses.dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention over one cached low-rank latent per token plus one rotated
    key part shared by all heads (models/latent_attention.py)."""

    heads: int
    dim: int                      # unrotated query/key dims per head
    rot_dim: int                  # rotated query/key dims per head
    vdim: int                     # value dims per head
    kv_rank: int                  # latent size
    scale: float                  # on the scores
    rope_base: float
    q_rank: Optional[int] = None  # low-rank query; None = direct projection
    window: Optional[int] = None  # keys visible, self included; None = all
    head_gate: bool = True        # sigmoid gate per head on the output
    rope_scaling: RotaryScaling = None
    rope_half: bool = False       # dimension i turns with i + rot_dim/2, else 2i with 2i + 1
    sink: bool = False            # learned logit per head in the denominator

    def params(self, w: int) -> int:
        qdim = self.heads * (self.dim + self.rot_dim)
        n = self.q_rank * (w + 1 + qdim) if self.q_rank else w * qdim
        n += w * (self.kv_rank + self.rot_dim) + self.kv_rank
        n += self.kv_rank * self.heads * (self.dim + self.vdim) + self.heads * self.vdim * w
        return n + (w * self.heads if self.head_gate else 0) + (self.heads if self.sink else 0)


@dataclasses.dataclass(frozen=True)
class GroupedAttentionSpec:
    """Attention over cached keys and values shared by groups of query heads
    (models/grouped_attention.py)."""

    heads: int
    kv_heads: int
    dim: int                        # query/key size per head
    vdim: int                       # value size per head
    scale: float                    # on the scores
    softcap: Optional[float] = None  # scores -> softcap * tanh(score / softcap)
    window: Optional[int] = None    # keys visible, self included; None = all
    chunk: Optional[int] = None     # only keys of the query's own chunk, positions / chunk
    keep_first: int = 0             # first tokens that stay visible beyond the window
    bias: bool = True               # on the query, key and value projections
    sink: bool = True               # learned logit per head in the denominator
    kv_from: Optional[int] = None   # the layer whose keys and values are used
    conv: int = 0                   # taps of the short convolutions on q, k, v; 0 = none
    qk_norm: bool = False           # RMS norm of query and key heads, learned weight
    row_norm: bool = False          # the same over all query (key) heads at once
    v_norm: bool = False            # RMS norm of value heads, no weight
    rotary: Optional[RotarySpec] = None
    q_temp: Optional[QueryTemperature] = None
    head_temp: bool = False         # learned factor per head on the scores
    talk: bool = False              # a head's scores are a learned mix of all heads'
    distance_bias: Optional[DistanceBias] = None
    sigmoid: bool = False           # weights sigmoid(score + learned offset), not normalized
    head_gate: bool = False         # sigmoid gate per head on the output
    out_bias: bool = False

    def params(self, w: int) -> int:
        q, o = self.heads * self.dim, self.heads * self.vdim
        kv = 0 if self.kv_from is not None else self.kv_heads * (self.dim + self.vdim)
        n = (q + kv) * (w + self.bias + self.conv) + o * w + (w if self.out_bias else 0)
        n += 2 * self.dim if self.qk_norm else 0
        n += (self.heads + self.kv_heads) * self.dim if self.row_norm else 0
        n += self.heads ** 2 if self.talk else 0
        n += self.heads * (self.sink + self.head_temp + self.sigmoid)
        n += self.heads * self.distance_bias.buckets if self.distance_bias else 0
        return n + (self.heads * w if self.head_gate else 0)


@dataclasses.dataclass(frozen=True)
class GatedDeltaSpec:
    """Gated delta rule with one decay per head, or per head and key channel
    (models/gated_delta.py)."""

    heads: int                      # value heads, one state each
    kv_heads: int                   # query/key heads
    dim: int                        # query/key size per head
    vdim: int                       # value size per head
    conv: int                       # taps of the short convolutions
    decay_rank: int = 0             # inner size of the decay projection; 0 = direct
    gate_rank: int = 0              # inner size of the output gate's projection; 0 = direct
    head_decay: bool = False        # one decay per head, else one per head and key channel
    gate_silu: bool = False         # output gate silu, else sigmoid
    unit_eps: float = 1e-6          # in the unit vectors' sum of squares

    @property
    def decays(self) -> int:
        return self.heads * (1 if self.head_decay else self.dim)

    def params(self, w: int) -> int:
        qk, v = 2 * self.kv_heads * self.dim, self.heads * self.vdim
        n = (qk + v) * (w + self.conv) + self.heads * (w + 1) + self.vdim + v * w
        r, g = self.decay_rank, self.gate_rank
        n += (r * (w + self.decays) if r else w * self.decays) + self.decays
        return n + (g * (w + v) if g else w * v)


@dataclasses.dataclass(frozen=True)
class ClampedGluSpec:
    """g * sigmoid(alpha (g + cubic g^3)) * (clamp(up, +-limit) + offset),
    g = min(gate, limit)."""

    width: int
    limit: float
    alpha: float = 1.702
    offset: float = 1.0
    cubic: float = 0.0
    bias: bool = False              # on all three projections

    def params(self, w: int) -> int:
        return 3 * w * self.width + (2 * self.width + w if self.bias else 0)


def silu_glu(width: int) -> ClampedGluSpec:
    """silu(gate) * up."""
    return ClampedGluSpec(width, limit=math.inf, alpha=1.0, offset=0.0)


def gelu_glu(width: int, bias: bool = False) -> ClampedGluSpec:
    """gelu(gate) * up, the tanh form: 1 + tanh(z) = 2 sigmoid(2z)."""
    return ClampedGluSpec(
        width, limit=math.inf, alpha=2 * math.sqrt(2 / math.pi), offset=0.0, cubic=0.044715,
        bias=bias,
    )


@dataclasses.dataclass(frozen=True)
class ExpertsSpec:
    """Mixture of experts: each token uses ``top`` of ``experts`` GLUs, weighted by the
    softmax over the chosen router logits or by their normed sigmoids, and the shared one
    (models/experts.py)."""

    experts: int
    top: int
    expert: ClampedGluSpec
    shared: Optional[ClampedGluSpec] = None
    router_bias: bool = True
    sigmoid: bool = False           # scores are the logits' sigmoids
    correction: bool = False        # learned, on the scores in the choice only
    scale: float = 1.0              # on the weights

    @property
    def width(self) -> int:
        """Feed-forward width a token uses."""
        return self.top * self.expert.width + (self.shared.width if self.shared else 0)

    def params(self, w: int) -> int:
        each = w + self.router_bias + self.correction + self.expert.params(w)
        return self.experts * each + (self.shared.params(w) if self.shared else 0)


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: Union[LatentAttentionSpec, GroupedAttentionSpec, GatedDeltaSpec]
    mlp: Union[None, ClampedGluSpec, ExpertsSpec] = None
    sandwich: bool = False  # mixer, then mlp, each normed on its way in and out
    mlp_norm: bool = False  # side by side, the mlp on a norm of its own
    norm_out: bool = False  # mixer, then mlp, each normed on its way out only
    gated: bool = False     # sigmoid gates on both results, from what they were made of
    weights_of: Optional[int] = None  # the layer whose weights are used


@dataclasses.dataclass(frozen=True)
class LoopSpec:
    """Layers [start, stop) run ``times`` times in a row on the same weights."""

    start: int
    stop: int
    times: int


@dataclasses.dataclass
class ModelConfig:
    name: str = "llama3-8b"
    vocab_size: int = 128256
    hidden_size: int = 4096
    intermediate_size: int = 14336
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    # Qwen2-family attention bias on the QKV projection
    attention_bias: bool = False
    # MoE (Mixtral): 0 experts = dense
    num_experts: int = 0
    num_experts_per_tok: int = 2
    dtype: str = "bfloat16"
    # models/registry key; "" picks llama or mixtral by num_experts
    architecture: str = ""
    # designs whose layers differ from each other list them; the head/MLP
    # sizes above are then unused
    layers: Tuple[LayerSpec, ...] = ()
    loop: Optional[LoopSpec] = None
    # per-layer token embedding: dims per layer, 0 = none
    token_side_dim: int = 0
    # on every sublayer's output
    residual_mult: float = 1.0
    # what a layer hands on is a learned mix of all layers' results so far
    depth_average: bool = False
    # sinusoidal positions added to the embedding: the base, None = none
    position_base: Optional[float] = None
    # on the token embedding
    embed_scale: float = 1.0
    # logits -> cap * tanh(logits / cap)
    logit_softcap: Optional[float] = None
    # on the logits
    logit_scale: float = 1.0

    @property
    def layer_runs(self) -> Tuple[Tuple[int, bool], ...]:
        """(layer, enters a loop pass) in execution order: one entry, and
        one cache, per layer and pass."""
        n = len(self.layers) or self.num_layers
        if self.loop is None:
            return tuple((i, False) for i in range(n))
        lo, hi = self.loop.start, self.loop.stop
        runs = [(i, False) for i in range(lo)]
        for _ in range(self.loop.times):
            runs += [(i, i == lo) for i in range(lo, hi)]
        return tuple(runs + [(i, False) for i in range(hi, n)])

    @property
    def is_moe(self) -> bool:
        return self.num_experts > 0

    def params_bytes(self, dtype_bytes: int = 2) -> int:
        if self.layers:
            return self._listed_layer_params() * dtype_bytes
        h, i, v, L = self.hidden_size, self.intermediate_size, self.vocab_size, self.num_layers
        kvh = self.num_kv_heads * self.head_dim
        qh = self.num_heads * self.head_dim
        attn = h * qh + 2 * h * kvh + qh * h
        mlp = 3 * h * i
        if self.is_moe:
            mlp = self.num_experts * 3 * h * i + h * self.num_experts
        per_layer = attn + mlp + 2 * h
        total = L * per_layer + 2 * v * h + h
        return total * dtype_bytes

    def _listed_layer_params(self) -> int:
        w, v = self.hidden_size, self.vocab_size
        total = v * w * (1 if self.tie_embeddings else 2) + w
        for i, layer in enumerate(self.layers):
            if layer.weights_of is not None:
                continue
            total += w + layer.mixer.params(w)
            total += layer.mlp.params(w) if layer.mlp else 0
            total += w if layer.mlp and (layer.mlp_norm or layer.norm_out) else 0
            total += (w * w + w) * (2 if layer.mlp else 1) if layer.gated else 0
            if layer.sandwich:
                total += w + (2 * w if layer.mlp else 0)
            if self.depth_average:
                total += i + 2
            if self.token_side_dim:
                total += 2 * w * self.token_side_dim + w + v * self.token_side_dim
        return total + (2 * w * w if self.loop else 0)


def _fetolix(name: str, *, width: int, heads: int, layers: int, ff: int,
             kv_rank: int, q_rank: int, dim: int, rot_dim: int, vdim: int,
             window: int, vocab: int, side: int, limit: float = 7.0,
             loop: Optional[LoopSpec] = None, full_every: int = 4,
             **kw) -> ModelConfig:
    """Every ``full_every``-th layer sees all keys with a direct query; the
    others see a window with a low-rank query."""
    def mixer(i: int) -> LatentAttentionSpec:
        full = i % full_every == full_every - 1
        return LatentAttentionSpec(
            heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank,
            scale=(dim + rot_dim) ** -0.5, rope_base=1e6 if full else 1e4,
            q_rank=None if full else q_rank, window=None if full else window,
        )

    return ModelConfig(
        name=name, architecture="Fetolix", vocab_size=vocab, hidden_size=width,
        intermediate_size=ff, num_layers=layers, num_heads=heads,
        num_kv_heads=1, head_dim=dim + rot_dim, tie_embeddings=True,
        layers=tuple(
            LayerSpec(mixer(i), ClampedGluSpec(ff, limit)) for i in range(layers)
        ),
        loop=loop, token_side_dim=side, **kw,
    )


def _tezinex(name: str, *, width: int, layers: int, ff: int, heads: int, kv_heads: int,
             dim: int, vdim: int, window: int, keep_first: int, d_heads: int, d_kv_heads: int,
             d_dim: int, d_vdim: int, rank: int, vocab: int, conv: int = 4,
             attn_every: int = 4, share: int = 2, **kw) -> ModelConfig:
    """Every ``attn_every``-th layer is windowed attention, the others delta
    layers; of ``share`` consecutive attention layers all use the first one's keys."""
    delta = GatedDeltaSpec(d_heads, d_kv_heads, d_dim, d_vdim, conv, rank, rank)

    def mixer(i: int):
        nth, at = divmod(i, attn_every)
        if at != attn_every - 1:
            return delta
        owner = (nth - nth % share) * attn_every + attn_every - 1
        return GroupedAttentionSpec(
            heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5,
            softcap=50.0, window=window, keep_first=keep_first,
            kv_from=None if owner == i else owner,
        )

    return ModelConfig(
        name=name, architecture="Tezinex", vocab_size=vocab, hidden_size=width,
        intermediate_size=ff, num_layers=layers, num_heads=heads, num_kv_heads=kv_heads,
        head_dim=dim, tie_embeddings=True, residual_mult=0.5, depth_average=True,
        position_base=10000.0, logit_softcap=30.0,
        layers=tuple(LayerSpec(mixer(i), silu_glu(ff), sandwich=True) for i in range(layers)),
        **kw,
    )


def _lobuvik(name: str, *, width: int, layers: int, heads: int, kv_heads: int, dim: int,
             vdim: int, conv: int, bias: DistanceBias, kv_rank: int, rot_dim: int, window: int,
             ff: int, experts: ExpertsSpec, vocab: int, **kw) -> ModelConfig:
    """Biased, latent and rotated attention in turn; a dense feed-forward in the first
    layer, experts in the others."""
    biased = GroupedAttentionSpec(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, bias=True,
        out_bias=True, sink=False, sigmoid=True, conv=conv, qk_norm=True, v_norm=True,
        distance_bias=bias, q_temp=QueryTemperature(0.1, 8192),
    )
    latent = LatentAttentionSpec(
        heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank,
        scale=(dim + rot_dim) ** -0.5, rope_base=1e6, rope_half=True,
        rope_scaling=YarnScaling(8.0, 4096, 32.0, 1.0), window=window, head_gate=False, sink=True,
    )
    rotated = GroupedAttentionSpec(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, softcap=50.0,
        window=window, bias=False, sink=False, head_temp=True, head_gate=True,
        rotary=RotarySpec(5e5, dim // 2, WavelengthScaling(8.0, 1.0, 4.0, 8192)),
    )
    mixers = (biased, latent, rotated)
    return ModelConfig(
        name=name, architecture="Lobuvik", vocab_size=vocab, hidden_size=width,
        intermediate_size=ff, num_layers=layers, num_heads=heads, num_kv_heads=kv_heads,
        head_dim=dim, layers=tuple(
            LayerSpec(mixers[i % 3], gelu_glu(ff) if i == 0 else experts, mlp_norm=True)
            for i in range(layers)
        ), **kw,
    )


def _noganex(name: str, *, width: int, layers: int, heads: int, kv_heads: int, dim: int,
             vdim: int, chunk: int, rotary: RotarySpec, d_heads: int, d_kv_heads: int,
             d_dim: int, d_vdim: int, ff: int, experts: ExpertsSpec, vocab: int, conv: int = 4,
             logit_scale: float = 0.25, **kw) -> ModelConfig:
    """Chunked attention with a dense feed-forward and delta layers with experts in turn;
    every second delta layer uses the one before's weights."""
    attention = LayerSpec(GroupedAttentionSpec(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, chunk=chunk,
        bias=False, sink=False, row_norm=True, rotary=rotary, talk=True,
    ), gelu_glu(ff, bias=True), norm_out=True, gated=True)
    delta = LayerSpec(GatedDeltaSpec(
        d_heads, d_kv_heads, d_dim, d_vdim, conv, head_decay=True, gate_silu=True,
    ), experts, norm_out=True, gated=True)

    def layer(i: int) -> LayerSpec:
        if i % 2 == 0:
            return attention
        return delta if i % 4 == 1 else dataclasses.replace(delta, weights_of=i - 2)

    return ModelConfig(
        name=name, architecture="Noganex", vocab_size=vocab, hidden_size=width,
        intermediate_size=ff, num_layers=layers, num_heads=heads, num_kv_heads=kv_heads,
        head_dim=dim, layers=tuple(layer(i) for i in range(layers)), logit_scale=logit_scale,
        **kw,
    )


def _corrected_experts(experts: int, top: int, ff: int, shared: int, scale: float) -> ExpertsSpec:
    return ExpertsSpec(
        experts, top, silu_glu(ff), silu_glu(shared), router_bias=False, sigmoid=True,
        correction=True, scale=scale,
    )


PRESETS = {
    "llama3-8b": ModelConfig(),
    # Llama-2 family: same architecture, smaller rope base / context / vocab
    "llama2-7b": ModelConfig(
        name="llama2-7b", vocab_size=32000, hidden_size=4096,
        intermediate_size=11008, num_layers=32, num_heads=32,
        num_kv_heads=32, rope_theta=10000.0, rms_eps=1e-5, max_position=4096,
    ),
    "llama2-13b": ModelConfig(
        name="llama2-13b", vocab_size=32000, hidden_size=5120,
        intermediate_size=13824, num_layers=40, num_heads=40,
        num_kv_heads=40, rope_theta=10000.0, max_position=4096,
    ),
    # Qwen2: GQA + QKV bias (the one architectural delta from Llama)
    "qwen2-7b": ModelConfig(
        name="qwen2-7b", vocab_size=152064, hidden_size=3584,
        intermediate_size=18944, num_layers=28, num_heads=28,
        num_kv_heads=4, rope_theta=1000000.0, rms_eps=1e-6,
        max_position=8192, attention_bias=True,
    ),
    "llama3-70b": ModelConfig(
        name="llama3-70b",
        hidden_size=8192,
        intermediate_size=28672,
        num_layers=80,
        num_heads=64,
        num_kv_heads=8,
    ),
    "mixtral-8x7b": ModelConfig(
        name="mixtral-8x7b",
        vocab_size=32000,
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=32,
        num_heads=32,
        num_kv_heads=8,
        rope_theta=1000000.0,
        num_experts=8,
        num_experts_per_tok=2,
    ),
    # Fetolix at the layer sizes of an 8B-class dense model (random weights):
    # width and head count of llama3-8b, a 512-wide latent
    "fetolix-8b": _fetolix(
        "fetolix-8b", width=4096, heads=32, layers=24, ff=14336, kv_rank=512,
        q_rank=1536, dim=128, rot_dim=64, vdim=128, window=4096, vocab=128256,
        side=64, loop=LoopSpec(4, 12, 2),
    ),
    # half the width, 16 heads
    "fetolix-2b": _fetolix(
        "fetolix-2b", width=2048, heads=16, layers=16, ff=8192, kv_rank=512,
        q_rank=768, dim=128, rot_dim=64, vdim=128, window=1024, vocab=32000,
        side=64, loop=LoopSpec(4, 8, 2),
    ),
    "tiny-fetolix": _fetolix(
        "tiny-fetolix", width=48, heads=3, layers=4, ff=72, kv_rank=24,
        q_rank=20, dim=12, rot_dim=8, vdim=10, window=19, vocab=300, side=6,
        limit=1.5, loop=LoopSpec(1, 3, 2), full_every=2, max_position=4096,
        dtype="float32",
    ),
    # Tezinex at the layer sizes of an 8B-class dense model (random weights):
    # width, heads and feed-forward of llama3-8b
    "tezinex-8b": _tezinex(
        "tezinex-8b", width=4096, layers=32, ff=14336, heads=32, kv_heads=8, dim=128,
        vdim=128, window=4096, keep_first=16, d_heads=32, d_kv_heads=32, d_dim=128,
        d_vdim=128, rank=128, vocab=128256,
    ),
    # half the width, 16 heads
    "tezinex-2b": _tezinex(
        "tezinex-2b", width=2048, layers=20, ff=8192, heads=16, kv_heads=8, dim=128,
        vdim=128, window=1024, keep_first=4, d_heads=16, d_kv_heads=16, d_dim=128,
        d_vdim=128, rank=64, vocab=32000,
    ),
    "tiny-tezinex": _tezinex(
        "tiny-tezinex", width=44, layers=6, ff=60, heads=6, kv_heads=3, dim=10, vdim=14,
        window=21, keep_first=3, d_heads=4, d_kv_heads=2, d_dim=12, d_vdim=18, rank=7,
        vocab=300, conv=3, attn_every=2, max_position=4096, dtype="float32",
    ),
    # Lobuvik with the layer sizes of an 8B-class dense model per token (random weights):
    # width, heads and active feed-forward of llama3-8b
    "lobuvik-8b": _lobuvik(
        "lobuvik-8b", width=4096, layers=30, heads=32, kv_heads=8, dim=128, vdim=128, conv=4,
        bias=DistanceBias(64, 512), kv_rank=512, rot_dim=64, window=4096, ff=14336,
        experts=ExpertsSpec(32, 4, ClampedGluSpec(2560, 7.0), ClampedGluSpec(4096, 7.0)),
        vocab=128256,
    ),
    # half the width, 16 heads
    "lobuvik-2b": _lobuvik(
        "lobuvik-2b", width=2048, layers=18, heads=16, kv_heads=8, dim=128, vdim=128, conv=4,
        bias=DistanceBias(32, 256), kv_rank=512, rot_dim=64, window=1024, ff=8192,
        experts=ExpertsSpec(16, 4, ClampedGluSpec(1536, 7.0), ClampedGluSpec(2048, 7.0)),
        vocab=32000,
    ),
    "tiny-lobuvik": _lobuvik(
        "tiny-lobuvik", width=44, layers=4, heads=6, kv_heads=3, dim=12, vdim=10, conv=3,
        bias=DistanceBias(12, 50), kv_rank=20, rot_dim=6, window=23, ff=52,
        experts=ExpertsSpec(5, 2, ClampedGluSpec(18, 1.5), ClampedGluSpec(22, 2.0)),
        vocab=300, max_position=4096, dtype="float32",
    ),
    # Noganex with the layer sizes of an 8B-class dense model per token (random weights):
    # width, heads and active feed-forward of llama3-8b
    "noganex-8b": _noganex(
        "noganex-8b", width=4096, layers=28, heads=32, kv_heads=8, dim=128, vdim=128,
        chunk=4096, rotary=RotarySpec(5e5, 128, YarnScaling(4.0, 8192, 32.0, 1.0)), d_heads=32,
        d_kv_heads=16, d_dim=128, d_vdim=128, ff=14336,
        experts=_corrected_experts(32, 4, 2560, 4096, 2.5), vocab=128256,
    ),
    # half the width, 16 heads
    "noganex-2b": _noganex(
        "noganex-2b", width=2048, layers=18, heads=16, kv_heads=8, dim=128, vdim=128,
        chunk=1024, rotary=RotarySpec(5e5, 64, YarnScaling(4.0, 4096, 32.0, 1.0)), d_heads=16,
        d_kv_heads=8, d_dim=128, d_vdim=128, ff=8192,
        experts=_corrected_experts(16, 4, 1536, 2048, 2.5), vocab=32000,
    ),
    "tiny-noganex": _noganex(
        "tiny-noganex", width=44, layers=4, heads=6, kv_heads=2, dim=12, vdim=10, chunk=23,
        rotary=RotarySpec(1e4, 8, YarnScaling(3.0, 64, 8.0, 1.0)), d_heads=6, d_kv_heads=3,
        d_dim=10, d_vdim=14, conv=3, ff=52, experts=_corrected_experts(5, 2, 18, 22, 1.7),
        vocab=300, max_position=4096, dtype="float32",
    ),
    # tiny GPU config: real head_dim/GQA shape for the CDNA4 kernels at
    # test scale (kernels require head_dim 128)
    "tiny-gpu": ModelConfig(
        name="tiny-gpu",
        vocab_size=512,
        hidden_size=256,
        intermediate_size=512,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=128,
        max_position=2048,
        dtype="bfloat16",
    ),
    # tiny GPU config with Qwen2-style attention bias
    "tiny-gpu-bias": ModelConfig(
        name="tiny-gpu-bias",
        vocab_size=512,
        hidden_size=256,
        intermediate_size=512,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=128,
        max_position=2048,
        attention_bias=True,
        dtype="bfloat16",
    ),
    # tiny configs for CPU tests
    # tiny bias variant (Qwen2-shaped attention for CPU tests)
    "tiny-bias": ModelConfig(
        name="tiny-bias",
        vocab_size=512,
        hidden_size=64,
        intermediate_size=128,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=16,
        max_position=4096,
        attention_bias=True,
        dtype="float32",
    ),
    "tiny": ModelConfig(
        name="tiny",
        vocab_size=512,
        hidden_size=64,
        intermediate_size=128,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=16,
        max_position=4096,
        dtype="float32",
    ),
    "tiny-moe": ModelConfig(
        name="tiny-moe",
        vocab_size=512,
        hidden_size=64,
        intermediate_size=128,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=16,
        max_position=512,
        num_experts=4,
        num_experts_per_tok=2,
        dtype="float32",
    ),
}


@dataclasses.dataclass
class EngineConfig:
    # a PRESETS name, or "auto": the checkpoint's own config.json
    model: str = "llama3-8b"
    # overrides the model's dtype ("bfloat16" | "float32")
    dtype: Optional[str] = None
    device: str = "cuda"                 # "cuda" (ROCm) or "cpu"
    kv_block_size: int = 16
    # KV pool: fraction of free HBM to claim (288 GB/GPU on MI355X), or an
    # explicit block count for tests
    gpu_memory_utilization: float = 0.85
    num_kv_blocks: Optional[int] = None
    # models with recurrent state: sequences that hold a state at a time (None:
    # max_batch_size, less if they would take over half of the memory budget)
    num_state_slots: Optional[int] = None
    max_batch_size: int = 2048
    # chunked-prefill token budget per step: 16384 measured ~7% faster
    # wave p50 than 8192 at 1k concurrency —
    # fewer, larger steps amortize per-step host+launch cost; activations
    # at 16k tokens are ~1 GB against 288 GB HBM
    max_prefill_tokens: int = 16384
    max_model_len: int = 8192
    max_queue: int = 65536
    enforce_eager: bool = False          # True disables hipGraph capture
    # launch decode step t+1 from GPU-resident sampled tokens before step t
    # syncs (hides per-step host time); auto-disabled for TP and whenever a
    # grammar-constrained decode is running
    async_scheduling: bool = True
    # fold forced grammar byte runs (MID scaffolding, schema literals) into
    # one prefill chunk instead of sequential masked decode steps
    grammar_fold: bool = True
    tensor_parallel: int = 1
    seed: int = 0
    request_timeout_s: float = 600.0
    # HF-named safetensors dir; None = random-init (no network here)
    checkpoint_path: Optional[str] = None
    # HF tokenizer.json; defaults to <checkpoint_path>/tokenizer.json when
    # present, else the byte-level tokenizer (synthetic workloads)
    tokenizer_path: Optional[str] = None

    def model_config(self) -> ModelConfig:
        if self.model == "auto":
            from ..models.configs import read_model_config

            if self.checkpoint_path is None:
                raise ValueError('model="auto" needs checkpoint_path')
            cfg = read_model_config(self.checkpoint_path)
        elif self.model in PRESETS:
            cfg = PRESETS[self.model]
        else:
            raise KeyError(f"unknown model preset {self.model!r}; have {sorted(PRESETS)}")
        return dataclasses.replace(cfg, dtype=self.dtype) if self.dtype else cfg
