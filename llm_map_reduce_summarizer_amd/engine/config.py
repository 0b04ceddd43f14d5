"""Model presets for the on-node engine.

The reference never runs a model locally (its map/reduce calls go to hosted
APIs: ``llm_executor.py:250-409``); BASELINE.json names Llama-3-8B for the
map stage and Llama-3-70B (fp8, TP=8) for the aggregator.  Shapes are the
public Llama-3 configs; weights are random-init (seeded)
because no checkpoints are available offline.  ``tiny*`` presets keep the
real vocabulary and head_dim=128 (what the HIP attention kernels are built
for) so CPU tests and GPU smoke runs exercise the same code paths.
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Optional, Tuple, Union

# The engine's default chunked-prefill slice length (tokens; engine/engine.py LLMEngine ``prefill_chunk``).
# Defined here, next to the model presets, so the planner (parallel/plan.py) prices the slice length the
# engine actually runs without importing the engine; tests/test_plan.py fails if the two drift.
PREFILL_CHUNK = 8192


@dataclass(frozen=True)
class ModelConfig:
    name: str
    vocab_size: int = 128256
    hidden: int = 4096
    n_layers: int = 32
    n_heads: int = 32
    n_kv_heads: int = 8
    head_dim: int = 128
    ffn: int = 14336
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 40960
    init_std: float = 0.02
    # Llama-3.1 "llama3" RoPE frequency scaling: (factor, low_freq_factor, high_freq_factor,
    # original_max_position_embeddings); None = plain RoPE
    rope_scaling: Optional[Tuple[float, float, float, int]] = None

    @property
    def qkv_dim(self) -> int:
        return (self.n_heads + 2 * self.n_kv_heads) * self.head_dim

    def n_params(self) -> int:
        per_layer = (self.hidden * self.qkv_dim + self.n_heads * self.head_dim * self.hidden
                     + 3 * self.hidden * self.ffn + 2 * self.hidden)
        return self.n_layers * per_layer + 2 * self.vocab_size * self.hidden + self.hidden

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return 2 * self.n_layers * self.n_kv_heads * self.head_dim * dtype_bytes


# ------------------------------------------------------------------ hybrid attention / state-space models
@dataclass(frozen=True)
class AttnSpec:
    """Grouped-query attention without rotation: query head h reads kv head h // (heads // kv_heads).  ``bias``:
    q / k / v projections carry one; ``qk_norm``: RMS norm over the WHOLE q (and k) projection before the split
    into heads; ``head_gate``: head h's output is multiplied by sigmoid(W_g x)_h; ``q_temp`` = (coef, every):
    queries at position p are multiplied by 1 + coef * ln(floor((p + 1) / every) + 1)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[Tuple[float, float]] = None
    bias: bool = True
    qk_norm: bool = True
    head_gate: bool = True

    def __post_init__(self):
        if self.heads <= 0 or self.kv_heads <= 0 or self.heads % self.kv_heads:
            raise ValueError("attention: %d query heads do not group over %d kv heads" % (self.heads, self.kv_heads))


@dataclass(frozen=True)
class SSMSpec:
    """Mamba-2 (state-space duality): head h uses B / C group h // (heads // groups); ``conv`` taps of the causal
    short convolution; the gated output norm runs in ``norm_groups`` equal parts."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    def __post_init__(self):
        if self.heads % self.groups or self.inner % self.norm_groups or self.conv < 1:
            raise ValueError("state-space mixer: heads %d / groups %d / norm_groups %d / conv %d do not fit"
                             % (self.heads, self.groups, self.norm_groups, self.conv))

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """Channels of the short convolution: x, B and C."""
        return self.inner + 2 * self.groups * self.state

    @property
    def in_rows(self) -> int:
        """Rows of the input projection: z | x | B | C | dt."""
        return self.inner + self.channels + self.heads


@dataclass(frozen=True)
class YarnSpec:
    """YaRN interpolation of rotary frequencies: pairs that turn fewer than ``slow`` times over ``original`` positions
    are slowed down by ``factor``, those that turn more than ``fast`` times are kept, with a linear ramp between; cosine
    and sine are multiplied by 0.1 ln(factor) + 1."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotarySpec:
    """Rotate-half positions on ``dims`` dimensions: pair (i, i + dims / 2) turns by position * base^(-2 i / dims)."""
    dims: int
    base: float
    scaling: Optional[YarnSpec] = None

    def __post_init__(self):
        if self.dims <= 0 or self.dims % 2:
            raise ValueError("rotary positions need an even number of dimensions, got %d" % self.dims)


@dataclass(frozen=True)
class LatentSpec:
    """Latent attention: keys and values of every head are expanded from one normed latent of ``kv_rank`` per token
    (plus one rotated key part of ``rot.dims`` shared by the heads), queries from a normed latent of ``q_rank``.  Only
    the latent and the rotated part are cached.  ``kv_from``: the layer whose cache this one reads instead of having
    its own."""
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    rot: RotarySpec
    scale: float
    kv_from: Optional[int] = None

    @property
    def rot_dim(self) -> int:
        return self.rot.dims


@dataclass(frozen=True)
class DeltaSpec:
    """Gated delta rule: head h uses query / key head h // (heads // kv_heads); ``conv`` taps of the causal short
    convolutions of q, k and v; one decay and one step size per head; head-wise output norm with a silu gate."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    def __post_init__(self):
        if self.kv_heads <= 0 or self.heads % self.kv_heads or self.conv < 1:
            raise ValueError("delta mixer: heads %d / kv_heads %d / conv %d do not fit"
                             % (self.heads, self.kv_heads, self.conv))

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """Channels of the short convolutions: q, k and v."""
        return 2 * self.kv_heads * self.dim + self.inner


@dataclass(frozen=True)
class GeluSpec:
    """Plain feed-forward: W_down gelu(W_up h), the tanh form of gelu."""
    ff: int


@dataclass(frozen=True)
class BigramSpec:
    """A second embedding, indexed by the pair (previous token, token): row (previous * mul_prev + token * mul_cur)
    mod ``buckets``, and row ``buckets`` for a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class GLUSpec:
    """Clamped gated linear unit: g = min(g, limit), u = clamp(u, -limit, limit), y = g sigmoid(alpha g) (u + shift)."""
    ff: int
    limit: float
    alpha: float = 1.702
    shift: float = 1.0


@dataclass(frozen=True)
class LayerSpec:
    """One pre-norm layer: the mixers given (attention beside a state-space mixer, or latent attention, or a delta rule)
    on the same normed input, summed (attention and state-space mixer with their scales), and an optional feed-forward
    -- after the mixers behind a norm of its own, or, ``parallel``, on the mixers' input and added with them."""
    attn: Optional[AttnSpec] = None
    ssm: Optional[SSMSpec] = None
    mlp: Optional[Union[GLUSpec, GeluSpec]] = None
    attn_scale: float = 1.0
    ssm_scale: float = 1.0
    latent: Optional[LatentSpec] = None
    delta: Optional[DeltaSpec] = None
    parallel: bool = False

    def __post_init__(self):
        if all(m is None for m in (self.attn, self.ssm, self.latent, self.delta)):
            raise ValueError("a layer needs a mixer")
        if self.mlp is not None and isinstance(self.mlp, GeluSpec) != self.parallel:
            raise ValueError("a parallel layer has a plain feed-forward, a sequential one a gated one")


@dataclass(frozen=True)
class HybridConfig:
    """A decoder whose layers are listed one by one (engine/hybrid.py HybridModel): fp32 residual stream; the scaled
    embedding plus sinusoidal absolute positions (``pos_base``), or plus a bigram embedding and an RMS norm
    (``bigram``); the model's RMS norms multiply by (``norm_offset`` + weight)."""
    name: str
    vocab_size: int
    hidden: int
    layers: Tuple[LayerSpec, ...]
    rms_eps: float = 1e-6
    embed_scale: float = 1.0
    pos_base: Optional[float] = 10000.0
    norm_offset: float = 1.0
    max_position: int = 131072
    init_std: float = 0.02
    bigram: Optional[BigramSpec] = None
    tp_shardable = False  # recurrent mixers, whole-projection norms and shared latents are not sharded

    def __post_init__(self):
        for i, la in enumerate(self.layers):
            s = la.latent
            if s is None or s.kv_from is None:
                continue
            j = s.kv_from
            o = self.layers[j].latent if 0 <= j < i else None
            if o is None or o.kv_from is not None:
                raise ValueError("layer %d takes its latents from layer %r, which has none of its own before it" % (i, j))
            if (o.kv_rank, o.rot) != (s.kv_rank, s.rot):
                raise ValueError("layers %d and %d share latents of different form" % (i, j))

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    def n_params(self) -> int:
        n = 2 * self.vocab_size * self.hidden + self.hidden
        if self.bigram is not None:
            n += (self.bigram.buckets + 1) * self.hidden + self.hidden
        for la in self.layers:
            n += self.hidden
            if la.attn is not None:
                a = la.attn
                n += self.hidden * (a.heads * (a.dim + a.vdim + 1) + a.kv_heads * (a.dim + a.vdim))
            if la.ssm is not None:
                n += self.hidden * (la.ssm.in_rows + la.ssm.inner) + la.ssm.channels * (la.ssm.conv + 1)
            if la.latent is not None:
                s = la.latent
                n += s.q_rank * (self.hidden + 1 + s.heads * (s.dim + s.rot_dim))
                n += s.heads * (s.kv_rank * (s.dim + s.vdim) + s.vdim * self.hidden)
                if s.kv_from is None:
                    n += (s.kv_rank + s.rot_dim) * self.hidden + s.kv_rank
            if la.delta is not None:
                d = la.delta
                n += self.hidden * (d.channels + 2 * d.inner + 2 * d.heads) + d.channels * d.conv + 2 * d.heads + d.vdim
            if isinstance(la.mlp, GLUSpec):
                n += 3 * self.hidden * la.mlp.ff + self.hidden
            elif la.mlp is not None:
                n += 2 * self.hidden * la.mlp.ff
        return n

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        n = sum(la.attn.kv_heads * (la.attn.dim + la.attn.vdim) for la in self.layers if la.attn is not None)
        n += sum(la.latent.kv_rank + la.latent.rot_dim for la in self.layers
                 if la.latent is not None and la.latent.kv_from is None)
        return dtype_bytes * n

    def state_bytes_per_seq(self) -> int:
        """fp32 recurrent state and convolution taps of one sequence."""
        n = sum(la.ssm.inner * la.ssm.state + la.ssm.channels * (la.ssm.conv - 1) for la in self.layers
                if la.ssm is not None)
        n += sum(la.delta.inner * la.delta.dim + la.delta.channels * (la.delta.conv - 1) for la in self.layers
                 if la.delta is not None)
        return 4 * n


AnyConfig = Union[ModelConfig, HybridConfig]


def _merulorn(name, vocab, hidden, pattern, ssm, attn, side, ff, limit=7.0, scales=(0.75, 0.7), **kw) -> HybridConfig:
    """``pattern``: one letter per layer, m = mamba2, p = attention beside a state-space mixer, upper case = with a
    feed-forward."""
    glu = GLUSpec(ff, limit)
    layers = tuple(LayerSpec(attn if c in "pP" else None, side if c in "pP" else ssm, glu if c.isupper() else None,
                             *(scales if c in "pP" else (1.0, 1.0))) for c in pattern)
    return HybridConfig(name, vocab, hidden, layers, **kw)


def _muzozen(name, vocab, hidden, pattern, latent, delta, ff, bigram, **kw) -> HybridConfig:
    """``pattern``: one letter per layer, l = latent attention, s = latent attention over the latents of the last l,
    d = delta rule, upper case = with a feed-forward."""
    layers, own = [], None
    for i, c in enumerate(pattern):
        mlp = GeluSpec(ff) if c.isupper() else None
        if c in "dD":
            layers.append(LayerSpec(delta=delta, mlp=mlp, parallel=True))
        else:
            layers.append(LayerSpec(latent=replace(latent, kv_from=own if c in "sS" else None), mlp=mlp, parallel=True))
            own = i if c in "lL" else own
    return HybridConfig(name, vocab, hidden, tuple(layers), pos_base=None, norm_offset=0.0, bigram=bigram, **kw)


PRESETS = {
    "llama3-8b": ModelConfig("llama3-8b"),
    "llama3-70b": ModelConfig("llama3-70b", hidden=8192, n_layers=80, n_heads=64, n_kv_heads=8, ffn=28672),
    # Llama-3.1: same shapes, 128k positions with the "llama3" RoPE scaling -- the model for a single-pass
    # reduce over a whole day of summaries (--no-hierarchical on 24 h: ~100k-token prompt)
    "llama3.1-8b": ModelConfig("llama3.1-8b", max_position=131072, rope_scaling=(8.0, 1.0, 4.0, 8192)),
    "llama3.1-70b": ModelConfig("llama3.1-70b", hidden=8192, n_layers=80, n_heads=64, n_kv_heads=8, ffn=28672,
                                max_position=131072, rope_scaling=(8.0, 1.0, 4.0, 8192)),
    # test / smoke configs (real vocab, head_dim 128)
    "tiny": ModelConfig("tiny", hidden=256, n_layers=2, n_heads=2, n_kv_heads=1, ffn=512, max_position=8192),
    "tiny-gqa4": ModelConfig("tiny-gqa4", hidden=512, n_layers=2, n_heads=8, n_kv_heads=2, ffn=1024,
                             max_position=8192),
    # GQA 3:1 (Llama-3.2-3B's ratio, 24 / 8): the attention kernels' per-query-head fallback
    "tiny-gqa3": ModelConfig("tiny-gqa3", hidden=768, n_layers=2, n_heads=6, n_kv_heads=2, ffn=1024,
                             max_position=8192),
    # 8 KV heads (GQA 2:1) with heads / ffn / vocab divisible by 8: the TP=4 / TP=8 sharding paths of an
    # 8-GPU node (one or two KV heads per rank, 16032-row vocab shards, 8-way KV hand-off) on CPU ranks
    "tiny-kv8": ModelConfig("tiny-kv8", hidden=512, n_layers=2, n_heads=16, n_kv_heads=8, ffn=1024,
                            max_position=8192),
    # Merulorn designs (engine/hybrid.py).  merulorn-8b: layers of the width, head and FFN sizes of llama3-8b
    # (32 x 128 query heads over 8 kv heads, FFN 14336) with Mamba-2 mixers of inner size 8192 / 4096 (state 128),
    # 7.9e9 parameters to llama3-8b's 8.0e9
    "merulorn-8b": _merulorn("merulorn-8b", 128256, 4096, "mPPmPPmP" * 4,
                             ssm=SSMSpec(128, 64, 128, 8, 4, 8), side=SSMSpec(64, 64, 128, 8, 4, 8),
                             attn=AttnSpec(32, 8, 128, 128, 128 ** -0.5, (0.1, 1024.0)), ff=14336, embed_scale=64.0),
    "tiny-merulorn": _merulorn("tiny-merulorn", 128256, 192, "mPMp",
                               ssm=SSMSpec(4, 40, 24, 2, 4, 2), side=SSMSpec(3, 32, 40, 1, 3, 1),
                               attn=AttnSpec(6, 2, 48, 32, 48 ** -0.5, (0.2, 32.0)), ff=320, limit=2.0,
                               embed_scale=8.0, max_position=8192),
    # Muzozen designs (engine/hybrid.py).  muzozen-8b: 32 layers of llama3-8b's width with 32 heads of 128 (+ 64
    # rotated) over 512-wide latents and 32 x 128 delta heads, 7.9e9 parameters
    "muzozen-8b": _muzozen("muzozen-8b", 128256, 4096, "LSDD" * 8,
                           latent=LatentSpec(32, 128, 128, 1536, 512,
                                             RotarySpec(64, 500000.0, YarnSpec(8.0, 8192, 32.0, 1.0)), 192 ** -0.5),
                           delta=DeltaSpec(32, 16, 128, 128, 4), ff=18432, bigram=BigramSpec(65536, 8191, 127),
                           embed_scale=8.0),
    "tiny-muzozen": _muzozen("tiny-muzozen", 128256, 192, "LdSD",
                             latent=LatentSpec(4, 48, 32, 72, 96, RotarySpec(24, 10000.0, YarnSpec(2.0, 512, 16.0, 1.0)),
                                               0.12),
                             delta=DeltaSpec(4, 2, 40, 24, 3), ff=320, bigram=BigramSpec(1021, 13, 5), embed_scale=4.0,
                             max_position=8192),
}


def get_model_config(name: str, **overrides) -> AnyConfig:
    key = name.lower()
    if key not in PRESETS:
        raise ValueError("unknown model %r (known: %s)" % (name, ", ".join(sorted(PRESETS))))
    cfg = PRESETS[key]
    return replace(cfg, **overrides) if overrides else cfg
