"""Model architecture configs (random-init; shapes of the public checkpoints).

Llama-3 shapes: public HF ``config.json`` of meta-llama/Meta-Llama-3-8B / -70B
(rope_theta 5e5; Llama-3.1 adds the "llama3" rope scaling, kept optional here).
Mixtral-8x7B: transformers ``MixtralConfig`` defaults (SURVEY.md §2.5 model table).
"""
from __future__ import annotations

from dataclasses import asdict, dataclass, field, replace


@dataclass(frozen=True)
class ModelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    intermediate_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    head_dim: int = 128
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    # MoE (Mixtral): 0 experts = dense MLP
    num_experts: int = 0
    top_k: int = 2
    rope_scaling: dict | None = field(default=None, hash=False, compare=False)
    eos_token_id: int = 128001
    # further end-of-sequence ids (HF eos_token_id lists, e.g. Llama-3.1-Instruct's
    # [128001, 128008, 128009]: <|eot_id|> must stop generation too)
    extra_eos_ids: tuple = field(default=(), hash=False, compare=False)

    @property
    def eos_ids(self) -> tuple:
        return (self.eos_token_id, *self.extra_eos_ids)

    @property
    def is_moe(self) -> bool:
        return self.num_experts > 0

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    def num_params(self) -> int:
        H, I, V, L = self.hidden_size, self.intermediate_size, self.vocab_size, self.num_layers
        attn = H * (self.q_size + 2 * self.kv_size) + self.q_size * H
        mlp = 3 * H * I * (self.num_experts if self.is_moe else 1)
        router = H * self.num_experts if self.is_moe else 0
        norms = 2 * H
        emb = V * H * (1 if self.tie_embeddings else 2)
        return L * (attn + mlp + router + norms) + emb + H

    def active_params(self) -> int:
        if not self.is_moe:
            return self.num_params()
        dense = replace(self, num_experts=0)
        extra = self.num_layers * 3 * self.hidden_size * self.intermediate_size * (self.top_k - 1)
        return dense.num_params() + extra + self.num_layers * self.hidden_size * self.num_experts

    def weight_bytes(self, dtype_bytes: int = 2) -> int:
        return self.num_params() * dtype_bytes

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return 2 * self.num_layers * self.kv_size * dtype_bytes

    def flops_per_token(self) -> int:
        """Matmul FLOPs of one forward token (2 * active params, attention excluded)."""
        return 2 * self.active_params()

    def to_dict(self) -> dict:
        return asdict(self)


@dataclass(frozen=True)
class YarnSpec:
    """Stretched rotary frequencies: pairs that turn less than ``slow`` times in ``original`` positions turn
    ``factor`` times slower, pairs that turn more than ``fast`` times as before, a ramp between them; cos
    and sin times 0.1 ln(factor) + 1."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotarySpec:
    """Rotary positions of ``dims`` dimensions in pairs (2i, 2i + 1)."""
    base: float
    dims: int
    scaling: YarnSpec | None = None


@dataclass(frozen=True)
class AttentionSpec:
    """Softmax-attention mixer of a hybrid decoder layer."""
    heads: int
    kv_heads: int
    dim: int                 # query / key head size
    vdim: int                # value head size
    scale: float             # score scale
    rot_base: float
    rot_dims: int            # leading dims of a head that rotate (pairs 2i, 2i + 1)
    v_mix: bool = False      # values mixed with the first v_mix layer's
    scaling: YarnSpec | None = None
    window: int = 0          # a token sees itself and the window - 1 tokens before it (0: all)
    head_norm: bool = False  # query / key norm per head, one weight for all heads (else over the whole rows)
    tied_kv: bool = False    # the values are the projected keys (before norm and rotation)
    sink: bool = True        # a number per head joins the softmax's denominator
    gate_elem: bool = False  # output gate per value element (else per head)

    @property
    def rot(self) -> RotarySpec:
        return RotarySpec(self.rot_base, self.rot_dims, self.scaling)

    def params(self, width: int) -> int:
        norms = 2 * self.dim if self.head_norm else (self.heads + self.kv_heads) * self.dim
        return self.macs(width) + norms + self.heads * self.sink + int(self.v_mix)

    def macs(self, width: int) -> int:
        qk, v = (self.heads + self.kv_heads) * self.dim, 0 if self.tied_kv else self.kv_heads * self.vdim
        gates = self.heads * (self.vdim if self.gate_elem else 1)
        return width * (qk + v + gates + self.heads * self.vdim)


@dataclass(frozen=True)
class GLASpec:
    """Gated-linear-attention mixer: a [dim, vdim] state per head with a decay per key channel."""
    heads: int
    dim: int
    vdim: int
    tau: float               # decay = sigmoid(z) ** (1 / tau)
    rank: int                # inner size of the decay projection

    def params(self, width: int) -> int:
        hk, hv = self.heads * self.dim, self.heads * self.vdim
        return width * (2 * hk + 3 * hv + self.rank) + hk * (self.rank + 1) + self.vdim

    def macs(self, width: int) -> int:
        hk, hv = self.heads * self.dim, self.heads * self.vdim
        return width * (2 * hk + 3 * hv + self.rank) + hk * self.rank + 2 * hk * self.vdim

    def state_elems(self) -> int:
        return self.heads * self.dim * self.vdim


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Softmax-attention mixer over cached latents."""
    heads: int
    dim: int                 # query / key head size (without a rotated part)
    vdim: int                # value head size
    rank: int                # latent size
    scale: float             # score scale
    window: int = 0          # a token sees itself and the window - 1 tokens before it (0: all)
    sink: bool = True        # a number per head joins the softmax's denominator
    gate: bool = True        # output gate, one per value element
    q_rank: int = 0          # queries through a normed latent of this size (0: straight from the input)
    rot: RotarySpec | None = None  # rotated part of queries and keys; a key's is one for all heads, cached
    kv_from: int = -1        # layer whose cached latents and rotated keys this one reads (-1: its own)

    @property
    def rot_dim(self) -> int:
        return self.rot.dims if self.rot else 0

    @property
    def cached(self) -> int:
        """Values kept per token."""
        return 0 if self.kv_from >= 0 else self.rank + self.rot_dim

    def params(self, width: int) -> int:
        n = self.macs(width) + self.q_rank + self.heads * self.sink
        return n + (self.rank if self.kv_from < 0 else 0)

    def macs(self, width: int) -> int:
        hq, hv = self.heads * (self.dim + self.rot_dim), self.heads * self.vdim
        q = self.q_rank * (width + hq) if self.q_rank else width * hq
        return q + width * (self.cached + hv * (1 + self.gate)) + self.rank * (self.heads * self.dim + hv)


@dataclass(frozen=True)
class SSDSpec:
    """Selective-state-space mixer (Mamba-2): a [state, vdim] state per head with one decay per head,
    behind a short convolution."""
    heads: int
    vdim: int
    state: int
    groups: int              # B and C are shared by heads / groups heads
    taps: int                # of the convolution
    norm_groups: int         # equal parts of the output norm

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """Convolved channels: x, B and C."""
        return self.inner + 2 * self.groups * self.state

    def params(self, width: int) -> int:
        return (width * (2 * self.inner + 2 * self.groups * self.state + self.heads) + width * self.inner +
                self.channels * (self.taps + 1) + 3 * self.heads + self.inner)

    def macs(self, width: int) -> int:
        return (width * (3 * self.inner + 2 * self.groups * self.state + self.heads) + self.channels * self.taps +
                2 * self.inner * self.state)

    def state_elems(self) -> int:
        return self.inner * self.state + (self.taps - 1) * self.channels


@dataclass(frozen=True)
class DeltaSpec:
    """Generalized-delta-rule mixer: a [dim, dim] state per head with a decay and a removal rate per key
    channel."""
    heads: int
    dim: int
    rank: int                # inner size of the decay projection

    def params(self, width: int) -> int:
        n = self.heads * self.dim
        return width * (6 * n + self.rank) + n * (self.rank + 3)

    def macs(self, width: int) -> int:
        n = self.heads * self.dim
        return width * (6 * n + self.rank) + n * self.rank + 3 * n * self.dim

    def state_elems(self) -> int:
        return self.heads * self.dim * self.dim


@dataclass(frozen=True)
class MoESpec:
    """Mixture of gated experts.

    ``scores`` "sigmoid": each token goes through the ``top`` experts with the largest sigmoid scores, its input
    times the score; beside them a shared expert (``shared`` 0: none) with a sigmoid gate per token.
    "softmax": scores over all experts, the weights on the experts' outputs as they are.  The last ``identity``
    of the scored outputs give the token itself back.  A number per output (``correction``) joins the score where
    experts are chosen, and only there; the outputs form ``groups`` equal groups of neighbours, and the choice is
    from the ``keep`` groups with the largest best one."""
    experts: int
    top: int
    ff: int
    shared: int = 0
    scores: str = "sigmoid"
    identity: int = 0
    groups: int = 1
    keep: int = 1
    correction: bool = False
    limit: float = 0.0       # clamped gated unit with this bound (0: silu(gate) up)

    @property
    def outputs(self) -> int:
        """Router outputs that are experts."""
        return self.experts + self.identity

    def params(self, width: int) -> int:
        return (width * (self.outputs + 3 * self.experts * self.ff + 3 * self.shared + bool(self.shared)) +
                self.outputs * self.correction)

    def macs(self, width: int) -> int:
        used = 3 * self.top * self.ff * self.experts // self.outputs
        return width * (self.outputs + used + 3 * self.shared + bool(self.shared))


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec | GLASpec | LatentAttentionSpec | SSDSpec | DeltaSpec
    ff: int = 0              # feed-forward width (0: none)
    limit: float = 0.0       # clamp of a gated feed-forward (designs that have one)
    moe: MoESpec | None = None  # experts instead of the feed-forward
    weights_of: int = -1     # layer whose weights this one uses (-1: its own); its cache is its own


@dataclass(frozen=True)
class HybridConfig(ModelConfig):
    """A decoder whose layers are listed one by one (``layers``).  The uniform fields of ``ModelConfig``
    hold the largest layer's sizes."""
    layers: tuple = ()

    def __post_init__(self):
        # replace(num_layers=n) keeps the first n layers
        object.__setattr__(self, "layers", self.layers[:self.num_layers])

    @property
    def attention(self) -> tuple:
        """Mixers that keep pages."""
        return tuple(la.mixer for la in self.layers if isinstance(la.mixer, (AttentionSpec, LatentAttentionSpec)))

    @property
    def recurrent(self) -> tuple:
        """Mixers that keep a state."""
        return tuple(la.mixer for la in self.layers if isinstance(la.mixer, (GLASpec, SSDSpec, DeltaSpec)))

    def active_params(self) -> int:
        return self.num_params()

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(m.cached if isinstance(m, LatentAttentionSpec) else m.kv_heads * (m.dim + m.vdim)
                   for m in self.attention) * dtype_bytes

    def state_bytes_per_seq(self) -> int:
        return 4 * sum(m.state_elems() for m in self.recurrent)


@dataclass(frozen=True)
class KosesunConfig(HybridConfig):
    """Kosesun: attention and gated linear attention on hyper-connection streams, squared-relu
    feed-forward."""
    streams: int = 1
    embed_scale: float = 1.0
    logit_softcap: float = 0.0

    def num_params(self) -> int:
        W, S, n = self.hidden_size, self.streams, 2 * self.vocab_size * self.hidden_size + self.hidden_size
        for la in self.layers:
            sub = 1 + bool(la.ff)
            n += la.mixer.params(W) + 2 * W * la.ff + sub * (W + S * (S + 2))
        return n

    def flops_per_token(self) -> int:
        W = self.hidden_size
        return 2 * (self.vocab_size * W + sum(la.mixer.macs(W) + 2 * W * la.ff for la in self.layers))


@dataclass(frozen=True)
class RegesunConfig(HybridConfig):
    """Regesun: windowed latent attention, selective state space and generalized delta rule, a norm
    before and behind every sublayer with a layer scale, learned positions (``max_position`` of them),
    clamped gated feed-forward."""

    def num_params(self) -> int:
        W = self.hidden_size
        n = (2 * self.vocab_size + self.max_position + 1) * W
        for la in self.layers:
            n += la.mixer.params(W) + 3 * W * la.ff + 3 * W * (1 + bool(la.ff))
        return n

    def flops_per_token(self) -> int:
        W = self.hidden_size
        return 2 * (self.vocab_size * W + sum(la.mixer.macs(W) + 3 * W * la.ff for la in self.layers))


@dataclass(frozen=True)
class NafazenConfig(HybridConfig):
    """Nafazen: latent attention with a rotated key part, on layers' own or an earlier layer's latents, dense
    (xIELU) and mixture-of-experts feed-forwards, norms behind the sublayers only, soft-capped logits."""
    embed_scale: float = 1.0
    logit_softcap: float = 0.0

    def __post_init__(self):
        super().__post_init__()
        for i, m in enumerate(self.attention):
            if m.kv_from < 0:
                continue
            src = self.layers[m.kv_from].mixer if m.kv_from < i else None
            if src is None or src.kv_from >= 0 or (src.rank, src.rot) != (m.rank, m.rot):
                raise ValueError(f"layer {i}: layer {m.kv_from} has no latents of its own for it")

    def _count(self, moe) -> int:
        W = self.hidden_size
        n = 2 * self.vocab_size * W + 1
        for la in self.layers:
            n += la.mixer.params(W) + 1 + bool(la.ff or la.moe)
            n += moe(la.moe) if la.moe else 2 * W * la.ff + 2 * bool(la.ff)
        return n

    def num_params(self) -> int:
        return self._count(lambda e: e.params(self.hidden_size))

    def active_params(self) -> int:
        return self._count(lambda e: e.macs(self.hidden_size))

    def flops_per_token(self) -> int:
        W = self.hidden_size
        return 2 * (self.vocab_size * W + sum(la.mixer.macs(W) + (la.moe.macs(W) if la.moe else 2 * W * la.ff)
                                              for la in self.layers))


@dataclass(frozen=True)
class DibedraConfig(HybridConfig):
    """Dibedra: windowed attention whose values are its keys, beside the feed-forward (dense or experts in groups,
    some of them the identity) on one normed input; dynamic-tanh norms; layers may use another's weights."""
    logit_scale: float = 1.0

    def __post_init__(self):
        super().__post_init__()
        for i, la in enumerate(self.layers):
            j = la.weights_of
            if j >= 0 and (j >= len(self.layers) or self.layers[j].weights_of >= 0 or replace(self.layers[j], weights_of=j) != la):
                raise ValueError(f"layer {i}: layer {j} has no weights of its own for it")

    def _count(self, layer) -> int:
        # embedding, head, last norm
        return (2 * self.vocab_size + 2) * self.hidden_size + 1 + sum(layer(la) for la in self.layers)

    def num_params(self) -> int:
        W = self.hidden_size
        return self._count(lambda la: 0 if la.weights_of >= 0 else la.mixer.params(W) + 2 * W + 1 +
                           (la.moe.params(W) if la.moe else 2 * W * la.ff))

    def active_params(self) -> int:
        W = self.hidden_size
        return self._count(lambda la: la.mixer.params(W) + 2 * W + 1 + (la.moe.macs(W) if la.moe else 2 * W * la.ff))

    def flops_per_token(self) -> int:
        W = self.hidden_size
        return 2 * (self.vocab_size * W + sum(la.mixer.macs(W) + (la.moe.macs(W) if la.moe else 2 * W * la.ff)
                                              for la in self.layers))


def _hybrid(cls, name: str, vocab: int, width: int, layers, eps: float, **kw):
    """``cls`` over listed layers, the uniform fields from the largest attention layer."""
    layers = tuple(layers)
    att = [la.mixer for la in layers if isinstance(la.mixer, (AttentionSpec, LatentAttentionSpec))]
    return cls(
        name=name, vocab_size=vocab, hidden_size=width,
        intermediate_size=max((la.moe.ff if la.moe else la.ff for la in layers), default=0),
        num_layers=len(layers), num_heads=max((m.heads for m in att), default=1),
        num_kv_heads=max((getattr(m, "kv_heads", 1) for m in att), default=1),
        head_dim=max((m.dim for m in att), default=64), rms_eps=eps, layers=layers,
        **{"max_position": 131072, "eos_token_id": -1, **kw})


def kosesun_config(name: str, vocab: int, width: int, layers, streams: int, embed_scale: float, logit_softcap: float,
                   eps: float = 1e-5, **kw) -> KosesunConfig:
    return _hybrid(KosesunConfig, name, vocab, width, layers, eps, streams=streams, embed_scale=embed_scale,
                   logit_softcap=logit_softcap, **kw)


def regesun_config(name: str, vocab: int, width: int, layers, max_position: int, eps: float = 1e-5, **kw) -> RegesunConfig:
    return _hybrid(RegesunConfig, name, vocab, width, layers, eps, max_position=max_position, **kw)


def nafazen_config(name: str, vocab: int, width: int, layers, embed_scale: float, logit_softcap: float, eps: float = 1e-5,
                   **kw) -> NafazenConfig:
    return _hybrid(NafazenConfig, name, vocab, width, layers, eps, embed_scale=embed_scale, logit_softcap=logit_softcap, **kw)


def dibedra_config(name: str, vocab: int, width: int, layers, logit_scale: float = 1.0, eps: float = 1e-5, **kw) -> DibedraConfig:
    return _hybrid(DibedraConfig, name, vocab, width, layers, eps, logit_scale=logit_scale, **kw)


LLAMA3_8B = ModelConfig(
    name="llama3-8b", vocab_size=128256, hidden_size=4096, intermediate_size=14336,
    num_layers=32, num_heads=32, num_kv_heads=8, rope_theta=500000.0, max_position=8192)

LLAMA3_70B = ModelConfig(
    name="llama3-70b", vocab_size=128256, hidden_size=8192, intermediate_size=28672,
    num_layers=80, num_heads=64, num_kv_heads=8, rope_theta=500000.0, max_position=8192)

# Llama-3.1: same shapes, 128k context through the "llama3" RoPE frequency scaling
# (public HF config.json of meta-llama/Llama-3.1-8B / -70B)
_LLAMA31_ROPE = {"rope_type": "llama3", "factor": 8.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                 "original_max_position_embeddings": 8192}
LLAMA31_8B = replace(LLAMA3_8B, name="llama3.1-8b", max_position=131072, rope_scaling=_LLAMA31_ROPE)
LLAMA31_70B = replace(LLAMA3_70B, name="llama3.1-70b", max_position=131072, rope_scaling=_LLAMA31_ROPE)

MIXTRAL_8X7B = ModelConfig(
    name="mixtral-8x7b", vocab_size=32000, hidden_size=4096, intermediate_size=14336,
    num_layers=32, num_heads=32, num_kv_heads=8, rope_theta=1e6, max_position=32768,
    num_experts=8, top_k=2, eos_token_id=2)

# tiny shapes for CPU unit tests / GPU smoke (same code paths: GQA 4, head_dim 128)
TINY_LLAMA = ModelConfig(
    name="tiny-llama", vocab_size=512, hidden_size=256, intermediate_size=512, num_layers=2,
    num_heads=4, num_kv_heads=1, max_position=2048, eos_token_id=1)

TINY_MIXTRAL = ModelConfig(
    name="tiny-mixtral", vocab_size=512, hidden_size=256, intermediate_size=256, num_layers=2,
    num_heads=4, num_kv_heads=1, max_position=2048, num_experts=4, top_k=2, eos_token_id=1)

# CPU rehearsals of the 8-rank bench (bench.py --gpus 8 over gloo): 8 q heads so TP = 8 shards them
# (the one kv head is replicated), 8 experts so EP = 8 gives every rank one
TINY_LLAMA_8H = replace(TINY_LLAMA, name="tiny-llama-8h", num_heads=8)
TINY_MIXTRAL_8E = replace(TINY_MIXTRAL, name="tiny-mixtral-8e", num_experts=8)

def _kosesun(name: str, width: int, ff: int, n_layers: int, vocab: int, heads: int, kv_heads: int, dim: int, vdim: int,
             gla: GLASpec, **kw) -> KosesunConfig:
    """One recurrent layer in three, attention elsewhere, four streams."""
    att = AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, rot_base=500000.0,
                        rot_dims=dim // 2, v_mix=True)
    layers = [LayerSpec(gla if i % 3 == 1 else att, ff) for i in range(n_layers)]
    return kosesun_config(name, vocab, width, layers, streams=4, embed_scale=width ** 0.5, logit_softcap=30.0, **kw)


# layers of the size of the Llama-3 presets' (same width, query / key / value sizes, feed-forward
# parameters); the tiny one is for tests and demos
KOSESUN_8B = _kosesun("kosesun-8b", width=4096, ff=21504, n_layers=32, vocab=128256, heads=32, kv_heads=8, dim=128,
                      vdim=128, gla=GLASpec(heads=16, dim=128, vdim=256, tau=16.0, rank=16))
KOSESUN_1B = _kosesun("kosesun-1b", width=2048, ff=8192, n_layers=18, vocab=128256, heads=16, kv_heads=4, dim=128,
                      vdim=64, gla=GLASpec(heads=8, dim=128, vdim=128, tau=16.0, rank=16))
TINY_KOSESUN = _kosesun("tiny-kosesun", width=256, ff=384, n_layers=4, vocab=512, heads=6, kv_heads=2, dim=32, vdim=48,
                        gla=GLASpec(heads=3, dim=24, vdim=40, tau=8.0, rank=12), max_position=2048)


def _regesun(name: str, width: int, ff: int, n_layers: int, vocab: int, ssd: SSDSpec, latent: LatentAttentionSpec,
             delta: DeltaSpec, limit: float, max_position: int) -> RegesunConfig:
    """State space, windowed latent attention and delta rule in turn, a feed-forward in every layer."""
    mixers = (ssd, latent, delta)
    return regesun_config(name, vocab, width, [LayerSpec(mixers[i % 3], ff, limit) for i in range(n_layers)], max_position)


# layers of the size of the Kosesun presets' (same width, feed-forward parameters, vocabulary)
REGESUN_8B = _regesun("regesun-8b", width=4096, ff=14336, n_layers=32, vocab=128256,
                      ssd=SSDSpec(heads=64, vdim=128, state=128, groups=8, taps=4, norm_groups=8),
                      latent=LatentAttentionSpec(heads=32, dim=128, vdim=128, rank=512, scale=128 ** -0.5, window=4096),
                      delta=DeltaSpec(heads=32, dim=128, rank=64), limit=7.0, max_position=32768)
REGESUN_1B = _regesun("regesun-1b", width=2048, ff=5376, n_layers=18, vocab=128256,
                      ssd=SSDSpec(heads=64, vdim=64, state=128, groups=1, taps=4, norm_groups=1),
                      latent=LatentAttentionSpec(heads=16, dim=128, vdim=64, rank=256, scale=128 ** -0.5, window=1024),
                      delta=DeltaSpec(heads=32, dim=64, rank=32), limit=7.0, max_position=32768)
TINY_REGESUN = _regesun("tiny-regesun", width=256, ff=320, n_layers=4, vocab=512,
                        ssd=SSDSpec(heads=4, vdim=40, state=24, groups=2, taps=3, norm_groups=2),
                        latent=LatentAttentionSpec(heads=5, dim=24, vdim=32, rank=72, scale=0.2, window=40),
                        delta=DeltaSpec(heads=3, dim=56, rank=12), limit=2.0, max_position=2048)


def _nafazen(name: str, width: int, ff: int, n_layers: int, vocab: int, heads: int, dim: int, rot_dim: int, vdim: int,
             rank: int, q_rank: int, moe: MoESpec, **kw) -> NafazenConfig:
    """Four layers in turn: stretched positions and a dense feed-forward, plain positions and experts, twice;
    the last reads the second's latents."""
    def att(scaling=None, kv_from=-1):
        return LatentAttentionSpec(heads=heads, dim=dim, vdim=vdim, rank=rank, scale=(dim + rot_dim) ** -0.5, sink=False,
                                   gate=False, q_rank=q_rank, rot=RotarySpec(500000.0, rot_dim, scaling), kv_from=kv_from)

    yarn = YarnSpec(factor=4.0, original=4096, fast=32.0, slow=1.0)
    turn = lambda i: (LayerSpec(att(yarn), ff), LayerSpec(att(), moe=moe), LayerSpec(att(yarn), ff),  # noqa: E731
                      LayerSpec(att(kv_from=i - 2), moe=moe))[i % 4]
    return nafazen_config(name, vocab, width, [turn(i) for i in range(n_layers)], embed_scale=width ** 0.5,
                          logit_softcap=30.0, **kw)


# attention and feed-forward sizes of the Regesun presets' order
NAFAZEN_8B = _nafazen("nafazen-8b", width=4096, ff=14336, n_layers=32, vocab=128256, heads=32, dim=128, rot_dim=64, vdim=128,
                      rank=512, q_rank=1536, moe=MoESpec(experts=8, top=2, ff=1792, shared=3584))
NAFAZEN_1B = _nafazen("nafazen-1b", width=2048, ff=8192, n_layers=16, vocab=128256, heads=16, dim=64, rot_dim=64, vdim=64,
                      rank=256, q_rank=768, moe=MoESpec(experts=16, top=2, ff=768, shared=1536))
TINY_NAFAZEN = _nafazen("tiny-nafazen", width=192, ff=200, n_layers=4, vocab=512, heads=5, dim=24, rot_dim=16, vdim=40,
                        rank=72, q_rank=56, moe=MoESpec(experts=6, top=2, ff=40, shared=72), max_position=2048)


def _dibedra(name: str, width: int, ff: int, n_layers: int, vocab: int, heads: int, kv_heads: int, dim: int, window: int,
             moe: MoESpec, **kw) -> DibedraConfig:
    """Four layers in turn: a dense feed-forward, experts, the same dense layer, and the experts' once more."""
    att = AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, rot_base=500000.0, rot_dims=dim,
                        scaling=YarnSpec(factor=4.0, original=4096, fast=32.0, slow=1.0), window=window, head_norm=True,
                        tied_kv=True, sink=False, gate_elem=True)
    turn = lambda i: LayerSpec(att, *(() if i % 2 else (ff,)), moe=moe if i % 2 else None,  # noqa: E731
                               weights_of=i - 2 if i % 4 > 1 else -1)
    return dibedra_config(name, vocab, width, [turn(i) for i in range(n_layers)], logit_scale=0.5, **kw)


# head sizes of the Llama's, feed-forwards of the Kosesun presets' and experts of the Nafazen presets' sizes (two of
# them per token where the scores are even)
DIBEDRA_8B = _dibedra("dibedra-8b", width=4096, ff=21504, n_layers=32, vocab=128256, heads=32, kv_heads=8, dim=128, window=4096,
                      moe=MoESpec(experts=8, top=3, ff=1792, scores="softmax", identity=4, groups=3, keep=2, correction=True,
                                  limit=7.0))
DIBEDRA_1B = _dibedra("dibedra-1b", width=2048, ff=8192, n_layers=16, vocab=128256, heads=16, kv_heads=4, dim=128, window=1024,
                      moe=MoESpec(experts=16, top=3, ff=768, scores="softmax", identity=8, groups=6, keep=3, correction=True,
                                  limit=7.0))
TINY_DIBEDRA = _dibedra("tiny-dibedra", width=192, ff=200, n_layers=5, vocab=512, heads=6, kv_heads=2, dim=24, window=40,
                        moe=MoESpec(experts=5, top=2, ff=40, scores="softmax", identity=1, groups=3, keep=2, correction=True,
                                    limit=2.0), max_position=2048)

PRESETS = {c.name: c for c in (LLAMA3_8B, LLAMA3_70B, LLAMA31_8B, LLAMA31_70B, MIXTRAL_8X7B, TINY_LLAMA,
                                TINY_MIXTRAL, TINY_LLAMA_8H, TINY_MIXTRAL_8E, KOSESUN_8B, KOSESUN_1B,
                                TINY_KOSESUN, REGESUN_8B, REGESUN_1B, TINY_REGESUN, NAFAZEN_8B, NAFAZEN_1B,
                                TINY_NAFAZEN, DIBEDRA_8B, DIBEDRA_1B, TINY_DIBEDRA)}
# accepted aliases (MLflow tags / CR annotations use HF-ish names)
ALIASES = {
    "meta-llama/Meta-Llama-3-8B": "llama3-8b", "llama-3-8b": "llama3-8b", "Llama-3-8B": "llama3-8b",
    "meta-llama/Meta-Llama-3-70B": "llama3-70b", "llama-3-70b": "llama3-70b", "Llama-3-70B": "llama3-70b",
    "meta-llama/Llama-3.1-8B": "llama3.1-8b", "meta-llama/Meta-Llama-3.1-8B": "llama3.1-8b",
    "meta-llama/Llama-3.1-70B": "llama3.1-70b", "meta-llama/Meta-Llama-3.1-70B": "llama3.1-70b",
    "mistralai/Mixtral-8x7B-v0.1": "mixtral-8x7b", "Mixtral-8x7B": "mixtral-8x7b",
}


def get_config(name: str, **overrides) -> ModelConfig:
    key = ALIASES.get(name, name)
    if key not in PRESETS:
        raise KeyError(f"unknown model '{name}' (known: {sorted(PRESETS)})")
    cfg = PRESETS[key]
    return replace(cfg, **overrides) if overrides else cfg
