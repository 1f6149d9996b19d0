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

    def params(self, width: int) -> int:
        qk, v = (self.heads + self.kv_heads) * self.dim, self.kv_heads * self.vdim
        return width * (qk + v + self.heads + self.heads * self.vdim) + qk + self.heads + int(self.v_mix)

    def macs(self, width: int) -> int:
        return width * ((self.heads + self.kv_heads) * self.dim + (self.kv_heads + self.heads) * self.vdim + self.heads)


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


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec | GLASpec
    ff: int = 0              # squared-relu feed-forward width (0: none)


@dataclass(frozen=True)
class HybridConfig(ModelConfig):
    """A decoder whose layers are listed one by one (``layers``), on hyper-connection streams
    (Kosesun).  The uniform fields of ``ModelConfig`` hold the largest layer's sizes."""
    layers: tuple = ()
    streams: int = 1
    embed_scale: float = 1.0
    logit_softcap: float = 0.0

    def __post_init__(self):
        # replace(num_layers=n) keeps the first n layers
        object.__setattr__(self, "layers", self.layers[:self.num_layers])

    @property
    def attention(self) -> tuple:
        return tuple(la.mixer for la in self.layers if isinstance(la.mixer, AttentionSpec))

    @property
    def recurrent(self) -> tuple:
        return tuple(la.mixer for la in self.layers if isinstance(la.mixer, GLASpec))

    def num_params(self) -> int:
        W, S, n = self.hidden_size, self.streams, 2 * self.vocab_size * self.hidden_size + self.hidden_size
        for la in self.layers:
            sub = 1 + bool(la.ff)
            n += la.mixer.params(W) + 2 * W * la.ff + sub * (W + S * (S + 2))
        return n

    def active_params(self) -> int:
        return self.num_params()

    def flops_per_token(self) -> int:
        W = self.hidden_size
        return 2 * (self.vocab_size * W + sum(la.mixer.macs(W) + 2 * W * la.ff for la in self.layers))

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(m.kv_heads * (m.dim + m.vdim) for m in self.attention) * dtype_bytes

    def state_bytes_per_seq(self) -> int:
        return sum(m.heads * m.dim * m.vdim for m in self.recurrent) * 4


def hybrid_config(name: str, vocab: int, width: int, layers, streams: int, embed_scale: float, logit_softcap: float,
                  eps: float = 1e-5, **kw) -> HybridConfig:
    layers = tuple(layers)
    att = [la.mixer for la in layers if isinstance(la.mixer, AttentionSpec)]
    return HybridConfig(
        name=name, vocab_size=vocab, hidden_size=width, intermediate_size=max((la.ff for la in layers), default=0),
        num_layers=len(layers), num_heads=max((m.heads for m in att), default=1),
        num_kv_heads=max((m.kv_heads for m in att), default=1), head_dim=max((m.dim for m in att), default=64),
        rms_eps=eps, layers=layers, streams=streams, embed_scale=embed_scale, logit_softcap=logit_softcap,
        **{"max_position": 131072, "eos_token_id": -1, **kw})


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
             gla: GLASpec, **kw) -> HybridConfig:
    """One recurrent layer in three, attention elsewhere, four streams."""
    att = AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, rot_base=500000.0,
                        rot_dims=dim // 2, v_mix=True)
    layers = [LayerSpec(gla if i % 3 == 1 else att, ff) for i in range(n_layers)]
    return hybrid_config(name, vocab, width, layers, streams=4, embed_scale=width ** 0.5, logit_softcap=30.0, **kw)


# layers of the size of the Llama-3 presets' (same width, query / key / value sizes, feed-forward
# parameters); the tiny one is for tests and demos
KOSESUN_8B = _kosesun("kosesun-8b", width=4096, ff=21504, n_layers=32, vocab=128256, heads=32, kv_heads=8, dim=128,
                      vdim=128, gla=GLASpec(heads=16, dim=128, vdim=256, tau=16.0, rank=16))
KOSESUN_1B = _kosesun("kosesun-1b", width=2048, ff=8192, n_layers=18, vocab=128256, heads=16, kv_heads=4, dim=128,
                      vdim=64, gla=GLASpec(heads=8, dim=128, vdim=128, tau=16.0, rank=16))
TINY_KOSESUN = _kosesun("tiny-kosesun", width=256, ff=384, n_layers=4, vocab=512, heads=6, kv_heads=2, dim=32, vdim=48,
                        gla=GLASpec(heads=3, dim=24, vdim=40, tau=8.0, rank=12), max_position=2048)

PRESETS = {c.name: c for c in (LLAMA3_8B, LLAMA3_70B, LLAMA31_8B, LLAMA31_70B, MIXTRAL_8X7B, TINY_LLAMA,
                                TINY_MIXTRAL, TINY_LLAMA_8H, TINY_MIXTRAL_8E, KOSESUN_8B, KOSESUN_1B,
                                TINY_KOSESUN)}
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
