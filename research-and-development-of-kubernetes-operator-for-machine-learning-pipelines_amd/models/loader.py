"""Checkpoint loading: Hugging Face ``config.json`` + ``*.safetensors`` -> our model layout.

The operator hands a predictor its MLflow artifact URI (``s3://mlflow/<rel>``, reference
``mlflow_operator.py:125-127``).  When that artifact is reachable as a local directory
(``file://`` URI, a plain path, or ``s3://mlflow/<rel>`` under ``MLOP_ARTIFACT_ROOT``)
holding a Llama / Mixtral checkpoint in the HF layout, the runtime serves those weights;
otherwise it random-initialises the architecture named by the CR / MLflow tags (the
benchmark configuration: no checkpoints are downloadable here).

Layout mapping (HF name -> ours; TP sharding then reuses ``load_shard_from``):
  model.embed_tokens / lm_head / model.norm       -> embed / lm_head / final_norm
  self_attn.{q,k,v}_proj                         -> qkv  ([q; k; v] rows, rotate-half RoPE as HF)
  self_attn.o_proj                               -> o
  input_layernorm / post_attention_layernorm     -> in_norm / post_norm
  mlp.{gate,up}_proj                             -> gate_up (rows interleaved in groups of 16:
                                                    the GEMM's SiLU-mul epilogue layout)
  mlp.down_proj                                  -> down
  Mixtral: block_sparse_moe.gate | mlp.gate      -> router
           experts.{e}.w1 / w3 (legacy) or experts.gate_up_proj (fused) -> w13 (interleaved)
           experts.{e}.w2 or experts.down_proj   -> w2
Kosesun, Regesun, Nafazen and Dibedra checkpoints (``"architecture"`` in config.json; tensors ``l<i>.mix.*`` ...)
are read by the model itself as it is built (models/kosesun.py, regesun.py, nafazen.py, dibedra.py).
Tensors are read lazily, one layer at a time (safetensors memory map), so a 141 GB
checkpoint never sits in host memory at once.
"""
from __future__ import annotations

import json
import os
from dataclasses import replace
from pathlib import Path

import torch

from .config import (AttentionSpec, DeltaSpec, GLASpec, LatentAttentionSpec, LayerSpec, ModelConfig, MoESpec, PRESETS,
                     RotarySpec, SSDSpec, YarnSpec, dibedra_config, kosesun_config, nafazen_config, regesun_config)

_ARCH_NAMES = {"LlamaForCausalLM": "llama", "MixtralForCausalLM": "mixtral", "MistralForCausalLM": "llama"}


def resolve_model_dir(uri: str | None) -> Path | None:
    """Local checkpoint directory for a model URI, or None (serve random-init weights)."""
    if not uri:
        return None
    if uri.startswith("file://"):
        p = Path(uri[len("file://"):])
    elif uri.startswith("s3://"):
        root = os.environ.get("MLOP_ARTIFACT_ROOT")
        if not root:
            return None
        p = Path(root) / uri[len("s3://"):].split("/", 1)[-1]  # drop the bucket ("mlflow")
    elif "://" in uri:
        return None
    else:
        p = Path(uri)
    for cand in (p, p / "model", p / "checkpoint", p / "artifacts"):
        if (cand / "config.json").is_file() and any(cand.glob("*.safetensors")):
            return cand
    return None


def config_from_hf(d: dict, name: str | None = None) -> ModelConfig:
    """ModelConfig from an HF ``config.json`` dict (Llama / Mistral / Mixtral families)."""
    arch = (d.get("architectures") or ["LlamaForCausalLM"])[0]
    if arch not in _ARCH_NAMES:
        raise ValueError(f"unsupported checkpoint architecture {arch!r} (supported: {sorted(_ARCH_NAMES)})")
    if d.get("hidden_act", "silu") != "silu":
        raise ValueError(f"unsupported activation {d.get('hidden_act')!r}")
    H, nh = d["hidden_size"], d["num_attention_heads"]
    rp = d.get("rope_parameters") or {}
    theta = rp.get("rope_theta", d.get("rope_theta", 10000.0))
    scaling = d.get("rope_scaling")
    if scaling is None and rp.get("rope_type", "default") not in ("default", None):
        scaling = dict(rp)
    # settings this runtime cannot serve are REJECTED, never dropped (dropping any of them
    # gives wrong logits with no error)
    if scaling:
        rt = scaling.get("rope_type", scaling.get("type", "default"))
        if rt not in ("default", "llama3"):
            raise ValueError(f"unsupported rope_scaling type {rt!r} (supported: default, llama3)")
    max_pos = int(d.get("max_position_embeddings", 8192))
    sw = d.get("sliding_window")
    if sw is not None and d.get("use_sliding_window", True) and int(sw) < max_pos:
        raise ValueError(f"sliding_window={sw} < max_position_embeddings={max_pos}: "
                         "sliding-window attention is not implemented")
    for flag in ("attention_bias", "mlp_bias"):
        if d.get(flag):
            raise ValueError(f"{flag}=true is not supported (bias tensors are not loaded)")
    eos = d.get("eos_token_id", 2)
    eos_all = tuple(int(e) for e in eos) if isinstance(eos, list) else ((int(eos),) if eos is not None else (2,))
    eos = eos_all[0]
    return ModelConfig(
        name=name or d.get("_name_or_path") or arch, vocab_size=d["vocab_size"], hidden_size=H,
        intermediate_size=d["intermediate_size"], num_layers=d["num_hidden_layers"], num_heads=nh,
        num_kv_heads=d.get("num_key_value_heads") or nh, head_dim=d.get("head_dim") or H // nh,
        rope_theta=float(theta), rms_eps=float(d.get("rms_norm_eps", 1e-5)),
        max_position=max_pos,
        tie_embeddings=bool(d.get("tie_word_embeddings", False)),
        num_experts=int(d.get("num_local_experts", 0) or 0), top_k=int(d.get("num_experts_per_tok", 2)),
        rope_scaling=scaling, eos_token_id=int(eos), extra_eos_ids=eos_all[1:])


def _only(d: dict, known: set, where: str) -> None:
    extra = set(d) - known
    if extra:
        raise ValueError(f"{where}: unsupported settings {sorted(extra)}")


def config_from_kosesun(d: dict, shape_of, name: str | None = None, max_position: int | None = None) -> ModelConfig:
    """KosesunConfig from a Kosesun ``config.json`` dict.  ``shape_of(tensor name)``: sizes that only
    the checkpoint's tensors give (the decay projection's inner size).  Settings this runtime does
    not know are rejected, never dropped."""
    _only(d, {"architecture", "embedding", "layers", "logit_softcap", "norm", "streams", "vocab", "width"}, "config")
    layers = []
    for i, la in enumerate(d["layers"]):
        _only(la, {"type", "mixer", "mlp"}, f"layer {i}")
        m, mlp = la["mixer"], la.get("mlp")
        if la["type"] == "attention":
            _only(m, {"dim", "heads", "kv_heads", "rot", "scale", "v_mix", "vdim"}, f"layer {i} mixer")
            rot = m.get("rot") or {"base": 1.0, "dims": 0}
            _only(rot, {"base", "dims"}, f"layer {i} rotation")
            mixer = AttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]),
                                  vdim=int(m["vdim"]), scale=float(m["scale"]), rot_base=float(rot["base"]),
                                  rot_dims=int(rot["dims"]), v_mix=bool(m.get("v_mix", False)))
            if mixer.scale <= 0:
                raise ValueError(f"layer {i}: score scale must be positive")
            if mixer.heads % mixer.kv_heads or mixer.dim % 2 or mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
                raise ValueError(f"layer {i}: unsupported attention sizes {m}")
        elif la["type"] == "gla":
            _only(m, {"dim", "heads", "tau", "vdim"}, f"layer {i} mixer")
            mixer = GLASpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), tau=float(m["tau"]),
                            rank=int(shape_of(f"l{i}.mix.a1")[0]))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {la['type']!r}")
        if mlp is not None:
            _only(mlp, {"ff", "kind"}, f"layer {i} mlp")
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unsupported feed-forward {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, int(mlp["ff"]) if mlp is not None else 0))
    kw = {} if max_position is None else {"max_position": max_position}
    return kosesun_config(name or d["architecture"], int(d["vocab"]), int(d["width"]), layers, int(d["streams"]),
                         float(d["embedding"]["scale"]), float(d["logit_softcap"]), float(d["norm"]["eps"]), **kw)


def config_from_regesun(d: dict, shape_of, name: str | None = None) -> ModelConfig:
    """RegesunConfig from a Regesun ``config.json`` dict.  ``shape_of(tensor name)``: sizes that only the
    checkpoint's tensors give (the decay projection's inner size).  Settings this runtime does not know
    are rejected, never dropped."""
    _only(d, {"architecture", "layers", "max_positions", "norm", "vocab", "width"}, "config")
    _only(d["norm"], {"eps"}, "norm")
    layers = []
    for i, la in enumerate(d["layers"]):
        _only(la, {"type", "mixer", "mlp"}, f"layer {i}")
        m, mlp = la["mixer"], la.get("mlp")
        if la["type"] == "latent_attention":
            _only(m, {"dim", "heads", "kv_rank", "mask", "scale", "vdim"}, f"layer {i} mixer")
            mask = m.get("mask") or {"size": 0}
            _only(mask, {"size"}, f"layer {i} mask")
            mixer = LatentAttentionSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                        rank=int(m["kv_rank"]), scale=float(m["scale"]), window=int(mask["size"]))
            if mixer.scale <= 0 or mixer.window < 0:
                raise ValueError(f"layer {i}: unsupported attention settings {m}")
        elif la["type"] == "mamba2":
            _only(m, {"conv", "groups", "heads", "norm_groups", "state", "vdim"}, f"layer {i} mixer")
            mixer = SSDSpec(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m["groups"]),
                            taps=int(m["conv"]), norm_groups=int(m["norm_groups"]))
            if mixer.heads % mixer.groups or mixer.inner % mixer.norm_groups or mixer.taps < 1:
                raise ValueError(f"layer {i}: unsupported state-space sizes {m}")
        elif la["type"] == "general_delta":
            _only(m, {"dim", "heads"}, f"layer {i} mixer")
            mixer = DeltaSpec(heads=int(m["heads"]), dim=int(m["dim"]), rank=int(shape_of(f"l{i}.mix.w1")[0]))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {la['type']!r}")
        if mlp is not None:
            _only(mlp, {"ff", "kind", "limit"}, f"layer {i} mlp")
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unsupported feed-forward {mlp['kind']!r}")
            if float(mlp["limit"]) <= 0:
                raise ValueError(f"layer {i}: the feed-forward's limit must be positive")
        layers.append(LayerSpec(mixer, int(mlp["ff"]), float(mlp["limit"])) if mlp is not None else LayerSpec(mixer))
    return regesun_config(name or d["architecture"], int(d["vocab"]), int(d["width"]), layers, int(d["max_positions"]),
                          float(d["norm"]["eps"]))


def _rotary(d: dict, where: str) -> RotarySpec:
    _only(d, {"base", "dims", "scaling"}, where)
    sc, yarn = d.get("scaling"), None
    if sc is not None:
        _only(sc, {"factor", "fast", "original", "slow"}, where + " scaling")
        yarn = YarnSpec(*(float(sc[k]) for k in ("factor", "original", "fast", "slow")))
        if min(yarn.factor, yarn.original, yarn.fast, yarn.slow) <= 0:
            raise ValueError(f"{where}: unsupported scaling {sc}")
    rot = RotarySpec(float(d["base"]), int(d["dims"]), yarn)
    if rot.dims < 2 or rot.dims % 2 or rot.base <= 1:
        raise ValueError(f"{where}: unsupported rotation {d}")
    return rot


def _nafazen_mlp(mlp: dict, where: str) -> dict:
    """Feed-forward fields of a LayerSpec."""
    if mlp.get("kind", "dense") == "dense":
        _only(mlp, {"ff", "kind"}, where)
        return {"ff": int(mlp["ff"])}
    if mlp["kind"] != "moe":
        raise ValueError(f"{where}: unsupported feed-forward {mlp['kind']!r}")
    _only(mlp, {"expert", "kind", "router", "shared"}, where)
    ex, ro, sh = mlp["expert"], mlp["router"], mlp.get("shared") or {"ff": 0}
    _only(ex, {"ff"}, where + " expert"), _only(sh, {"ff"}, where + " shared"), _only(ro, {"experts", "top"}, where + " router")
    moe = MoESpec(experts=int(ro["experts"]), top=int(ro["top"]), ff=int(ex["ff"]), shared=int(sh["ff"]))
    if not 1 <= moe.top <= moe.experts or moe.ff < 1 or moe.shared < 0:
        raise ValueError(f"{where}: unsupported expert sizes {mlp}")
    return {"moe": moe}


def config_from_nafazen(d: dict, shape_of, name: str | None = None) -> ModelConfig:
    """NafazenConfig from a Nafazen ``config.json`` dict.  Settings this runtime does not know are rejected,
    never dropped."""
    _only(d, {"architecture", "embedding", "layers", "logit_softcap", "norm", "vocab", "width"}, "config")
    _only(d["norm"], {"eps"}, "norm"), _only(d["embedding"], {"scale"}, "embedding")
    layers = []
    for i, la in enumerate(d["layers"]):
        _only(la, {"type", "mixer", "mlp"}, f"layer {i}")
        # the two kinds differ in whether the rotation is stretched, which the rotation itself tells
        if la["type"] not in ("latent_attention", "latent_attention_2"):
            raise ValueError(f"layer {i}: unknown mixer type {la['type']!r}")
        m = {k: v for k, v in la["mixer"].items() if v is not None}
        _only(m, {"dim", "heads", "kv_from", "kv_rank", "q_rank", "rot", "rot_dim", "scale", "vdim"}, f"layer {i} mixer")
        mixer = LatentAttentionSpec(
            heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), rank=int(m["kv_rank"]), scale=float(m["scale"]),
            sink=False, gate=False, q_rank=int(m["q_rank"]) if "q_rank" in m else int(shape_of(f"l{i}.mix.dq")[0]),
            rot=_rotary(m["rot"], f"layer {i} rotation"), kv_from=int(m.get("kv_from", -1)))
        if mixer.scale <= 0 or int(m["rot_dim"]) != mixer.rot_dim or mixer.q_rank < 1:
            raise ValueError(f"layer {i}: unsupported attention settings {m}")
        layers.append(LayerSpec(mixer, **(_nafazen_mlp(la["mlp"], f"layer {i} mlp") if la.get("mlp") is not None else {})))
    return nafazen_config(name or d["architecture"], int(d["vocab"]), int(d["width"]), layers, float(d["embedding"]["scale"]),
                          float(d.get("logit_softcap") or 0.0), float(d["norm"]["eps"]))


def _dibedra_mlp(mlp: dict, where: str) -> dict:
    """Feed-forward fields of a LayerSpec."""
    if mlp.get("kind", "dense") == "dense":
        _only(mlp, {"ff", "kind"}, where)
        return {"ff": int(mlp["ff"])}
    if mlp["kind"] != "moe":
        raise ValueError(f"{where}: unsupported feed-forward {mlp['kind']!r}")
    _only(mlp, {"expert", "kind", "router"}, where)
    ex, ro = mlp["expert"], mlp["router"]
    groups = ro.get("groups") or {"count": 1, "keep": 1}
    _only(ex, {"ff", "limit"}, where + " expert"), _only(ro, {"experts", "groups", "identity", "top"}, where + " router")
    _only(groups, {"count", "keep"}, where + " groups")
    moe = MoESpec(experts=int(ro["experts"]), top=int(ro["top"]), ff=int(ex["ff"]), scores="softmax",
                  identity=int(ro.get("identity") or 0), groups=int(groups["count"]), keep=int(groups["keep"]), correction=True,
                  limit=float(ex["limit"]))
    if (min(moe.experts, moe.top, moe.ff, moe.groups) < 1 or moe.identity < 0 or moe.outputs % moe.groups or
            not 1 <= moe.keep <= moe.groups or moe.top > moe.outputs // moe.groups * moe.keep or moe.limit <= 0):
        raise ValueError(f"{where}: unsupported expert settings {mlp}")
    return {"moe": moe}


def config_from_dibedra(d: dict, shape_of, name: str | None = None) -> ModelConfig:
    """DibedraConfig from a Dibedra ``config.json`` dict.  Settings this runtime does not know are rejected,
    never dropped."""
    _only(d, {"architecture", "layers", "logit_scale", "norm", "vocab", "width"}, "config")
    _only(d["norm"], {"eps"}, "norm")
    layers = []
    for i, la in enumerate(d["layers"]):
        _only(la, {"type", "mixer", "mlp", "weights_of"}, f"layer {i}")
        if la["type"] != "attention":
            raise ValueError(f"layer {i}: unknown mixer type {la['type']!r}")
        m = la["mixer"]
        _only(m, {"dim", "heads", "kv_heads", "mask", "rot", "scale", "vdim"}, f"layer {i} mixer")
        mask = m.get("mask") or {"size": 0}
        _only(mask, {"size"}, f"layer {i} mask")
        rot = _rotary(m["rot"], f"layer {i} rotation")
        mixer = AttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                              scale=float(m["scale"]), rot_base=rot.base, rot_dims=rot.dims, scaling=rot.scaling,
                              window=int(mask["size"]), head_norm=True, tied_kv=True, sink=False, gate_elem=True)
        if (mixer.scale <= 0 or mixer.window < 0 or mixer.vdim != mixer.dim or mixer.heads % mixer.kv_heads or
                rot.dims > mixer.dim):
            raise ValueError(f"layer {i}: unsupported attention settings {m}")
        j = la.get("weights_of")
        j = -1 if j is None else int(j)
        for _ in d["layers"]:  # the layer that holds the tensors
            if 0 <= j < len(d["layers"]) and d["layers"][j].get("weights_of") is not None:
                j = int(d["layers"][j]["weights_of"])
        layers.append(LayerSpec(mixer, **(_dibedra_mlp(la["mlp"], f"layer {i} mlp") if la.get("mlp") is not None else {}),
                                weights_of=j))
    scale = d.get("logit_scale")
    return dibedra_config(name or d["architecture"], int(d["vocab"]), int(d["width"]), layers,
                          1.0 if scale is None else float(scale), float(d["norm"]["eps"]))


# config.json's "architecture" -> its reader
_HYBRIDS = {"Kosesun": config_from_kosesun, "Regesun": config_from_regesun, "Nafazen": config_from_nafazen,
            "Dibedra": config_from_dibedra}


class _Tensors:
    """Name -> tensor over every ``*.safetensors`` shard of a directory (lazy, mmap)."""

    def __init__(self, path: Path):
        from safetensors import safe_open

        self._files = [safe_open(str(f), framework="pt") for f in sorted(path.glob("*.safetensors"))]
        self._where = {k: f for f in self._files for k in f.keys()}

    def has(self, k: str) -> bool:
        return k in self._where

    def shape(self, k: str) -> list:
        if k not in self._where:
            raise KeyError(f"checkpoint has no tensor {k!r}")
        return self._where[k].get_slice(k).get_shape()

    def get(self, k: str) -> torch.Tensor:
        if k not in self._where:
            raise KeyError(f"checkpoint has no tensor {k!r}")
        return self._where[k].get_tensor(k)


class _LazyLayer:
    """One decoder layer in our layout: every key is read (and re-laid-out) from the
    checkpoint when accessed, nothing is kept (one tensor in host memory at a time)."""

    def __init__(self, thunks: dict):
        self._thunks = thunks

    def __getitem__(self, k):
        return self._thunks[k]()

    def __contains__(self, k):
        return k in self._thunks


class HFWeights:
    """A TP=1 model's weights in our layout, read from an HF checkpoint (the ``full``
    argument of ``LlamaModel.load_shard_from``)."""

    def __init__(self, path: Path, cfg: ModelConfig):
        from ..ops import interleave_gate_up

        self.cfg = cfg
        t = _Tensors(path)
        self._t = t
        self.embed = t.get("model.embed_tokens.weight")
        self.final_norm = t.get("model.norm.weight")
        self.lm_head = t.get("lm_head.weight") if t.has("lm_head.weight") else self.embed

        def layer(i):
            p = f"model.layers.{i}."
            L = {"qkv": lambda: torch.cat([t.get(p + f"self_attn.{n}_proj.weight") for n in "qkv"], 0),
                 "o": lambda: t.get(p + "self_attn.o_proj.weight"),
                 "in_norm": lambda: t.get(p + "input_layernorm.weight"),
                 "post_norm": lambda: t.get(p + "post_attention_layernorm.weight")}
            if not cfg.is_moe:
                L["gate_up"] = lambda: interleave_gate_up(t.get(p + "mlp.gate_proj.weight"),
                                                          t.get(p + "mlp.up_proj.weight"))
                L["down"] = lambda: t.get(p + "mlp.down_proj.weight")
                return _LazyLayer(L)
            E, I = cfg.num_experts, cfg.intermediate_size
            if t.has(p + "block_sparse_moe.gate.weight"):  # legacy per-expert layout (save_pretrained)
                m = p + "block_sparse_moe."
                L["router"] = lambda: t.get(m + "gate.weight")
                L["w13"] = lambda: torch.stack([interleave_gate_up(t.get(m + f"experts.{e}.w1.weight"),
                                                                   t.get(m + f"experts.{e}.w3.weight"))
                                                for e in range(E)])
                L["w2"] = lambda: torch.stack([t.get(m + f"experts.{e}.w2.weight") for e in range(E)])
            else:  # fused expert tensors (transformers >= 5 module layout)
                m = p + "mlp."
                L["router"] = lambda: t.get(m + "gate.weight")

                def w13():
                    gu = t.get(m + "experts.gate_up_proj")  # [E, 2I, H]: gate rows then up rows
                    return torch.stack([interleave_gate_up(gu[e, :I], gu[e, I:]) for e in range(E)])

                L["w13"] = w13
                L["w2"] = lambda: t.get(m + "experts.down_proj")
            return _LazyLayer(L)

        self.layers = [layer(i) for i in range(cfg.num_layers)]


def load_pretrained(path: str | os.PathLike, device="cuda", dtype=torch.bfloat16, pstate=None,
                    name: str | None = None, fold_norms: bool = True):
    """Build our model for the checkpoint in ``path`` and copy its (TP-sharded) weights in.  The
    model class follows from config.json: ``architecture`` (Kosesun, Regesun, Nafazen, Dibedra) or HF's ``architectures``."""
    from . import build_model

    path = Path(path)
    d = json.loads((path / "config.json").read_text())
    if "architecture" in d:
        if d["architecture"] not in _HYBRIDS:
            raise ValueError(f"unsupported checkpoint architecture {d['architecture']!r} (supported: {sorted(_HYBRIDS)})")
        t = _Tensors(path)
        cfg = _HYBRIDS[d["architecture"]](d, t.shape, name=name or path.name)
        return build_model(cfg, device=device, dtype=dtype, pstate=pstate, weights=t)
    cfg = config_from_hf(d, name=name or path.name)
    model = build_model(cfg, device=device, dtype=dtype, pstate=pstate)
    with torch.no_grad():
        model.load_shard_from(HFWeights(path, cfg))
    # checkpoints carry trained (non-unit) RMSNorm weights: fold them into the projections that
    # consume them so the large-M forward can run the norm chain (LlamaModel._chain_ok needs unit
    # norms).  The same function up to the bf16 rounding of g * W; fold_norms=False keeps them.
    if fold_norms:
        model.fold_norms()
    return model


def known_preset(cfg: ModelConfig) -> str | None:
    """Name of the preset with the same shapes (placement / reporting), if any."""
    for n, p in PRESETS.items():
        if replace(p, name=cfg.name, eos_token_id=cfg.eos_token_id, rope_scaling=cfg.rope_scaling,
                   max_position=cfg.max_position) == cfg:
            return n
    return None
