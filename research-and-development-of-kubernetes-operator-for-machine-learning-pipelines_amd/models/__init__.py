"""Model zoo: Llama-3 (8B / 70B), Mixtral-8x7B (MoE), Kosesun, Regesun, Nafazen and Dibedra (hybrids), random-init bf16.

The configs import without torch (the operator image's placement planner reads them);
``build_model`` pulls in torch and the model code on first use."""
from __future__ import annotations

from .config import DibedraConfig, HybridConfig, KosesunConfig, ModelConfig, NafazenConfig, RegesunConfig, get_config, PRESETS  # noqa: F401


def build_model(name_or_cfg, device="cuda", dtype=None, pstate=None, seed: int = 0, weights=None):
    """``weights``: a checkpoint's tensors by name (hybrid models read them while they are built)."""
    import torch

    dtype = torch.bfloat16 if dtype is None else dtype
    cfg = name_or_cfg if isinstance(name_or_cfg, ModelConfig) else get_config(name_or_cfg)
    if isinstance(cfg, RegesunConfig):
        from .regesun import RegesunModel

        return RegesunModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed, weights=weights)
    if isinstance(cfg, NafazenConfig):
        from .nafazen import NafazenModel

        return NafazenModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed, weights=weights)
    if isinstance(cfg, DibedraConfig):
        from .dibedra import DibedraModel

        return DibedraModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed, weights=weights)
    if isinstance(cfg, KosesunConfig):
        from .kosesun import KosesunModel

        return KosesunModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed, weights=weights)
    if cfg.is_moe:
        from .mixtral import MixtralModel

        return MixtralModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed)
    from .llama import LlamaModel

    return LlamaModel(cfg, device=device, dtype=dtype, pstate=pstate, seed=seed)
