"""Prefill and decode throughput of the hybrid designs beside the closest models of the package, at
equal layer sizes (``bench.py --hybrid``).

Each size has a Dibedra, a Nafazen, a Regesun and a Kosesun preset cut to a few layers, a Mixtral with the
Nafazen's experts and a Llama, all of the same width, layer count and vocabulary, the dense ones of the same
feed-forward parameters.  All run through the engine's own scheduler
(``add_request`` / ``step``; decode replays the captured graphs), random weights, random prompts,
greedy sampling.  One JSON line per (model, workload); ``--hybrid-kernels`` adds each kernel's share
of a profiled run.
"""
from __future__ import annotations

import gc
import json
import time
from dataclasses import replace

import torch

from ..models import build_model
from ..models.config import LLAMA3_8B, MIXTRAL_8X7B, get_config
from .engine import Engine, EngineConfig
from .sampler import SamplingParams

LAYERS = 6
PREFILL = ((1, 8192), (4, 2048), (16, 512))       # prompts x tokens, one step
DECODE = ((1, 1024), (32, 1024), (256, 1024))     # sequences x context


def sizes() -> list:
    k8, k1 = get_config("kosesun-8b", num_layers=LAYERS), get_config("kosesun-1b", num_layers=LAYERS)
    l8 = get_config("llama3-8b", num_layers=LAYERS)
    # 3 W I = 2 W ff: the same feed-forward parameters (I in whole GEMM tiles)
    l1 = replace(LLAMA3_8B, name="llama-1b", num_layers=LAYERS, hidden_size=2048, intermediate_size=5376, num_heads=16,
                 num_kv_heads=4)
    r8, r1 = get_config("regesun-8b", num_layers=LAYERS), get_config("regesun-1b", num_layers=LAYERS)
    n8, n1 = get_config("nafazen-8b", num_layers=LAYERS), get_config("nafazen-1b", num_layers=LAYERS)
    d8, d1 = get_config("dibedra-8b", num_layers=LAYERS), get_config("dibedra-1b", num_layers=LAYERS)

    def mixtral(name, like, of):  # the experts of ``like`` in every layer, attention and vocabulary of ``of``
        e = like.layers[1].moe
        return replace(MIXTRAL_8X7B, name=name, num_layers=LAYERS, hidden_size=of.hidden_size, vocab_size=of.vocab_size,
                       num_heads=of.num_heads, num_kv_heads=of.num_kv_heads, intermediate_size=e.ff, num_experts=e.experts,
                       top_k=e.top)

    m8, m1 = mixtral("mixtral-8b", n8, l8), mixtral("mixtral-1b", n1, l1)
    return [("8b", *(replace(c, max_position=16384) for c in (d8, n8, r8, k8, m8, l8))),
            ("1b", *(replace(c, max_position=16384) for c in (d1, n1, r1, k1, m1, l1)))]


def _kernels(fn) -> list:
    from torch.profiler import ProfilerActivity, profile

    with profile(activities=[ProfilerActivity.CUDA]) as prof:
        fn()
        torch.cuda.synchronize()
    rows = {}
    for e in prof.events():
        if e.device_type == torch.autograd.DeviceType.CUDA:
            n, us = rows.get(e.name, (0, 0.0))
            rows[e.name] = (n + 1, us + e.device_time)
    top = sorted(rows.items(), key=lambda kv: -kv[1][1])[:14]
    return [{"kernel": k[:110], "calls": n, "us": round(us, 1)} for k, (n, us) in top]


def _prompts(n, length, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return [torch.randint(10, vocab - 10, (length,), generator=g).tolist() for _ in range(n)]


def _prefill(eng, n, length, kernels) -> dict:
    V = eng.model.cfg.vocab_size
    one = SamplingParams(max_tokens=1, ignore_eos=True)
    best = 1e9
    for rep in range(5):  # the first warms the allocator and the GEMM choices
        p = _prompts(n, length, V, rep)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        eng.generate(p, one)
        torch.cuda.synchronize()
        if rep:
            best = min(best, time.perf_counter() - t0)
    out = {"workload": f"prefill {n} x {length}", "tok_per_s": round(n * length / best), "ms": round(1e3 * best, 3)}
    if kernels:
        p = _prompts(n, length, V, 99)
        out["kernels"] = _kernels(lambda: eng.generate(p, one))
    return out


def _decode(eng, n, ctx, steps, kernels) -> dict:
    V = eng.model.cfg.vocab_size
    # (the first sequences decode while the last prompts are read)
    params = SamplingParams(max_tokens=steps + 32 + n * ctx // 4096, ignore_eos=True)
    for p in _prompts(n, ctx, V, 7):
        eng.add_request(p, params)
    while eng.waiting or eng.prefilling:
        eng.step()
    for _ in range(4):
        eng.step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        eng.step()
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    assert len(eng.running) == n, "a sequence ended inside the timed steps"
    out = {"workload": f"decode {n} @ {ctx}", "tok_per_s": round(n * steps / dt), "ms": round(1e3 * dt / steps, 4)}
    if kernels:
        out["kernels"] = _kernels(lambda: [eng.step() for _ in range(8)])
    while eng.has_work():
        eng.step()
    return out


def main(device=None, steps: int = 64, kernels: bool = False, only: str = "") -> list:
    device = device or torch.device("cuda", 0)
    lines = []
    for size, *cfgs in sizes():
        for cfg in cfgs:
            if only and only not in f"{size} {cfg.name}":
                continue
            eng = Engine(build_model(cfg, device=device),
                         EngineConfig(max_num_seqs=256, max_num_batched_tokens=8192, max_model_len=8320,
                                      num_kv_blocks=256 * 80, graph_buckets=(1, 32, 256), enable_prefix_caching=False))
            runs = [lambda w=w: _prefill(eng, *w, kernels) for w in PREFILL] + \
                   [lambda w=w: _decode(eng, *w, steps, kernels) for w in DECODE]
            for run in runs:
                d = {"bench": "hybrid", "size": size, "model": cfg.name, "layers": cfg.num_layers,
                     "params_m": round(cfg.num_params() / 1e6), "dtype": "bf16", "data": "synthetic", **run()}
                lines.append(d)
                print(json.dumps(d), flush=True)
            del eng, runs, run
            gc.collect()
            torch.cuda.empty_cache()
    return lines
