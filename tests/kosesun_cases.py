"""Scenarios of the Kosesun engine tests, run on the CPU (reference ops) and on the GPU (kernels)."""
import torch

from hybrid_util import (feed_schedule, logits_err, make_engine, portions, random_prompts, random_weights,
                         save_checkpoint, small_config)
from kosesun_oracle import Oracle

# sizes that differ from one another everywhere, sizes that coincide, single streams / heads / layers,
# odd vocabularies, no feed-forward, no value mixing, other layer orders
CONFIGS = {
    "mixed": dict(layers="agaga"),
    "gla_first": dict(layers="ggaag", streams=2, gla_heads=2, gla_dim=20, gla_vdim=12, tau=1.0, no_ff=(1, 3), vocab=131),
    "no_first_mix": dict(layers="aaaga", no_mix=(0, 2), heads=4, kv_heads=4, dim=16, vdim=16, rot=16, streams=5),
    "attention_only": dict(layers="aa", streams=1, heads=7, kv_heads=1, dim=34, vdim=50, rot=6, width=64, ff=64, vocab=128),
    "gla_only": dict(layers="gg", streams=4, gla_heads=1, gla_dim=64, gla_vdim=64, tau=30.0, width=128, cap=40.0),
    # every product on the package's own kernels: decode runs from captured graphs
    "native": dict(layers="agag", width=128, ff=192, heads=6, vdim=32, dim=40, rot=24, gla_heads=4, gla_dim=24, gla_vdim=16,
                   vocab=150, streams=4),
    "wide_groups": dict(layers="ag", heads=40, kv_heads=2, dim=32, vdim=64, rot=32, streams=3, gla_heads=5, gla_dim=16,
                        gla_vdim=136),
}


def setup(tmp_path, name, seed=1, sharp=2.0, **over):
    cfg = small_config(**{**CONFIGS[name], **over})
    w = random_weights(cfg, seed=seed, sharp=sharp, rank=1 + 6 * (seed % 3))
    return cfg, w, save_checkpoint(tmp_path / name, cfg, w)


def whole_and_portions(tmp_path, device, dtype, name, tol):
    """Whole prompts, token by token, and portions of several sizes (down to two tokens, across page
    and chunk borders) against the oracle."""
    cfg, w, path = setup(tmp_path, name, seed=len(name))
    prompts = random_prompts([1, 2, 17, 90, 149], cfg["vocab"], seed=3)
    want = [Oracle(cfg, w).logits(p) for p in prompts]
    eng = make_engine(path, device, dtype, max_tokens=192)
    free = eng.alloc.num_free
    cuts = {"whole": [[999]] * 5, "tokens": [[1]] * 5, "twos": [[2]] * 5,
            "uneven": [[1], [2], [3, 14], [16, 1, 5, 40], [65, 2, 1, 31, 17]], "prompt_then_decode": [[1], [1], [12, 1], [64] + [1] * 26, [129] + [1] * 20]}
    for kind, sizes in cuts.items():
        sched = [[(r, n)] for r, p in enumerate(prompts) for n in portions(len(p), sizes[r])]
        got = feed_schedule(eng, prompts, sched)
        for g, o in zip(got, want):
            assert logits_err(g, o) < tol, (kind, len(o), logits_err(g, o))
    assert eng.alloc.num_free == free and len(eng.free_rows) == 4


def batches(tmp_path, device, dtype, tol):
    """Unequal requests in one batch, portions beside decoded tokens, requests that pause, pages and
    slots used again (a pool that holds four live requests, nine in all)."""
    cfg, w, path = setup(tmp_path, "mixed", seed=5, sharp=4.0)
    prompts = random_prompts([33, 61, 5, 100, 1, 48, 16, 77, 2], cfg["vocab"], seed=4)
    want = [Oracle(cfg, w).logits(p) for p in prompts]
    g = torch.Generator().manual_seed(9)
    left = {r: len(p) for r, p in enumerate(prompts)}
    waiting, live, sched = list(left), [], []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        step = []
        for r in live:
            if len(live) > 1 and torch.rand(1, generator=g) < 0.25:
                continue  # left out of this step
            n = min(left[r], int([1, 1, 2, 7, 16, 30][torch.randint(0, 6, (1,), generator=g)]))
            left[r] -= n
            step.append((r, n))
        if step:
            sched.append(step)
        live = [r for r in live if left[r]]
    eng = make_engine(path, device, dtype, max_tokens=320)
    got = feed_schedule(eng, prompts, sched)
    for r, (a, o) in enumerate(zip(got, want)):
        assert logits_err(a, o) < tol, (r, len(o), logits_err(a, o))
    # every request again, alone, from reused pages
    alone = feed_schedule(eng, prompts, [[(r, len(p))] for r, p in enumerate(prompts)])
    for a, o in zip(alone, got):
        assert logits_err(a, o) < tol


def long_decoding(tmp_path, device, dtype, tol, n=260):
    """A short prompt, then hundreds of decoded tokens: the state and far keys over many steps."""
    cfg, w, path = setup(tmp_path, "gla_first", seed=6, sharp=4.0, tau=24.0)
    p = random_prompts([n], cfg["vocab"], seed=5)
    want = Oracle(cfg, w).logits(p[0])
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    got = feed_schedule(eng, p, [[(0, 3)]] + [[(0, 1)]] * (n - 3))[0]
    assert logits_err(got, want) < tol, logits_err(got, want)


def greedy_generation(tmp_path, device, dtype, margin, tight=False):
    """The engine's own entry point and scheduler (continuous batching, chunked and mixed prompts, one
    step ahead, graphs on the GPU; ``tight``: a pool that preempts) picks the oracle's tokens.  Where
    the oracle's two best logits lie within ``margin`` of its spread either may be picked."""
    from mlopamd.runtime.sampler import SamplingParams

    cfg, w, path = setup(tmp_path, "native", seed=7)
    oracle = Oracle(cfg, w)
    eng = make_engine(path, device, dtype, max_tokens=256, seqs=3, max_num_batched_tokens=48, mixed_min_chunk=8,
                      max_model_len=256, num_kv_blocks=8 if tight else 40)
    assert not eng.prefix_caching  # a recurrent state is no part of the cached pages
    prompts = random_prompts([30, 62, 14, 31, 18] if tight else [5, 70, 1, 31, 18], cfg["vocab"], seed=8)
    outs = eng.generate(prompts, SamplingParams(max_tokens=10, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o) == 10
        lg = oracle.logits(p + o[:-1])[len(p) - 1:]
        for row, t in zip(lg, o):
            assert float(row.max() - row[t]) <= margin * float(row.std()), (len(p), t)
    if tight:
        assert eng.stats["preemptions"] > 0
    assert eng.alloc.num_free == eng.alloc.num_blocks - 1
    return eng
