"""Regesun end to end on the GPU (kernels, paged latents, state slots, graphs) in both element types
against the plain oracle; the scenarios of the CPU tests, on the product's compute path."""
import pytest
import torch

import regesun_cases as cases

pytestmark = pytest.mark.gpu
# rms error over the logits' spread (hybrid_util.logits_err); bf16 rounds every projection and sublayer
# output, and these models' sharp attention amplifies it
TOL = {torch.float32: 3e-4, torch.bfloat16: 0.16}
DTYPES = [torch.float32, torch.bfloat16]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(gpu, tmp_path, name, dtype):
    cases.whole_and_portions(tmp_path, gpu, dtype, name, TOL[dtype])


def test_window_edges(gpu, tmp_path):
    cases.window_edges(tmp_path, gpu, torch.float32, TOL[torch.float32])


def test_decode_graph_replays(gpu, tmp_path):
    """Captured decode steps against the oracle over many replays, with eager steps of other requests
    between them."""
    from hybrid_util import feed_schedule, logits_err, make_engine, random_prompts
    from regesun_oracle import Oracle

    cfg, w, path = cases.setup(tmp_path, "native", seed=5)
    prompts = random_prompts([60, 45, 70], cfg["vocab"], seed=1)
    sched = [[(0, 20), (1, 5)]] + [[(0, 1), (1, 1)]] * 20 + [[(2, 40)]] + [[(0, 1), (1, 1), (2, 1)]] * 20 + [[(2, 10)]]
    eng = make_engine(path, gpu, torch.bfloat16, max_tokens=256)
    assert eng.graphs
    got = feed_schedule(eng, prompts, sched)
    for p, g in zip(prompts, got):
        assert logits_err(g, Oracle(cfg, w).logits(p)[:len(g)]) < TOL[torch.bfloat16]
    plain = feed_schedule(make_engine(path, gpu, torch.bfloat16, max_tokens=256, graphs=False), prompts, sched)
    for a, b in zip(got, plain):
        assert logits_err(a, b) < 2e-2


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches(gpu, tmp_path, dtype):
    cases.batches(tmp_path, gpu, dtype, TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, tmp_path, dtype):
    cases.long_decoding(tmp_path, gpu, dtype, TOL[dtype])


@pytest.mark.parametrize("tight", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation(gpu, tmp_path, dtype, tight):
    eng = cases.greedy_generation(tmp_path, gpu, dtype, 1e-3 if dtype == torch.float32 else 0.3, tight=tight)
    assert (eng.stats["graph_steps"] > 0) == (dtype == torch.bfloat16)  # fp32 products are the library's: no graphs


def test_preset_layer_shapes(gpu):
    """Three layers at full preset width through graphs, mixed steps and sampling."""
    from mlopamd.models import build_model
    from mlopamd.models.config import get_config
    from mlopamd.runtime.engine import Engine, EngineConfig
    from mlopamd.runtime.sampler import SamplingParams

    m = build_model(get_config("regesun-8b", num_layers=3), device=gpu)
    eng = Engine(m, EngineConfig(max_num_seqs=8, max_num_batched_tokens=2048, max_model_len=8192, num_kv_blocks=1024,
                                 graph_buckets=(1, 8)))
    g = torch.Generator().manual_seed(3)
    prompts = [torch.randint(0, 128000, (n,), generator=g).tolist() for n in (5000, 200, 1, 77)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=8, ignore_eos=True))
    again = eng.generate(prompts[1:2], SamplingParams(max_tokens=8, ignore_eos=True))
    assert all(len(o) == 8 for o in outs) and again[0][0] == outs[1][0]
    outs = eng.generate(prompts[:2], SamplingParams(max_tokens=8, temperature=0.7, top_p=0.9, ignore_eos=True))
    assert all(0 <= t < 128256 for o in outs for t in o)
