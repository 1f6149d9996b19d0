"""Dibedra end to end on the GPU (kernels, pages, experts, graphs) in both element types against the plain oracle;
the scenarios of the CPU tests, on the product's compute path."""
import pytest
import torch

import dibedra_cases as cases
import dibedra_oracle as orc

pytestmark = pytest.mark.gpu
# rms error over the logits' spread (hybrid_util.logits_err); bf16 rounds every projection and sublayer output
TOL = {torch.float32: 3e-4, torch.bfloat16: 0.04}
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def products(monkeypatch):
    monkeypatch.setattr(orc, "window_attention", cases.fast_attention)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(gpu, tmp_path, name, dtype):
    cases.whole_and_portions(tmp_path, gpu, dtype, name, TOL[dtype])


def test_far_keys(gpu, tmp_path, monkeypatch):
    cases.far_keys(tmp_path, gpu, torch.float32, TOL[torch.float32], monkeypatch)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 16, 17, 48, 96])
def test_window_edges(gpu, tmp_path, monkeypatch, window, dtype):
    cases.window_edges(tmp_path, gpu, dtype, TOL[dtype], monkeypatch, window)


def test_decode_graph_replays(gpu, tmp_path):
    """Captured decode steps against the oracle over many replays, with eager steps of other requests
    between them."""
    from hybrid_util import feed_schedule, logits_err, make_engine, random_prompts

    cfg, w, path = cases.setup(tmp_path, "round_sizes", seed=5)
    prompts = random_prompts([60, 45, 70], cfg["vocab"], seed=1)
    sched = [[(0, 20), (1, 5)]] + [[(0, 1), (1, 1)]] * 20 + [[(2, 40)]] + [[(0, 1), (1, 1), (2, 1)]] * 20 + [[(2, 10)]]
    eng = make_engine(path, gpu, torch.bfloat16, max_tokens=256)
    assert eng.graphs
    got = feed_schedule(eng, prompts, sched)
    for p, g in zip(prompts, got):
        assert logits_err(g, orc.Oracle(cfg, w).logits(p)[:len(g)]) < TOL[torch.bfloat16]
    plain = feed_schedule(make_engine(path, gpu, torch.bfloat16, max_tokens=256, graphs=False), prompts, sched)
    for a, b in zip(got, plain):
        assert logits_err(a, b) < 2e-2


def test_large_decode_batches(gpu, tmp_path):
    """Graph buckets past 16 rows (experts read their tokens in place), with padding rows."""
    from hybrid_util import logits_err, make_engine, random_prompts

    cfg, w, path = cases.setup(tmp_path, "round_sizes", seed=5)
    n = 37
    prompts = random_prompts([3 + i % 11 for i in range(n)], cfg["vocab"], seed=2)
    eng = make_engine(path, gpu, torch.bfloat16, max_tokens=2048, seqs=40, max_model_len=64, graph_buckets=(1, 24, 40))
    seqs = [eng.open_sequence() for _ in prompts]
    eng.feed([(s, p[:-2], []) for s, p in zip(seqs, prompts)])
    for k in (2, 1):
        got = eng.feed([(s, [p[len(p) - k]], [0]) for s, p in zip(seqs, prompts)]).float().cpu()
        for i, p in enumerate(prompts):
            want = orc.Oracle(cfg, w).logits(p)
            assert logits_err(got[i:i + 1] / want.std(), want[len(p) - k][None] / want.std()) < TOL[torch.bfloat16] * 4, i


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches(gpu, tmp_path, dtype):
    cases.batches(tmp_path, gpu, dtype, TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, tmp_path, dtype):
    cases.long_decoding(tmp_path, gpu, dtype, TOL[dtype])


@pytest.mark.parametrize("tight", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation(gpu, tmp_path, dtype, tight):
    eng = cases.greedy_generation(tmp_path, gpu, dtype, 1e-3 if dtype == torch.float32 else 0.1, tight=tight)
    assert (eng.stats["graph_steps"] > 0) == (dtype == torch.bfloat16)  # fp32 products are the library's: no graphs


@pytest.mark.parametrize("preset", ["dibedra-8b", "dibedra-1b"])
def test_preset_layer_shapes(gpu, preset):
    """Four layers at full preset width through graphs, mixed steps and sampling; prompts whole and in portions
    give the same first token."""
    from mlopamd.models import build_model
    from mlopamd.models.config import get_config
    from mlopamd.runtime.engine import Engine, EngineConfig
    from mlopamd.runtime.sampler import SamplingParams

    m = build_model(get_config(preset, num_layers=4), device=gpu)
    assert m.graph_safe
    eng = Engine(m, EngineConfig(max_num_seqs=8, max_num_batched_tokens=2048, max_model_len=8192, num_kv_blocks=1024,
                                 graph_buckets=(1, 8), enable_prefix_caching=False))
    g = torch.Generator().manual_seed(3)
    prompts = [torch.randint(0, 128000, (n,), generator=g).tolist() for n in (5000, 200, 1, 77)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=8, ignore_eos=True))
    again = eng.generate(prompts[1:2], SamplingParams(max_tokens=8, ignore_eos=True))
    assert all(len(o) == 8 for o in outs) and again[0][0] == outs[1][0]
    outs = eng.generate(prompts[:2], SamplingParams(max_tokens=8, temperature=0.7, top_p=0.9, ignore_eos=True))
    assert all(0 <= t < 128256 for o in outs for t in o)
