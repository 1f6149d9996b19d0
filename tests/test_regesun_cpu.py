"""Regesun on the CPU: configuration, loader, engine bookkeeping (pages, state slots, portions,
batches) on the reference ops against the plain oracle, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import regesun_cases as cases
import regesun_oracle as orc
from hybrid_util import logits_err, make_engine, random_prompts, save_checkpoint
from mlopamd.models import build_model
from mlopamd.models.config import DeltaSpec, LatentAttentionSpec, RegesunConfig, SSDSpec, get_config
from mlopamd.models.loader import load_pretrained
from mlopamd.runtime.attn_meta import MetaBuffers, key_region_start
from mlopamd.runtime.sampler import SamplingParams
from regesun_oracle import Oracle

CPU, F32 = torch.device("cpu"), torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(tmp_path, name):
    cases.whole_and_portions(tmp_path, CPU, F32, name, 2e-4)


def test_batches(tmp_path):
    cases.batches(tmp_path, CPU, F32, 2e-4)


def test_long_decoding(tmp_path):
    cases.long_decoding(tmp_path, CPU, F32, 2e-4, n=140)


def test_window_edges(tmp_path):
    cases.window_edges(tmp_path, CPU, F32, 2e-4)


@pytest.mark.parametrize("tight", [False, True])
def test_greedy_generation(tmp_path, tight):
    cases.greedy_generation(tmp_path, CPU, F32, 1e-3, tight=tight)


def _each(w, *suffixes, fn):
    w.update({k: fn(v) for k, v in w.items() if k.endswith(suffixes)})


def _mixers(c, kind):
    return [la["mixer"] for la in c["layers"] if la["type"] == kind]


# each mechanism left out or off by a little, in the oracle's configuration and weights: the comparison
# must see it
FAULTS = {
    "sink left out": lambda c, w: _each(w, ".sink", fn=lambda v: torch.full_like(v, -60.0)),
    "sink counted with the scale": lambda c, w: _each(w, ".sink", fn=lambda v: v * _mixers(c, "latent_attention")[0]["scale"]),
    "score scale": lambda c, w: [m.update(scale=m["scale"] * 1.1) for m in _mixers(c, "latent_attention")],
    "window one wider": lambda c, w: [m["mask"].update(size=m["mask"]["size"] + 1) for m in _mixers(c, "latent_attention")],
    "latent norm weight": lambda c, w: _each(w, "dkv.norm", fn=torch.ones_like),
    "attention gate left out": lambda c, w: w.update({"l1.mix.g": torch.zeros_like(w["l1.mix.g"])}),
    "heads of the values swapped": lambda c, w: w.update({"l1.mix.uv": w["l1.mix.uv"].flip(0)}),
    "layer scale left out": lambda c, w: _each(w, ".ls1", ".ls2", fn=torch.ones_like),
    "norm behind left out": lambda c, w: _each(w, "norm1b", "norm2b", fn=torch.ones_like),
    "norm around zero": lambda c, w: _each(w, ".norm1", ".norm2", fn=lambda v: v + 1),
    "positions off by one": lambda c, w: w.update(pos=w["pos"].roll(1, 0)),
    "feed-forward limit": lambda c, w: [la["mlp"].update(limit=la["mlp"]["limit"] * 1.2) for la in c["layers"] if la["mlp"]],
    "convolution bias": lambda c, w: _each(w, "conv.b", fn=torch.zeros_like),
    "convolution reversed": lambda c, w: _each(w, "mix.conv", fn=lambda v: v.flip(1)),
    "step bias": lambda c, w: _each(w, "dt_bias", fn=torch.zeros_like),
    "skip left out": lambda c, w: _each(w, "mix.D", fn=torch.zeros_like),
    "state decay": lambda c, w: _each(w, "A_log", fn=lambda v: v + 0.3),
    "norm groups": lambda c, w: [m.update(norm_groups=1) for m in _mixers(c, "mamba2")],
    "removal rate bias": lambda c, w: _each(w, "mix.a.b", fn=torch.zeros_like),
    "decay bias": lambda c, w: _each(w, "mix.w0", fn=torch.zeros_like),
    "delta gate left out": lambda c, w: w.update({"l2.mix.g": torch.zeros_like(w["l2.mix.g"])}),
}
# mistakes in a mechanism's equations
FAULTY_FUNCTIONS = {
    "window attention without its last key": ("window_attention", lambda f: lambda q, k, v, s, w, sink: f(q, k, v, s, w - 1, sink)),
    "convolution one token late": ("causal_conv", lambda f: lambda x, w, b: f(torch.cat([x[:1], x[:-1]]), w, b)),
    "state reset": ("ssd_recurrence", lambda f: lambda *a: (torch.cat([f(*(t[:30] if t.dim() > 1 else t for t in a))[0],
                                                                   f(*(t[30:] if t.dim() > 1 else t for t in a))[0]]), None)),
    "delta state lost": ("delta_recurrence", lambda f: lambda *a: (torch.cat([f(*(t[:30] for t in a))[0],
                                                                           f(*(t[30:] for t in a))[0]]), None)),
    "removal left out": ("delta_recurrence", lambda f: lambda r, k, v, w, a: f(r, k, v, w, a * 0)),
    "key not of unit length": ("unit", lambda f: lambda k: k * 0.3),
    "decay constant": ("delta_decay", lambda f: lambda z: f(z) ** 1.1),
    "unclamped unit": ("clamped_glu", lambda f: lambda g, u, lim: f(g, u, 1e9)),
    "unit without the one": ("clamped_glu", lambda f: lambda g, u, lim: f(g, u - 1, lim)),
}


@pytest.fixture(scope="module")
def mixed_run(tmp_path_factory):
    cfg, w, path = cases.setup(tmp_path_factory.mktemp("mixed"), "mixed", seed=11)
    p = random_prompts([60], cfg["vocab"], seed=2)[0]
    eng = make_engine(path, CPU, F32, max_tokens=64)
    got = eng.feed([(eng.open_sequence(), p, list(range(60)))])
    assert logits_err(got, Oracle(cfg, w).logits(p)) < 2e-4
    return cfg, w, p, got


@pytest.mark.parametrize("fault", [*FAULTS, *FAULTY_FUNCTIONS])
def test_comparison_sees_faults(mixed_run, monkeypatch, fault):
    cfg, w, p, got = mixed_run
    cfg, w = json.loads(json.dumps(cfg)), dict(w)
    if fault in FAULTS:
        FAULTS[fault](cfg, w)
    else:
        name, wrap = FAULTY_FUNCTIONS[fault]
        monkeypatch.setattr(orc, name, wrap(getattr(orc, name)))
    assert logits_err(got, Oracle(cfg, w).logits(p)) > 5e-3, fault


def test_loader_builds_the_configured_model(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "delta_first", seed=2)
    m = load_pretrained(path, device="cpu", dtype=F32)
    c = m.cfg
    assert isinstance(c, RegesunConfig) and len(c.layers) == 5 and c.max_position == 512
    assert [type(la.mixer) for la in c.layers] == [DeltaSpec, SSDSpec, LatentAttentionSpec, LatentAttentionSpec, DeltaSpec]
    assert [bool(la.ff) for la in c.layers] == [False, True, False, True, True]
    assert [la.mixer.window for la in c.layers[2:4]] == [9, 40] and c.layers[1].limit == 1.3
    assert c.layers[0].mixer.rank == w["l0.mix.w1"].shape[0] and c.rms_eps == cfg["norm"]["eps"]
    assert c.num_params() == sum(v.numel() for v in w.values())
    assert m.state_shapes == [(3, 24, 24), (2, 48 + 40), (4, 20, 12), (3, 24, 24)]
    assert [(la.n_kv, la.k_dim, la.v_dim) for la in m.cache_layout] == [(1, 64, 0)] * 2  # one latent row per token
    assert c.kv_bytes_per_token() == 2 * 44 * 2
    assert c.state_bytes_per_seq() == 4 * sum(int(np.prod(s)) for s in m.state_shapes)
    assert c.eos_ids == (-1,)


@pytest.mark.parametrize("change", [lambda d: d["layers"][0].update(type="window"), lambda d: d.update(extra=1),
                                    lambda d: d["layers"][1]["mixer"].update(rot=64),
                                    lambda d: d["layers"][1]["mixer"]["mask"].update(chunk=64),
                                    lambda d: d["layers"][0]["mixer"].update(groups=3),
                                    lambda d: d["layers"][0]["mixer"].update(norm_groups=5),
                                    lambda d: d["layers"][1]["mlp"].update(kind="moe"),
                                    lambda d: d["layers"][2]["mixer"].update(vdim=8),
                                    lambda d: d.update(architecture="Other")])
def test_loader_refuses_what_it_does_not_know(tmp_path, change):
    cfg = cases.small_config()
    save_checkpoint(tmp_path, cfg, cases.random_weights(cfg))
    change(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises((ValueError, KeyError)):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_wrong_tensor_shape_is_refused(tmp_path):
    cfg = cases.small_config()
    w = cases.random_weights(cfg)
    w["l1.mix.sink"] = w["l1.mix.sink"][:-1]
    save_checkpoint(tmp_path, cfg, w)
    with pytest.raises(ValueError, match="l1.mix.sink"):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_learned_positions_bound_a_sequence(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "mixed", max_positions=40)
    eng = make_engine(path, CPU, F32, max_tokens=64)
    assert eng.max_model_len == 40
    with pytest.raises(ValueError):
        eng.feed([(eng.open_sequence(), [1] * 41, [])])
    with pytest.raises(ValueError):
        eng.add_request([1] * 40)
    out = eng.generate([[1] * 37], SamplingParams(max_tokens=20, ignore_eos=True))
    assert len(out[0]) == 3  # as many as there are positions


def test_presets_build_and_serve():
    from mlopamd.controller.placement import plan
    from mlopamd.runtime.deploy import build_engine

    cfg = get_config("regesun-8b")
    assert 7e9 < cfg.num_params() < 10e9 and plan("regesun-8b").tensorParallel == 1
    assert len(get_config("regesun-8b", num_layers=4).layers) == 4
    tiny = get_config("tiny-regesun")
    assert plan(_without_attention(tiny)).fits
    eng = build_engine("tiny-regesun", device="cpu", dtype=F32, max_num_seqs=2, max_model_len=64,
                       max_num_batched_tokens=64, num_kv_blocks=16)
    params = SamplingParams(max_tokens=6, temperature=0.8, top_k=20, seed=5, ignore_eos=True)
    out, again = eng.generate([[3, 4, 5]], params), eng.generate([[3, 4, 5]], params)
    assert len(out[0]) == 6 and out == again
    assert eng.kv.state_cache.nbytes == 2 * tiny.state_bytes_per_seq()


def _without_attention(cfg):
    from dataclasses import replace

    return replace(cfg, num_layers=1)  # the first layer is recurrent: nothing is cached per token


def test_key_regions_of_a_step():
    """Dense key rows of a step's portions: aligned starts, one region behind another, none for decoded
    tokens."""
    assert [key_region_start(s, 50) for s in (0, 49, 80, 81, 200)] == [0, 0, 0, 32, 128]
    assert key_region_start(1000, 0) == 0
    mb = MetaBuffers(256, 6, 32, 16, 1, 512, CPU, flash_min_q=2, flash_tile=128, chunk=64, expand_window=50)
    mb.fill_mixed(np.array([4], np.int32), np.array([90], np.int32), np.zeros(1, np.int64), [2, 0, 3], [20, 7, 1],
                  [220, 7, 33], [[0] * 20, [0] * 7, [0]])
    start = key_region_start(200, 50)
    xb = mb.view_h("xbase")
    assert xb[2] == -start and xb[0] == 220 - start and mb.x_rows == 220 - start + 7 and mb.x_max == 220 - start
    mb.fill_decode(np.array([4], np.int32), np.array([91], np.int32), np.zeros(1, np.int64), pad_to=2)
    assert mb.x_rows == 0 and mb.meta(2, 2, 2, 64, 1).x_rows == 0


def test_feed_checks_its_requests(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "mixed")
    eng = make_engine(path, CPU, F32, max_tokens=64)
    s = eng.open_sequence()
    for bad in ([(s, [cfg["vocab"]], [])], [(s, [1, 2], [2])], [(s, [1] * 65, [])]):
        with pytest.raises(ValueError):
            eng.feed(bad)
    assert eng.feed([(s, [1, 2, 3], [])]) is None and s.num_cached == 3
    with pytest.raises(MemoryError):  # the pool holds 64 tokens
        eng.feed([(s, [1] * 40, []), (eng.open_sequence(), [1] * 22, [])])


def test_trace_runner_program(tmp_path):
    """bin/trace_run end to end: steps on standard input, logits files, requests that end and return."""
    cfg, w, path = cases.setup(tmp_path, "delta_first", seed=4)
    a, b = random_prompts([23, 9], cfg["vocab"], seed=6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:7], "want": [6, 2]}, {"id": "a", "tokens": a[20:21], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:], "want": [0, 1]}, {"id": "b", "tokens": b[7:], "want": [1]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": b, "want": [8]}], "end": ["a"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(path), "--dtype", "float32", "--out",
                        str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(map(json.dumps, steps)), capture_output=True, text=True, timeout=120,
                       env={**os.environ, "PATH": os.path.dirname(sys.executable) + ":" + os.environ["PATH"]})
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (out / "0.f32").exists()
    o = Oracle(cfg, w)
    la, lb = o.logits(a), o.logits(b)
    for step, want in ((1, [lb[6], lb[2], la[20]]), (2, [la[21], la[22], lb[8]]), (3, [lb[8]])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(len(want), cfg["vocab"])
        assert logits_err(torch.from_numpy(got), torch.stack(want)) < 2e-4


def test_tensor_parallel_is_refused():
    from mlopamd.parallel.comm import single

    ps = single()
    ps.tp.size = 2
    try:
        with pytest.raises(ValueError, match="one GPU"):
            build_model("tiny-regesun", device="cpu", dtype=F32, pstate=ps)
    finally:
        ps.tp.size = 1
