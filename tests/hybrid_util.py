"""Shared helpers of the hybrid decoders' tests: small random Kosesun checkpoints, and one step's metadata
with scattered pages."""
import json
import math

import numpy as np
import torch

from mlopamd.runtime.attn_meta import MetaBuffers, plan_partitions
from mlopamd.runtime.kv_cache import BLOCK_SIZE, blocks_needed


def rel_err(got, want):
    """Largest difference over the largest magnitude."""
    got, want = got.double().cpu(), want.double().cpu()
    return float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))


class Step:
    """Rows with ``q_lens[i]`` new tokens on top of a context that ends at ``ctx[i]`` tokens, on
    shuffled pages, one-token rows first (as the engine orders them)."""

    def __init__(self, q_lens, ctx, device, n_kv=1, chunk=64, min_part=None, part_dim=64, seed=0, expand_window=None):
        order = sorted(range(len(q_lens)), key=lambda i: q_lens[i] != 1)
        self.q_lens, self.ctx = [q_lens[i] for i in order], [ctx[i] for i in order]
        n = len(q_lens)
        rng = np.random.default_rng(seed)
        self.rows = rng.permutation(n + 2)[:n].astype(np.int32)
        longest = max(self.ctx)
        mb = MetaBuffers(max(sum(q_lens), 4), n + 2, blocks_needed(longest), 16, n_kv, longest, device, flash_min_q=2,
                         flash_tile=128, part_dim=part_dim, chunk=chunk, expand_window=expand_window)
        pages = rng.permutation(sum(blocks_needed(c) for c in self.ctx)) + 1
        self.num_blocks = len(pages) + 1
        o = 0
        for row, c in zip(self.rows, self.ctx):
            k = blocks_needed(c)
            mb.bt_h[row, :k] = pages[o:o + k]
            o += k
        B = sum(q == 1 for q in self.q_lens)
        self.T, nt, nl = mb.fill_mixed(self.rows[:B], np.array(self.ctx[:B], dtype=np.int32), np.zeros(B, np.int64),
                                       self.rows[B:], self.q_lens[B:], self.ctx[B:], [[0] * q for q in self.q_lens[B:]])
        mb.upload()
        part, nparts = (plan_partitions(nt, n_kv, longest) if min_part is None else
                        (min_part, -(-longest // min_part)))
        self.mb = mb
        self.meta = mb.meta(self.T, nt, nl, part, nparts, mb.npt)

    def starts(self):
        return np.concatenate([[0], np.cumsum(self.q_lens)])

    def scatter(self, cache, i, x, upto):
        """Write rows [0, upto) of x [n, heads, d] as sequence i's cached tokens."""
        for t in range(upto):
            blk = int(self.mb.bt_h[self.rows[i], t // BLOCK_SIZE])
            cache[blk, :, t % BLOCK_SIZE, :x.shape[2]] = x[t].to(cache.device, cache.dtype)


def small_config(seed=0, layers="agaga", width=72, vocab=150, streams=3, heads=6, kv_heads=2, dim=24, vdim=20, rot=16,
                 gla_heads=3, gla_dim=12, gla_vdim=28, tau=5.0, ff=104, no_ff=(), no_mix=(), eps=3e-5, cap=11.0, scale=None):
    """config.json dictionary; ``layers``: a = attention, g = gla."""
    out = []
    for i, c in enumerate(layers):
        if c == "a":
            mixer = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "rot": {"base": 8000.0, "dims": rot},
                     "scale": scale or 1.3 * dim ** -0.5, "v_mix": i not in no_mix, "vdim": vdim}
        else:
            mixer = {"dim": gla_dim, "heads": gla_heads, "tau": tau, "vdim": gla_vdim}
        out.append({"type": "attention" if c == "a" else "gla", "mixer": mixer,
                    "mlp": None if i in no_ff else {"ff": ff, "kind": "dense"}})
    return {"architecture": "Kosesun", "embedding": {"scale": 3.7}, "layers": out, "logit_softcap": cap,
            "norm": {"eps": eps}, "streams": streams, "vocab": vocab, "width": width}


def random_weights(cfg, seed=0, rank=7, sharp=2.0):
    """Random bf16 weights of a config, sized so that every mechanism matters in the logits."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg["width"], cfg["streams"]
    w = {}

    def lin(name, o, i, gain=1.0):
        w[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, mean, std):
        w[name] = mean + std * torch.randn(n, generator=g)

    lin("embed", cfg["vocab"], W, math.sqrt(W) / cfg["embedding"]["scale"])
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        if la["type"] == "attention":
            nq, nk, nv = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            lin(p + "mix.q", nq, W), lin(p + "mix.k", nk, W), lin(p + "mix.v", nv, W)
            vec(p + "mix.q.norm", nq, sharp, 0.2), vec(p + "mix.k.norm", nk, 1.0, 0.2)
            vec(p + "mix.sink", m["heads"], 1.0, 1.5)
            lin(p + "mix.g", m["heads"], W), lin(p + "mix.o", W, m["heads"] * m["vdim"])
            if m["v_mix"]:
                w[p + "mix.vmix"] = torch.tensor(0.3 + 0.1 * i)
        else:
            hk, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            lin(p + "mix.q", hk, W), lin(p + "mix.k", hk, W), lin(p + "mix.v", hv, W), lin(p + "mix.g", hv, W)
            lin(p + "mix.o", W, hv), lin(p + "mix.a1", rank, W), lin(p + "mix.a2", hk, rank, 2.0)
            vec(p + "mix.a2.b", hk, 2.0, 2.0), vec(p + "mix.norm", m["vdim"], 1.0, 0.2)
        for q in (1, 2):
            vec(p + f"hc{q}.in", S, 1.0 / S, 0.2), vec(p + f"hc{q}.out", S, 1.0, 0.3)
            w[p + f"hc{q}.mix"] = torch.eye(S) * 0.8 + 0.1 * torch.randn(S, S, generator=g)
            vec(p + f"norm{q}", W, 0.0, 0.2)
        if la["mlp"]:
            lin(p + "mlp.up", la["mlp"]["ff"], W), lin(p + "mlp.down", W, la["mlp"]["ff"])
    vec("final.norm", W, 0.0, 0.2)
    lin("head", cfg["vocab"], W, 4.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


def save_checkpoint(path, cfg, weights):
    from safetensors.torch import save_file

    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in weights.items()}, str(path / "model.safetensors"))
    return path


def make_engine(path, device, dtype, max_tokens=1024, seqs=4, graphs=True, **kw):
    from mlopamd.models.loader import load_pretrained
    from mlopamd.runtime.engine import Engine, EngineConfig

    model = load_pretrained(path, device=device, dtype=dtype)
    kw = {"max_num_seqs": seqs, "max_num_batched_tokens": max_tokens, "max_model_len": max_tokens,
          "num_kv_blocks": blocks_needed(max_tokens) + 1, "graph_buckets": (1, 2, 4), "max_step_logits": max_tokens + 8,
          "use_graphs": graphs, **kw}
    return Engine(model, EngineConfig(**kw))


def feed_schedule(eng, prompts, schedule):
    """``schedule``: steps of [(request, tokens)]; every position's logits, per request.  A request is
    closed when its tokens are through."""
    seqs, at, out = {}, {}, {r: [] for r, _ in enumerate(prompts)}
    for step in schedule:
        entries = []
        for r, n in step:
            if r not in seqs:
                seqs[r], at[r] = eng.open_sequence(), 0
            entries.append((seqs[r], prompts[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
        logits, o = eng.feed(entries).float().cpu(), 0
        for r, n in step:
            out[r].append(logits[o:o + n])
            o += n
            if at[r] == len(prompts[r]):
                eng.close_sequence(seqs.pop(r))
    return [torch.cat(out[r]) for r in range(len(prompts))]


def portions(n, sizes):
    """Cut n tokens into the repeated ``sizes``."""
    out, i = [], 0
    while n:
        k = min(n, sizes[i % len(sizes)])
        out.append(k)
        n, i = n - k, i + 1
    return out


def random_prompts(lens, vocab, seed=0):
    g = torch.Generator().manual_seed(seed)
    return [torch.randint(0, vocab, (n,), generator=g).tolist() for n in lens]


def logits_err(got, want):
    """rms over the vocabulary of the mean-free difference, over the logits' spread: the worst
    position, or four times the average over all positions if that is more."""
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.std()
    return float(max(e.max(), 4 * e.mean()))
