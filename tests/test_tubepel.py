"""Tubepel on the engine against the plain float64 oracle (tubepel_oracle.py).

Every test builds its own small configuration and random checkpoint, loads it
through the framework's config reader and weight loader, runs it through the
engine (scheduler, paged cache, decode graphs on the GPU) and compares logits
with the oracle run on whole sequences; the mechanisms are also tested alone at
the level of the ops. The CPU cases run the torch reference ops; the `gpu`
cases run the HIP kernels in fp32 and bf16.
"""

import io
import json
import os
import random

import numpy as np
import pytest
import torch

import tubepel_oracle as O
from sutro_amd.engine.config import EngineConfig
from sutro_amd.engine.engine import LLMEngine
from sutro_amd.engine.request import SamplingParams
from sutro_amd.models.registry import spec_from_dir
from sutro_amd.ops import hybrid as hops

BACKENDS = [
    pytest.param(("cpu", torch.float32), id="cpu"),
    pytest.param(("cuda", torch.float32), id="gpu-fp32", marks=pytest.mark.gpu),
    pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu),
]


@pytest.fixture(params=BACKENDS)
def backend(request):
    return request.param


def limit(dtype):
    return 5e-5 if dtype == torch.float32 else 6e-2


def row_errors(got, want):
    """Per position: root mean square of the difference (mean over the
    vocabulary taken off), relative to the spread of the expected logits."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    ref = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()


# ------------------------------------------------------------- configs ------

def config_a():
    """Sizes that are multiples of 8 nowhere; three streams; a looped middle
    (three passes) with all three mixers; a window of 11 that keeps 3 tokens
    and one of 6 that keeps none; values wider and narrower than keys; dense,
    routed (with and without a shared expert) and absent feed-forwards."""
    m1 = O.moe_cfg(20, 5, 3, shared_ff=12)
    m2 = O.moe_cfg(12, 6, 2)
    return O.make_config(44, 270, [
        O.layer("latent_attention_2", O.latent_cfg(3, 12, 6, 10, 18, 22, base=500.0),
                O.dense_cfg(50)),
        O.layer("attention", O.attn_cfg(6, 2, 10, 14, 11, 3, 6, base=300.0), m1),
        O.layer("latent_attention", O.latent_cfg(2, 6, 10, 14, 12, 10, scale=0.4),
                m2),
        O.layer("latent_attention_2", O.latent_cfg(5, 6, 2, 6, 26, 20), None),
        O.layer("attention", O.attn_cfg(3, 3, 12, 6, 6, 0, 12, scale=0.5), m1),
    ], streams=3, loop=(1, 4, 3), eps=1e-5)


def config_b():
    """One head, one stream, one expert a token and one expert at all, a loop
    over every layer, a vocabulary below the byte alphabet, a window of one
    token that keeps the first, and one wider than any sequence."""
    return O.make_config(36, 50, [
        O.layer("attention", O.attn_cfg(1, 1, 6, 10, 1, 1, 2, base=7.0),
                O.moe_cfg(28, 4, 1)),
        O.layer("latent_attention", O.latent_cfg(1, 10, 4, 18, 6, 12, base=50.0),
                O.moe_cfg(8, 1, 1, shared_ff=20)),
        O.layer("attention", O.attn_cfg(2, 1, 8, 8, 500, 2, 0), O.dense_cfg(40)),
    ], streams=1, loop=(0, 3, 2), eps=2e-4)


def config_c():
    """Sizes the matrix-core kernels take (pages of 32, head and latent sizes
    multiples of 8, widths multiples of 64); four streams; a loop over the last
    layer alone; kept tokens that cross a page's edge."""
    return O.make_config(128, 300, [
        O.layer("latent_attention", O.latent_cfg(6, 24, 16, 40, 48, 88, base=2000.0),
                O.moe_cfg(64, 13, 4, shared_ff=64)),
        O.layer("attention", O.attn_cfg(8, 2, 48, 64, 45, 35, 32), O.dense_cfg(192)),
        O.layer("latent_attention_2", O.latent_cfg(2, 64, 64, 32, 64, 136),
                O.moe_cfg(128, 7, 2)),
        O.layer("attention", O.attn_cfg(4, 4, 64, 32, 33, 5, 64), None),
    ], streams=4, loop=(2, 4, 2), eps=1e-6)


def config_far():
    """Attention whose scores spread so far that one key takes nearly all the
    weight: a wrong, missing or stale key changes the row altogether."""
    return O.make_config(64, 120, [
        O.layer("latent_attention", O.latent_cfg(4, 16, 8, 16, 32, 24, scale=1.1),
                None),
        O.layer("attention", O.attn_cfg(4, 2, 16, 16, 37, 9, 16, scale=1.2), None),
        O.layer("latent_attention_2", O.latent_cfg(2, 8, 8, 32, 24, 32, scale=1.3),
                None),
    ], streams=2, loop=(0, 2, 2))


_CACHE = {}


def checkpoint(tmp_path_factory, name, cfg_fn, seed=0):
    key = (name, seed)
    if key not in _CACHE:
        cfg = cfg_fn()
        w = O.make_weights(cfg, seed=seed)
        path = O.save_checkpoint(str(tmp_path_factory.mktemp(name)), cfg, w)
        _CACHE[key] = (path, cfg, w, {})
    return _CACHE[key]


def oracle_logits(ck, tokens):
    path, cfg, w, memo = ck
    key = tuple(tokens)
    if key not in memo:
        memo[key] = O.forward(cfg, w, list(tokens))
    return memo[key]


def engine(ck, backend, page=8, blocks=64, max_seqs=4, budget=4096, **kw):
    device, dtype = backend
    cfg = EngineConfig(spec=spec_from_dir(ck[0]), device=device, dtype=dtype,
                       kv_block_size=page, max_model_len=page * (blocks - 1),
                       max_num_seqs=max_seqs, num_kv_blocks=blocks,
                       max_tokens_per_step=budget, **kw)
    return LLMEngine(cfg)


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(3, cfg["vocab"], (n,), generator=g).tolist()


def replay(eng, seqs, schedule):
    """Run `schedule` (a list of steps, each a list of (name, count)) and
    return name -> logits of every position [len, vocab]."""
    live, at, out = {}, {k: 0 for k in seqs}, {k: [] for k in seqs}
    for step in schedule:
        entries = []
        for name, n in step:
            if name not in live:
                live[name] = eng.new_replay_request()
            lo = at[name]
            entries.append((live[name], seqs[name][lo:lo + n], list(range(n))))
            at[name] = lo + n
        logits = eng.replay_step(entries)
        k = 0
        for name, n in step:
            # a graph's output buffer is written again by its next replay
            out[name].append(logits[k:k + n].clone())
            k += n
        for name, _ in step:
            if at[name] == len(seqs[name]) and name in live:
                eng.finish_replay_request(live.pop(name))
    return {k: torch.cat(v) for k, v in out.items() if v}


def check(ck, got, seqs, dtype, names=None, tol=None):
    """Every position within the limit; in bf16, where the smallest
    configurations amplify rounding a little now and then, within three times
    it and the median position within it."""
    for name in names or got:
        want = oracle_logits(ck, seqs[name])
        assert got[name].shape == want.shape
        rows = row_errors(got[name], want)
        lim = tol or limit(dtype)
        worst = lim if dtype == torch.float32 or tol else 3 * lim
        assert float(rows.max()) < worst, \
            f"{name}: error {float(rows.max())} at {int(rows.argmax())}"
        assert len(rows) < 4 or float(rows.median()) < lim, \
            f"{name}: median error {float(rows.median())}"


def page_of(cfg_fn):
    return 32 if cfg_fn is config_c else 8


# ------------------------------------------------ whole prompts, decoding ---

@pytest.mark.parametrize("cfg_fn", [config_a, config_b, config_c])
def test_whole_prompt(tmp_path_factory, backend, cfg_fn):
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend, page=page_of(cfg_fn), blocks=24)
    seqs = {"s": tokens_for(ck[1], 130 if cfg_fn is config_c else 45, 1)}
    got = replay(eng, seqs, [[("s", len(seqs["s"]))]])
    check(ck, got, seqs, backend[1])


@pytest.mark.parametrize("cfg_fn", [config_a, config_b, config_c])
def test_layer_streams_match(tmp_path_factory, backend, cfg_fn):
    """The sum of the fp32 streams after every layer run (a looped layer counts
    each time) against the oracle's: a fault shows in the layer that makes
    it."""
    device, dtype = backend
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend, page=page_of(cfg_fn))
    toks = tokens_for(ck[1], 23, 9)
    want = []
    O.forward(ck[1], ck[2], toks, streams=want)
    eng.model.layer_taps = []
    replay(eng, {"s": toks}, [[("s", 23)]])
    taps = eng.model.layer_taps
    eng.model.layer_taps = None
    lp = ck[1]["loop"]
    assert len(taps) == len(want) == len(ck[1]["layers"]) + \
        (lp["times"] - 1) * (lp["stop"] - lp["start"])
    for i, (g, e) in enumerate(zip(taps, want)):
        err = (g.double().cpu() - e).norm(dim=-1) / e.norm(dim=-1)
        assert float(err.max()) < (2e-5 if dtype == torch.float32 else 8e-2), \
            f"layer run {i}: {float(err.max())}"


@pytest.mark.parametrize("cfg_fn", [config_a, config_b])
def test_first_tokens(tmp_path_factory, backend, cfg_fn):
    """Sequences of one, two and three tokens, alone and decoded one by one."""
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend)
    seqs = {f"n{n}": tokens_for(ck[1], n, 10 + n) for n in (1, 2, 3)}
    got = replay(eng, seqs, [[("n1", 1)], [("n2", 2)], [("n3", 3)]])
    check(ck, got, seqs, backend[1])
    got = replay(eng, seqs, [[("n3", 1), ("n2", 1)], [("n3", 1), ("n2", 1)],
                             [("n3", 1)]])
    check(ck, got, seqs, backend[1], names=["n2", "n3"])


@pytest.mark.parametrize("cfg_fn", [config_a, config_b, config_c])
def test_prefill_then_token_by_token(tmp_path_factory, backend, cfg_fn):
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend, page=page_of(cfg_fn), blocks=24)
    n = 100 if cfg_fn is config_c else 45
    seqs = {"s": tokens_for(ck[1], n, 1)}
    got = replay(eng, seqs, [[("s", 9)]] + [[("s", 1)]] * (n - 9))
    check(ck, got, seqs, backend[1])


@pytest.mark.parametrize("cfg_fn,page", [(config_a, 8), (config_a, 32),
                                         (config_b, 4), (config_c, 32),
                                         (config_c, 16)])
def test_portions_of_many_sizes(tmp_path_factory, backend, cfg_fn, page):
    """Prompt pieces of 2, 3, 1, 11, 2, 5 ... tokens: cuts inside pages,
    windows and the kept tokens."""
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend, page=page, blocks=24)
    seqs = {"s": tokens_for(ck[1], 62, 2)}
    sizes = [2, 3, 1, 11, 2, 5, 1, 1, 13, 2, 8, 7, 2, 4]
    assert sum(sizes) == 62
    got = replay(eng, seqs, [[("s", n)] for n in sizes])
    check(ck, got, seqs, backend[1])


@pytest.mark.parametrize("cfg_fn", [config_a, config_c])
def test_long_decoding(tmp_path_factory, backend, cfg_fn):
    """A short prompt and 150 decoded tokens: page borders, the window's edge
    and the kept tokens' pass under single-token steps."""
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    eng = engine(ck, backend, page=page_of(cfg_fn), blocks=24)
    seqs = {"s": tokens_for(ck[1], 154, 3)}
    got = replay(eng, seqs, [[("s", 4)]] + [[("s", 1)]] * 150)
    check(ck, got, seqs, backend[1])


@pytest.mark.parametrize("page", [8, 32])
def test_far_keys_through_the_engine(tmp_path_factory, backend, page):
    """Peaked attention over 200 tokens: most rows hang on a single key, far
    away, at a page border or at the window's edge; whole, in portions with
    cuts around page borders, and decoded."""
    ck = checkpoint(tmp_path_factory, "config_far", config_far)
    seqs = {"s": tokens_for(ck[1], 200, 17)}
    dtype = backend[1]
    # bf16 scores of this size are only good to a few percent
    tol = 5e-4 if dtype == torch.float32 else 0.35
    sizes = [31, 2, 30, 1, 1, 31, 2, 62]
    for schedule in ([200], sizes + [1] * (200 - sum(sizes))):
        eng = engine(ck, backend, page=page, blocks=40)
        got = replay(eng, seqs, [[("s", n)] for n in schedule])
        check(ck, got, seqs, dtype, tol=tol)


# ------------------------------------------------ random configurations -----

def random_config(seed):
    """Widths, streams, the order and number of layers, the loop, head counts,
    key, value and latent sizes, windows, kept tokens, rotations, expert counts
    and choices: all drawn."""
    rnd = random.Random(seed)
    n = rnd.randint(2, 5)
    layers = []
    for _ in range(n):
        kind = rnd.choice(["attention", "latent_attention",
                           "latent_attention_2"])
        base = rnd.choice([50.0, 10000.0, 500000.0])
        if kind == "attention":
            G, dk = rnd.choice([1, 2, 3]), rnd.choice([8, 12, 32, 72])
            mixer = O.attn_cfg(
                G * rnd.choice([1, 2, 3]), G, dk, rnd.choice([8, 20, 32, 96]),
                rnd.choice([2, 9, 17, 32, 40]), rnd.choice([0, 1, 4, 33]),
                rnd.choice([0, 2, dk // 2, dk]), base=base)
        else:
            mixer = O.latent_cfg(
                rnd.choice([1, 3, 8]), rnd.choice([8, 20, 32]),
                rnd.choice([2, 8, 16, 24]), rnd.choice([4, 16, 40]),
                rnd.choice([5, 24, 64]), rnd.choice([8, 36, 64, 160]),
                scale=rnd.choice([0.1, 0.3]), base=base)
        r = rnd.random()
        mlp = None
        if r < 0.3:
            mlp = O.dense_cfg(rnd.choice([24, 64, 100, 33]))
        elif r < 0.85:
            E = rnd.choice([1, 3, 8])
            mlp = O.moe_cfg(rnd.choice([24, 40, 64, 72]), E,
                            rnd.randint(1, min(E, 4)),
                            shared_ff=rnd.choice([0, 16, 64]))
        layers.append(O.layer(kind, mixer, mlp))
    start = rnd.randint(0, n - 1)
    loop = rnd.choice([None, (start, rnd.randint(start + 1, n),
                              rnd.choice([1, 2, 3]))])
    return O.make_config(
        rnd.choice([64, 96, 136, 50]), rnd.choice([300, 512, 777]), layers,
        streams=rnd.choice([1, 2, 3, 4, 5, 9]), loop=loop,
        eps=rnd.choice([1e-6, 1e-5]))


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8, 9, 10])
def test_random_configurations(tmp_path_factory, backend, seed):
    ck = checkpoint(tmp_path_factory, f"random{seed}",
                    lambda: random_config(seed), seed=seed)
    eng = engine(ck, backend, page=[8, 32][seed % 2], blocks=24)
    seqs = {"a": tokens_for(ck[1], 48, seed), "b": tokens_for(ck[1], 33, seed + 50),
            "c": tokens_for(ck[1], 7, seed + 90)}
    got = replay(eng, seqs, [
        [("a", 21), ("b", 1)], [("a", 1), ("b", 2), ("c", 3)],
        [("b", 27), ("a", 2), ("c", 1)], [("a", 24), ("b", 1), ("c", 1)],
        [("b", 1), ("c", 2)], [("b", 1)]])
    check(ck, got, seqs, backend[1])


# ----------------------------------------------------- batches, reuse -------

MIXED = [
    [("a", 13), ("b", 1)],
    [("a", 1), ("b", 1), ("c", 2)],
    [("b", 6), ("c", 1), ("d", 20), ("a", 1)],
    [("a", 20), ("c", 1), ("d", 1)],
    [("b", 9), ("d", 1), ("c", 5), ("a", 5)],
    [("d", 4)],
]


@pytest.mark.parametrize("cfg_fn,page", [(config_a, 8), (config_c, 32)])
def test_mixed_batch_equals_each_alone(tmp_path_factory, backend, cfg_fn, page):
    """Unequal requests in one batch (prompt pieces beside single tokens,
    requests that sit out a step) give what each gives alone."""
    ck = checkpoint(tmp_path_factory, cfg_fn.__name__, cfg_fn)
    dtype = backend[1]
    seqs = {"a": tokens_for(ck[1], 40, 4), "b": tokens_for(ck[1], 17, 5),
            "c": tokens_for(ck[1], 9, 6), "d": tokens_for(ck[1], 26, 7)}
    # with and without captured decode steps (eager: one batch for all rows)
    for kw in ({}, {"enforce_eager": True}):
        eng = engine(ck, backend, page=page, blocks=24, **kw)
        got = replay(eng, seqs, MIXED)
        check(ck, got, seqs, dtype)
    alone = replay(engine(ck, backend, page=page, blocks=24), seqs,
                   [[(k, len(v))] for k, v in seqs.items()])
    for k in seqs:
        e = row_errors(got[k], alone[k].double().cpu())
        assert float(e.max()) < limit(dtype)


def test_pages_and_slots_are_reused(tmp_path_factory, backend):
    """Two sequence slots and a pool of six pages serve eight requests one
    after another; what a freed page held must not leak into the next
    request."""
    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    eng = engine(ck, backend, page=8, blocks=7, max_seqs=2)
    seqs = {f"r{i}": tokens_for(ck[1], 9 + 3 * (i % 4), 20 + i) for i in range(8)}
    names = list(seqs)
    schedule = []
    for i in range(0, 8, 2):
        a, b = names[i], names[i + 1]
        la, lb = len(seqs[a]), len(seqs[b])
        schedule += [[(a, 5), (b, 2)], [(a, la - 5), (b, 1)], [(b, lb - 3)]]
    got = replay(eng, seqs, schedule)
    check(ck, got, seqs, backend[1])
    assert eng.kv.allocator.num_free == 6
    with pytest.raises(MemoryError):
        replay(eng, {"x": [3] * 40, "y": [4] * 16}, [[("x", 40), ("y", 16)]])


def test_cache_layout(tmp_path_factory):
    """Every layer RUN holds pages of its own; latent layers hold one row of
    latent and rotated key part; there is no recurrent state."""
    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    eng = engine(ck, ("cpu", torch.float32))
    assert eng.spec.runs == ((0, 0), (1, 0), (2, 0), (3, 0), (1, 1), (2, 1),
                             (3, 1), (1, 2), (2, 2), (3, 2), (4, 0))
    kv, st = eng.model.cache_layout()
    att, l2, l3 = (2, 10, 14), (1, 10 + 10, 0), (1, 20 + 2, 0)
    assert kv == [(1, 22 + 6, 0), att, l2, l3, att, l2, l3, att, l2, l3,
                  (3, 12, 6)]
    assert st == [None] * 11 and eng.kv.state is None
    assert len({eng.kv.k_cache[i].data_ptr() for i in range(11)}) == 11


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_decode_graph_replays_equal_eager_steps(tmp_path_factory, dtype):
    """Single-token steps run as captured hipGraphs. Many replays with prompt
    pieces of other requests and host synchronisation between them must give,
    every time, what an engine that captures nothing gives (up to rounding: a
    graph pads its batch and its block tables)."""
    ck = checkpoint(tmp_path_factory, "config_c", config_c)
    seqs = {"a": tokens_for(ck[1], 60, 1), "b": tokens_for(ck[1], 45, 2),
            "c": tokens_for(ck[1], 38, 3)}
    schedule = [[("a", 20)], [("a", 1)], [("a", 1), ("b", 30)],
                [("a", 1), ("b", 1)], [("c", 33), ("a", 1)]]
    schedule += [[("a", 1), ("b", 1), ("c", 1)]] * 5 + [[("a", 31), ("b", 8)]]
    graphs = engine(ck, ("cuda", dtype), page=32, blocks=24)
    assert graphs.graph_runner is not None
    eager = engine(ck, ("cuda", dtype), page=32, blocks=24, enforce_eager=True)
    assert eager.graph_runner is None
    got, want = replay(graphs, seqs, schedule), replay(eager, seqs, schedule)
    for k in seqs:
        rows = row_errors(got[k], want[k].double().cpu())
        assert float(rows.max()) < (1e-5 if dtype == torch.float32 else 3e-2), k


# ------------------------------------------------- mechanisms on their own --

def _bf(x):
    return x.to(torch.bfloat16).double()


@pytest.mark.parametrize("T,S,W", [(5, 1, 44), (9, 2, 36), (7, 3, 50), (6, 4, 256),
                                   (4, 5, 1100), (3, 6, 64), (3, 7, 12),
                                   (3, 8, 2048), (5, 9, 40), (2, 16, 130),
                                   (300, 4, 1024)])
def test_streams_mix_read_and_write(backend, T, S, W):
    """The fused kernel against the two equations: a first read of equal
    streams; the first update, which takes all streams from one row; updates
    with a plain result, with gathered and weighted expert rows and with a
    shared expert's row; a last one that does not write."""
    device, dtype = backend
    g = torch.Generator().manual_seed(S + W)
    eps = 1e-5

    def f32(*shape, mean=0.0):
        return (torch.randn(*shape, generator=g) + mean)

    M, b, a, nw = f32(S, S), f32(S), f32(S), f32(W, mean=1.0)
    e0 = f32(T, W)
    y, y2 = _bf(f32(T, W)), _bf(f32(T, W))
    rows = _bf(f32(3 * T, W))
    k = 2
    pos = torch.randint(3 * T, (T, k), generator=g).int()
    pw = torch.rand(T, k, generator=g)
    dev = lambda t: t.float().to(device)                       # noqa: E731
    act = lambda t: t.to(dtype).to(device)                     # noqa: E731
    htol = 2e-5 if dtype == torch.float32 else 2e-2

    def close(got, want, tol):
        err = (got.double().cpu() - want).abs().max() / want.abs().max()
        assert float(err) < tol

    def read(X):
        u = O.bundle_read(X, a.double())
        return O.rms(u, nw.double(), eps)

    h = torch.empty(T, W, dtype=dtype, device=device)
    x = torch.full((T, S, W), 1e6, device=device)
    nwd, ad = dev(nw), dev(a)
    X = e0.double().expand(S, T, W)
    hops.hyper_rmsnorm(x, dev(e0), in_w=ad, norm_w=nwd, eps=eps, h_out=h)
    close(h, read(X), htol)
    assert float(x.min()) == 1e6                 # nothing was written
    gathered = (rows[pos.long()] * pw.double().unsqueeze(-1)).sum(1)
    plain = rows[pos.long()].sum(1) * 0.75
    for n, (kw, r) in enumerate([
            (dict(x_in=dev(e0), y=act(y)), y),
            (dict(y=act(y)), y),
            (dict(rows=act(rows), padpos=pos.to(device), wts=dev(pw)), gathered),
            (dict(rows=act(rows), padpos=pos.to(device), wts=0.75,
                  y2=act(y2)), plain + y2)]):
        X = O.bundle_write(X, M.double(), b.double(), r)
        X = X / X.abs().max()
        hops.hyper_rmsnorm(x, mix=dev(M), out=dev(b), in_w=ad, norm_w=nwd,
                           eps=eps, h_out=h, **kw)
        x /= x.abs().max()
        close(x.transpose(0, 1), X, 2e-5 * (n + 1))
        hops.hyper_rmsnorm(x, in_w=ad, norm_w=nwd, eps=eps, h_out=h)
        close(h, read(X), htol * (n + 1))
    before = x.clone()
    hops.hyper_rmsnorm(x, y=act(y), mix=dev(M), out=dev(b), in_w=ad,
                       norm_w=nwd, eps=eps, h_out=h, write=False)
    close(h, read(O.bundle_write(X, M.double(), b.double(), y)), htol * 5)
    assert torch.equal(x, before)


@pytest.mark.parametrize("T,n", [(3, 40), (5, 33), (1, 1), (64, 512)])
def test_squared_relu(backend, T, n):
    device, dtype = backend
    g = torch.Generator().manual_seed(n)
    z = _bf(torch.randn(T, n, generator=g) * 3)
    got = hops.relu_sq(z.to(dtype).to(device))
    want = O.relu_squared(z)
    tol = 1e-6 if dtype == torch.float32 else 4e-3
    assert bool(((got.double().cpu() - want).abs() <= tol * want).all())


def _scrambled_pages(T, page, g, extra=2):
    """(number of blocks, table [ceil(T / page)]) with pages out of order."""
    need = (T + page - 1) // page
    return need + extra, (torch.randperm(need + extra - 1, generator=g)
                          + 1)[:need].int()


def _window_attention(device, dtype, q, k, v, scale, window, keep, page,
                      pieces, sink=None, gate=None):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] of one sequence through
    `local_attention`, piece by piece. Returns [T, H, dv] on the CPU."""
    T, H, dk = q.shape
    G, dv = v.shape[1:]
    g = torch.Generator().manual_seed(T + page)
    n_blocks, table = _scrambled_pages(T, page, g)
    # what stale pages hold must not matter
    kc = torch.full((n_blocks, G, page, dk), 3.0, dtype=dtype, device=device)
    vc = torch.full((n_blocks, G, page, dv), 9.0, dtype=dtype, device=device)
    got, done = [], 0
    for n in pieces:
        pos = torch.arange(done, done + n)
        blk, off = table[pos // page].long().to(device), (pos % page).to(device)
        kc[blk, :, off] = k[done:done + n].to(dtype).to(device)
        vc[blk, :, off] = v[done:done + n].to(dtype).to(device)
        qq = q[done:done + n].to(dtype).to(device).contiguous()
        pad = 8
        proj = torch.zeros(n, pad + H * dv, dtype=dtype, device=device)
        if gate is not None:
            proj[:, pad:] = gate[done:done + n].reshape(n, -1).to(dtype).to(device)
        out = torch.zeros(n, 8 + H * dv, dtype=dtype, device=device)
        done += n
        tiles = {}
        if n > 1:
            tiles = dict(
                tile_seq=torch.zeros((n + 31) // 32, dtype=torch.int32, device=device),
                tile_q0=torch.arange(0, n, 32, dtype=torch.int32, device=device),
                prefill_rows=n)
        hops.local_attention(
            qq, kc, vc, table[None].to(device),
            torch.tensor([done], dtype=torch.int32, device=device),
            torch.tensor([0, n], dtype=torch.int32, device=device), scale, 0,
            window, proj, pad if gate is not None else -1, out, 8, 1.0,
            token_seq=torch.zeros(n, dtype=torch.int32, device=device),
            sink=sink is not None, keep_first=keep, gate_n=dv,
            sink_w=None if sink is None else sink.float().to(device), **tiles)
        assert float(out[:, :8].abs().max()) == 0.0
        got.append(out[:, 8:].float().cpu())
    return torch.cat(got).view(T, H, dv)


def _want_window(q, k, v, scale, window, keep, sink=None, gate=None):
    T, H = q.shape[:2]
    G = k.shape[1]
    mask = O.sees(T, window, keep)
    o = torch.stack([O.attend(q[:, a], k[:, a * G // H], v[:, a * G // H], scale,
                              mask, None if sink is None else sink[a])
                     for a in range(H)], dim=1)
    return o if gate is None else o * torch.sigmoid(gate)


SHAPES = [(4, 6, 2, 10, 14), (32, 4, 1, 24, 40), (32, 8, 2, 64, 64),
          (32, 3, 3, 128, 96), (16, 4, 2, 40, 24), (32, 2, 2, 72, 200)]


@pytest.mark.parametrize("mode", ["prompt", "pieces", "decoded"])
@pytest.mark.parametrize("page,H,G,dk,dv", SHAPES)
def test_window_edges_and_kept_tokens_stand_out(backend, mode, page, H, G, dk,
                                                dv):
    """One key is made to score far above all others, so a row's output is
    (nearly) that key's value if and only if the row sees it: the first tokens
    just inside and just outside the kept ones, keys on both sides of page
    borders, rows just inside and just outside the window."""
    device, dtype = backend
    T, scale = 130, 0.25
    for window, keep, star in ((40, 5, 4), (40, 5, 5), (33, 35, 34), (33, 35, 35),
                               (17, 0, 0), (64, 1, 31), (64, 1, 32), (1, 2, 1),
                               (500, 3, 60)):
        g = torch.Generator().manual_seed(page + dk + star)
        q = torch.randn(T, H, dk, generator=g, dtype=torch.float64) * 0.3
        k = torch.randn(T, G, dk, generator=g, dtype=torch.float64) * 0.3
        v = _bf(torch.randn(T, G, dv, generator=g))
        u = torch.zeros(dk, dtype=torch.float64)
        u[(star + 3) % dk] = 1.0
        k[star] += 14.0 * u
        q += 7.0 * u
        q, k = _bf(q), _bf(k)
        if mode == "prompt":
            pieces = [T]
        elif mode == "pieces":
            cuts = sorted({2, max(star, 3), star + 2, min(star + window, 126),
                           min(star + window + 2, 128)} - {0})
            pieces = [b - a for a, b in zip([0] + cuts, cuts + [T])]
        else:
            pieces = [3] + [1] * (T - 3)
        got = _window_attention(device, dtype, q, k, v, scale, window, keep,
                                page, pieces)
        want = _want_window(q, k, v, scale, window, keep)
        err = float((got.double() - want).abs().max() / want.abs().max())
        assert err < (1e-4 if dtype == torch.float32 else 2e-2), \
            (window, keep, star, err)
        # the test shows what it means to
        seen = O.sees(T, window, keep)[:, star]
        off = (want[:, 0] - v[star, 0]).abs().amax(-1)
        assert float(off[seen].max()) < 0.3
        assert not bool((~seen).any()) or float(off[~seen].min()) > 0.3


@pytest.mark.parametrize("mode", ["prompt", "decoded"])
@pytest.mark.parametrize("page,H,G,dk,dv", SHAPES)
def test_learned_sinks_and_elementwise_gates(backend, mode, page, H, G, dk, dv):
    """Sinks from far below to far above the scores (a large one takes nearly
    all the weight; it is not scaled and carries no value), different per
    head, with an elementwise gate; a first token has nothing but itself and
    the sink."""
    device, dtype = backend
    T = 70
    g = torch.Generator().manual_seed(dk + dv)
    q, k, v, gate = (_bf(torch.randn(T, n, d, generator=g))
                     for n, d in ((H, dk), (G, dk), (G, dv), (H, dv)))
    sink = _bf(torch.linspace(-9.0, 5.0, H) if H > 1 else torch.tensor([2.0]))
    scale = 0.3 * dk ** -0.5
    pieces = [T] if mode == "prompt" else [2] + [1] * (T - 2)
    for kw in (dict(sink=sink), dict(sink=sink, gate=gate), dict(gate=gate),
               dict(sink=torch.zeros(H, dtype=torch.float64) + 40.0)):
        got = _window_attention(device, dtype, q, k, v, scale, 19, 4, page,
                                pieces, **kw).double()
        want = _want_window(q, k, v, scale, 19, 4, **kw)
        # a large sink leaves a tiny result: compare with its own size
        err = float((got - want).abs().max() / want.abs().max())
        assert err < (1e-4 if dtype == torch.float32 else 2e-2), (sorted(kw), err)


@pytest.mark.parametrize("adjacent", [True, False])
@pytest.mark.parametrize("H,dk,rd,R", [(3, 12, 6, 22), (4, 8, 16, 64),
                                       (1, 5, 2, 7), (16, 64, 32, 128),
                                       (3, 16, 64, 576), (2, 8, 48, 32)])
def test_latent_rows_and_both_pairings(backend, adjacent, H, dk, rd, R):
    """The cache row (normed latent | rotated key part, the latter not normed)
    and the rotated query parts in either pairing; other cache rows and the
    folded queries stay as they are."""
    device, dtype = backend
    g = torch.Generator().manual_seed(R)
    T, N, base = 12, 20, 3000.0
    tab = hops.rope_table(torch.arange(T).to(device),
                          hops.yarn_inv_freq(rd, base, None)[0].to(device))
    off = 8
    proj = _bf(torch.randn(T, off + R + rd + 4 + H * (dk + rd), generator=g))
    w = _bf(torch.rand(R, generator=g) + 0.5)
    pd = proj.to(dtype).to(device)
    q = pd[:, off + R + rd + 4:].unflatten(1, (H, dk + rd))
    cache = torch.full((N, R + rd), 5.0, dtype=dtype, device=device)
    qa = torch.full((T, H, R + rd), 6.0, dtype=dtype, device=device)
    rows = torch.randperm(N, generator=g)[:T]
    hops.latent_prep(pd, off, R, w.float().to(device), 1e-4, tab, cache,
                     rows.to(device), q, dk, qa, adjacent=adjacent)
    rot = {"dims": rd, "base": base}
    c = O.rms(proj[:, off:off + R], w, 1e-4)
    kr = O.turn(proj[:, off + R:off + R + rd], rot, adjacent)
    tol = 3e-5 if dtype == torch.float32 else 3e-2
    got = cache.double().cpu()
    assert float((got[rows] - torch.cat([c, kr], 1)).abs().max()) < tol
    rest = [i for i in range(N) if i not in set(rows.tolist())]
    assert float((got[rest] - 5.0).abs().max()) == 0.0
    qr = proj[:, off + R + rd + 4:].view(T, H, dk + rd)[..., dk:]
    want = torch.stack([O.turn(qr[:, a], rot, adjacent) for a in range(H)], 1)
    assert float((qa[..., R:].double().cpu() - want).abs().max()) < tol
    assert float((qa[..., :R].float() - 6.0).abs().max()) == 0.0


@pytest.mark.parametrize("T,E,top", [(40, 8, 1), (7, 5, 5), (300, 130, 6), (1, 3, 2)])
def test_router_keeps_the_scores(backend, T, E, top):
    device, _ = backend
    g = torch.Generator().manual_seed(E)
    z = torch.randn(T, E, generator=g) * 2
    idx, w = hops.moe_route(z.to(device), top, 1, 1, renorm=False)
    s, order = torch.sigmoid(z.double()).sort(dim=-1, descending=True)
    assert torch.equal(idx.long().cpu(), order[:, :top])
    assert float((w.double().cpu() - s[:, :top]).abs().max()) < 1e-6


@pytest.mark.parametrize("T,W,ff,E,top,shared", [
    (50, 44, 20, 5, 3, 12), (9, 36, 28, 4, 1, 0), (300, 128, 64, 12, 4, 64),
    (1, 64, 64, 3, 2, 8), (2600, 64, 128, 4, 2, 0), (5, 40, 24, 1, 1, 16),
    (3100, 32, 24, 7, 3, 0), (900, 128, 192, 3, 1, 64)])
def test_experts_read_weighted_inputs(backend, T, W, ff, E, top, shared):
    """Router, dispatch with row weights, both expert GEMMs and the shared
    expert against the per-token formulas. The weight must reach the input:
    an expert is not linear, so weighing its result is far off."""
    device, dtype = backend
    from sutro_amd.models.hybrid_spec import RoutedExpertsSpec
    from sutro_amd.models.layers import RoutedExperts

    g = torch.Generator().manual_seed(T + W)
    spec = RoutedExpertsSpec(ff=ff, experts=E, top=top, router="sigmoid",
                             act="silu_glu", shared_ff=shared,
                             shared_gate=False, renorm=False, weigh_input=True)
    mod = RoutedExperts(spec, W, dtype).to(device).requires_grad_(False)
    w = {}
    for e in [f"e{i}" for i in range(E)] + (["shared"] if shared else []):
        f = shared if e == "shared" else ff
        for n, shape, std in (("gate", (f, W), 1.5 * W ** -0.5),
                              ("up", (f, W), 1.5 * W ** -0.5),
                              ("down", (W, f), f ** -0.5)):
            w[f"{e}.{n}"] = _bf(torch.randn(*shape, generator=g) * std)
    w["router"] = _bf(torch.randn(E, W, generator=g) * W ** -0.5)
    params = dict(mod.named_parameters())
    targets = mod.param_targets("", "")
    assert {k.lstrip(".") for k in targets} == set(w)
    with torch.no_grad():
        for ck, (pname, dim, start, length, _) in targets.items():
            dst = params[pname].narrow(dim, start, length)
            src = w[ck.lstrip(".")]
            if dst.dim() == src.dim() + 1:
                dst = dst.squeeze(dim)
            dst.copy_(src.to(dst.dtype))
    h = _bf(torch.randn(T, W, generator=g))
    hd = h.to(dtype).to(device)
    rows, padpos, wts, idw = mod(hd)
    assert idw is None and wts == 1.0
    got = rows[padpos.long()].float().sum(1)
    if shared:
        y2, _, sg = mod.shared_forward(hd)
        assert sg == -1
        got = got + y2.float()
    fc = {"router": {"top": top}, "shared": bool(shared)}
    want = O.routed(h, {"m." + k: v for k, v in w.items()}, "m.", fc)
    err = float((got.double().cpu() - want).abs().max() / want.abs().max())
    assert err < (1e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("neighbours", [True, False])
@pytest.mark.parametrize("mode", ["prompt", "decoded"])
def test_far_latents_stand_out(backend, neighbours, mode):
    """One latent layer whose queries and one far token's key agree in the
    part that is not rotated: all later rows read that token, across pages and
    the 64-key steps of the matrix-core kernel; and without it they read
    something else."""
    device, dtype = backend
    T, H, R, rd, page, scale = 150, 5, 72, 24, 32, 0.25
    g = torch.Generator().manual_seed(3)
    rot = {"dims": rd, "base": 100.0}
    for star in (0, 31, 64, 127):
        q = torch.randn(T, H, R + rd, generator=g, dtype=torch.float64) * 0.3
        c = torch.randn(T, R + rd, generator=g, dtype=torch.float64) * 0.3
        c[star, 5] += 12.0
        q[..., 5] += 6.0
        c[:, R:] = O.turn(c[:, R:], rot, neighbours)
        for a in range(H):
            q[:, a, R:] = O.turn(q[:, a, R:], rot, neighbours)
        q, c = _bf(q), _bf(c)
        n_blocks, table = _scrambled_pages(T, page, g)
        cache = torch.full((n_blocks, 1, page, R + rd), 3.0, dtype=dtype,
                           device=device)
        got, done = [], 0
        for n in [T] if mode == "prompt" else [5] + [1] * (T - 5):
            pos = torch.arange(done, done + n)
            cache[table[pos // page].long().to(device), 0,
                  (pos % page).to(device)] = c[done:done + n].to(dtype).to(device)
            qq = q[done:done + n].to(dtype).to(device).contiguous()
            done += n
            out = torch.zeros(n, H * R, dtype=dtype, device=device)
            tiles = {} if n == 1 else dict(
                tile_seq=torch.zeros((n + 31) // 32, dtype=torch.int32, device=device),
                tile_q0=torch.arange(0, n, 32, dtype=torch.int32, device=device),
                prefill_rows=n)
            hops.local_attention(
                qq, cache, cache[..., :R], table[None].to(device),
                torch.tensor([done], dtype=torch.int32, device=device),
                torch.tensor([0, n], dtype=torch.int32, device=device), scale,
                0, 0, qq.view(n, -1), -1, out, 0, 1.0,
                token_seq=torch.zeros(n, dtype=torch.int32, device=device),
                **tiles)
            got.append(out.double().cpu())
        got = torch.cat(got).view(T, H, R)
        want = torch.stack([O.attend(q[:, a], c, c[:, :R], scale, O.sees(T))
                            for a in range(H)], dim=1)
        err = float((got - want).abs().max() / want.abs().max())
        assert err < (1e-4 if dtype == torch.float32 else 2e-2), (star, err)
        assert float((want[T - 1, 0] - c[star, :R]).abs().max()) < 0.3
        if star:
            assert float((want[star - 1, 0] - c[star, :R]).abs().max()) > 1.0


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 2, 2), (1, 2, 4), (1, 3, 2)])
def test_loops(tmp_path_factory, backend, loop):
    """Loops at the start, in the middle and at the end, of one and several
    layers, passed once and often; prompts and decoding."""
    def cfg():
        return O.make_config(40, 90, [
            O.layer("attention", O.attn_cfg(2, 1, 8, 8, 7, 2, 4),
                    O.moe_cfg(16, 3, 2)),
            O.layer("latent_attention", O.latent_cfg(2, 8, 4, 8, 12, 16), None),
            O.layer("latent_attention_2", O.latent_cfg(1, 8, 8, 8, 20, 8),
                    O.dense_cfg(24)),
        ], loop=loop)
    ck = checkpoint(tmp_path_factory, f"loop{loop}", cfg)
    eng = engine(ck, backend, blocks=24)
    assert len(eng.spec.runs) == 3 + (
        (loop[2] - 1) * (loop[1] - loop[0]) if loop else 0)
    seqs = {"s": tokens_for(ck[1], 30, 8)}
    got = replay(eng, seqs, [[("s", 11)], [("s", 2)]] + [[("s", 1)]] * 17)
    check(ck, got, seqs, backend[1])


# ------------------------------------------------ the framework's own path --

@pytest.mark.parametrize("lagged", [False, True])
def test_greedy_generation_through_scheduler(tmp_path_factory, backend, lagged):
    """Requests go through add_request / step(): the scheduler cuts prompts by
    its own token budget, batches prefill with decode and samples greedily
    (with `lagged`, a step's tokens are read by the host one step later).
    Every generated token must be the oracle's argmax given the same prefix
    (ties within rounding excepted)."""
    device, dtype = backend
    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    eng = engine(ck, backend, budget=16, blocks=40, async_decode=lagged)
    prompts = [tokens_for(ck[1], n, 30 + n) for n in (21, 5, 34, 2, 13)]
    reqs = [eng.add_request(p, SamplingParams(max_tokens=12, temperature=0.0))
            for p in prompts]
    steps = 0
    while eng.has_work():
        eng.step()
        steps += 1
        assert steps < 400
    checked = 0
    for p, r in zip(prompts, reqs):
        assert r.finished and len(r.output_token_ids) >= 1
        seq = p + r.output_token_ids
        logits = oracle_logits(ck, seq[:-1])
        spread = float(logits.std())
        for n, tok in enumerate(r.output_token_ids):
            row = logits[len(p) - 1 + n, :eng.tokenizer.vocab_size]
            best = int(row.argmax())
            margin = float(row[best] - row[tok]) / spread
            assert tok == best or margin < 5 * limit(dtype), (n, tok, best)
            checked += 1
    assert checked >= 20


def test_replay_tool_writes_the_wanted_logits(tmp_path_factory, monkeypatch,
                                              capsys):
    """The replay program on a checkpoint directory: wanted rows in entry
    order, one file a step that wants something, `done` lines."""
    from sutro_amd.engine import replay as tool

    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    a, b = tokens_for(ck[1], 20, 1), tokens_for(ck[1], 6, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:15], "want": [0, 14]}],
         "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []},
                                {"id": "a", "tokens": a[15:16], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[16:], "want": [3, 1]},
                                {"id": "b", "tokens": b[2:], "want": [2]}],
         "end": ["a", "b"]}]
    out = str(tmp_path_factory.mktemp("replayed"))
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "\n".join(json.dumps(s) for s in steps) + "\n"))
    assert tool.main(["--model", ck[0], "--dtype", "float32", "--out", out,
                      "--max-tokens", "128", "--device", "cpu"]) == 0
    lines = capsys.readouterr().out.split("\n")
    assert [x for x in lines if x.startswith("done")] == [
        "done 0", "done 1", "done 2"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32"]
    V = ck[1]["vocab"]
    la, lb = oracle_logits(ck, a), oracle_logits(ck, b)
    for name, want in (("0", la[[0, 14]]),
                       ("2", torch.stack([la[19], la[17], lb[4]]))):
        got = np.fromfile(os.path.join(out, name + ".f32"), "<f4").reshape(-1, V)
        assert float(row_errors(torch.from_numpy(got), want).max()) < 1e-4


def test_service_job_on_a_checkpoint_directory(tmp_path_factory, local_client):
    """A checkpoint directory is a model name for the job service too."""
    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    job = local_client.infer(["alpha", "beta gamma"], model=ck[0],
                             sampling_params={"max_tokens": 4, "temperature": 0},
                             stay_attached=False)
    out = local_client.await_job_completion(job, timeout=120)
    assert out is not None and len(out) == 2


def test_cli_generates_from_a_checkpoint_directory(tmp_path_factory):
    from click.testing import CliRunner

    from sutro_amd.cli import cli

    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    res = CliRunner().invoke(cli, ["generate", "--model", ck[0], "--prompt",
                                   "hello there", "--prompt", "two",
                                   "--max-tokens", "5", "--temperature", "0",
                                   "--device", "cpu", "--max-model-len", "256"])
    assert res.exit_code == 0, res.output
    lines = [json.loads(x) for x in res.output.strip().splitlines()]
    assert [x["prompt"] for x in lines] == ["hello there", "two"]


def test_registry_reads_every_size_from_the_config(tmp_path_factory):
    from sutro_amd.models.hybrid_spec import (AttnMixerSpec, HybridSpec,
                                              LatentAttnMixerSpec,
                                              tubepel_spec)
    from sutro_amd.models.registry import get_model_spec, safetensors_shapes

    ck = checkpoint(tmp_path_factory, "config_a", config_a)
    spec = get_model_spec(ck[0])
    assert isinstance(spec, HybridSpec) and spec.arch == "tubepel"
    assert [type(l.mixer) for l in spec.layers] == [
        LatentAttnMixerSpec, AttnMixerSpec, LatentAttnMixerSpec,
        LatentAttnMixerSpec, AttnMixerSpec]
    a = spec.layers[0].mixer
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank) == (
        3, 12, 6, 10, 18, 22)
    assert not a.rot_adjacent and not a.out_gate and a.rot_base == 500.0
    assert spec.layers[2].mixer.rot_adjacent
    assert spec.layers[2].mixer.scale == 0.4
    m = spec.layers[1].mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim) == (6, 2, 10, 14)
    assert (m.window, m.keep_first, m.rot_dims, m.rot_base) == (11, 3, 6, 300.0)
    assert m.sink and m.sink_learned and m.out_gate and m.gate_elements
    assert not m.qk_norm and not m.bias
    assert spec.layers[4].mixer.keep_first == 0
    e = spec.layers[1].moe
    assert (e.ff, e.experts, e.top, e.shared_ff) == (20, 5, 3, 12)
    assert e.router == "sigmoid" and not e.renorm and e.weigh_input
    assert not e.shared_gate and spec.layers[2].moe.shared_ff == 0
    assert spec.layers[0].ff == 50 and spec.layers[0].ff_kind == "relu2"
    assert spec.layers[3].ff == 0 and spec.layers[3].moe is None
    assert spec.loop == (1, 4, 3) and not spec.loop_reenter
    assert spec.streams == 3 and spec.norm_eps == 1e-5
    assert not spec.tie_embeddings
    assert spec.param_count() == sum(v.numel() for v in ck[2].values())

    # a query rank the config leaves out is the tensor's row count
    cfg = json.loads(json.dumps(ck[1]))
    for l in cfg["layers"]:
        l["mixer"].pop("q_rank", None)
    again = tubepel_spec(cfg, tensor_shapes=safetensors_shapes(ck[0]))
    assert again.layers == spec.layers

    def broken(change):
        bad = json.loads(json.dumps(ck[1]))
        change(bad)
        with pytest.raises(ValueError):
            tubepel_spec(bad)

    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=4))
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=9))
    broken(lambda c: c["layers"][0].update(type="unheard_of"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="unheard_of"))
    broken(lambda c: c["loop"].update(stop=9))
    broken(lambda c: c.update(streams=0))


def test_loading_is_strict_but_knows_unused_tensors(tmp_path_factory):
    """A layer without a feed-forward may carry that sublayer's norm and stream
    weights; any other surplus or missing tensor is an error."""
    cfg = config_a()
    w = O.make_weights(cfg, seed=4)
    extra = dict(w)
    extra["l3.norm2"] = torch.ones(44, dtype=O.F64)
    for n, shape in (("in", (3,)), ("out", (3,)), ("mix", (3, 3))):
        extra["l3.hc2." + n] = torch.ones(*shape, dtype=O.F64)
    path = O.save_checkpoint(str(tmp_path_factory.mktemp("extra")), cfg, extra)
    eng = engine((path, cfg, extra, {}), ("cpu", torch.float32))
    toks = tokens_for(cfg, 12, 1)
    got = replay(eng, {"s": toks}, [[("s", 12)]])
    assert float(row_errors(got["s"], O.forward(cfg, w, toks)).max()) < 1e-4
    # the mix matrix is indexed [from, to]
    assert torch.equal(eng.model.layers[1].hc2.w_mix.double(), w["l1.hc2.mix"])
    for change in (lambda d: d.pop("l1.mix.sink"), lambda d: d.pop("l2.hc2.mix"),
                   lambda d: d.update({"l0.mix.g": torch.ones(30, 44)})):
        bad = dict(w)
        change(bad)
        path = O.save_checkpoint(str(tmp_path_factory.mktemp("bad")), cfg, bad)
        with pytest.raises(ValueError):
            engine((path, cfg, bad, {}), ("cpu", torch.float32))
