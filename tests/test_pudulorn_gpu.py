"""Pudulorn on the GPU: whole models through the engine's step function and cache
manager against the plain implementation: whole prompts, token-by-token
decoding, portions down to two tokens, mixed batches with pages used again,
random schedules, long decoding across many windows and chunks, keys just inside
and just outside every window and chunk, layers that read other layers' latents,
the first tokens of a sequence, other orders and sizes, and greedy generation
through the entry point and the scheduler."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

from conftest import ROOT
from pudulorn_util import (BLOCK_SIZE, CONFIGS, RouterLog, config, dense, edit, latent, moe, pairs, plain_greedy, plain_logits,
                           plain_logits_routed_alike, plain_sensitivity, random_config, write_model)
from trace_util import Trace, compare, compare_with_alone, random_tokens, random_trace, replay

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]

# bfloat16 against the 64-bit plain model on the same rounded weights (and the engine's choice of experts), of a
# row's largest logit.  Measured: a trace's median 1.2e-2 at worst, rows 2.7e-2; single rows that are far more
# sensitive than the rest get an allowance of eight times what a rounding step of the weights moves them by (up to
# four to five times are measured).
TOL16 = dict(rtol=0.0, atol=2e-2, median=2e-2)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: {dt: write_model(str(tmp_path_factory.mktemp(f"pudulorn{name}_{dt}")), cfg, seed=11 + ord(name), dtype=dt)
                   for dt in DTYPES} for name, cfg in CONFIGS.items()}


LENGTHS = {"a": 1, "b": 7, "c": 33, "d": 70, "e": 130}


def requests_for(name, extra=None):
    lens = dict(LENGTHS, **(extra or {}))
    return {rid: random_tokens(n, CONFIGS[name]["vocab"], seed=700 + i) for i, (rid, n) in enumerate(sorted(lens.items()))}


def run_and_check(folder, dtype, t, label, block_size, alone=False, tol16=TOL16, **kw):
    """Replay the trace and compare every row with the plain model."""
    with RouterLog() as log:
        got = replay(folder, dtype, t, block_size=block_size, **kw)
    slack = None
    if dtype == "float32":
        want = plain_logits(folder, t.requests)
    else:      # 16-bit: with the experts the engine chose (requests that were fed in full)
        fed = {rid: toks[:t.fed[rid]] for rid, toks in t.requests.items() if t.fed[rid]}
        chosen = log.by_request(t)
        want = plain_logits_routed_alike(folder, fed, chosen)
        slack = {rid: 8.0 * s.numpy() for rid, s in plain_sensitivity(folder, fed, chosen).items()}
    compare(t, got, want, dtype, label, tol=None if dtype == "float32" else tol16, slack=slack)
    if alone and dtype == "float32":
        compare_with_alone(t, got, folder, dtype, label)
    return got


def check(folders, name, dtype, t, label, **kw):
    return run_and_check(folders[name][dtype], dtype, t, label, BLOCK_SIZE[name], **kw)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_whole_prompts(folders, name, dtype):
    for rid, toks in requests_for(name).items():
        t = Trace({rid: toks})
        t.step([(rid, len(toks))], end=[rid])
        check(folders, name, dtype, t, f"whole {name} {rid}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_prefill_then_token_by_token(folders, name, dtype):
    for rid, toks in requests_for(name).items():
        if len(toks) < 33:
            continue
        t = Trace({rid: toks})
        t.step([(rid, len(toks) - 30)], want="last")
        for _ in range(30):
            t.step([(rid, 1)])
        check(folders, name, dtype, t, f"decode {name} {rid}", alone=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_every_token_alone_from_the_first(folders, name, dtype):
    toks = requests_for(name)["d"]
    t = Trace({"d": toks})
    for _ in toks:
        t.step([("d", 1)])
    check(folders, name, dtype, t, f"one by one {name}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_portions_down_to_two_tokens(folders, name, dtype):
    sizes = [7, 2, 5, 3, 16, 2, 31, 4, 2, 9]
    for rid, toks in requests_for(name).items():
        if len(toks) < 9:
            continue
        t = Trace({rid: toks})
        left, i = len(toks), 0
        while left:
            n = min(sizes[i % len(sizes)], left)
            if left - n == 1:
                n += 1
            t.step([(rid, n)])
            left -= n
            i += 1
        check(folders, name, dtype, t, f"portions {name} {rid}", alone=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_mixed_batches_with_pages_used_again(folders, name, dtype):
    reqs = requests_for(name, {"f": 90, "g": 12, "h": 50})
    t = Trace(reqs)
    t.step([("d", 40), ("a", 1)], end=["a"])
    t.step([("d", 2), ("b", 4), ("c", 20)])
    t.step([("d", 1), ("b", 1), ("c", 2), ("e", 30)])
    t.step([("b", 1), ("c", 1), ("e", 7)])                              # d sits this one out
    t.step([("d", 27), ("b", 1), ("c", 10)], end=["b", "c"])
    t.step([("e", 1), ("f", 64), ("g", 3)], end=["d"])                  # f and g take the pages of b and c
    t.step([("e", 2), ("f", 1), ("g", 2), ("h", 33)])
    for _ in range(5):
        t.step([("e", 1), ("f", 1), ("g", 1), ("h", 1)])
    t.step([("e", 85), ("f", 20), ("g", 2), ("h", 12)], end=["e", "f", "g", "h"])
    total = sum(64 * -(-len(v) // 64) for v in reqs.values())
    assert t.max_tokens < total, "the pool is meant to be too small for all requests at once"
    check(folders, name, dtype, t, f"mixed {name}", alone=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_random_schedules(folders, name, dtype):
    for seed in range(4):
        rng = random.Random(31 * seed + ord(name))
        reqs, t = random_trace(rng, CONFIGS[name]["vocab"], 150)
        check(folders, name, dtype, t, f"random schedule {name} {seed}", alone=True)


@pytest.mark.parametrize("name", ["A", "C"])
def test_long_decoding(folders, name):
    """400 tokens: most as portions that end inside pages, windows and chunks, the last 150 one by one: every
    window and chunk passes over decoded tokens several times."""
    toks = random_tokens(400, CONFIGS[name]["vocab"], seed=1)
    t = Trace({"x": toks})
    t.step([("x", 131)], want="last")
    t.step([("x", 119)], want="last")
    for _ in range(150):
        t.step([("x", 1)])
    check(folders, name, "float32", t, "long decoding")


def test_pages_behind_windows_and_chunks_are_used_again(tmp_path):
    """A model whose layers all forget: 500 tokens of one request run on pools of a few pages, portions and
    single tokens, and the pages come back with every window and chunk passed."""
    cfg = config(90, 64, [latent(2, 16, 16, 16, 32, 32, window=20, mlp=dense(64)), pairs(4, 2, 16, 32, chunk=24),
                          latent(3, 8, 16, 12, 24, 32, window=37, kv_from=0)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=6, dtype="float32")
    toks = random_tokens(500, 90, seed=8)
    t = Trace({"x": toks})
    left, i = 500, 0
    while left > 60:
        n = (9, 2, 14, 5, 1, 20)[i % 6]
        t.step([("x", n)])
        left, i = left - n, i + 1
    for _ in range(left):
        t.step([("x", 1)])
    run_and_check(folder, "float32", t, "few pages", 8, cache_groups=[(9, 8), (8, 8)], max_model_len=512)


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_in_several_partitions(tmp_path, dtype):
    """1,300 tokens through attention on the matrix cores and row by row, without masks and with long ones, with
    scales large enough that a query's weight lies on a few keys anywhere before it; portions that end
    inside pages and tiles, then single tokens."""
    cfg = config(211, 96, [latent(4, 32, 16, 32, 40, 64, scale=0.5, mlp=moe(6, 2, 48, 32)),
                           pairs(4, 2, 32, 64, scale=0.5, chunk=900, mlp=dense(80)),
                           latent(2, 24, 10, 40, 20, 36, scale=0.5, base=1e6, window=700),
                           pairs(3, 3, 10, 24, scale=0.6, chunk=640),
                           pairs(2, 1, 16, 32, scale=0.6)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=13, dtype=dtype)
    toks = random_tokens(1300, 211, seed=6)
    t = Trace({"x": toks})
    for n in (511, 3, 258, 490):
        t.step([("x", n)], want="last")
    for _ in range(38):
        t.step([("x", 1)])
    run_and_check(folder, dtype, t, "far keys", 16, tol16=dict(rtol=0.0, atol=2e-2, median=4e-2))


# One token is made to stand out: a feature that no other token has is what its key consists of, and what its
# value carries to the logits.  Which positions it can be seen from is then read off the logits.
def _marked_latent(ts, rot):
    """Token 96 alone has a large last feature; the latent's first value is that feature, every query asks for it."""
    e = ts["embed"]
    e[:, -1], e[:, -2] = 0.0, 3.0          # a constant the queries are made of
    e[96] *= 0.1
    e[96, -1], e[96, -2] = 8.0, 3.0
    for n in ("l0.norm1", "l0.norm2"):
        if n in ts:
            ts[n].zero_()
    ts["l0.mix.dkv"][0] = 0.0
    ts["l0.mix.dkv"][0, -1] = 20.0
    ts["l0.mix.dq"][0] = 0.0
    ts["l0.mix.dq"][0, -2] = 20.0
    ts["l0.mix.uq"] *= 0.05
    ts["l0.mix.uq"][:, 0] = 0.5
    ts["l0.mix.uk"] *= 0.1
    ts["l0.mix.uk"][:, 0] = 0.5


def _marked_pairs(ts):
    """The same for a head's first map; its second map is left flat."""
    e = ts["embed"]
    e[:, -1], e[:, -2] = 0.0, 3.0
    e[96] *= 0.1
    e[96, -1], e[96, -2] = 8.0, 3.0
    ts["l0.norm1"].zero_()
    dim = ts["l0.mix.q.norm"].numel()
    for n in ("q", "k"):
        ts[f"l0.mix.{n}.norm"].fill_(1.0)
        w = ts[f"l0.mix.{n}"].view(-1, 2, dim, e.shape[1])
        w *= 0.02
        w[:, 0, dim - 1, -2 if n == "q" else -1] = 10.0     # the last value of a map does not turn


def seen_from(folder, toks, mark_at, run):
    """Positions (after the mark) whose logits move when the token at ``mark_at`` is replaced by another marked one."""
    out = []
    for other in (False, True):
        seq = list(toks)
        seq[mark_at] = 96 if other else 95
        out.append(run(seq))
    moved = np.abs(out[0] - out[1]).max(-1) / np.abs(out[0]).max()
    return moved


@pytest.mark.parametrize("sizes", [(64, 16), (36, 8)])       # matrix cores, row by row
@pytest.mark.parametrize("window", [1, 2, 16, 33, 64, 100])
def test_the_edge_of_a_window(tmp_path, window, sizes):
    """A key is seen up to window - 1 positions later and not one further, in a prompt and decoded alone, at page
    borders and elsewhere."""
    kv, rot = sizes
    cfg = config(97, 64, [latent(2, 16, rot, 16, 24, kv, scale=1.0, base=1e5, window=window)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=4, dtype="float32")
    edit(folder, lambda ts: _marked_latent(ts, rot))
    toks = random_tokens(260, 95, seed=2)

    def whole(seq):
        t = Trace({"x": seq})
        t.step([("x", len(seq))])
        return run_and_check(folder, "float32", t, "whole", 16)[0]

    def in_steps(seq):
        t = Trace({"x": seq})
        t.step([("x", 80)])
        t.step([("x", 37)])
        while t.fed["x"] < len(seq):
            t.step([("x", 1)])
        got = run_and_check(folder, "float32", t, "in steps", 16)
        return np.concatenate([got[s] for s in sorted(got)])

    for at in (0, 15, 16, 70, 112):
        for run in (whole, in_steps):
            moved = seen_from(folder, toks, at, run)
            last = at + window - 1
            assert (moved[:at] == 0).all() and (moved[last + 1:] == 0).all(), f"mark at {at}: seen where it must not be"
            assert moved[last] > 1e-3, f"mark at {at}: not seen from {last}, the window's last position"


@pytest.mark.parametrize("sizes", [(32, 64), (10, 24)])
@pytest.mark.parametrize("chunk", [1, 7, 16, 50, 64])
def test_the_edge_of_a_chunk(tmp_path, chunk, sizes):
    """A key is seen from the rest of its chunk and from no position of the next, in a prompt, in portions cut inside
    chunks, and decoded alone."""
    dim, vdim = sizes
    cfg = config(97, 64, [pairs(4, 2, dim, vdim, scale=1.0, chunk=chunk, dims=dim - 2, diff=0.3)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=5, dtype="float32")
    edit(folder, _marked_pairs)
    toks = random_tokens(260, 95, seed=3)

    def whole(seq):
        t = Trace({"x": seq})
        t.step([("x", len(seq))])
        return run_and_check(folder, "float32", t, "whole", 16)[0]

    def in_steps(seq):
        t = Trace({"x": seq})
        t.step([("x", 61)])
        t.step([("x", 2)])
        t.step([("x", 57)])
        while t.fed["x"] < len(seq):
            t.step([("x", 1)])
        got = run_and_check(folder, "float32", t, "in steps", 16)
        return np.concatenate([got[s] for s in sorted(got)])

    for at in (0, chunk - 1, chunk, 66, 3 * chunk + chunk // 2):
        for run in (whole, in_steps):
            moved = seen_from(folder, toks, at, run)
            last = at // chunk * chunk + chunk - 1
            assert (moved[:at] == 0).all() and (moved[last + 1:] == 0).all(), f"mark at {at}: seen where it must not be"
            assert moved[last] > 1e-3, f"mark at {at}: not seen from {last}, the chunk's last position"


@pytest.mark.parametrize("windows", [(12, 40), (40, 12), (12, None), (None, 12), (20, 20)])
@pytest.mark.parametrize("kv", [32, 28])
def test_a_reader_sees_the_sources_latents_within_its_own_window(tmp_path, windows, kv):
    """The source's window decides nothing about the reader's: the pages are kept for the wider of the two."""
    rot = 16
    own, reader = windows
    cfg = config(97, 64, [latent(2, 16, rot, 16, 24, kv, window=own, mlp=dense(64)),
                          latent(3, 8, rot, 12, 20, kv, window=reader, kv_from=0, scale=0.8, mlp=moe(4, 2, 24)),
                          latent(1, 12, rot, 20, 16, kv, window=reader, kv_from=0)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=9, dtype="float32")
    reqs = {"x": random_tokens(120, 97, seed=1), "y": random_tokens(50, 97, seed=2)}
    t = Trace(reqs)
    t.step([("x", 55)])
    t.step([("x", 2), ("y", 30)])
    for _ in range(20):
        t.step([("x", 1), ("y", 1)])
    t.step([("x", 43)], end=["x", "y"])
    run_and_check(folder, "float32", t, f"windows {windows}", 8, alone=True)


@pytest.mark.parametrize("name", ["A", "C"])
def test_what_a_position_depends_on(folders, name):
    """Changing one token changes the logits from its position on and, bit for bit, nothing before."""
    toks = random_tokens(120, CONFIGS[name]["vocab"], seed=5)
    other = list(toks)
    other[50] = (toks[50] + 1) % CONFIGS[name]["vocab"]
    outs = []
    for seq in (toks, other):
        t = Trace({"x": seq})
        t.step([("x", 45)])
        t.step([("x", 30)])
        for _ in range(45):
            t.step([("x", 1)])
        got = replay(folders[name]["float32"], "float32", t, block_size=BLOCK_SIZE[name])
        outs.append(np.concatenate([got[s] for s in sorted(got)]))
    moved = np.abs(outs[0] - outs[1]).max(-1)
    assert (moved[:50] == 0.0).all() and moved[50] > 1e-5 and (moved[50:58] > 1e-6).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_second_maps_that_take_off_nearly_all_or_nothing(tmp_path, dtype):
    """lambda near one, at zero and below: the sums of both maps nearly cancel where they look at the same keys (the
    norm then blows up what is left), or the second map does not count."""
    for n, (lq1, lq2, diff) in enumerate(((0.0, 0.0, 0.95), (-2.0, 0.0, 0.6), (1.0, 2.0, 0.1), (0.0, 0.0, 0.02))):
        cfg = config(131, 64, [pairs(4, 2, 16, 32, chunk=40, diff=diff, mlp=dense(64)), pairs(3, 1, 6, 10, diff=diff)])
        folder = write_model(str(tmp_path / f"m{n}"), cfg, seed=17, dtype=dtype)

        def change(ts):
            for i in (0, 1):
                for a, v in (("lq1", lq1), ("lq2", lq2)):
                    t = ts[f"l{i}.mix.{a}"]
                    t.zero_()
                    t[0] = v
                    ts[f"l{i}.mix.{a.replace('q', 'k')}"].fill_(1.0)
        edit(folder, change)
        toks = random_tokens(90, 131, seed=9)
        t = Trace({"x": toks})
        t.step([("x", 51)])
        t.step([("x", 2)])
        for _ in range(37):
            t.step([("x", 1)])
        run_and_check(folder, dtype, t, f"take off {n}", 8, tol16=dict(rtol=0.0, atol=2e-2, median=4e-2))


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_given_shape_of_things_is_not_assumed(tmp_path, dtype):
    """Sizes that are equal, or 1, in one model and not in another: one head and many, value heads wider and narrower
    than the keys, a latent wider than the stream, one expert, all experts at once, a window and a chunk of one
    position, a rotation of two values, a head that is all rotated or not at all, a vocabulary of few ids."""
    cases = [
        [latent(1, 2, 2, 1, 1, 3, window=1, mlp=moe(1, 1, 1, 1)), pairs(1, 1, 2, 1, chunk=1)],
        [latent(7, 4, 6, 10, 5, 90, window=300, mlp=moe(4, 4, 12, 20)), latent(2, 0, 6, 3, 9, 90, kv_from=0, mlp=dense(7)),
         pairs(5, 5, 12, 3, chunk=500)],
        [pairs(9, 1, 4, 30, chunk=13, mlp=dense(200)), latent(3, 5, 0, 9, 16, 16, window=13), latent(1, 40, 4, 40, 40, 40, scale=0.05)],
        [latent(16, 8, 16, 8, 16, 16, window=30, mlp=moe(33, 5, 8)), pairs(32, 2, 16, 16, chunk=30, mlp=moe(2, 1, 60, 30)),
         latent(2, 16, 16, 80, 33, 16, window=5, kv_from=0)],
    ]
    for n, layers in enumerate(cases):
        cfg = config((11, 97, 64, 300)[n], 40, layers, eps=1e-3)
        folder = write_model(str(tmp_path / f"m{n}"), cfg, seed=5 + n, dtype=dtype)
        toks = random_tokens(45, cfg["vocab"], seed=3)
        t = Trace({"x": toks})
        t.step([("x", 20)])
        t.step([("x", 2)])
        for _ in range(23):
            t.step([("x", 1)])
        run_and_check(folder, dtype, t, f"one of everything {n}", 8, tol16=dict(rtol=0.0, atol=2e-2, median=4e-2))


@pytest.mark.parametrize("dtype", DTYPES)
def test_wide_layers_and_steps_of_every_size(tmp_path, dtype):
    """Layers as wide as a small real model's: products of few rows in two chunks, steps of 17 to 64 rows
    (partial sums), of more than 64 rows (the vendor library), experts with few rows and with many."""
    cfg = config(1000, 512, [latent(8, 64, 64, 64, 192, 64, window=120, mlp=dense(1024, 2.0)),
                             pairs(8, 4, 64, 128, chunk=150, mlp=moe(4, 2, 256, 512)),
                             latent(8, 32, 64, 48, 128, 64, window=64, kv_from=0, mlp=moe(8, 3, 128, 128)),
                             pairs(2, 2, 128, 256, chunk=70)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=2, dtype=dtype)
    reqs = {"x": random_tokens(330, 1000, seed=1), "y": random_tokens(60, 1000, seed=2), "z": random_tokens(20, 1000, seed=3)}
    t = Trace(reqs)
    t.step([("x", 200)])
    t.step([("x", 12), ("y", 40)])
    t.step([("x", 100), ("z", 2)])
    for n in (1, 5, 8, 2):
        t.step([("x", n), ("y", 1), ("z", 3)])
    t.step([("x", 2)], end=["x", "y", "z"])
    run_and_check(folder, dtype, t, "wide layers", 16)


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations_under_random_schedules(tmp_path, seed):
    rng = random.Random(5000 + seed)
    cfg = random_config(rng)
    folder = write_model(str(tmp_path / "m"), cfg, seed=seed, dtype="float32")
    reqs, t = random_trace(rng, cfg["vocab"], rng.choice([60, 150, 250]))
    run_and_check(folder, "float32", t, f"random configuration {seed}", rng.choice([4, 8, 16]))


# ------------------------------------------------------------------- generation
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_entry_point(folders, name, dtype):
    import lyapunov_engine_amd as L

    folder = folders[name][dtype]
    prompts = [random_tokens(n, CONFIGS[name]["vocab"], seed=60 + n) for n in (3, 19, 40)]
    llm = L.LLM(folder, dtype=dtype, num_blocks=96, block_size=BLOCK_SIZE[name], max_num_batched_tokens=32)
    outs = llm.generate(prompts, L.SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    for prompt, o in zip(prompts, outs):
        assert o.finished and o.prompt_tokens == prompt and len(o.output_tokens) == 12
        want, margins = plain_greedy(folder, prompt, 12)
        close = [i for i, m in enumerate(margins) if m < (1e-3 if dtype == "float32" else 0.5)]
        upto = close[0] if close else 12
        assert o.output_tokens[:upto] == want[:upto]


def test_generation_with_and_without_recorded_steps_and_with_preemption(folders):
    """Recorded steps run the attention, the router and the norms at the ends of products again and again with other
    tokens, windows and chunks; the same tokens come out as from eager steps and the plain model."""
    import lyapunov_engine_amd as L

    folder = folders["C"]["float32"]
    prompts = [random_tokens(n, CONFIGS["C"]["vocab"], seed=80 + n) for n in (5, 30, 61, 12)]
    sp = L.SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True)
    plain = [plain_greedy(folder, p, 20) for p in prompts]
    for kw in (dict(enable_graphs=True, num_blocks=64), dict(enable_graphs=False, num_blocks=64),
               dict(enable_graphs=True, num_blocks=12, max_num_batched_tokens=24)):   # few pages: preemption
        outs = L.LLM(folder, dtype="float32", block_size=16, max_model_len=96, **kw).generate(prompts, sp)
        for o, (want, margins) in zip(outs, plain):
            upto = next((i for i, m in enumerate(margins) if m < 1e-4), 20)
            assert o.output_tokens[:upto] == want[:upto], kw


def test_recorded_steps_give_the_logits_of_eager_ones(folders):
    """The same decode steps through a recorded graph, replayed with other tokens, contexts and batch
    sizes (padded rows too), and through the eager step, across the ends of chunks."""
    from lyapunov_engine_amd.engine.core import EngineCore, StepEntry
    from lyapunov_engine_amd.engine.graphs import StepGraphs

    for name in ("A", "B", "C"):
        V = CONFIGS[name]["vocab"]
        core = EngineCore.from_folder(folders[name]["float32"], dtype="float32", device="cuda:0", num_blocks=128,
                                      block_size=BLOCK_SIZE[name], num_state_slots=4, max_model_len=128)
        graphs = StepGraphs(core.runner, max_batch=4)
        toks = {s: random_tokens(60, V, seed=90 + s) for s in range(3)}
        for s in toks:
            core.cache.add(s)
            core.cache.extend(s, 17 + s)
            core.step([StepEntry(s, toks[s][:17 + s], 0, [])])
            core.cache.commit(s, 17 + s)
        for i in range(12):
            live = list(toks)[:1 + i % 3]
            entries = []
            for s in live:
                at = core.cache.length(s)
                core.cache.extend(s, at + 1)
                entries.append(StepEntry(s, [toks[s][at]], at, [0]))
            eager = core.step(entries).float().cpu()
            recorded = graphs.step(entries).float().cpu()       # the same slots are written once more with the same values
            for s, e in zip(live, entries):
                core.cache.commit(s, e.start + 1)
            scale = max(1.0, float(eager.abs().max()))
            assert float((eager - recorded).abs().max()) < 2e-5 * scale, f"{name}, step {i}"


def test_command_line_generate(folders):
    folder = folders["A"]["float32"]
    prompt = random_tokens(9, CONFIGS["A"]["vocab"], seed=8)
    want, _ = plain_greedy(folder, prompt, 8)
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "lyapunov"), "generate", "--model", folder,
                           "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "8", "--temperature", "0",
                           "--dtype", "float32", "--block-size", "4", "--num-blocks", "32"],
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert proc.stdout.strip().splitlines()[-1].split() == [str(t) for t in want]


def test_trace_runner_as_a_program(folders, tmp_path):
    folder = folders["A"]["float32"]
    toks = random_tokens(30, CONFIGS["A"]["vocab"], seed=4)
    steps = [{"step": 0, "entries": [{"id": "r", "tokens": toks[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "r", "tokens": toks[17:18], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "r", "tokens": toks[18:], "want": [11]}], "end": ["r"]}]
    out = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                           "--out", str(out), "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = plain_logits(folder, {"r": toks})["r"].numpy()
    for step, rows in ((0, [0, 16]), (1, [17]), (2, [29])):
        got = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(rows), -1)
        assert np.abs(got - want[rows]).max() < 5e-4 * max(1.0, np.abs(want[rows]).max())
