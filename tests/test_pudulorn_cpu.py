"""Pudulorn without a GPU: the plain mechanisms on cases worked out by hand, the
configuration, the model as built (names, running order, cache groups), and how
pages come back behind windows and chunks."""
import copy
import math
import random

import pytest
import torch

from plain import pudulorn_plain as DP
from pudulorn_util import CONFIGS, config, dense, latent, moe, pairs, random_config, write_model

F = torch.float64


def built(cfg):
    from lyapunov_engine_amd.config.registry import architecture_of
    from lyapunov_engine_amd.models.decoder import build_model

    arch = architecture_of(cfg)
    return build_model(arch.to_spec(arch.config_class.from_dict(cfg)))


# ------------------------------------------------------------ plain mechanisms
def test_norms():
    x = torch.tensor([[3.0, 4.0]], dtype=F)
    r = math.sqrt(12.5 + 0.5)
    assert torch.allclose(DP.unit_rms(x, 0.5), torch.tensor([[3 / r, 4 / r]], dtype=F))
    w = torch.tensor([0.0, -0.5], dtype=F)
    assert torch.allclose(DP.shifted_rms_norm(x, w, 0.5), torch.tensor([[3 / r, 2 / r]], dtype=F))
    assert torch.allclose(DP.rms_norm(x, w, 0.5), torch.tensor([[0.0, -2 / r]], dtype=F))


def test_halves_turn_together():
    v = torch.tensor([[1.0, 2.0, 3.0, 4.0, 5.0]], dtype=F)
    p = torch.tensor([3])
    out = DP.rotate_halves(v, p, 100.0, 4)
    for i, a in ((0, 3.0), (1, 3.0 / 10)):
        assert math.isclose(float(out[0, i]), v[0, i] * math.cos(a) - v[0, i + 2] * math.sin(a))
        assert math.isclose(float(out[0, i + 2]), v[0, i + 2] * math.cos(a) + v[0, i] * math.sin(a))
    assert float(out[0, 4]) == 5.0
    assert torch.equal(DP.rotate_halves(v, torch.tensor([0]), 100.0, 4), v)


def test_who_sees_whom():
    w = DP.window_mask(6, 3)
    assert [w[5].tolist(), w[1].tolist()] == [[False, False, False, True, True, True], [True, True, False, False, False, False]]
    assert DP.window_mask(4, 1).tolist() == torch.eye(4).bool().tolist()
    c = DP.chunk_mask(7, 3)
    assert c[2].tolist() == [True, True, True, False, False, False, False]
    assert c[3].tolist() == [False, False, False, True, False, False, False]
    assert c[5].tolist() == [False, False, False, True, True, True, False]
    assert torch.equal(DP.chunk_mask(5, None), torch.ones(5, 5).tril().bool()) and torch.equal(DP.window_mask(5, 9), DP.chunk_mask(5, 9))


def test_softmax_over_what_is_seen():
    q, k = torch.tensor([[1.0], [1.0], [1.0]], dtype=F), torch.tensor([[2.0], [3.0], [9.0]], dtype=F)
    v = torch.tensor([[10.0], [20.0], [30.0]], dtype=F)
    o = DP.softmax_attention(q, k, v, 0.5, DP.window_mask(3, 2))
    e2, e3, e9 = math.exp(1.0), math.exp(1.5), math.exp(4.5)
    assert [round(float(x), 12) for x in o[:, 0]] == [10.0, round((10 * e2 + 20 * e3) / (e2 + e3), 12),
                                                     round((20 * e3 + 30 * e9) / (e3 + e9), 12)]


def test_one_map_is_taken_off_the_other():
    w = {"lq1": torch.tensor([0.5, 1.0], dtype=F), "lk1": torch.tensor([2.0, -1.0], dtype=F),
         "lq2": torch.tensor([1.0, 0.0], dtype=F), "lk2": torch.tensor([-0.7, 3.0], dtype=F)}
    lam = math.exp(0.0) - math.exp(-0.7) + 0.25
    assert math.isclose(float(DP.take_off(w, 0.25)), lam)
    # one token: every softmax is 1, both sums are the value itself, so o = (1 - lambda) v, normed and gated
    g = torch.Generator().manual_seed(0)
    m = dict(heads=2, kv_heads=1, dim=2, vdim=3, scale=1.0, diff=0.25, rot=dict(base=10.0, dims=2))
    for n, s in (("q", (8, 4)), ("k", (4, 4)), ("v", (3, 4)), ("g", (6, 4)), ("o", (4, 6)), ("q.norm", (2,)), ("k.norm", (2,))):
        w[n] = torch.randn(s, generator=g, dtype=F)
    h = torch.randn(1, 4, generator=g, dtype=F)
    v = (w["v"] @ h[0]) * (1 - lam)
    o = v / torch.sqrt(v.pow(2).mean() + 1e-6) * 0.75
    want = w["o"] @ (torch.cat((o, o)) * torch.sigmoid(w["g"] @ h[0]))
    assert torch.allclose(DP.differential_attention(h, w, m, 1e-6)[0], want)


def test_limits_of_the_gated_feed_forward():
    one = torch.eye(1, dtype=F)
    w = dict(gate=one, up=one.clone(), down=one.clone())
    for x in (-9.0, -1.0, 0.5, 9.0):
        g, u = min(x, 2.0), max(min(x, 2.0), -2.0)
        want = g / (1 + math.exp(-1.702 * g)) * (u + 1)
        assert math.isclose(float(DP.limited_ff(torch.tensor([[x]], dtype=F), w, 2.0)), want, rel_tol=1e-12)


def test_experts_and_their_weights():
    g = torch.Generator().manual_seed(2)
    w = {"router": torch.randn(4, 3, generator=g, dtype=F), "shared.sg": torch.randn(1, 3, generator=g, dtype=F)}
    for e in ["e0", "e1", "e2", "e3", "shared"]:
        for n, s in (("gate", (5, 3)), ("up", (5, 3)), ("down", (3, 5))):
            w[f"{e}.{n}"] = torch.randn(s, generator=g, dtype=F)
    h = torch.randn(2, 3, generator=g, dtype=F)
    got = DP.expert_ff(h, w, dict(router=dict(experts=4, top=2, scale=3.0), shared=dict(ff=5)))
    for t in range(2):
        z = [float(w["router"][e] @ h[t]) for e in range(4)]
        s = [math.exp(x) / sum(math.exp(y) for y in z) for x in z]
        best = sorted(range(4), key=lambda e: -s[e])[:2]
        want = sum(3.0 * s[e] * DP.gated_ff(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])[0] for e in best)
        share = 1 / (1 + math.exp(-float(w["shared.sg"][0] @ h[t])))
        want = want + share * DP.gated_ff(h[t:t + 1], w["shared.gate"], w["shared.up"], w["shared.down"])[0]
        assert torch.allclose(got[t], want)


def test_a_reader_uses_the_sources_latents_and_its_own_everything_else(tmp_path):
    """Changing the source's dkv moves the reader; the reader has no dkv to change; the source's window does not bind it."""
    cfg = config(40, 16, [latent(1, 4, 4, 4, 6, 8, window=2), latent(2, 6, 4, 3, 5, 8, window=5, kv_from=0)])
    folder = write_model(str(tmp_path / "m"), cfg, seed=1, dtype="float32")
    c, w = DP.load_folder(folder)
    toks = [3, 9, 1, 7, 30, 22]
    h = torch.randn(6, 16, generator=torch.Generator().manual_seed(3), dtype=F)
    m0, m1 = c["layers"][0]["mixer"], c["layers"][1]["mixer"]
    kept = DP.latents_of(h, DP.sub(w, "l0.mix."), m0, 1e-6)
    a = DP.latent_attention(h, DP.sub(w, "l1.mix."), m1, 1e-6, kept)
    b = DP.latent_attention(h, DP.sub(w, "l1.mix."), m1, 1e-6, (kept[0] * 2, kept[1]))
    assert not torch.allclose(a, b) and "l1.mix.dkv" not in w and "l1.mix.dkv.norm" not in w
    seen = [(a != DP.latent_attention(h, DP.sub(w, "l1.mix."), m1, 1e-6, (kept[0].index_fill(0, torch.tensor([1]), 5.0), kept[1]))).any(-1)]
    assert seen[0].tolist() == [False, True, True, True, True, True]      # five positions: its own window
    assert DP.forward(toks, w, c).shape == (6, 40)


# --------------------------------------------------------------- configuration
def test_configuration_errors_name_the_missing_key():
    from lyapunov_engine_amd.config import ConfigError, PudulornConfig

    good = CONFIGS["A"]
    assert PudulornConfig.from_dict(PudulornConfig.from_dict(good).to_dict()) == PudulornConfig.from_dict(good)
    for path, key in (((), "width"), ((), "vocab"), (("norm",), "eps"), (("layers", 0, "mixer"), "scale"),
                      (("layers", 0, "mixer"), "kv_rank"), (("layers", 0, "mixer"), "q_rank"), (("layers", 0, "mixer", "rot"), "base"),
                      (("layers", 0, "mixer", "mask"), "size"), (("layers", 1, "mixer"), "diff"), (("layers", 1, "mixer"), "kv_heads"),
                      (("layers", 0, "mlp"), "limit"), (("layers", 1, "mlp", "router"), "scale"),
                      (("layers", 1, "mlp", "expert"), "ff"), (("layers", 1, "mlp", "shared"), "ff"), (("layers", 2), "type")):
        bad = copy.deepcopy(good)
        d = bad
        for p in path:
            d = d[p]
        del d[key]
        with pytest.raises(ConfigError, match=key):
            PudulornConfig.from_dict(bad)
    for change, match in ((lambda d: d["layers"][0].update(type="something"), "something"),
                          (lambda d: d["layers"][0]["mlp"].update(kind="other"), "other"),
                          (lambda d: d["layers"][1]["mlp"]["router"].update(top=6), "6 of 5"),
                          (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=9), "9"),
                          (lambda d: d["layers"][1]["mixer"].update(kv_heads=4), "6 query heads over 4"),
                          (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "size"),
                          (lambda d: d["layers"][0]["mlp"].update(limit=0.0), "limit"),
                          (lambda d: d["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
                          (lambda d: d["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
                          (lambda d: d["layers"][2]["mixer"].update(kv_rank=44), "other sizes"),
                          (lambda d: d["layers"][2]["mixer"]["rot"].update(base=7.0), "another rotation"),
                          (lambda d: d["layers"][5]["mixer"].update(kv_from=2), "own")):
        bad = copy.deepcopy(good)
        change(bad)
        with pytest.raises(ConfigError, match=match):
            PudulornConfig.from_dict(bad)


def test_built_model_names_order_and_groups(tmp_path):
    model = built(CONFIGS["A"])
    names = model.expected_tensors()
    shapes = {n: s for n, (s, _) in names.items()}
    assert shapes["l0.mix.dq"] == (18, 72) and shapes["l0.mix.uq"] == (36, 18) and shapes["l0.mix.dkv"] == (48, 72)
    assert shapes["l2.mix.uk"] == (36, 40) and shapes["l2.mix.uv"] == (60, 40) and shapes["l2.mix.dq.norm"] == (30,)
    assert shapes["l1.mix.q"] == (6 * 2 * 10, 72) and shapes["l1.mix.k"] == (3 * 2 * 10, 72) and shapes["l1.mix.v"] == (78, 72)
    assert shapes["l1.mix.g"] == (6 * 26, 72) and shapes["l1.mix.lq2"] == (10,) and shapes["l1.mix.k.norm"] == (10,)
    assert shapes["l1.mlp.shared.sg"] == (1, 72) and shapes["l2.mlp.shared.up"] == (44, 72) and shapes["l1.mlp.e4.down"] == (72, 28)
    assert shapes["head"] == (203, 72) and shapes["embed"] == (203, 72)
    for absent in ("l2.mix.dkv", "l2.mix.dkv.norm", "l5.mix.dkv", "l3.norm2", "l3.mlp.up", "l0.mix.sink", "l1.mlp.router.b", "l1.mlp.e5.up"):
        assert absent not in names, absent
    assert model.ignorable("l3.norm2")
    assert [(c.layer, c.cache, c.writes) for c in model.schedule] == [
        (0, 0, True), (1, 1, True), (2, 0, False), (3, 3, True), (4, 4, True), (5, 4, False)]
    groups = model.cache_layout().groups
    assert [(g.spec.window, g.spec.chunk, g.spec.keeps_all, g.buffers) for g in groups] == [
        (50, 0, False, (0,)),           # the source's window is 21, its reader's 50
        (0, 24, False, (1,)), (0, 7, False, (3,)),
        (0, 0, True, (4,))]             # the reader of layer 4 sees everything
    assert groups[1].spec.tensors[0].shape == (6, -1, 10) and groups[1].spec.tensors[1].shape == (3, 26, -1)
    folder = write_model(str(tmp_path / "m"), CONFIGS["A"], seed=1, dtype="float32")
    cfg, tensors = DP.load_folder(folder)
    assert set(tensors) == set(names)
    assert DP.forward([1, 2, 3], tensors, cfg).shape == (3, 203)


def test_tensors_are_bound(tmp_path):
    from lyapunov_engine_amd.weights.loader import FolderSource, WeightError, check_tensors, load_weights

    cfg = CONFIGS["A"]
    folder = write_model(str(tmp_path / "m"), cfg, seed=1, dtype="bfloat16")
    model = load_weights(built(cfg), FolderSource(folder), torch.bfloat16, "cpu", max_positions=64)
    _, w = DP.load_folder(folder)
    first, reader, pair = model.layers[0], model.layers[2], model.layers[1]
    assert torch.equal(first.mixer.down_proj.double(), torch.cat([w["l0.mix.dq"], w["l0.mix.dkv"]]))
    assert torch.equal(reader.mixer.down_proj.double(), w["l2.mix.dq"]) and reader.mixer.kv_norm_f is None
    assert torch.equal(reader.mixer.uk_t[1].double(), w["l2.mix.uk"][12:24].T)
    assert torch.equal(pair.mixer.in_proj.double(), torch.cat([w[f"l1.mix.{n}"] for n in "qkvg"]))
    assert math.isclose(pair.mixer.take_off, float(DP.take_off(DP.sub(w, "l1.mix."), 0.25)), rel_tol=1e-12)
    assert torch.equal(first.norm1.multiplier, 1.0 + w["l0.norm1"].float())
    # gates and ups of the dense layer in runs of eight where its width allows (100: it does not, 52: it does not)
    assert torch.equal(first.ffn.gate_up_proj.double(), torch.cat([w["l0.mlp.gate"], w["l0.mlp.up"]])) and first.ffn.interleave == 0
    experts, other = pair.ffn, reader.ffn
    assert torch.equal(experts.router_f.double(), torch.cat([w["l1.mlp.router"], w["l1.mlp.shared.sg"]]))
    # a shared expert of the experts' size is one more matrix behind theirs; another size is kept apart
    assert experts.shared_folded and torch.equal(experts.down[5].double(), w["l1.mlp.shared.down"])
    assert not other.shared_folded and other.shared_down.shape == (72, 44) and other.gate_up.shape[0] == 7
    shapes = {n: tuple(t.shape) for n, t in w.items()}
    check_tensors(built(cfg), shapes)
    for name, shape in (("l1.mix.lq1", (9,)), ("l0.mix.dq", (17, 72)), ("l1.mlp.shared.sg", (72,))):
        with pytest.raises(WeightError, match=name):
            check_tensors(built(cfg), dict(shapes, **{name: shape}))


def test_random_configurations_build():
    for seed in range(40):
        cfg = random_config(random.Random(seed))
        model = built(cfg)
        readers = [c for c in model.schedule if not c.writes]
        assert len(readers) == sum("kv_from" in l["mixer"] for l in cfg["layers"])


def test_random_weights_mode(tmp_path):
    from lyapunov_engine_amd.weights import write_random_model

    write_random_model(dict(CONFIGS["C"]), str(tmp_path / "r"), seed=3, dtype="bfloat16")
    cfg, w = DP.load_folder(str(tmp_path / "r"))
    assert abs(float(w["l0.norm1"].mean())) < 0.1, "norm weights lie around zero"
    assert DP.forward([5, 6], w, cfg).shape == (2, 320)


# ------------------------------------------------------------------- the cache
def test_what_one_buffer_keeps_for_calls_of_different_reach():
    from lyapunov_engine_amd.parts.base import SLOT, PagedSpec, PageTensor

    t, other = (PageTensor("latent", (SLOT, 8)),), (PageTensor("latent", (SLOT, 9)),)
    assert PagedSpec(t, 10).covering(PagedSpec(t, 25)) == PagedSpec(t, 25) == PagedSpec(t, 25).covering(PagedSpec(t, 10))
    assert PagedSpec(t, 10).covering(PagedSpec(t)).keeps_all and PagedSpec(t).covering(PagedSpec(t, chunk=4)).keeps_all
    assert PagedSpec(t, chunk=6).covering(PagedSpec(t, chunk=6)) == PagedSpec(t, chunk=6)
    assert PagedSpec(t, chunk=6).covering(PagedSpec(t, chunk=9)) == PagedSpec(t, 9)
    assert PagedSpec(t, chunk=30).covering(PagedSpec(t, 10, 3)) == PagedSpec(t, 30, 3)
    with pytest.raises(ValueError, match="two contents"):
        PagedSpec(t).covering(PagedSpec(other))
    with pytest.raises(ValueError, match="not both"):
        PagedSpec(t, 4, chunk=4)


def test_pages_behind_a_chunk_come_back():
    from lyapunov_engine_amd.cache.manager import CacheManager, GroupConfig

    m = CacheManager([GroupConfig(8, 4, chunk=6)], 2)
    m.add(0)
    m.extend(0, 5), m.commit(0, 5)
    assert m.table(0) == [0, 1]                  # the next token, 5, is of the first chunk
    m.extend(0, 6), m.commit(0, 6)
    assert m.table(0) == [-1, 1]                 # token 6 begins a chunk; page 1 holds tokens 4 to 7
    m.extend(0, 11), m.commit(0, 11)
    assert m.table(0) == [-1, 1, 2]
    m.extend(0, 12), m.commit(0, 12)
    assert m.table(0) == [-1, -1, -1]            # token 12 begins a chunk at a page's first slot
    m.extend(0, 13), m.commit(0, 13)
    assert m.table(0)[:3] == [-1, -1, -1] and m.table(0)[3] >= 0 and m.num_free_pages(0) == 7
    m.check()
    for bad in (GroupConfig(4, 4, window=3, chunk=3), GroupConfig(4, 4, chunk=-1)):
        with pytest.raises(Exception):
            CacheManager([bad], 1)


@pytest.mark.parametrize("seed", range(4))
def test_random_growth_with_chunks_keeps_what_is_seen(seed):
    """Whatever the portions, every token that a later one can see has its page, and no other whole page is held."""
    from lyapunov_engine_amd.cache.manager import CacheManager, GroupConfig

    rng = random.Random(seed)
    page, chunk = rng.choice([1, 2, 4, 16]), rng.choice([1, 3, 8, 17, 40])
    m = CacheManager([GroupConfig(200, page, chunk=chunk)], 1)
    m.add(0)
    n = 0
    while n < 150:
        n += rng.randint(1, 12)
        m.extend(0, n)
        m.commit(0, n)
        table, lo = m.table(0), n - n % chunk
        for i, p in enumerate(table):
            assert (p >= 0) == ((i + 1) * page > lo), (n, i, table)
        m.check()
    m.free(0)
    assert m.num_free_pages(0) == 200


def test_position_reach_of_a_model_that_forgets():
    from lyapunov_engine_amd.engine.core import EngineCore

    some = built(config(50, 16, [latent(1, 4, 4, 4, 4, 8, window=6), pairs(1, 1, 4, 4, chunk=9)]))
    assert EngineCore.reach(some, 4, 8, None, 500) == 500, "windows and chunks bind no request's length"
    keeps = built(config(50, 16, [latent(1, 4, 4, 4, 4, 8, window=6), pairs(1, 1, 4, 4)]))
    assert EngineCore.reach(keeps, 4, 8, None, 500) == 32


def test_bounds_of_what_is_seen():
    from lyapunov_engine_amd.kernels import ops

    for window, chunk in ((0, 0), (10, 0), (0, 10), (1, 0), (0, 1), (0, 32)):
        for tokens in (1, 64):
            most = 0
            for first in range(0, 150):
                last = first + tokens - 1
                lo = max(0, first - window + 1) if window else (first - first % chunk if chunk else 0)
                most = max(most, last + 1 - lo // 16 * 16)
            assert most <= ops.visible_keys(149 + tokens, window, chunk, tokens)
    assert ops.visible_keys(7, 100, 0) == 7
    assert ops.paired_attn_fits_matrix_cores(48, 80) and not ops.paired_attn_fits_matrix_cores(40, 80)
    assert not ops.paired_attn_fits_matrix_cores(144, 80) and not ops.paired_attn_fits_matrix_cores(64, 272)
