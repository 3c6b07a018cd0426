"""Panodra without a GPU: the plain implementation pinned on cases worked out by
hand, the stretched rotation's table, configuration errors, and the built
model's tensor names, running order, cache groups and random weights."""
import copy
import math

import pytest
import torch

from panodra_util import CONFIGS, config, dense, latent, moe, write_model
from plain import panodra_plain as PP

F = torch.float64


def built(cfg):
    from lyapunov_engine_amd.config.registry import architecture_of
    from lyapunov_engine_amd.models.decoder import build_model

    arch = architecture_of(cfg)
    return build_model(arch.to_spec(arch.config_class.from_dict(cfg)))


# ------------------------------------------------------- the plain mechanisms
def test_the_norm_bends_every_feature_by_itself():
    x = torch.tensor([[0.5, -2.0]], dtype=F)
    y = PP.tanh_norm(x, torch.tensor(3.0, dtype=F), torch.tensor([2.0, 1.0], dtype=F), torch.tensor([0.1, -0.2], dtype=F))
    assert torch.allclose(y, torch.tensor([[2 * math.tanh(1.5) + 0.1, math.tanh(-6.0) - 0.2]], dtype=F))
    other = PP.tanh_norm(torch.tensor([[0.5, 77.0]], dtype=F), torch.tensor(3.0, dtype=F), torch.tensor([2.0, 1.0], dtype=F),
                         torch.tensor([0.1, -0.2], dtype=F))
    assert other[0, 0] == y[0, 0], "a feature does not depend on its neighbours"


def test_latent_norm_has_eps_inside_the_root():
    x = torch.tensor([[3.0, 4.0]], dtype=F)
    assert math.isclose(float(PP.rms_norm(x, torch.ones(2, dtype=F), 3.5)[0, 0]), 3 / 4.0)


def test_activations():
    z = torch.tensor([-2.0, 0.0, 3.0], dtype=F)
    assert PP.squared_relu(z).tolist() == [0.0, 0.0, 9.0]
    assert torch.allclose(PP.silu(z), torch.tensor([-2 / (1 + math.exp(2.0)), 0.0, 3 / (1 + math.exp(-3.0))], dtype=F))


def test_pair_rotation_by_hand_and_by_distance():
    v = torch.tensor([[1.0, 2.0, 3.0, 4.0, 9.0]], dtype=F)
    rot = dict(base=100.0, dims=4)
    a0, a1 = 3 * 1.0, 3 * 100.0 ** -0.5
    got = PP.rotate_pairs(v, torch.tensor([3]), rot)[0]
    want = [1 * math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + 1 * math.sin(a0),
            3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1), 9.0]
    assert torch.allclose(got, torch.tensor(want, dtype=F))
    g = torch.Generator().manual_seed(1)
    q, k = torch.randn(1, 8, generator=g, dtype=F), torch.randn(1, 8, generator=g, dtype=F)
    rot = dict(base=50.0, dims=8, scaling=dict(factor=4.0, original=32, fast=4.0, slow=1.0))
    dot = lambda a, b: float((PP.rotate_pairs(q, torch.tensor([a]), rot) * PP.rotate_pairs(k, torch.tensor([b]), rot)).sum())
    assert math.isclose(dot(9, 4), dot(105, 100), rel_tol=1e-9)
    assert not math.isclose(dot(9, 4), dot(9, 5), rel_tol=1e-3)


def test_stretched_frequencies_by_hand():
    """16 dimensions, base 10^4, 1,000 positions: the pair that turns 16 times has number
    16 ln(1000 / (32 pi)) / (2 ln 10^4) = 1.9953..., the one that turns twice 3.8014...: pairs 0 and 1
    keep their frequency, pairs from 4 on are divided, 2 and 3 lie a third and two thirds between."""
    sc = dict(factor=5.0, original=1000, fast=16.0, slow=2.0)
    plain = [10000.0 ** (-2 * i / 16) for i in range(8)]
    got = PP.stretched_frequencies(10000.0, 16, sc)
    share = [0.0, 0.0, 1 / 3, 2 / 3, 1.0, 1.0, 1.0, 1.0]
    assert math.floor(16 * math.log(1000 / (2 * math.pi * 16)) / (2 * math.log(1e4))) == 1
    assert math.ceil(16 * math.log(1000 / (2 * math.pi * 2)) / (2 * math.log(1e4))) == 4
    for f, p, s in zip(got, plain, share):
        assert math.isclose(f, p / 5 * s + p * (1 - s), rel_tol=1e-12)
    assert math.isclose(PP.rotation_gain(sc), 0.1 * math.log(5.0) + 1.0) and PP.rotation_gain(None) == 1.0


@pytest.mark.parametrize("case", [
    dict(dims=16, base=10000.0, sc=dict(factor=5.0, original=1000, fast=16.0, slow=2.0)),
    dict(dims=64, base=500000.0, sc=dict(factor=8.0, original=4096, fast=32.0, slow=1.0)),
    dict(dims=10, base=100.0, sc=dict(factor=3.0, original=40, fast=6.0, slow=0.5)),
    dict(dims=6, base=1000.0, sc=dict(factor=2.0, original=20, fast=32.0, slow=16.0)),   # both borders cut off at 0
    dict(dims=4, base=10.0, sc=dict(factor=7.0, original=100000, fast=1.0, slow=0.01)),  # the upper one at dims - 1
    dict(dims=2, base=50.0, sc=dict(factor=1.0, original=64, fast=8.0, slow=1.0)),       # nothing to stretch: gain 1
])
def test_the_position_table_follows_the_stretch(case):
    from lyapunov_engine_amd.parts.rope import RotaryEncoding

    dims, sc = case["dims"], case["sc"]
    enc = RotaryEncoding(dims, case["base"], 5000, scaling=dict(sc, rope_type="yarn"), precise=True)
    table = enc.build_table()
    assert table.shape == (5000, dims)
    freq = PP.stretched_frequencies(case["base"], dims, sc)
    gain = PP.rotation_gain(sc)
    for pos in (0, 1, 7, 333, 4999):
        for i in range(dims // 2):
            assert abs(float(table[pos, i]) - gain * math.cos(pos * freq[i])) < 1e-6
            assert abs(float(table[pos, dims // 2 + i]) - gain * math.sin(pos * freq[i])) < 1e-6
    # without the 64-bit table the scaling is refused rather than left out
    with pytest.raises(ValueError):
        RotaryEncoding(dims, case["base"], 16, scaling=dict(sc, rope_type="yarn")).build_table()


def test_softmax_with_and_without_a_sink():
    q = torch.tensor([[[1.0]], [[1.0]]], dtype=F)
    k = torch.tensor([[[2.0]], [[3.0]]], dtype=F)
    v = torch.tensor([[[10.0]], [[20.0]]], dtype=F)
    e2, e3, es = math.exp(1.0), math.exp(1.5), math.exp(0.7)
    o = PP.causal_softmax_attention(q, k, v, 0.5, torch.tensor([0.7], dtype=F))
    assert math.isclose(float(o[0, 0, 0]), 10 * e2 / (e2 + es))
    assert math.isclose(float(o[1, 0, 0]), (10 * e2 + 20 * e3) / (e2 + e3 + es))
    o = PP.causal_softmax_attention(q, k, v, 0.5, None)
    assert math.isclose(float(o[0, 0, 0]), 10.0) and math.isclose(float(o[1, 0, 0]), (10 * e2 + 20 * e3) / (e2 + e3))


def test_experts_by_the_table():
    g = torch.Generator().manual_seed(2)
    w = {"table": torch.tensor([[0, 2], [2, 1], [1, 0]], dtype=torch.int32)}
    for e in range(3):
        for n, s in (("gate", (4, 3)), ("up", (4, 3)), ("down", (3, 4))):
            w[f"e{e}.{n}"] = torch.randn(s, generator=g, dtype=F)
    h = torch.randn(4, 3, generator=g, dtype=F)
    got = PP.table_experts(h, [1, 1, 0, 2], w)
    for t, pair in enumerate(((2, 1), (2, 1), (0, 2), (1, 0))):
        want = sum(0.5 * (PP.silu(h[t] @ w[f"e{e}.gate"].T) * (h[t] @ w[f"e{e}.up"].T)) @ w[f"e{e}.down"].T for e in pair)
        assert torch.allclose(got[t], want)


def test_a_pass_begins_with_the_stream_beside_the_embedding():
    x, x0 = torch.tensor([[1.0, 2.0]], dtype=F), torch.tensor([[10.0, 20.0]], dtype=F)
    w = torch.tensor([[1.0, 0.0, 0.0, 1.0], [0.0, 3.0, 0.5, 0.0]], dtype=F)
    assert PP.enter_pass(x, x0, w).tolist() == [[21.0, 11.0]]
    assert PP.layer_order(4, dict(start=1, stop=3, times=2)) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert PP.layer_order(2, None) == [(0, False), (1, False)]


def test_logits_are_scaled_and_then_capped():
    table = torch.tensor([[1.0, 0.0], [0.0, 100.0]], dtype=F)
    z = PP.capped_logits(torch.tensor([[2.0, 3.0]], dtype=F), table, 0.5, 4.0)
    assert torch.allclose(z, torch.tensor([[4 * math.tanh(1.0 / 4), 4 * math.tanh(150.0 / 4)]], dtype=F))


# ------------------------------------------------------------- configuration
def test_configuration_errors_name_the_missing_key():
    from lyapunov_engine_amd.config import ConfigError, PanodraConfig

    good = CONFIGS["A"]
    assert PanodraConfig.from_dict(PanodraConfig.from_dict(good).to_dict()) == PanodraConfig.from_dict(good)
    for path, key in (((), "width"), ((), "vocab"), (("norm",), "eps"), (("loop",), "times"), (("layers", 0, "mixer"), "scale"),
                      (("layers", 0, "mixer"), "kv_rank"), (("layers", 0, "mixer", "rot"), "base"),
                      (("layers", 0, "mixer", "rot", "scaling"), "original"), (("layers", 0, "mlp"), "ff"),
                      (("layers", 1, "mlp", "router"), "top"), (("layers", 1, "mlp", "expert"), "ff"), (("layers", 2), "type")):
        bad = copy.deepcopy(good)
        d = bad
        for p in path:
            d = d[p]
        del d[key]
        with pytest.raises(ConfigError, match=key):
            PanodraConfig.from_dict(bad)
    for change, match in ((lambda d: d["layers"][0].update(type="something"), "something"),
                          (lambda d: d["layers"][0]["mlp"].update(kind="other"), "other"),
                          (lambda d: d["layers"][1]["mlp"]["router"].update(top=6), "6 of 5"),
                          (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=9), "9"),
                          (lambda d: d["loop"].update(stop=9), "loop"), (lambda d: d.update(logit_softcap=-1.0), "softcap")):
        bad = copy.deepcopy(good)
        change(bad)
        with pytest.raises(ConfigError, match=match):
            PanodraConfig.from_dict(bad)


def test_optional_constants_may_be_absent():
    model = built(config(50, 16, [latent(1, 4, 4, 4, 8)], scale=None, cap=None))
    assert model.head.scale == 1.0 and model.head.cap == 0.0 and model.stream_entry is None
    names = set(model.expected_tensors())
    assert "loop.in" not in names and "l0.norm2" not in names and model.ignorable("l0.norm2.alpha")


# ------------------------------------------------------------------ the model
def test_built_model_names_order_and_groups(tmp_path):
    model = built(CONFIGS["A"])
    names = model.expected_tensors()
    shapes = {n: s for n, (s, _) in names.items()}
    assert shapes["loop.in"] == (72, 144) and shapes["l0.norm1.alpha"] == () and shapes["final.norm.b"] == (72,)
    assert shapes["l0.mix.q"] == (2 * 18, 72) and shapes["l0.mix.dkv"] == (48, 72) and shapes["l0.mix.sink"] == (2,)
    assert shapes["l1.mix.uk"] == (36, 24) and shapes["l1.mix.uv"] == (60, 24) and shapes["l1.mix.o"] == (72, 60)
    assert shapes["l1.mlp.table"] == (203, 2) and shapes["l1.mlp.e4.down"] == (72, 28) and shapes["l0.mlp.up"] == (100, 72)
    for absent in ("l1.mix.sink", "l3.norm2", "l3.mlp.up", "head", "l1.mlp.e5.up", "l1.mlp.router", "l0.mix.dq"):
        assert absent not in names, absent
    assert [(c.layer, c.cache, c.enter) for c in model.schedule] == [
        (0, 0, False), (1, 1, True), (2, 2, False), (1, 3, True), (2, 4, False), (1, 5, True), (2, 6, False), (3, 7, False)]
    layout = model.cache_layout()
    assert [(g.spec.tensors[0].shape, g.buffers) for g in layout.groups] == [
        ((-1, 48), (0,)), ((-1, 38), (1, 3, 5)), ((-1, 46), (2, 4, 6)), ((-1, 34), (7,))]
    assert not layout.states and not layout.part_states
    # layers whose tables are alike in size are sorted together; these two differ in their numbers of experts
    assert [len(g) for g in model._step_groups] == [1, 1]
    c = built(config(90, 32, [latent(1, 8, 8, 8, 16, mlp=moe(6, 2, 8)), latent(1, 8, 8, 8, 16, mlp=dense(8)),
                              latent(1, 8, 8, 8, 16, sink=False, mlp=moe(6, 2, 24))], loop=(0, 3, 2)))
    assert [len(g) for g in c._step_groups] == [2]
    folder = write_model(str(tmp_path / "m"), CONFIGS["A"], seed=1, dtype="float32")
    cfg, tensors = PP.load_folder(folder)
    assert set(tensors) == set(names)
    assert PP.forward([1, 2, 3], tensors, cfg).shape == (3, 203)


def test_tensors_are_bound_and_a_bad_table_is_refused(tmp_path):
    from lyapunov_engine_amd.weights.loader import DictSource, FolderSource, WeightError, check_tensors, load_weights

    cfg = CONFIGS["A"]
    folder = write_model(str(tmp_path / "m"), cfg, seed=1, dtype="bfloat16")
    model = load_weights(built(cfg), FolderSource(folder), torch.bfloat16, "cpu", max_positions=64)
    _, w = PP.load_folder(folder)
    assert torch.equal(model.stream_entry.stream_half.double(), w["loop.in"][:, :72])
    assert torch.equal(model.stream_entry.first_half.double(), w["loop.in"][:, 72:])
    mix = model.layers[0].mixer
    assert torch.equal(mix.down_proj.double(), torch.cat([w["l0.mix.q"], w["l0.mix.dkv"]]))
    assert torch.equal(mix.uk_t[1].double(), w["l0.mix.uk"][10:20].T) and torch.equal(mix.sink_f.double(), w["l0.mix.sink"])
    assert model.layers[1].mixer.sink_f is None and model.layers[0].norm1.map.alpha == float(w["l0.norm1.alpha"])
    experts = model.layers[1].ffn
    assert experts.table.dtype == torch.int32 and torch.equal(experts.gate_up[3].double(), torch.cat([w["l1.mlp.e3.gate"], w["l1.mlp.e3.up"]]))
    tensors = {n: (t if not t.is_floating_point() else t.float()) for n, t in w.items()}
    tensors["l1.mlp.table"] = tensors["l1.mlp.table"].clone()
    tensors["l1.mlp.table"][7, 1] = 5
    with pytest.raises(ValueError, match="5"):
        load_weights(built(cfg), DictSource(tensors), torch.float32, "cpu", max_positions=64)
    shapes = {n: tuple(t.shape) for n, t in w.items()}
    check_tensors(built(cfg), shapes)
    for name, shape in (("loop.in", (72, 143)), ("l0.norm1.alpha", (1,)), ("l1.mlp.table", (203, 3))):
        with pytest.raises(WeightError, match=name):
            check_tensors(built(cfg), dict(shapes, **{name: shape}))


def test_random_weights_mode_writes_tables(tmp_path):
    from lyapunov_engine_amd.weights import write_random_model

    write_random_model(dict(CONFIGS["C"]), str(tmp_path / "r"), seed=3, dtype="bfloat16")
    cfg, w = PP.load_folder(str(tmp_path / "r"))
    t = w["l0.mlp.table"]
    assert t.dtype == torch.int32 and t.shape == (320, 3) and int(t.min()) == 0 and int(t.max()) == 11
    assert all(len(set(row)) == 3 for row in t.tolist()), "a row's experts differ"
    assert PP.forward([5, 6], w, cfg).shape == (2, 320)


def test_a_call_that_enters_needs_an_entry():
    from lyapunov_engine_amd.config import LayerCall
    from lyapunov_engine_amd.config.registry import architecture_of
    from lyapunov_engine_amd.models.decoder import build_model
    import dataclasses

    cfg = config(50, 16, [latent(1, 4, 4, 4, 8)])
    arch = architecture_of(cfg)
    spec = arch.to_spec(arch.config_class.from_dict(cfg))
    with pytest.raises(ValueError, match="enters"):
        build_model(dataclasses.replace(spec, schedule=(LayerCall(0, 0, enter=True),)))


def test_which_latent_sizes_the_matrix_cores_take():
    from lyapunov_engine_amd.kernels import ops

    assert ops.latent_attn_fits_matrix_cores(64, 32) and ops.latent_attn_fits_matrix_cores(512, 64)
    assert not ops.latent_attn_fits_matrix_cores(40, 16) and not ops.latent_attn_fits_matrix_cores(64, 8)
    assert not ops.latent_attn_fits_matrix_cores(512, 256), "a tile in float would not fit"
