"""The kernels behind Panodra's mechanisms, each alone against the plain
implementation (tests/plain/panodra_plain.py): the stream read through a tanh
(by the row kernel, at the end of a product of few rows, at the end of the
experts' weighted sum), the squared relu, the preparation of direct queries and
latents, attention over latents without a sink, the pairs that a table names
sorted for several layers at once, the gated experts, and scaled and capped
logits with their maxima."""

import numpy as np
import pytest
import torch

from plain import panodra_plain as PP

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
DEV = "cuda:0"


def tdt(dtype):
    return torch.float32 if dtype == "float32" else torch.bfloat16


def close(got, want, dtype, what="", floor=1.0, tol=None):
    got, want = got.double().cpu(), want.double().cpu()
    tol = tol if tol is not None else (2e-5 if dtype == "float32" else 1e-2)
    scale = max(floor, float(want.abs().max()))
    err = float((got - want).abs().max())
    assert err <= tol * scale, f"{what}: max error {err:.3e} at scale {scale:.3f}"


def ints(a):
    return torch.tensor(np.asarray(a, dtype=np.int32), device=DEV)


def bend(H, seed, alpha=0.7):
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(seed)
    w, b = 1 + 0.3 * torch.randn(H, generator=g), 0.4 * torch.randn(H, generator=g)
    bent = lambda x: PP.tanh_norm(x, torch.tensor(alpha, dtype=torch.float64), w.double(), b.double())
    return ops.StreamMap(w.to(DEV), b.to(DEV), alpha), bent


# --------------------------------------------------------- the stream's map
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [70, 256, 2052])      # one feature a thread; four; several workgroups a row
@pytest.mark.parametrize("kind", ["bent", "as it is"])
def test_stream_rows(dtype, H, kind):
    """Every form of what is still to be added, on the stream itself and on another base, kept and not
    kept, all rows and picked ones (twice the same, out of order)."""
    from lyapunov_engine_amd.kernels import ops

    T = 7
    g = torch.Generator().manual_seed(H)
    h0, base = torch.randn(T, H, generator=g) * 3, torch.randn(T, H, generator=g) * 3
    parts = torch.randn(3, T, H, generator=g)
    y = torch.randn(T, H, generator=g).to(tdt(dtype))
    smap, f = (bend(H, 1) if kind == "bent" else (ops.StreamMap(), lambda x: x))
    for what, delta, add in (("nothing", None, 0.0), ("activations", y, y.double()), ("float", y.float(), y.double()),
                             ("partial sums", parts, parts.double().sum(0))):
        for other in (False, True):
            d = None if delta is None else delta.to(DEV)
            if other:
                d = ops.Restart(base.to(DEV), d)
            want = (base if other else h0).double() + add
            h = h0.to(DEV)
            out = ops.stream_next(h, d, smap, tdt(dtype))
            close(out, f(want), dtype, f"{what}, other base {other}")
            close(h, want, "float32", f"stream after {what}, other base {other}")
            h = h0.to(DEV)
            close(ops.stream_next(h, d, smap, tdt(dtype), keep=False), f(want), dtype, f"{what}, not kept")
            rows = [5, 0, 5]
            h = h0.to(DEV)
            out = ops.stream_next(h, d, smap, tdt(dtype), rows=ints(rows))
            close(out, f(want[rows]), dtype, f"{what}, picked rows")
            assert torch.equal(h.cpu(), h0), "picked rows leave the stream alone"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 2, 8, 9, 16])
@pytest.mark.parametrize("N,K", [(192, 128), (200, 64), (24, 192), (3088, 256)])   # paired or not; 16 rows a workgroup from 3,072 on
def test_product_of_few_rows_that_ends_in_the_norm(dtype, M, N, K):
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(N + M)
    x, w = torch.randn(M, K, generator=g).to(tdt(dtype)), (torch.randn(N, K, generator=g) * K ** -0.5).to(tdt(dtype))
    h0, base = torch.randn(M, N, generator=g) * 2, torch.randn(M, N, generator=g) * 2
    prod = x.double() @ w.double().T
    for smap, f, what in ((*bend(N, 2, -0.8), "bent"), (ops.StreamMap(), lambda v: v, "as it is")):
        for other in (False, True):
            p = ops.linear(x.to(DEV), w.to(DEV), pending=True)
            assert isinstance(p, ops.PendingLinear)
            want = (base if other else h0).double() + prod
            h = h0.to(DEV)
            out = ops.stream_next(h, ops.Restart(base.to(DEV), p) if other else p, smap, tdt(dtype))
            close(out, f(want), dtype, f"{what}, other base {other}")
            close(h, want, "float32", "the stream", tol=2e-5)
            h = h0.to(DEV)
            out2 = ops.stream_next(h, ops.Restart(base.to(DEV), p) if other else p, smap, tdt(dtype), keep=False)
            assert torch.equal(out, out2) and torch.equal(h.cpu(), h0)
            rows = [M - 1, 0]
            h = h0.to(DEV)
            out = ops.stream_next(h, ops.Restart(base.to(DEV), p) if other else p, smap, tdt(dtype), rows=ints(rows))
            close(out, f(want[rows]), dtype, f"{what}, picked rows")
            assert torch.equal(h.cpu(), h0)


def test_a_sizes_mismatch_is_an_error():
    from lyapunov_engine_amd.kernels import ops

    smap, _ = bend(64, 1)
    h = torch.zeros(2, 72, device=DEV)
    with pytest.raises(ops.KernelError):
        ops.stream_next(h, None, smap, torch.float32)
    with pytest.raises(ops.KernelError):
        ops.stream_next(torch.zeros(2, 64, device=DEV), torch.zeros(3, 64, device=DEV), smap, torch.float32)
    with pytest.raises(ops.KernelError):
        ops.stream_next(torch.zeros(2, 64, device=DEV), ops.Restart(torch.zeros(3, 64, device=DEV), None), smap, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 9, 40, 64, 70, 200])
@pytest.mark.parametrize("N,K", [(192, 128), (100, 72)])
def test_squared_relu(dtype, M, N, K):
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g).to(tdt(dtype)), (torch.randn(N, K, generator=g) * K ** -0.5).to(tdt(dtype))
    want = PP.squared_relu(x.double() @ w.double().T)
    close(ops.linear_relu2(x.to(DEV), w.to(DEV)), want, dtype, f"{M} rows", tol=2e-5 if dtype == "float32" else 2e-2)
    z = torch.tensor([-3.0, -0.0, 0.0, 0.5, 2.0]).to(tdt(dtype))
    assert ops.activation(z.to(DEV), "relu2").cpu().float().tolist() == [0.0, 0.0, 0.0, 0.25, 4.0]


# --------------------------------------------------- around latent attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(3, 10, 14, 24, 10), (2, 7, 9, 25, 8), (4, 32, 16, 64, 16), (1, 0, 6, 300, 6), (5, 12, 0, 40, 0),
                                   (40, 64, 64, 512, 64)])
def test_direct_queries_and_latents_prepared_together(dtype, sizes):
    from lyapunov_engine_amd.kernels import ops
    from lyapunov_engine_amd.parts.rope import RotaryEncoding

    H, dim, rot, kv, dims = sizes
    T, page = 11, 4
    g = torch.Generator().manual_seed(kv)
    wide = H * (dim + rot)
    x = (torch.randn(T, wide + kv + rot, generator=g) * 2).to(tdt(dtype))
    wkv = 1 + 0.3 * torch.randn(kv, generator=g)
    pos = torch.tensor([0, 1, 2, 3, 40, 41, 42, 43, 44, 45, 500], dtype=torch.int32)
    slots = torch.tensor([8, 9, 10, 11, 0, 1, 2, 3, 4, 5, -1], dtype=torch.int32)        # the last row is padding
    sc = dict(factor=3.0, original=128, fast=8.0, slow=1.0)
    table = None
    if dims:
        enc = RotaryEncoding(dims, 500.0, 1024, scaling=dict(sc, rope_type="yarn"), precise=True)
        enc.materialize(DEV, tdt(dtype))
        table = enc.table
    qa = torch.full((T, H, kv + rot), -7.0, dtype=tdt(dtype), device=DEV)
    pages = torch.full((3, page, kv + rot), -9.0, dtype=tdt(dtype), device=DEV)
    ops.latent_direct_prep(x.to(DEV), wkv.to(DEV), pos.to(DEV), table, slots.to(DEV), qa, pages, num_heads=H, dim=dim, kv_rank=kv,
                           rot_dim=rot, eps=1e-5)
    xd = x.double()
    want_c = PP.rms_norm(xd[:, wide:wide + kv], wkv.double(), 1e-5)
    want_r = xd[:, wide + kv:]
    want_q = xd[:, :wide].view(T, H, dim + rot)[..., dim:]
    if dims:
        turn = dict(base=500.0, dims=dims, scaling=sc)
        want_r, want_q = PP.rotate_pairs(want_r, pos, turn), PP.rotate_pairs(want_q, pos, turn)
    flat = pages.view(-1, kv + rot).cpu()
    for t in range(T - 1):
        close(flat[int(slots[t]), :kv], want_c[t], dtype, f"latent of row {t}")
        if rot:
            close(flat[int(slots[t]), kv:], want_r[t], dtype, f"key part of row {t}")
    assert float((flat[[6, 7]] + 9.0).abs().max()) == 0.0, "slots of no row stay as they were"
    if rot:
        close(qa[..., kv:], want_q, dtype, "queries")
    assert float((qa[..., :kv] + 7.0).abs().max()) == 0.0


KERNELS = ["rows", "cores", "cores in partitions"]


def run_attention(kernel, dtype, keys, qa, scale, kv, rot, page, sink=None, seed=0):
    """One request whose keys lie in shuffled pages of a pool filled with NaN; qa's rows are its last."""
    from lyapunov_engine_amd.kernels import ops

    n, m, H = keys.shape[0], qa.shape[0], qa.shape[1]
    blocks = -(-n // page)
    ids = np.random.RandomState(seed).permutation(blocks + 3)[:blocks]
    pages = torch.full((blocks + 3, page, kv + rot), float("nan"), dtype=tdt(dtype))
    for j in range(n):
        pages[ids[j // page], j % page] = keys[j]
    out = torch.full((m, H, kv), float("nan"), dtype=tdt(dtype), device=DEV)
    args = (qa.to(DEV), pages.to(DEV), ints([ids]), ints([0, m]), ints(np.arange(n - m, n)), ints([n]),
            None if sink is None else sink.to(DEV), scale, out)
    if kernel == "rows":
        return ops.latent_attn_rows(*args, kv_rank=kv, rot_dim=rot)
    launch = ops.latent_attn_launch(m, 1, H, n, tdt(dtype), kv, rot, n_parts=3 if "partitions" in kernel else 1)
    part_o = torch.full((max(1, launch["part_o"]),), float("nan"), device=DEV)
    part_ml = torch.full((max(1, launch["part_ml"]),), float("nan"), device=DEV)
    return ops.latent_attn(*args, launch, part_o, part_ml, kv_rank=kv, rot_dim=rot)


def plain_attention(keys, qa, scale, kv, sink=None):
    """Every head's key is the page row, its value the row's first kv values."""
    n, m, H = keys.shape[0], qa.shape[0], qa.shape[1]
    q = torch.zeros(n, H, qa.shape[2], dtype=torch.float64)
    q[n - m:] = qa.double()
    k = keys.double()[:, None, :].expand(n, H, -1)
    return PP.causal_softmax_attention(q, k, k[..., :kv], scale, None if sink is None else sink.double())[n - m:]


@pytest.mark.parametrize("kernel", KERNELS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(37, 3, 64, 16, 4, 37), (300, 2, 32, 16, 16, 5), (513, 1, 48, 16, 16, 70), (700, 4, 16, 0, 16, 1),
                                   (1, 5, 64, 32, 16, 1)])
def test_attention_without_a_sink(dtype, shape, kernel):
    n, H, kv, rot, page, m = shape
    g = torch.Generator().manual_seed(n)
    keys = torch.randn(n, kv + rot, generator=g).to(tdt(dtype))
    qa = torch.randn(m, H, kv + rot, generator=g).to(tdt(dtype))
    scale = (kv + rot) ** -0.5
    got = run_attention(kernel, dtype, keys, qa, scale, kv, rot, page)
    close(got, plain_attention(keys, qa, scale, kv), dtype, f"no sink {shape}", floor=1e-3)
    # a row that sees one key has that key's value, whatever its score
    if m == n:
        close(got[0], keys[0, :kv].double().expand(H, kv), dtype, "the first row")
    # a sink far below changes nothing, one far above takes everything
    low = run_attention(kernel, dtype, keys, qa, scale, kv, rot, page, sink=torch.full((H,), -80.0))
    close(low, got.cpu(), dtype, "a sink far below", floor=1e-3, tol=1e-5)
    high = run_attention(kernel, dtype, keys, qa, scale, kv, rot, page, sink=torch.full((H,), 60.0))
    assert float(high.abs().max()) < 1e-6


@pytest.mark.parametrize("kernel", KERNELS)
@pytest.mark.parametrize("dtype", DTYPES)
def test_without_a_sink_one_planted_key_is_found_anywhere(dtype, kernel):
    n, H, kv, rot, page = 900, 2, 32, 16, 16
    g = torch.Generator().manual_seed(3)
    keys = (torch.randn(n, kv + rot, generator=g) * 0.1).to(tdt(dtype))
    for where in (0, 1, 15, 16, 17, 63, 64, 255, 256, 319, 320, 600, 898, 899):
        qa = (keys[where].float() * 400.0)[None, None, :].repeat(1, H, 1).to(tdt(dtype))
        got = run_attention(kernel, dtype, keys, qa, 1.0, kv, rot, page, seed=where)
        want = plain_attention(keys, qa, 1.0, kv)
        close(got, want, dtype, f"planted key at {where}", floor=1e-3)
        assert torch.allclose(want[0, 0], keys[where, :kv].double(), atol=0.05)


@pytest.mark.parametrize("dtype", DTYPES)
def test_merge_and_value_projection_without_a_sink(dtype):
    """Steps of few rows: the partitions merged and multiplied by the heads' value matrices in one
    kernel; a padded request (context 0) beside a live one leaves finite rows."""
    from lyapunov_engine_amd.kernels import ops

    n, H, kv, rot, vdim, page = 700, 3, 64, 32, 40, 16
    g = torch.Generator().manual_seed(8)
    keys = torch.randn(n, kv + rot, generator=g).to(tdt(dtype))
    qa = torch.randn(2, H, kv + rot, generator=g).to(tdt(dtype))
    w = torch.randn(H, vdim, kv, generator=g).to(tdt(dtype))
    blocks = -(-n // page)
    pages = torch.zeros(blocks, page, kv + rot, dtype=tdt(dtype))
    pages.view(-1, kv + rot)[:n] = keys
    scale = (kv + rot) ** -0.5
    merged = plain_attention(keys, qa[:1], scale, kv)
    if dtype == "bfloat16":
        merged = merged.to(torch.bfloat16).double()
    want = torch.stack([merged[0, h] @ w[h].double().T for h in range(H)])
    launch = ops.latent_attn_launch(2, 2, H, n, tdt(dtype), kv, rot, n_parts=4)
    part_o = torch.full((launch["part_o"],), float("nan"), device=DEV)
    part_ml = torch.full((launch["part_ml"],), float("nan"), device=DEV)
    mixed = torch.full((2, H, kv), float("nan"), dtype=tdt(dtype), device=DEV)
    table = ints([list(range(blocks)), [-1] * blocks])
    args = (qa.to(DEV), pages.to(DEV), table, ints([0, 1, 2]), ints([n - 1, 0]), ints([n, 0]), None, scale)
    ops.latent_attn(*args, mixed, launch, part_o, part_ml, kv_rank=kv, rot_dim=rot, merge=False)
    out = torch.empty(2, H, vdim, dtype=tdt(dtype), device=DEV)
    ops.latent_heads_out(w.to(DEV), out, kv_rank=kv, rot_dim=rot, part_o=part_o, part_ml=part_ml, n_parts=launch["n_parts"])
    close(out[0], want, dtype, "merged and projected", floor=1e-3)
    assert torch.isfinite(out.float()).all()
    ops.latent_attn(*args, mixed, launch, part_o, part_ml, kv_rank=kv, rot_dim=rot)      # the merging pass by itself
    close(mixed[0], merged[0], dtype, "merged", floor=1e-3)
    assert torch.isfinite(mixed.float()).all()


# ------------------------------------------------------------ table experts
@pytest.mark.parametrize("shape", [(1, 50, 1, 1, 1), (3, 97, 5, 2, 9), (2, 300, 40, 4, 130), (4, 64, 3, 3, 700), (2, 40, 512, 8, 33)])
def test_pairs_of_a_table_sorted_for_several_layers(shape):
    from lyapunov_engine_amd.kernels import ops

    L, V, E, top, T = shape
    g = torch.Generator().manual_seed(T)
    tables = torch.stack([torch.rand(V, E, generator=g).argsort(1)[:, :top].to(torch.int32) for _ in range(L)])
    tokens = torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    plans = ops.MoePlan.from_tables(tables.to(DEV), tokens.to(DEV), E)
    assert len(plans) == L
    for layer, plan in enumerate(plans):
        expert = tables[layer][tokens.long()].flatten().numpy()
        order = np.argsort(expert, kind="stable")                       # in the order of the pairs within an expert
        assert plan.sorted_pair.cpu().numpy().tolist() == order.tolist()
        assert plan.place_of.cpu().numpy()[order].tolist() == list(range(T * top))
        off = np.concatenate([[0], np.cumsum(np.bincount(expert, minlength=E))])
        assert plan.expert_off.cpu().numpy().tolist() == off.tolist()
        tiles = [(e, r) for e in range(E) for r in range(off[e], off[e + 1], plan.tile_rows)]
        n = int(plan.n_tiles)
        assert n == len(tiles) <= plan.most_tiles
        assert list(zip(plan.tile_expert[:n].tolist(), plan.tile_row0[:n].tolist())) == tiles
        # what the chosen experts' own sort makes of the same choices
        other = ops.moe_sort(tables[layer][tokens.long()].contiguous().to(DEV), E)
        assert torch.equal(other.sorted_pair, plan.sorted_pair) and torch.equal(other.place_of, plan.place_of)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(1, 64, 32, 8, 2), (5, 72, 28, 5, 3), (33, 128, 64, 4, 1), (300, 96, 40, 3, 2), (400, 128, 64, 2, 2)])
def test_table_experts_against_the_plain_mixture(dtype, shape):
    """Few rows an expert and many; the gate has no limit and nothing is added to the up projection
    (values beyond +-7 on both sides), and the weighted sum goes onto the stream through the norm, or
    is carried out alone."""
    from lyapunov_engine_amd.kernels import ops

    T, H, I, E, top = shape
    V = 61
    g = torch.Generator().manual_seed(T + H)
    x = torch.randn(T, H, generator=g).to(tdt(dtype))
    w = {"table": torch.rand(V, E, generator=g).argsort(1)[:, :top].to(torch.int32)}
    for e in range(E):
        for n, s, k in (("gate", (I, H), 4.0), ("up", (I, H), 4.0), ("down", (H, I), 1.0)):
            w[f"e{e}.{n}"] = (torch.randn(s, generator=g) * k * s[1] ** -0.5).to(tdt(dtype))
    tokens = torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    want = PP.table_experts(x.double(), tokens.tolist(), {k: v if k == "table" else v.double() for k, v in w.items()})
    plan = ops.MoePlan.from_tables(w["table"][None].to(DEV), tokens.to(DEV), E)[0]
    gate_up = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(DEV)
    down = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(DEV)
    act = ops.moe_gemm(x.to(DEV), gate_up, plan, gated=True, limit=float("inf"), alpha=1.0, plus=0.0)
    pending = ops.PendingExperts(ops.moe_gemm(act, down, plan, gated=False), plan, None, T)
    tol = 2e-5 if dtype == "float32" else 3e-2
    close(pending.run()[0], want, dtype, "weighted sum", tol=tol)
    h0, base = torch.randn(T, H, generator=g), torch.randn(T, H, generator=g)
    smap, f = bend(H, 5, 0.4)
    for other in (False, True):
        h = h0.to(DEV)
        out = ops.stream_next(h, ops.Restart(base.to(DEV), pending) if other else pending, smap, tdt(dtype))
        total = (base if other else h0).double() + want
        close(h, total, dtype, "stream", tol=tol)
        close(out, f(total), dtype, "normed", tol=tol)
    rows = [T - 1, 0]
    close(ops.stream_next(h0.to(DEV), pending, smap, tdt(dtype), rows=ints(rows)), f((h0.double() + want)[rows]), dtype, "picked", tol=tol)
    # weights of their own instead of equal ones
    wts = torch.rand(T, top, generator=g)
    per = torch.stack([torch.stack([PP.expert(x[t:t + 1].double(), {k: v.double() for k, v in w.items()}, int(e))[0]
                                    for e in w["table"][int(tok)]]) for t, tok in enumerate(tokens)])
    h = h0.to(DEV)
    ops.stream_next(h, ops.PendingExperts(pending.y, plan, wts.to(DEV), T), smap, tdt(dtype))
    close(h, h0.double() + (per * wts.double()[..., None]).sum(1), dtype, "weights", tol=tol)


# ------------------------------------------------------------------- logits
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 8, 16, 20, 32, 40, 100])
@pytest.mark.parametrize("scale,cap", [(0.3, 15.0), (2.0, 0.0), (1.0, 5.0), (1.0, 0.0)])
def test_scaled_and_capped_logits(dtype, M, scale, cap):
    from lyapunov_engine_amd.kernels import ops

    V, K = 1003, 128
    g = torch.Generator().manual_seed(M)
    x, w = (torch.randn(M, K, generator=g) * 2).to(tdt(dtype)), torch.randn(V, K, generator=g).to(tdt(dtype))
    z = x.double() @ w.double().T * scale
    want = cap * torch.tanh(z / cap) if cap else z
    got, maxima = ops.lm_head(x.to(DEV), w.to(DEV), scale, cap)
    close(got, want, "float32", f"{M} rows, scale {scale}, cap {cap}", tol=2e-5)
    if maxima is not None:
        # the largest of the stored values and the first place it stands at (a cap makes large logits equal)
        val = maxima[..., 0].contiguous().view(torch.float32).cpu()
        idx = maxima[..., 1].cpu()
        best = got.cpu().max(-1).values
        assert torch.equal(val.max(-1).values, best)
        for m in range(M):
            first = int((got[m].cpu() == best[m]).nonzero()[0])
            assert int(idx[m][val[m] == best[m]].min()) == first
    # sizes the head's own kernels do not take
    x2, w2 = x[:, :100].contiguous(), w[:, :100].contiguous()
    z = x2.double() @ w2.double().T * scale
    got, maxima = ops.lm_head(x2.to(DEV), w2.to(DEV), scale, cap)
    assert maxima is None
    close(got, cap * torch.tanh(z / cap) if cap else z, "float32", "general product", tol=2e-5)


def test_logit_cap_in_place():
    from lyapunov_engine_amd.kernels import ops

    z = torch.linspace(-200, 200, 40001)
    got = ops.logit_cap(z.to(DEV), 0.5, 30.0).cpu()
    close(got, 30 * torch.tanh(z.double() * 0.5 / 30), "float32", "cap", tol=1e-6)
    assert float(got.max()) <= 30.0 and bool((got[1:] >= got[:-1]).all())
    close(ops.logit_cap(z.to(DEV), 0.25, 0.0).cpu(), z.double() * 0.25, "float32", "scale alone", tol=1e-6)
