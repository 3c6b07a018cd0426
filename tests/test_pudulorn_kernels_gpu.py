"""The kernels behind Pudulorn's mechanisms, each alone against the plain
implementation (tests/plain/pudulorn_plain.py): differential attention for
prompts and single tokens over shuffled pages, whole, in windows and in chunks, cut
into runs and partitions; the same row by row; latent attention within a window;
what prepares queries, keys, values and latents with rotated halves; the limited
gated product, alone and behind a norm; products behind a norm; the router whose
weights are shares of all, with the shared expert's gate; and the whole routed
part."""
import math

import numpy as np
import pytest
import torch

from plain import pudulorn_plain as DP

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
DEV = "cuda:0"


def tdt(dtype):
    return torch.float32 if dtype == "float32" else torch.bfloat16


def close(got, want, dtype, what="", floor=1.0, tol=None):
    got, want = got.double().cpu(), want.double().cpu()
    tol = tol if tol is not None else (2e-5 if dtype == "float32" else 1.2e-2)
    scale = max(floor, float(want.abs().max()))
    err = float((got - want).abs().max())
    assert err <= tol * scale, f"{what}: max error {err:.3e} at scale {scale:.3f}"


def ints(a):
    return torch.tensor(np.asarray(a, dtype=np.int32), device=DEV)


def first_seen(pos, window, chunk):
    return max(0, pos - window + 1) if window else (pos - pos % chunk if chunk else 0)


class Pages:
    """Block tables over shuffled pages for requests (tokens before the step, new tokens).  Pages that no token of
    the step sees any more are not in the tables; every slot that no request owns holds NaN."""

    def __init__(self, requests, bs, seed, window=0, chunk=0):
        self.requests, self.bs = requests, bs
        g = torch.Generator().manual_seed(seed)
        total = sum(-(-(a + n) // bs) for a, n in requests) + 3
        order = torch.randperm(total, generator=g).tolist()
        self.num, self.width = total, max(-(-(a + n) // bs) for a, n in requests) + 1
        self.table = np.full((len(requests), self.width), -1, dtype=np.int32)
        self.slots = []                      # per request: the pool slot of every token, or -1
        for b, (a, n) in enumerate(requests):
            lo = first_seen(a, window, chunk)
            slots = []
            for p in range(-(-(a + n) // bs)):
                page = order.pop() if (p + 1) * bs > lo else -1
                self.table[b, p] = page
                slots += [page * bs + s if page >= 0 else -1 for s in range(bs)]
            self.slots.append(slots[:a + n])
        self.q_start = np.concatenate([[0], np.cumsum([n for _, n in requests])]).astype(np.int32)
        self.ctx = np.asarray([a + n for a, n in requests], dtype=np.int32)
        self.positions = np.concatenate([np.arange(a, a + n) for a, n in requests]).astype(np.int32)
        self.T = int(self.q_start[-1])

    def device(self):
        return ints(self.table), ints(self.q_start), ints(self.positions), ints(self.ctx)

    def tiles(self):
        out = [(a + min(n, q0 + 64), b, q0) for b, (a, n) in enumerate(self.requests) if n > 1 for q0 in range(0, n, 64)]
        out.sort()
        return out


def paired_pools(pg, keys, values, dtype):
    """keys: per request [len, G, 2, D], values [len, G, V] -> the two pools, NaN where nobody lives."""
    G, D, V = keys[0].shape[1], keys[0].shape[3], values[0].shape[2]
    k = torch.full((pg.num, 2 * G, pg.bs, D), float("nan"), dtype=tdt(dtype))
    v = torch.full((pg.num, G, V, pg.bs), float("nan"), dtype=tdt(dtype))
    for slots, kk, vv in zip(pg.slots, keys, values):
        for t, s in enumerate(slots):
            if s >= 0:
                k[s // pg.bs, :, s % pg.bs] = kk[t].reshape(2 * G, D).to(tdt(dtype))
                v[s // pg.bs, :, :, s % pg.bs] = vv[t].to(tdt(dtype))
    return k.to(DEV), v.to(DEV)


def paired_case(pg, H, G, D, V, dtype, seed, window=0, chunk=0, take_off=0.45, post=0.7, eps=1e-3, gate=True, spike=None):
    """Random operands and the plain result of every row, [T, H V]."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g).to(tdt(dtype))
    q = rnd(pg.T, H, 2, D)
    keys, values = [rnd(a + n, G, 2, D) for a, n in pg.requests], [rnd(a + n, G, V) for a, n in pg.requests]
    z = torch.randn(pg.T, H * V, generator=g) if gate else None
    if spike is not None:
        spike(q, keys)
    scale = D ** -0.5
    want = torch.zeros(pg.T, H, V, dtype=torch.float64)
    for b, (a, n) in enumerate(pg.requests):
        L, r0 = a + n, int(pg.q_start[b])
        ok = (DP.window_mask(L, window) if window else DP.chunk_mask(L, chunk or None))[a:]
        for h in range(H):
            kh = h // (H // G)
            o = [DP.softmax_attention(q[r0:r0 + n, h, m].double(), keys[b][:, kh, m].double(), values[b][:, kh].double(), scale, ok)
                 for m in (0, 1)]
            want[r0:r0 + n, h] = DP.unit_rms(o[0] - take_off * o[1], eps) * post
    want = want.reshape(pg.T, H * V)
    if gate:
        want = want * torch.sigmoid(z.double())
    kpool, vpool = paired_pools(pg, keys, values, dtype)
    opts = dict(take_off=take_off, post=post, eps=eps, gate=z.to(DEV) if gate else None)
    return q.reshape(pg.T, H * 2 * D).to(DEV), kpool, vpool, scale, opts, want


MASKS = [(0, 0), (40, 0), (1, 0), (0, 50), (0, 7), (0, 64), (0, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mask", MASKS)
@pytest.mark.parametrize("heads,dims", [((4, 4), (16, 32)), ((8, 2), (32, 64)), ((6, 3), (48, 80)), ((5, 1), (32, 16)), ((2, 1), (128, 256))])
def test_differential_attention_of_prompts(dtype, mask, heads, dims):
    """Whole prompts, portions behind a context and portions of two tokens in one step, whole and in runs."""
    from lyapunov_engine_amd.kernels import ops

    (H, G), (D, V), (window, chunk) = heads, dims, mask
    pg = Pages([(0, 70), (90, 2), (37, 75), (0, 2), (130, 33)], 16, seed=H + D, window=window, chunk=chunk)
    q, kpool, vpool, scale, opts, want = paired_case(pg, H, G, D, V, dtype, seed=V + window + chunk, window=window, chunk=chunk)
    bt, q_start, _, ctx = pg.device()
    tiles = pg.tiles()
    seqs, q0s = ints([b for _, b, _ in tiles]), ints([q0 for _, _, q0 in tiles])
    sizes = dict(num_heads=H, num_kv_heads=G, dim=D, vdim=V, window=window, chunk=chunk)
    launch = ops.paired_prefill_launch(len(tiles), tiles[-1][0], tdt(dtype), **sizes)
    for parts in sorted({launch["parts"], 1, 2, 5}):
        n = len(tiles) * 64 * H * 2 * parts
        po, pm = torch.full((n * V,), float("nan"), device=DEV), torch.full((n * 2,), float("nan"), device=DEV)
        out = torch.full((pg.T, H * V), float("nan"), dtype=tdt(dtype), device=DEV)
        ops.paired_prefill(q, out, kpool, vpool, bt, q_start, ctx, seqs, q0s, len(tiles), dict(parts=parts), po, pm, scale=scale,
                           **sizes, **opts)
        close(out, want, dtype, f"{parts} runs", tol=3e-5 if dtype == "float32" else 2.5e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mask", MASKS + [(300, 0), (0, 400)])
@pytest.mark.parametrize("heads,dims", [((4, 4), (16, 32)), ((8, 2), (32, 64)), ((6, 3), (48, 80)), ((20, 1), (32, 16)), ((2, 1), (128, 256))])
def test_differential_attention_of_single_tokens(dtype, mask, heads, dims):
    """Requests of one token among others, all contexts from the first token on, in one partition and in several; a padded
    request among them."""
    from lyapunov_engine_amd.kernels import ops

    (H, G), (D, V), (window, chunk) = heads, dims, mask
    pg = Pages([(0, 1), (99, 1), (5, 3), (64, 1), (410, 1), (63, 1), (149, 1)], 16, seed=H + D, window=window, chunk=chunk)
    q, kpool, vpool, scale, opts, want = paired_case(pg, H, G, D, V, dtype, seed=V + window + chunk, window=window, chunk=chunk)
    bt, q_start, _, ctx = pg.device()
    ctx[3] = 0                                # a request of a recorded step that is only padding
    dec = ints([0, 1, 3, 4, 5, 6])
    rows = [int(pg.q_start[b]) for b in (0, 1, 4, 5, 6)]
    sizes = dict(num_heads=H, num_kv_heads=G, dim=D, vdim=V, window=window, chunk=chunk)
    bound = ops.visible_keys(411, window, chunk)
    least = 8 * 32 if V <= 128 else 4 * 32
    for launch in (ops.paired_decode_launch(6, 411, **sizes), dict(part_keys=least, max_parts=-(-bound // least)),
                   dict(part_keys=512, max_parts=1)):
        n = 6 * H * 2 * launch["max_parts"]
        po, pm = torch.full((n * V,), float("nan"), device=DEV), torch.full((n * 2,), float("nan"), device=DEV)
        out = torch.full((pg.T, H * V), float("nan"), dtype=tdt(dtype), device=DEV)
        ops.paired_decode(q, out, kpool, vpool, bt, q_start, ctx, dec, 6, launch, po, pm, scale=scale, **sizes, **opts)
        close(out[rows], want[rows], dtype, f"{launch}", tol=3e-5 if dtype == "float32" else 2.5e-2)
        assert (out[int(pg.q_start[3])] == 0).all(), "a padded request's row is written as zeros"
        assert out[int(pg.q_start[2]):int(pg.q_start[2]) + 3].isnan().all(), "rows of other requests are left alone"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bs", [1, 3, 4, 8, 12, 32])
@pytest.mark.parametrize("mask", [(0, 0), (21, 0), (0, 30)])
def test_differential_attention_at_other_page_sizes_and_without_a_gate(dtype, bs, mask):
    from lyapunov_engine_amd.kernels import ops

    window, chunk = mask
    H, G, D, V = 4, 2, 32, 48
    pg = Pages([(0, 50), (77, 1), (40, 9)], bs, seed=bs, window=window, chunk=chunk)
    q, kpool, vpool, scale, opts, want = paired_case(pg, H, G, D, V, dtype, seed=bs, window=window, chunk=chunk, gate=False)
    bt, q_start, _, ctx = pg.device()
    tiles = pg.tiles()
    sizes = dict(num_heads=H, num_kv_heads=G, dim=D, vdim=V, window=window, chunk=chunk)
    out = torch.full((pg.T, H * V), float("nan"), dtype=tdt(dtype), device=DEV)
    ops.paired_prefill(q, out, kpool, vpool, bt, q_start, ctx, ints([b for _, b, _ in tiles]), ints([q0 for _, _, q0 in tiles]),
                       len(tiles), dict(parts=1), scale=scale, **sizes, **opts)
    ops.paired_decode(q, out, kpool, vpool, bt, q_start, ctx, ints([1]), 1, dict(part_keys=256, max_parts=1), scale=scale, **sizes, **opts)
    close(out, want, dtype, f"pages of {bs}", tol=3e-5 if dtype == "float32" else 2.5e-2)


def test_one_key_among_many_stands_out():
    """A key far back, at page, tile, wave and partition borders, just inside and just outside the mask, dominates the first
    map where it is seen and does nothing where it is not."""
    from lyapunov_engine_amd.kernels import ops

    H, G, D, V, L = 2, 1, 32, 64, 700
    for window, chunk in ((0, 0), (300, 0), (0, 256)):
        lo = first_seen(L - 1, window, chunk)
        for at in sorted({0, lo - 1, lo, lo + 1, 511, 512, 527, 528, 639, 640, L - 2, L - 1}):
            if at < 0:
                continue
            pg = Pages([(L - 1, 1)], 16, seed=1, window=window, chunk=chunk)

            def spike(q, keys):
                keys[0][at, :, 0] = 6.0 * q[0, 0, 0] / q[0, 0, 0].norm()
            q, kpool, vpool, scale, opts, want = paired_case(pg, H, G, D, V, "float32", seed=3, window=window, chunk=chunk, spike=spike)
            bt, q_start, _, ctx = pg.device()
            sizes = dict(num_heads=H, num_kv_heads=G, dim=D, vdim=V, window=window, chunk=chunk)
            for most in (256, 512, 1024):
                parts = -(-ops.visible_keys(L, window, chunk) // most)
                n = H * 2 * parts
                out = torch.empty(1, H * V, device=DEV)
                ops.paired_decode(q, out, kpool, vpool, bt, q_start, ctx, None, 1, dict(part_keys=most, max_parts=parts),
                                  torch.empty(n * V, device=DEV), torch.empty(n * 2, device=DEV), scale=scale, **sizes, **opts)
                close(out, want, "float32", f"key {at}, mask {(window, chunk)}, partitions of {most}", tol=3e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mask", [(0, 0), (40, 0), (1, 0), (0, 50), (0, 7), (0, 1)])
@pytest.mark.parametrize("heads,dims", [((4, 2), (10, 24)), ((3, 3), (6, 7)), ((2, 1), (14, 300)), ((4, 4), (16, 32))])
def test_differential_attention_row_by_row(dtype, mask, heads, dims):
    from lyapunov_engine_amd.kernels import ops

    (H, G), (D, V), (window, chunk) = heads, dims, mask
    pg = Pages([(0, 40), (90, 1), (37, 12), (0, 2)], 4, seed=H + D, window=window, chunk=chunk)
    q, kpool, vpool, scale, opts, want = paired_case(pg, H, G, D, V, dtype, seed=V + chunk, window=window, chunk=chunk)
    bt, q_start, positions, ctx = pg.device()
    sums = torch.full((pg.T, H * 2 * V), float("nan"), device=DEV)
    ops.attn_rows(q, sums, kpool, vpool, bt, q_start, positions, ctx, num_heads=2 * H, num_kv_heads=2 * G, dim=D, vdim=V, scale=scale,
                  window=window, chunk=chunk, maps=2)
    out = ops.head_difference(sums, tdt(dtype), num_heads=H, vdim=V, **opts)
    close(out, want, dtype, "row by row")


def test_mismatches_are_errors():
    from lyapunov_engine_amd.kernels import ops

    pg = Pages([(0, 5)], 16, seed=1)
    q, kpool, vpool, scale, opts, _ = paired_case(pg, 4, 2, 16, 32, "float32", seed=1)
    bt, q_start, _, ctx = pg.device()
    out = torch.zeros(5, 4 * 32, device=DEV)
    sizes = dict(num_heads=4, num_kv_heads=2, dim=16, vdim=32)
    good = (q, out, kpool, vpool, bt, q_start, ctx, ints([0]), ints([0]), 1, dict(parts=1))
    for kw, args in ((dict(window=4, chunk=4), good), (dict(num_kv_heads=1), good), (dict(vdim=16), good),
                     ({}, (q[:, :64],) + good[1:]), ({}, good[:9] + (2, dict(parts=1))), ({}, good[:10] + (dict(parts=2),))):
        with pytest.raises(ops.KernelError):
            ops.paired_prefill(*args, scale=scale, **{**sizes, **kw}, **opts)
    with pytest.raises(ops.KernelError):
        ops.paired_decode(q, out, kpool, vpool, bt, q_start, ctx, None, 2, dict(part_keys=256, max_parts=1), scale=scale, **sizes, **opts)


# --------------------------------------------------------------- latent windows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 1, 2, 16, 40, 100, 1000])
@pytest.mark.parametrize("sizes", [(3, 32, 16), (12, 64, 32), (1, 16, 16), (70, 16, 0), (3, 20, 8)])   # the last: row by row
def test_latent_attention_within_a_window(dtype, window, sizes):
    """Prompts, portions and single tokens over shuffled pages of NaN, in one partition and in several."""
    from lyapunov_engine_amd.kernels import ops

    H, KV, RD = sizes
    pg = Pages([(0, 70), (150, 1), (37, 20), (0, 1), (210, 2), (99, 1)], 16, seed=H, window=window)
    g = torch.Generator().manual_seed(H + window)
    rnd = lambda *s: torch.randn(*s, generator=g).to(tdt(dtype))
    qa = rnd(pg.T, H, KV + RD)
    rows = [rnd(a + n, KV + RD) for a, n in pg.requests]
    pool = torch.full((pg.num * 16, KV + RD), float("nan"), dtype=tdt(dtype))
    for slots, r in zip(pg.slots, rows):
        for t, s in enumerate(slots):
            if s >= 0:
                pool[s] = r[t]
    pool = pool.view(pg.num, 16, KV + RD).to(DEV)
    scale = (KV + RD) ** -0.5 * 1.5
    want = torch.zeros(pg.T, H, KV, dtype=torch.float64)
    for b, (a, n) in enumerate(pg.requests):
        ok = DP.window_mask(a + n, window or None)[a:]
        r0 = int(pg.q_start[b])
        for h in range(H):
            want[r0:r0 + n, h] = DP.softmax_attention(qa[r0:r0 + n, h].double(), rows[b].double(), rows[b][:, :KV].double(), scale, ok)
    bt, q_start, positions, ctx = pg.device()
    args = (qa.to(DEV), pool, bt, q_start, positions, ctx, None, scale)
    out = torch.full((pg.T, H, KV), float("nan"), dtype=tdt(dtype), device=DEV)
    ops.latent_attn_rows(*args, out, kv_rank=KV, rot_dim=RD, window=window)
    close(out, want, dtype, "row by row")
    if not ops.latent_attn_fits_matrix_cores(KV, RD):
        return
    for n_parts in (None, 1, 2, 3):
        launch = ops.latent_attn_launch(pg.T, len(pg.requests), H, 212, tdt(dtype), KV, RD, n_parts=n_parts, window=window)
        po, pm = torch.full((max(1, launch["part_o"]),), float("nan"), device=DEV), torch.full((max(1, launch["part_ml"]),), float("nan"), device=DEV)
        out = torch.full((pg.T, H, KV), float("nan"), dtype=tdt(dtype), device=DEV)
        ops.latent_attn(*args, out, launch, po, pm, kv_rank=KV, rot_dim=RD, window=window)
        close(out, want, dtype, f"{launch}")


# --------------------------------------------------- queries, keys, values, latents
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(3, 10, 14, 18, 24, 10), (2, 7, 8, 20, 25, 8), (4, 32, 16, 64, 64, 16), (1, 0, 6, 33, 300, 4), (5, 12, 6, 8, 40, 0)])
def test_latents_and_query_parts_with_rotated_halves(dtype, sizes):
    from lyapunov_engine_amd.kernels import ops

    H, dim, rot, q_rank, kv, dims = sizes
    T, eps, base = 6, 1e-5, 300.0
    g = torch.Generator().manual_seed(kv)
    d = torch.randn(T, q_rank + kv + rot, generator=g).to(tdt(dtype))
    wq, wkv = 1 + 0.2 * torch.randn(q_rank, generator=g), 1 + 0.2 * torch.randn(kv, generator=g)
    pos = [0, 3, 1000, 17, 5, 9]
    angles = torch.arange(1001, dtype=torch.float64)[:, None] * torch.tensor([base ** (-2 * i / dims) for i in range(dims // 2)] if dims else [],
                                                                            dtype=torch.float64)
    table = torch.cat((angles.cos(), angles.sin()), 1).float().to(DEV) if dims else None
    slots = [7, 0, 3, -1, 11, 4]
    pages = torch.full((3, 4, kv + rot), 9.0, dtype=tdt(dtype), device=DEV)
    cq = torch.empty(T, q_rank, dtype=tdt(dtype), device=DEV)
    ops.latent_prep(d.to(DEV), wq.to(DEV), wkv.to(DEV), ints(pos), table, ints(slots), cq, pages, q_rank=q_rank, kv_rank=kv,
                    rot_dim=rot, eps=eps, pairing="halves")
    x = d.double()
    close(cq, DP.rms_norm(x[:, :q_rank], wq.double(), eps), dtype, "query latent")
    c = DP.rms_norm(x[:, q_rank:q_rank + kv], wkv.double(), eps)
    r = DP.rotate_halves(x[:, q_rank + kv:], torch.tensor(pos), base, dims)
    flat = pages.view(12, kv + rot)
    for t, s in enumerate(slots):
        if s >= 0:
            close(flat[s], torch.cat((c[t], r[t])), dtype, f"row {t}")
    assert (flat[[s for s in range(12) if s not in slots]] == 9.0).all()
    q = torch.randn(T, H * (dim + rot), generator=g).to(tdt(dtype))
    qa = torch.full((T, H, kv + rot), 5.0, dtype=tdt(dtype), device=DEV)
    ops.latent_query_rotate(q.to(DEV), ints(pos), table, qa, num_heads=H, dim=dim, rot_dim=rot, kv_rank=kv, pairing="halves")
    want = DP.rotate_halves(q.double().view(T, H, dim + rot)[:, :, dim:], torch.tensor(pos), base, dims)
    close(qa[:, :, kv:], want, dtype, "queries")
    assert (qa[:, :, :kv] == 5.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 5, 70])
@pytest.mark.parametrize("sizes", [(4, 2, 10, 26, 10), (3, 3, 14, 9, 6), (8, 2, 32, 64, 32), (2, 1, 64, 20, 64)])
def test_two_maps_a_head_prepared(dtype, T, sizes):
    """Keys of both maps beside values of half as many heads; slots nobody writes stay as they are."""
    from lyapunov_engine_amd.kernels import ops

    H, G, D, V, dims = sizes
    bs, base, eps = 4, 50.0, 1e-5
    g = torch.Generator().manual_seed(D)
    n = 2 * H * D + 2 * G * D + G * V + 3
    pre = torch.randn(T, n, generator=g) * 2
    wq, wk = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    pos = torch.randint(0, 200, (T,), generator=g)
    angles = torch.arange(200, dtype=torch.float64)[:, None] * torch.tensor([base ** (-2 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    table = torch.cat((angles.cos(), angles.sin()), 1).float().to(DEV)
    n_pages = -(-T // bs) + 2
    slots = torch.randperm(n_pages * bs, generator=g)[:T]
    if T > 1:
        slots[T // 2] = -1
    kpool = torch.full((n_pages, 2 * G, bs, D), 9.0, dtype=tdt(dtype), device=DEV)
    vpool = torch.full((n_pages, G, V, bs), 9.0, dtype=tdt(dtype), device=DEV)
    q, _ = ops.qkv_prepare(pre.to(DEV), tdt(dtype), num_heads=2 * H, num_kv_heads=2 * G, dim=D, vdim=V, slots=ints(slots), kpool=kpool,
                           vpool=vpool, page_size=bs, norm="head", q_weight=wq.to(DEV), k_weight=wk.to(DEV), eps=eps,
                           positions=ints(pos), table=table, pairing="halves", value_heads=G)
    x = pre.double()
    wantq = DP.rotate_halves(DP.rms_norm(x[:, :2 * H * D].view(T, H, 2, D), wq.double(), eps), pos, base, dims)
    wantk = DP.rotate_halves(DP.rms_norm(x[:, 2 * H * D:2 * (H + G) * D].view(T, G, 2, D), wk.double(), eps), pos, base, dims)
    wantv = x[:, 2 * (H + G) * D:2 * (H + G) * D + G * V].view(T, G, V)
    close(q, wantq.reshape(T, -1), dtype, "queries")
    k, v = torch.full((n_pages, 2 * G, bs, D), 9.0), torch.full((n_pages, G, V, bs), 9.0)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            k[s // bs, :, s % bs], v[s // bs, :, :, s % bs] = wantk[t].reshape(2 * G, D).float(), wantv[t].float()
    close(kpool, k, dtype, "keys")
    close(vpool, v, dtype, "values")


# ---------------------------------------------------------------- feed-forwards
def runs_of_eight(gate, up):
    I, K = gate.shape
    return torch.stack((gate.view(I // 8, 8, K), up.view(I // 8, 8, K)), 1).reshape(2 * I, K)


def pending_norm(M, K, dtype, seed):
    """A norm still to be carried out, as the product before it leaves it, and the normed rows in 64-bit."""
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(seed)
    h = torch.randn(M, K, generator=g) * 2
    x, w = torch.randn(M, 64, generator=g).to(tdt(dtype)), (torch.randn(K, 64, generator=g) / 8).to(tdt(dtype))
    nw = 1 + 0.3 * torch.randn(K, generator=g)
    p, delta = ops.rmsnorm_pending(h.to(DEV), nw.to(DEV), 1e-5, tdt(dtype), ops.PendingLinear(x.to(DEV), w.to(DEV), tdt(dtype)))
    assert p is not None and delta is None
    return p, DP.rms_norm(h.double() + x.double() @ w.double().T, nw.double(), 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 8, 9, 16, 17, 40, 64, 70, 200])
@pytest.mark.parametrize("I,K", [(96, 128), (1024, 192), (100, 72), (40, 64)])      # 100 and 72: no tiles of eight, or no few-rows kernel
def test_limited_gated_product(dtype, M, I, K):
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(M + I)
    x = torch.randn(M, K, generator=g).to(tdt(dtype))
    gate, up = ((torch.randn(I, K, generator=g) * 2.5 * K ** -0.5).to(tdt(dtype)) for _ in range(2))
    for limit, slope, plus in ((1.5, 1.702, 1.0), (math.inf, 1.0, 0.0), (0.4, 0.8, -0.5)):
        def want(v):
            a, b = torch.clamp(v @ gate.double().T, max=limit), torch.clamp(v @ up.double().T, min=-limit, max=limit)
            return a * torch.sigmoid(slope * a) * (b + plus)
        inter = 8 if I % 8 == 0 else 0
        w = (runs_of_eight(gate, up) if inter else torch.cat((gate, up))).to(DEV)
        tol = 2e-5 if dtype == "float32" else 2e-2
        close(ops.linear_glu(x.to(DEV), w, inter, limit, slope, plus), want(x.double()), dtype, f"limit {limit}", tol=tol)
        if M <= 16 and K % 64 == 0:
            p, normed = pending_norm(M, K, dtype, seed=M)
            close(ops.linear_glu(p, w, inter, limit, slope, plus), want(normed), dtype, f"behind a norm, limit {limit}", tol=tol)


@pytest.mark.parametrize("dtype", DTYPES)
def test_limited_gate_in_every_layout(dtype):
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(1)
    for T, I, n in ((3, 40, 0), (3, 40, 8), (5, 12, 4), (2, 7, 0), (700, 264, 8), (1, 8, 8)):
        gate, up = (3 * torch.randn(T, I, generator=g).to(tdt(dtype)) for _ in range(2))
        x = torch.stack((gate.view(T, I // n, n), up.view(T, I // n, n)), 2).reshape(T, 2 * I) if n else torch.cat((gate, up), 1)
        a, b = torch.clamp(gate.double(), max=1.2), torch.clamp(up.double(), -1.2, 1.2)
        close(ops.glu_clamped(x.to(DEV), 1.2, 1.702, 1.0, n), a * torch.sigmoid(1.702 * a) * (b + 1), dtype, f"{T} x {I} in runs of {n}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 8, 16])
@pytest.mark.parametrize("N,K", [(200, 128), (3088, 64), (24, 320)])
def test_products_behind_a_norm(dtype, M, N, K):
    from lyapunov_engine_amd.kernels import ops

    w = (torch.randn(N, K, generator=torch.Generator().manual_seed(N)) * K ** -0.5).to(tdt(dtype))
    for out_dtype in {torch.float32, tdt(dtype)}:
        p, normed = pending_norm(M, K, dtype, seed=M + N)
        got = ops.linear(p, w.to(DEV), out_dtype=out_dtype)
        assert got.dtype == out_dtype
        close(got, normed @ w.double().T, dtype, f"{M} x {N}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 7, 64, 300])
@pytest.mark.parametrize("E,top,K", [(16, 4, 96), (5, 5, 40), (1, 1, 64), (200, 6, 512), (64, 8, 130), (65, 3, 1024)])
def test_weights_are_shares_of_all_scores(dtype, T, E, top, K):
    """The choice, the weights and the shared expert's gate, with and without the sort, beside an always-used expert or not."""
    from lyapunov_engine_amd.kernels import ops

    g = torch.Generator().manual_seed(E + T)
    x = torch.randn(T, K, generator=g).to(tdt(dtype))
    w, sg = torch.randn(E, K, generator=g) * 1.5 * K ** -0.5, torch.randn(1, K, generator=g) * K ** -0.5
    z = x.double() @ w.double().T
    chosen, weight = DP.route(x.double(), w.double(), top, 2.5)
    share = torch.sigmoid(x.double() @ sg.double().T)[:, 0]
    srt = torch.sort(z, -1, descending=True).values
    clear = torch.ones(T, dtype=torch.bool) if top == E else (srt[:, top - 1] - srt[:, top]) > 1e-5
    for k in range(top - 1):
        clear &= (srt[:, k] - srt[:, k + 1]) > 1e-5
    assert int(clear.sum()) >= 0.9 * T
    for gated in (False, True):
        for always in (-1, E):
            for sort_for in (0, E + (always >= 0)):
                router = (torch.cat((w, sg)) if gated else w).to(DEV)
                idx, wgt, *rest = ops.moe_route_from(x.to(DEV), router, None, top, always, sort_for=sort_for, over_all=True, scale=2.5,
                                                     gated=gated)
                assert torch.equal(idx[:, :top].cpu().long()[clear], chosen[clear])
                close(wgt[:, :top][clear.to(DEV)], weight[clear], "float32", "weights")
                if always >= 0:
                    assert (idx[:, top] == E).all()
                    close(wgt[:, top], share if gated else torch.ones(T), "float32", "the always-used expert's weight")
                if sort_for:
                    plan = rest.pop(0)
                    order = plan.sorted_pair.long().cpu()
                    assert torch.equal(order, torch.sort(idx.reshape(-1).cpu(), stable=True).indices)
                if gated and always < 0:
                    close(rest.pop(0), share, "float32", "share")
                assert not rest


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [64, 320, 1024, 2052, 4096, 8192, 70, 8196])     # the last two: sum and norm apart
@pytest.mark.parametrize("T", [1, 33])
def test_the_experts_sum_that_ends_in_the_norm(dtype, H, T):
    """The weighted sum with and without a shared expert and its share, weights given and equal, onto the stream and
    through a norm in one kernel; picked rows leave the stream alone."""
    from lyapunov_engine_amd.kernels import ops
    from lyapunov_engine_amd.parts.base import StepContext
    from lyapunov_engine_amd.parts.norm import RMSNorm

    top, E = 3, 5
    g = torch.Generator().manual_seed(H + T)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int().to(DEV)
    plan = ops.moe_sort(idx, E)
    y = torch.randn(T * top, H, generator=g).to(tdt(dtype))
    place = plan.place_of.long().cpu().view(T, top)
    wgt, share = torch.rand(T, top, generator=g), torch.rand(T, generator=g)
    shared = torch.randn(T, H, generator=g).to(tdt(dtype))
    h0 = torch.randn(T, H, generator=g) * 2
    norm = RMSNorm(H, 1e-5, tensor="", one_plus=True)
    norm.weight = (0.3 * torch.randn(H, generator=g)).to(tdt(dtype)).to(DEV)
    ctx = StepContext(device=torch.device(DEV), dtype=tdt(dtype), T=T, B=1, token_ids=None, positions=None, q_start=None, ctx_len=None,
                      state_slots=None, logit_rows=None, R=0, groups=[])
    for w, s, f in ((wgt, shared, share), (wgt, None, None), (None, None, None), (wgt, shared, None)):
        want = h0.double() + ((torch.full((T, top), 1 / top) if w is None else w).double()[..., None] * y.double()[place]).sum(1)
        if s is not None:
            want = want + s.double() * (1.0 if f is None else f.double()[:, None])
        dev = lambda t: None if t is None else t.to(DEV)
        pending = lambda: ops.PendingExperts(y.to(DEV), plan, dev(w), T, dev(s), dev(f))
        h = h0.to(DEV)
        out = norm.forward(ctx, h, pending(), lazy=True)
        close(h, want, "float32", "the stream")
        normed = DP.shifted_rms_norm(want, norm.weight.double().cpu(), 1e-5)
        close(out, normed, dtype, "the norm")
        h = h0.to(DEV)
        close(norm.forward(ctx, h, pending(), rows=ints([T - 1, 0])), normed[[T - 1, 0]], dtype, "picked rows")
        assert torch.equal(h.cpu(), h0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(1, 16, 4, 128, 64, 128), (9, 5, 2, 72, 28, 28), (70, 12, 3, 128, 64, 96), (300, 6, 2, 256, 512, 512),
                                   (600, 3, 3, 64, 40, 20), (40, 7, 2, 512, 32, 0), (3, 1, 1, 40, 48, 50)])
def test_the_routed_part_against_the_plain_one(dtype, shape):
    from lyapunov_engine_amd.parts.base import StepContext
    from lyapunov_engine_amd.parts.routed_experts import RoutedExperts
    from lyapunov_engine_amd.weights.loader import DictSource  # noqa: F401

    T, E, top, H, I, S = shape
    g = torch.Generator().manual_seed(T + E)
    part = RoutedExperts(H, E, top, I, limit=math.inf, gate_slope=1.0, plus=0.0, router_bias=False, scores="all", scale=1.8,
                         shared_size=S, shared_limit=math.inf, shared_gate=S > 0)
    w = {}
    for ws in part.weight_specs():
        pieces = []
        for src in ws.sources:
            t = torch.randn(src.shape, generator=g) * (1.5 if ws.attr == "router" else 2.0) / math.sqrt(src.shape[-1])
            w[src.name] = t.to(tdt(dtype))
            pieces.append(w[src.name])
        joined = runs_of_eight(*pieces) if ws.interleave else torch.cat(pieces)
        setattr(part, ws.attr, joined.to(DEV))
    part.materialize(DEV, tdt(dtype))
    x = torch.randn(T, H, generator=g).to(tdt(dtype))
    ctx = StepContext(device=torch.device(DEV), dtype=tdt(dtype), T=T, B=1, token_ids=None, positions=None, q_start=None, ctx_len=None,
                      state_slots=None, logit_rows=None, R=0, groups=[])
    got = part.forward(ctx, x.to(DEV))
    wd = {k: v.double() for k, v in w.items()}
    want = DP.expert_ff(x.double(), wd, dict(router=dict(experts=E, top=top, scale=1.8), shared=dict(ff=S) if S else None))
    srt = torch.sort(x.double() @ wd["router"].T, -1, descending=True).values
    clear = torch.ones(T, dtype=torch.bool) if top == E else (srt[:, top - 1] - srt[:, top]) > 1e-4
    assert int(clear.sum()) >= 0.9 * T
    close(got[0][clear.to(DEV)], want[clear], dtype, f"{shape}", tol=2e-5 if dtype == "float32" else 2e-2)
