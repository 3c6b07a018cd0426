"""Differential attention: every head has two softmax maps over the same values,
and what the second sees is taken off the first.

Per token x at position p, with H query heads and G key/value heads (query head
h reads key/value head h // (H / G)), two maps of ``dim`` values a query or key
head side by side, values of ``vdim``:

    q = W_q x [H, 2, dim],  k = W_k x [G, 2, dim],  v = W_v x [G, vdim],  z = W_g x [H, vdim]    one product, 32-bit out
    q, k <- rms norm over every head's every map, one weight [dim] for all of them
    the first rotary_dim values of every map turn by p * f_i in pairs ("halves" or "neighbours")
    a_m = softmax over the visible keys of scale * q_m . k_m, applied to v          m = 1, 2
    lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff                                 one number for the layer
    o = a_1 - lambda a_2,   o <- o / sqrt(mean(o^2) + eps) * (1 - diff)             over every head's vdim values
    y = W_o (o * sigmoid(z))

A token sees the keys before it, those of a ``window``, or those of its own
chunk: the run of ``chunk`` positions, counted from position 0 of the sequence,
that it lies in.  Pages that no later token can see are given back.

Keys and values go to the request's pages first (keys [2 G][slot][dim], values
[G][vdim][slot]) and attention reads pages only, so a whole prompt, a portion
and a decoded token take one path.  Sizes in multiples of 16 (keys up to 128,
values up to 256) run on matrix-core kernels of their own, which keep both sums
in registers and finish the head; any other sizes take the row-by-row kernel,
which leaves the sums in 32-bit for one more kernel.
"""
from __future__ import annotations

from typing import Optional

import torch

from ..config.registry import MIXERS, POSITION_ENCODINGS
from ..config.specs import PartSpec
from ..kernels import ops
from .attention import AttentionWork
from .base import LayerCache, Mixer, PagedSpec, StepContext, WeightSource, WeightSpec

_WORK = AttentionWork()


@MIXERS.register("differential_attention")
class DifferentialAttention(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, dim: int, vdim: int, scale: float, diff: float,
                 eps: float, window: int = 0, chunk: int = 0, position: Optional[PartSpec] = None, pairing: str = "halves",
                 gate: bool = True, names: Optional[dict] = None):
        if num_heads <= 0 or num_kv_heads <= 0 or num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads do not split over {num_kv_heads} key/value heads")
        if dim <= 0 or vdim <= 0 or not scale > 0 or window < 0 or chunk < 0 or (window and chunk):
            raise ValueError(f"attention: heads of {dim}/{vdim}, scale {scale}, window {window}, chunk {chunk}")
        if pairing not in ops.PAIRINGS:
            raise ValueError(f"attention: pairing {pairing!r}; known: {sorted(ops.PAIRINGS)}")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.dim, self.vdim, self.scale, self.diff, self.eps = int(dim), int(vdim), float(scale), float(diff), float(eps)
        self.window, self.chunk, self.pairing, self.has_gate = int(window), int(chunk), pairing, bool(gate)
        self.position = POSITION_ENCODINGS.build(position) if position is not None else None
        if self.position is not None and self.position.rotary_dim > dim:
            raise ValueError("more rotated dimensions than a map has")
        n = dict(q="q", k="k", v="v", q_norm="q.norm", k_norm="k.norm", lq1="lq1", lk1="lk1", lq2="lq2", lk2="lk2", g="g", o="o")
        n.update(names or {})
        self.names = n
        self.matrix_cores = ops.paired_attn_fits_matrix_cores(self.dim, self.vdim)
        self.in_proj = self.o_proj = self.q_norm = self.k_norm = None
        self.lq1 = self.lk1 = self.lq2 = self.lk2 = None
        self.q_norm_f = self.k_norm_f = None
        self.take_off = 0.0          # lambda

    def weight_specs(self):
        n, H, G, C = self.names, self.num_heads, self.num_kv_heads, self.hidden_size
        sources = [WeightSource(n["q"], (H * 2 * self.dim, C)), WeightSource(n["k"], (G * 2 * self.dim, C)),
                   WeightSource(n["v"], (G * self.vdim, C))]
        if self.has_gate:
            sources.append(WeightSource(n["g"], (H * self.vdim, C)))
        specs = [WeightSpec("in_proj", tuple(sources)), WeightSpec("o_proj", (WeightSource(n["o"], (C, H * self.vdim)),)),
                 WeightSpec("q_norm", (WeightSource(n["q_norm"], (self.dim,)),), init="ones"),
                 WeightSpec("k_norm", (WeightSource(n["k_norm"], (self.dim,)),), init="ones")]
        return specs + [WeightSpec(a, (WeightSource(n[a], (self.dim,)),)) for a in ("lq1", "lk1", "lq2", "lk2")]

    def children(self):
        return {"rotary.": self.position} if self.position is not None else {}

    def materialize(self, device, dtype):
        super().materialize(device, dtype)
        self.q_norm_f, self.k_norm_f = self.q_norm.float().contiguous(), self.k_norm.float().contiguous()
        v = {a: getattr(self, a).double().cpu() for a in ("lq1", "lk1", "lq2", "lk2")}
        self.take_off = float(torch.exp((v["lq1"] * v["lk1"]).sum()) - torch.exp((v["lq2"] * v["lk2"]).sum())) + self.diff

    def cache_spec(self):
        return PagedSpec.keys_and_values(2 * self.num_kv_heads, self.dim, self.window, value_dim=self.vdim, chunk=self.chunk,
                                         value_heads=self.num_kv_heads)

    def step_planner(self):
        return _WORK if self.matrix_cores else None

    takes_pending_norm = True   # x may be an ops.PendingNorm: the fused product norms on its way in

    def forward(self, ctx: StepContext, x, cache: LayerCache):
        if not cache.writes:
            raise RuntimeError("this attention keeps its own keys and values")
        g, H, G = cache.group, self.num_heads, self.num_kv_heads
        pre = ops.linear(x, self.in_proj, out_dtype=torch.float32)
        q, _ = ops.qkv_prepare(
            pre, ctx.dtype, num_heads=2 * H, num_kv_heads=2 * G, dim=self.dim, vdim=self.vdim, slots=g.slot_mapping,
            kpool=cache.k, vpool=cache.v, page_size=g.page_size, norm="head", q_weight=self.q_norm_f, k_weight=self.k_norm_f,
            eps=self.eps, positions=ctx.positions, table=self.position.table if self.position is not None else None,
            pairing=self.pairing, value_heads=G)
        gate = pre[:, pre.shape[1] - H * self.vdim:] if self.has_gate else None
        finish = dict(take_off=self.take_off, post=1.0 - self.diff, eps=self.eps, gate=gate)
        if not self.matrix_cores:
            sums = torch.empty((ctx.T, H * 2 * self.vdim), dtype=torch.float32, device=q.device)
            ops.attn_rows(q, sums, cache.k, cache.v, g.block_tables, ctx.q_start, ctx.positions, ctx.ctx_len,
                          num_heads=2 * H, num_kv_heads=2 * G, dim=self.dim, vdim=self.vdim, scale=self.scale,
                          window=self.window, chunk=self.chunk, maps=2)
            out = ops.head_difference(sums, ctx.dtype, num_heads=H, vdim=self.vdim, **finish)
            return self._out(ctx, out)
        # a recorded step may hold rows that belong to no request: nothing writes them
        make = torch.zeros if ctx.fixed is not None and ctx.fixed.tokens else torch.empty
        out = make((ctx.T, H * self.vdim), dtype=ctx.dtype, device=q.device)
        sizes = dict(num_heads=H, num_kv_heads=G, dim=self.dim, vdim=self.vdim, window=self.window, chunk=self.chunk)
        work = ctx.plans[AttentionWork.key]
        meta = work.meta

        def spaces(launch):
            return [ctx.scratch(f"paired_{k}", launch[k]) if launch[k] else None for k in ("part_o", "part_ml")]

        if meta["n_tiles"]:
            launch = ops.paired_prefill_launch(meta["n_tiles"], meta["tile_keys"][1], ctx.dtype, **sizes)
            ops.paired_prefill(q, out, cache.k, cache.v, g.block_tables, ctx.q_start, ctx.ctx_len, work.arrays["tile_seq"],
                               work.arrays["tile_q0"], meta["n_tiles"], launch, *spaces(launch), scale=self.scale, **sizes,
                               **finish)
        if meta["n_dec"]:
            launch = ops.paired_decode_launch(meta["n_dec"], meta["max_ctx_dec"], **sizes)
            ops.paired_decode(q, out, cache.k, cache.v, g.block_tables, ctx.q_start, ctx.ctx_len, work.arrays.get("dec"),
                              meta["n_dec"], launch, *spaces(launch), scale=self.scale, **sizes, **finish)
        return self._out(ctx, out)

    def _out(self, ctx: StepContext, out):
        return ops.linear(out, self.o_proj, out_dtype=ctx.dtype, may_split=True, pending=True)
