"""Small Pudulorn models with random weights for the tests, and their logits by
the plain implementation (tests/plain/pudulorn_plain.py, 64-bit)."""
import json
import os

import torch

from plain import pudulorn_plain as DP
from ronupel_util import RouterLog  # noqa: F401  (the routed layers' choices, sorted by request)


def dense(ff, limit=1.5):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts, top, ff, shared=None, scale=2.0):
    d = dict(kind="moe", router=dict(experts=experts, top=top, scale=scale), expert=dict(ff=ff))
    if shared:
        d["shared"] = dict(ff=shared)
    return d


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, *, window=None, scale=None, base=10000.0, dims=None, kv_from=None, mlp=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
             scale=scale if scale is not None else (dim + rot_dim) ** -0.5)
    if rot_dim:
        m["rot"] = dict(base=base, dims=rot_dim if dims is None else dims)
    if window is not None:
        m["mask"] = dict(size=window)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=m, mlp=mlp)


def pairs(heads, kv_heads, dim, vdim, *, chunk=None, scale=None, diff=0.4, base=10000.0, dims=None, mlp=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else dim ** -0.5, diff=diff,
             rot=dict(base=base, dims=dim if dims is None else dims))
    if chunk is not None:
        m["mask"] = dict(size=chunk)
    return dict(type="attention", mixer=m, mlp=mlp)


def config(vocab, width, layers, *, eps=1e-6):
    return dict(architecture="Pudulorn", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)


def random_config(rng) -> dict:
    """A configuration drawn at random: width, vocabulary, one to six layers of either kind in any
    order, sizes that the matrix-core kernels take and others, windows and chunks from one position on,
    layers that read the latents of any earlier one, one expert and many, a shared expert of the experts'
    size, of another, or none."""
    width = rng.choice([48, 64, 72, 96, 128, 160, 192, 256])
    layers = []
    for i in range(rng.randint(1, 6)):
        kind = rng.random()
        if kind < 0.15:
            mlp = None
        elif kind < 0.55:
            mlp = dense(rng.choice([16, 40, 64, 100, 150, 320]), rng.choice([0.5, 1.0, 2.5, 7.0]))
        else:
            experts, ff = rng.choice([1, 2, 3, 5, 8, 16, 40]), rng.choice([8, 20, 32, 64, 96])
            mlp = moe(experts, rng.randint(1, min(experts, 5)), ff, rng.choice([None, ff, 24, 50, 128]), rng.choice([0.5, 1.0, 2.5]))
        if rng.random() < 0.5:
            heads, dim = rng.choice([1, 2, 3, 4, 6, 8]), rng.choice([0, 8, 10, 16, 32, 48])
            vdim, window = rng.choice([4, 8, 12, 16, 32, 40]), rng.choice([None, 1, 2, 7, 16, 33, 64, 100])
            base = rng.choice([100.0, 1e4, 2.5e5])
            own = [j for j, l in enumerate(layers) if l["type"] == "latent_attention" and "kv_from" not in l["mixer"]]
            if own and rng.random() < 0.5:
                j = rng.choice(own)
                m = layers[j]["mixer"]
                kv, rot, source = m["kv_rank"], m["rot_dim"], j
                base, dims = (m["rot"]["base"], m["rot"]["dims"]) if rot else (base, None)
            else:
                kv, rot = rng.choice([(16, 16), (32, 16), (48, 16), (64, 32), (96, 16), (16, 0), (48, 0), (20, 8), (40, 6), (72, 14)])
                source, dims = None, rng.choice([rot, rot, max(0, rot - 4)])
            if not rot and not dim:
                dim = 12
            layers.append(latent(heads, dim, rot, vdim, rng.choice([12, 24, 40, 64]), kv, window=window, base=base, dims=dims,
                                 scale=round((dim + rot) ** -0.5 * rng.uniform(0.7, 2.0), 4), kv_from=source, mlp=mlp))
        else:
            kv = rng.choice([1, 2, 3, 4])
            dim, vdim = rng.choice([(16, 16), (16, 32), (32, 16), (32, 48), (32, 64), (48, 80), (10, 24), (6, 7), (24, 18), (14, 40)])
            layers.append(pairs(kv * rng.choice([1, 1, 2, 3, 5]), kv, dim, vdim, chunk=rng.choice([None, 1, 3, 16, 24, 50, 64, 100]),
                                scale=round(dim ** -0.5 * rng.uniform(0.7, 1.5), 4), diff=rng.choice([0.2, 0.35, 0.7]),
                                base=rng.choice([100.0, 1e4]), dims=rng.choice([dim, dim, dim // 4 * 2]), mlp=mlp))
    return config(rng.randint(100, 600), width, layers, eps=rng.choice([1e-6, 1e-5]))


# Three configurations that differ in every size and option; none of their sizes coincide where a
# model's might by chance (plain and value sizes, heads and key/value heads, window and chunk and
# page, query rank and latent, experts and chosen ones, the shared expert and the others).
#   A: odd sizes (the row-by-row attention, the scalar paths), fewer rotated dimensions than there are in
#      some layers, a reader with a wider window than its source's and one that sees everything, a layer
#      without feed-forward, a shared expert of the experts' size
#   B: one head, one expert without a shared one, no masks, a head without a plain part, one without rotation
#   C: sizes in multiples of 16 (the matrix-core attention; products of few rows that end in the norm),
#      several query heads a key/value head, a reader with a narrower window than its source's, short chunks
CONFIGS = {
    "A": config(203, 72, [
        latent(2, 10, 8, 14, 18, 40, window=21, mlp=dense(100)),
        pairs(6, 3, 10, 26, chunk=24, diff=0.25, mlp=moe(5, 2, 28, 28, scale=1.7)),
        latent(3, 12, 8, 20, 30, 40, window=50, kv_from=0, scale=0.3, mlp=moe(7, 3, 36, 44)),
        pairs(2, 2, 14, 9, chunk=7, dims=6, base=500.0),
        latent(5, 6, 14, 8, 22, 36, window=9, dims=10, base=100.0, mlp=dense(52, 0.6)),
        latent(4, 8, 14, 16, 26, 36, dims=10, base=100.0, kv_from=4),
    ], eps=1e-5),
    "B": config(150, 64, [
        latent(1, 0, 16, 40, 20, 48, mlp=moe(1, 1, 48, scale=0.7)),
        pairs(1, 1, 16, 32, mlp=dense(72, 3.0)),
        latent(1, 24, 0, 12, 16, 16),
        pairs(6, 2, 32, 16, dims=8, mlp=moe(3, 3, 24, 40, scale=1.0)),
    ], eps=1e-6),
    "C": config(320, 128, [
        latent(4, 32, 16, 48, 96, 64, window=40, base=20000.0, mlp=dense(192)),
        pairs(8, 2, 32, 64, chunk=48, diff=0.3, mlp=moe(12, 3, 64, 96, scale=2.5)),
        latent(8, 16, 16, 32, 64, 64, window=17, base=20000.0, kv_from=0, mlp=moe(6, 2, 48, 48)),
        pairs(4, 4, 48, 80, chunk=20, dims=24, mlp=dense(256, 0.9)),
        pairs(6, 2, 16, 32, chunk=90, diff=0.6),
    ], eps=1e-6),
}
BLOCK_SIZE = {"A": 4, "B": 16, "C": 16}


def write_model(folder: str, cfg: dict, seed: int, dtype: str, std: float = 0.15) -> str:
    """config.json and model.safetensors with weights drawn so that faults show and rounding does not:
    attention that is not flat, second maps that take off a good part of the first, norm weights away from
    their neutral values (around zero where the design adds one), gates on both sides of zero."""
    from lyapunov_engine_amd.config.registry import architecture_of
    from lyapunov_engine_amd.models.decoder import build_model
    from lyapunov_engine_amd.weights.safetensors_io import write_safetensors

    arch = architecture_of(cfg)
    model = build_model(arch.to_spec(arch.config_class.from_dict(cfg)))
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, (shape, init) in model.expected_tensors().items():
        t = torch.randn(shape, generator=g)
        if init == "ones":
            t = 1.0 + 0.3 * t
        elif name.endswith(("norm1", "norm2", "final.norm")):
            t = 0.3 * t
        elif name.endswith((".lq1", ".lk1", ".lq2", ".lk2")):
            t = t.abs() * 0.7 * shape[-1] ** -0.5 if name[-3:] in ("lq2", "lk2") else t * 0.5 * shape[-1] ** -0.25
            if name.endswith(".lk2"):
                t = -t                            # what is taken off lies around one half of the first map
        elif name.endswith((".router", ".shared.sg")):
            t = t * 1.5 * shape[-1] ** -0.5
        elif name != "embed":
            t = t * std * (64.0 / shape[-1]) ** 0.5
        tensors[name] = t.to(torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    os.makedirs(folder, exist_ok=True)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors, metadata={"format": "pt"})
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return folder


_PLAIN: dict = {}


def _loaded(folder):
    if folder not in _PLAIN:
        _PLAIN[folder] = DP.load_folder(folder)
    return _PLAIN[folder]


def forget(folder):
    _PLAIN.pop(folder, None)


def plain_logits(folder: str, requests: dict) -> dict:
    """id -> [len, vocab] 64-bit logits of every whole request."""
    cfg, tensors = _loaded(folder)
    return {rid: DP.forward(toks, tensors, cfg) for rid, toks in requests.items()}


def plain_logits_routed_alike(folder: str, requests: dict, chosen: dict, clear: float = 0.4) -> dict:
    """As ``plain_logits`` with the experts the engine chose (id -> a tensor [len, top] per routed layer).  A 16-bit
    run may decide a close call the other way, which says nothing about its kernels; what it must not do is choose
    otherwise where the plain model's margin, on the same history, is clear: that is asserted here."""
    cfg, tensors = _loaded(folder)
    tops = [lc["mlp"]["router"]["top"] for lc in cfg["layers"] if lc.get("mlp") and lc["mlp"]["kind"] == "moe"]
    out = {}
    for rid, toks in requests.items():
        log = []
        picks = [c.long() for c in chosen[rid]]
        out[rid] = DP.forward(toks, tensors, cfg, choices=picks, log=log)
        for n, (z, mine, top) in enumerate(zip(log, picks, tops)):
            # every expert taken scores at least as much as the best one left, but for a close call
            taken = torch.zeros_like(z, dtype=torch.bool).scatter_(1, mine, True)
            assert int(taken.sum()) == taken.shape[0] * top, f"request {rid!r}, routed layer {n}: an expert chosen twice"
            if top == z.shape[1]:
                continue
            worst = z.masked_fill(~taken, float("inf")).min(-1).values
            best_left = z.masked_fill(taken, float("-inf")).max(-1).values
            gap = best_left - worst
            at = int(gap.argmax())
            assert float(gap[at]) < clear, (f"request {rid!r}, routed layer {n}, position {at}: chose {mine[at].tolist()} with "
                                            f"an expert left out that scores {float(gap[at]):.3f} more")
    return out


def plain_sensitivity(folder: str, requests: dict, chosen: dict, rel: float = 2.0 ** -9) -> dict:
    """id -> [len]: by how much a row's logits move when every matrix entry is changed by up to one rounding step of a
    16-bit number, the experts being those of ``chosen``.  Two maps of a head may nearly cancel, and what is left
    of them is normed: such a row carries its rounding many times enlarged, and this is the measure of it."""
    cfg, tensors = _loaded(folder)
    out = {}
    for rid, toks in requests.items():
        picks = [c.long() for c in chosen[rid]]
        base, worst = DP.forward(toks, tensors, cfg, choices=picks), 0.0
        for seed in (0, 1):
            g = torch.Generator().manual_seed(seed)
            moved = {k: v * (1.0 + rel * (2.0 * torch.rand(v.shape, generator=g, dtype=v.dtype) - 1.0)) if v.dim() >= 2 else v
                     for k, v in tensors.items()}
            worst = torch.clamp((DP.forward(toks, moved, cfg, choices=picks) - base).abs().max(-1).values, min=worst)
        out[rid] = worst
    return out


def plain_greedy(folder: str, prompt: list, n: int):
    """n greedy tokens after the prompt, and the margin between the best two logits at each."""
    toks, out, margins = list(prompt), [], []
    for _ in range(n):
        row = plain_logits(folder, {"g": toks})["g"][-1]
        top = torch.topk(row, 2)
        out.append(int(top.indices[0]))
        margins.append(float(top.values[0] - top.values[1]))
        toks.append(out[-1])
    return out, margins


def edit(folder, change):
    """Rewrite a written model's tensors: ``change(tensors)`` edits the dict name -> tensor in place."""
    from safetensors.torch import load_file

    from lyapunov_engine_amd.weights.safetensors_io import write_safetensors

    path = os.path.join(folder, "model.safetensors")
    tensors = dict(load_file(path))
    change(tensors)
    write_safetensors(path, tensors, metadata={"format": "pt"})
    forget(folder)
