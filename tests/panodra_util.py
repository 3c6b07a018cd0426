"""Small Panodra models with random weights for the tests, and their logits by
the plain implementation (tests/plain/panodra_plain.py, 64-bit)."""
import json
import os

import torch

from plain import panodra_plain as PP


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff):
    return dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))


def latent(heads, dim, rot_dim, vdim, kv_rank, *, scale=None, base=10000.0, dims=None, yarn=None, sink=True, mlp=None):
    """yarn: (factor, original, fast, slow) or None."""
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank,
             scale=scale if scale is not None else (dim + rot_dim) ** -0.5)
    if rot_dim:
        m["rot"] = dict(base=base, dims=rot_dim if dims is None else dims)
        if yarn is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return dict(type="latent_attention" if sink else "latent_attention_2", mixer=m, mlp=mlp)


def config(vocab, width, layers, *, loop=None, eps=1e-6, scale=1.0, cap=20.0):
    d = dict(architecture="Panodra", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)
    if scale is not None:
        d["logit_scale"] = scale
    if cap is not None:
        d["logit_softcap"] = cap
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def random_config(rng) -> dict:
    """A configuration drawn at random: width, vocabulary, one to six layers of either kind in any
    order, sizes that the matrix-core kernels take and others, rotations of the whole part or of some of
    it, stretched or not, one expert and many, looped stretches anywhere, caps and scales."""
    width = rng.choice([48, 64, 72, 96, 128, 160, 192, 256])
    layers = []
    for _ in range(rng.randint(1, 6)):
        kind = rng.random()
        if kind < 0.15:
            mlp = None
        elif kind < 0.55:
            mlp = dense(rng.choice([16, 40, 64, 100, 192, 320]))
        else:
            experts = rng.choice([1, 2, 3, 5, 8, 16, 40])
            mlp = moe(experts, rng.randint(1, min(experts, 5)), rng.choice([8, 20, 32, 64, 96]))
        # sizes of the prepared matrix-core libraries, or any for the row-by-row kernel
        kv, rot = rng.choice([(16, 16), (32, 16), (48, 16), (64, 16), (64, 32), (64, 64), (96, 16), (128, 32), (16, 0), (48, 0),
                              (20, 8), (40, 6), (72, 14), (25, 10)])
        yarn = None
        if rng.random() < 0.5:
            yarn = (rng.choice([1.0, 2.0, 4.0, 16.0]), rng.choice([32, 100, 1024]), rng.choice([8.0, 32.0]), rng.choice([0.5, 1.0, 2.0]))
        dim = rng.choice([0, 8, 10, 16, 32, 48]) if rot else rng.choice([8, 16, 30])
        layers.append(latent(rng.choice([1, 2, 3, 4, 6, 8]), dim, rot, rng.choice([4, 8, 12, 16, 32, 40]), kv,
                             scale=round((dim + rot) ** -0.5 * rng.uniform(0.7, 2.0), 4), base=rng.choice([100.0, 1e4, 2.5e5]),
                             yarn=yarn, sink=rng.random() < 0.5, mlp=mlp))
    loop = None
    if rng.random() < 0.7:
        start = rng.randint(0, len(layers) - 1)
        loop = (start, rng.randint(start + 1, len(layers)), rng.randint(1, 3))
    return config(rng.randint(100, 600), width, layers, loop=loop, eps=rng.choice([1e-6, 1e-5]),
                  scale=rng.choice([0.25, 0.5, 1.0, 2.0]), cap=rng.choice([None, 5.0, 15.0, 50.0]))


# Three configurations that differ in every size and option; none of their sizes coincide where a
# model's might by chance (plain and value sizes, heads x value size and width, latent and width,
# experts and chosen ones).
#   A: odd sizes (the row-by-row attention, the scalar paths), a loop in the middle that runs three
#      times, a layer without feed-forward, fewer rotated dimensions than the rotated part has in one
#      layer, five experts of which two are used, a stretch whose borders lie inside the pairs
#   B: one head, one expert, no loop, no scaling of logits, a head without a plain part
#   C: sizes in multiples of 64 (the products of few rows that end in the norm, the matrix-core
#      attention), a loop from the first layer on that runs twice, twelve experts of which three are used
CONFIGS = {
    "A": config(203, 72, [
        latent(2, 10, 8, 14, 40, yarn=(4.0, 64, 8.0, 1.0), mlp=dense(100)),
        latent(3, 12, 14, 20, 24, dims=10, base=500.0, sink=False, mlp=moe(5, 2, 28)),
        latent(5, 6, 10, 8, 36, base=100.0, scale=0.4, yarn=(3.0, 40, 6.0, 0.5), mlp=moe(7, 3, 36)),
        latent(2, 20, 6, 18, 28, sink=False),
    ], loop=(1, 3, 3), eps=1e-5, scale=0.6, cap=12.0),
    "B": config(150, 64, [
        latent(1, 0, 16, 40, 48, sink=False, mlp=moe(1, 1, 48)),
        latent(1, 24, 0, 12, 16, mlp=dense(72)),
        latent(6, 8, 16, 24, 64, yarn=(2.0, 1000, 32.0, 1.0), mlp=None),
    ], eps=1e-6, scale=1.0, cap=50.0),
    "C": config(320, 128, [
        latent(4, 32, 16, 48, 64, yarn=(8.0, 64, 32.0, 1.0), base=20000.0, mlp=moe(12, 3, 64)),
        latent(8, 16, 32, 16, 128, sink=False, mlp=dense(192)),
        latent(2, 64, 64, 64, 64, sink=False, base=1e6, mlp=moe(4, 2, 128)),
        latent(4, 16, 16, 32, 96, mlp=dense(256)),
    ], loop=(0, 2, 2), eps=1e-6, scale=0.3, cap=15.0),
}
BLOCK_SIZE = {"A": 4, "B": 16, "C": 16}


def write_model(folder: str, cfg: dict, seed: int, dtype: str, std: float = 0.15) -> str:
    """config.json and model.safetensors with weights drawn so that faults show and rounding does not
    (from a ``std`` of 0.25 on these models turn a rounding step into a change of everything): attention
    that is not flat, sinks of order one, norms that bend without being flat, weights and
    biases of the norms away from one and zero, a table whose rows name different experts."""
    from lyapunov_engine_amd.config.registry import architecture_of
    from lyapunov_engine_amd.models.decoder import build_model
    from lyapunov_engine_amd.weights.safetensors_io import write_safetensors

    arch = architecture_of(cfg)
    model = build_model(arch.to_spec(arch.config_class.from_dict(cfg)))
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, (shape, init) in model.expected_tensors().items():
        if init.startswith("choices:"):
            tensors[name] = torch.rand((shape[0], int(init[8:])), generator=g).argsort(dim=1)[:, :shape[1]].to(torch.int32).contiguous()
            continue
        t = torch.randn(shape, generator=g)
        if name.endswith(".alpha"):
            t = 0.6 + 0.15 * t
        elif init == "ones":
            t = 1.0 + 0.3 * t
        elif name.endswith(".b"):
            t = 0.3 * t
        elif name.endswith(".sink"):
            t = 1.5 * t
        elif name == "embed":
            t = t * 1.0
        elif name == "loop.in":
            t = t * 0.8 * shape[-1] ** -0.5
        else:
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
        _PLAIN[folder] = PP.load_folder(folder)
    return _PLAIN[folder]


def forget(folder):
    _PLAIN.pop(folder, None)


def plain_logits(folder: str, requests: dict) -> dict:
    """id -> [len, vocab] 64-bit logits of every whole request."""
    cfg, tensors = _loaded(folder)
    return {rid: PP.forward(toks, tensors, cfg) for rid, toks in requests.items()}


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
