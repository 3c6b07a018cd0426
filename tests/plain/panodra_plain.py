"""A plain, slow Panodra in torch on the CPU: whole sequences, no cache, no
pages, one function per mechanism.  It is what the engine is compared with and
shares no code with it (it imports nothing from the package; a model folder is
read with the safetensors library).

Panodra is a pre-norm decoder whose norms bend every feature through a tanh
instead of dividing by a row's size.  Its attention keeps one low-rank latent
and one rotated key part per token for all heads; one kind of layer stretches
the rotation's slow frequencies and has a learned sink in the softmax, the other
has neither.  The feed-forward is a dense layer with a squared relu, or a few of
many gated experts that a table picks by the token's id.  A stretch of layers
may run several times; every pass starts from a projection of the stream beside
the embedding's output.  Logits are the embedding's products, scaled and capped.
Everything here runs in the precision of the tensors it is given (the tests use
64-bit).

Notation: x the residual stream [n, width]; W matrices stored [out, in]; a
sequence's positions count from 0.
"""
from __future__ import annotations

import json
import math
import os

import torch


# ------------------------------------------------------------------ small parts
def tanh_norm(x: torch.Tensor, alpha: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """tanh(alpha x) * weight + bias, feature by feature; no statistics of the row."""
    return torch.tanh(alpha * x) * weight + bias


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * weight, the eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * weight


def squared_relu(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# --------------------------------------------------------------------- rotation
def stretched_frequencies(base: float, dims: int, scaling: dict | None) -> list:
    """base^(-2i/dims) for every pair i.  With ``scaling``: pairs that turn more than ``fast`` times
    within ``original`` positions keep their frequency, pairs that turn less than ``slow`` times have
    it divided by ``factor``, and between the two pair numbers (rounded outwards) the share of the
    divided frequency grows in a straight line."""
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return plain

    def pair_that_turns(t):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_that_turns(scaling["fast"])), 0)
    hi = min(math.ceil(pair_that_turns(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        share = (i - lo) / max(hi - lo, 0.001)
        share = min(max(share, 0.0), 1.0)
        out.append(f / scaling["factor"] * share + f * (1.0 - share))
    return out


def rotation_gain(scaling: dict | None) -> float:
    """What cosines and sines are multiplied by."""
    return 1.0 if scaling is None else 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(v: torch.Tensor, positions: torch.Tensor, rot: dict) -> torch.Tensor:
    """Neighbouring entries (2i, 2i+1) of the first ``rot["dims"]`` of the last axis turn by
    position * f_i (and are multiplied by the rotation's gain); the rest passes.  v [n, ..., D]."""
    dims = rot["dims"]
    out = v.clone()
    freq = torch.tensor(stretched_frequencies(rot["base"], dims, rot.get("scaling")), dtype=v.dtype)
    angle = positions.to(v.dtype)[:, None] * freq[None, :]
    shape = [v.shape[0]] + [1] * (v.dim() - 2) + [dims // 2]
    gain = rotation_gain(rot.get("scaling"))
    cos, sin = (gain * angle.cos()).reshape(shape), (gain * angle.sin()).reshape(shape)
    a, b = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = a * cos - b * sin
    out[..., 1:dims:2] = b * cos + a * sin
    return out


# -------------------------------------------------------------------- attention
def causal_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float,
                             sink: torch.Tensor | None) -> torch.Tensor:
    """One sequence, q and k [n, H, Dk], v [n, H, Dv]: weights_ij = exp(s_ij) over the sum of
    exp(s_ij') for j' <= i, plus exp(sink_h) where there is a sink; s = scale * q.k."""
    n, H = q.shape[0], q.shape[1]
    out = torch.zeros(n, H, v.shape[-1], dtype=q.dtype)
    ok = torch.ones(n, n).tril().bool()
    for h in range(H):
        s = ((q[:, h] @ k[:, h].T) * scale).masked_fill(~ok, float("-inf"))
        m = s.max(dim=-1).values
        if sink is not None:
            m = torch.maximum(m, sink[h])
        e = torch.exp(s - m[:, None])
        denom = e.sum(-1)
        if sink is not None:
            denom = denom + torch.exp(sink[h] - m)
        out[:, h] = (e / denom[:, None]) @ v[:, h]
    return out


def latent_attention(h: torch.Tensor, w: dict, m: dict, eps: float, sink: bool) -> torch.Tensor:
    """Queries straight from h; keys and values out of one normed latent per token, with one rotated
    key part for all heads.  w: the layer's 'mix.*' tensors by their short names."""
    n = h.shape[0]
    H, dim, rot, vdim, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(n)
    q = (h @ w["q"].T).reshape(n, H, dim + rot)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :rank], w["dkv.norm"], eps)
    k_plain = (c @ w["uk"].T).reshape(n, H, dim)
    v = (c @ w["uv"].T).reshape(n, H, vdim)
    q_rot, k_rot = q[..., dim:], down[:, None, rank:]
    if rot:
        q_rot, k_rot = rotate_pairs(q_rot, pos, m["rot"]), rotate_pairs(k_rot, pos, m["rot"])
    qq = torch.cat((q[..., :dim], q_rot), dim=-1)
    kk = torch.cat((k_plain, k_rot.expand(n, H, rot)), dim=-1)
    o = causal_softmax_attention(qq, kk, v, m["scale"], w["sink"] if sink else None)
    return o.reshape(n, H * vdim) @ w["o"].T


# ----------------------------------------------------------------- feed-forward
def dense_ff(h: torch.Tensor, w: dict) -> torch.Tensor:
    return squared_relu(h @ w["up"].T) @ w["down"].T


def expert(h: torch.Tensor, w: dict, e: int) -> torch.Tensor:
    return (silu(h @ w[f"e{e}.gate"].T) * (h @ w[f"e{e}.up"].T)) @ w[f"e{e}.down"].T


def table_experts(h: torch.Tensor, tokens, w: dict) -> torch.Tensor:
    """Row t goes to the experts that its token's row of the table names, each with weight 1 / top."""
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        row = [int(e) for e in w["table"][int(tok)]]
        for e in row:
            out[t] += expert(h[t:t + 1], w, e)[0] / len(row)
    return out


# ------------------------------------------------------------------------- ends
def enter_pass(x: torch.Tensor, x0: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """W [x; x0], the stream's half of the columns first."""
    return torch.cat((x, x0), dim=-1) @ w.T


def capped_logits(x: torch.Tensor, table: torch.Tensor, scale: float, cap: float | None) -> torch.Tensor:
    z = x @ table.T * scale
    return z if cap is None else cap * torch.tanh(z / cap)


# ------------------------------------------------------------------------- model
def layer_order(n_layers: int, loop) -> list:
    """[(layer, whether a pass begins right before it)] in running order."""
    if not loop:
        return [(i, False) for i in range(n_layers)]
    start, stop, times = loop["start"], loop["stop"], loop["times"]
    once = [(i, i == start) for i in range(start, stop)]
    return [(i, False) for i in range(start)] + once * times + [(i, False) for i in range(stop, n_layers)]


def sub(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def norm_of(x: torch.Tensor, tensors: dict, name: str) -> torch.Tensor:
    return tanh_norm(x, tensors[name + ".alpha"], tensors[name], tensors[name + ".b"])


def forward(tokens, tensors: dict, config: dict, trace: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one whole sequence.  ``trace`` collects the residual
    stream after every layer run."""
    eps = config["norm"]["eps"]
    x = tensors["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x0 = x
    for i, begins in layer_order(len(config["layers"]), config.get("loop")):
        lc, p = config["layers"][i], f"l{i}."
        if begins:
            x = enter_pass(x, x0, tensors["loop.in"])
        h = norm_of(x, tensors, p + "norm1")
        sink = {"latent_attention": True, "latent_attention_2": False}[lc["type"]]
        x = x + latent_attention(h, sub(tensors, p + "mix."), lc["mixer"], eps, sink)
        if lc.get("mlp"):
            h, w = norm_of(x, tensors, p + "norm2"), sub(tensors, p + "mlp.")
            x = x + (dense_ff(h, w) if lc["mlp"]["kind"] == "dense" else table_experts(h, tokens, w))
        if trace is not None:
            trace.append(x.clone())
    return capped_logits(norm_of(x, tensors, "final.norm"), tensors["embed"], config.get("logit_scale", 1.0),
                         config.get("logit_softcap"))


def load_folder(folder: str, dtype=torch.float64):
    from safetensors import safe_open

    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        for k in f.keys():
            t = f.get_tensor(k)
            tensors[k] = t.to(dtype) if t.is_floating_point() else t
    return config, tensors
