"""A plain, slow Pudulorn in torch on the CPU: whole sequences, no cache, no
pages, one function per mechanism.  It is what the engine is compared with and
shares no code with it (it imports nothing from the package; a model folder is
read with the safetensors library).

Pudulorn is a pre-norm decoder of two kinds of layer in any order.  One attends
through low-rank latents, queries included, within a sliding window, and may
read the latents another layer has stored.  The other is differential attention
within chunks of fixed length: two softmax maps per head over the same values,
of which one is taken off the other, normed and gated.  Feed-forwards are a
dense layer whose gate and up products are limited, or a few of many experts
whose softmax scores are used as they are, beside one that every token uses
through a gate of its own.  Everything here runs in the precision of the tensors
it is given (the tests use 64-bit).

Notation: x the residual stream [n, width]; W matrices stored [out, in]; a
sequence's positions count from 0.
"""
from __future__ import annotations

import json
import os

import torch

GATE_SLOPE = 1.702


# ------------------------------------------------------------------ small parts
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * weight


def shifted_rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The stored weight is the distance of the multiplier from one."""
    return unit_rms(x, eps) * (1.0 + weight)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def rotate_halves(v: torch.Tensor, positions: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """Entry i and entry i + dims/2 of the first ``dims`` of the last axis turn together by
    position * base^(-2i/dims); entries from ``dims`` on pass.  v [n, ..., D]."""
    half = dims // 2
    out = v.clone()
    shape = [v.shape[0]] + [1] * (v.dim() - 2)
    for i in range(half):
        a = (positions.to(v.dtype) * base ** (-2.0 * i / dims)).reshape(shape)
        out[..., i] = v[..., i] * a.cos() - v[..., i + half] * a.sin()
        out[..., i + half] = v[..., i + half] * a.cos() + v[..., i] * a.sin()
    return out


# ---------------------------------------------------------------- who sees whom
def window_mask(n: int, size) -> torch.Tensor:
    """[n, n]: row i sees column j when j is i itself or one of the size - 1 before it (None: every j <= i)."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def chunk_mask(n: int, size) -> torch.Tensor:
    """[n, n]: row i sees column j <= i of its own chunk of ``size`` positions, counted from position 0."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i // size == j // size)


def softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, ok: torch.Tensor) -> torch.Tensor:
    """One head: q, k [n, D], v [n, V], ok [n, n]."""
    s = ((q @ k.T) * scale).masked_fill(~ok, float("-inf"))
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return (e / e.sum(-1, keepdim=True)) @ v


def mask_size(m: dict):
    return m["mask"]["size"] if m.get("mask") else None


# -------------------------------------------------------------- latent attention
def latents_of(h: torch.Tensor, w: dict, m: dict, eps: float):
    """What a layer keeps per token: the normed latent [n, rank] and the rotated key part [n, rot_dim]."""
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :m["kv_rank"]], w["dkv.norm"], eps)
    r = down[:, m["kv_rank"]:]
    if m["rot_dim"]:
        r = rotate_halves(r, torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])
    return c, r


def latent_attention(h: torch.Tensor, w: dict, m: dict, eps: float, kept) -> torch.Tensor:
    """``kept``: the latents and rotated key parts that this layer reads, its own or another's."""
    n, H, dim, rot, vdim = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, r = kept
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(n, H, dim + rot)
    k_plain, v = (c @ w["uk"].T).reshape(n, H, dim), (c @ w["uv"].T).reshape(n, H, vdim)
    ok = window_mask(n, mask_size(m))
    out = torch.zeros(n, H, vdim, dtype=h.dtype)
    for a in range(H):
        q_rot = rotate_halves(q[:, a, dim:], torch.arange(n), m["rot"]["base"], m["rot"]["dims"]) if rot else q[:, a, dim:]
        out[:, a] = softmax_attention(torch.cat((q[:, a, :dim], q_rot), -1), torch.cat((k_plain[:, a], r), -1), v[:, a],
                                      m["scale"], ok)
    return out.reshape(n, H * vdim) @ w["o"].T


# -------------------------------------------------------- differential attention
def take_off(w: dict, diff: float) -> torch.Tensor:
    """How much of the second map is taken off the first: one number for the layer."""
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def differential_attention(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n, H, G, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(n)
    q = rms_norm((h @ w["q"].T).reshape(n, H, 2, dim), w["q.norm"], eps)
    k = rms_norm((h @ w["k"].T).reshape(n, G, 2, dim), w["k.norm"], eps)
    v = (h @ w["v"].T).reshape(n, G, vdim)
    if m.get("rot") and m["rot"]["dims"]:
        q = rotate_halves(q, pos, m["rot"]["base"], m["rot"]["dims"])
        k = rotate_halves(k, pos, m["rot"]["base"], m["rot"]["dims"])
    lam, ok = take_off(w, m["diff"]), chunk_mask(n, mask_size(m))
    out = torch.zeros(n, H, vdim, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        first, second = (softmax_attention(q[:, a, s], k[:, g, s], v[:, g], m["scale"], ok) for s in (0, 1))
        out[:, a] = unit_rms(first - lam * second, eps) * (1.0 - m["diff"])
    return (out.reshape(n, H * vdim) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ----------------------------------------------------------------- feed-forward
def limited_ff(h: torch.Tensor, w: dict, limit: float) -> torch.Tensor:
    """The gate has an upper limit, the up product one on both sides and one added."""
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w["down"].T


def gated_ff(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h: torch.Tensor, router: torch.Tensor, top: int, scale: float):
    """-> the chosen experts [n, top], best first, and their weights: scores over all experts, times scale."""
    s = torch.softmax(h @ router.T, dim=-1)
    best = torch.topk(s, top, dim=-1)
    return best.indices, best.values * scale


def expert_ff(h: torch.Tensor, w: dict, m: dict, choices: torch.Tensor | None = None) -> torch.Tensor:
    """``choices`` [n, top]: experts to use in place of the router's own (their scores stay the router's)."""
    chosen, weight = route(h, w["router"], m["router"]["top"], m["router"]["scale"])
    if choices is not None:
        chosen = choices
        weight = torch.softmax(h @ w["router"].T, dim=-1).gather(1, chosen) * m["router"]["scale"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, b in zip(chosen[t].tolist(), weight[t]):
            out[t] += b * gated_ff(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])[0]
    if m.get("shared"):
        share = torch.sigmoid(h @ w["shared.sg"].T)
        out = out + share * gated_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


# ------------------------------------------------------------------------- model
def sub(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(tokens, tensors: dict, config: dict, trace: list | None = None, choices: list | None = None,
            log: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one whole sequence.  ``trace`` collects the residual stream after every
    layer; ``choices`` gives the experts of every routed layer in their order (see ``expert_ff``), ``log``
    receives every routed layer's router logits."""
    eps = config["norm"]["eps"]
    x = tensors["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept, routed = {}, 0
    for i, lc in enumerate(config["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        h, w = shifted_rms_norm(x, tensors[p + "norm1"], eps), sub(tensors, p + "mix.")
        if lc["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                kept[i] = latents_of(h, w, m, eps)
            x = x + latent_attention(h, w, m, eps, kept[i if source is None else source])
        else:
            x = x + differential_attention(h, w, m, eps)
        if lc.get("mlp"):
            h, w = shifted_rms_norm(x, tensors[p + "norm2"], eps), sub(tensors, p + "mlp.")
            if lc["mlp"]["kind"] == "dense":
                x = x + limited_ff(h, w, lc["mlp"]["limit"])
            else:
                if log is not None:
                    log.append(h @ w["router"].T)
                x = x + expert_ff(h, w, lc["mlp"], None if choices is None else choices[routed])
                routed += 1
        if trace is not None:
            trace.append(x.clone())
    return shifted_rms_norm(x, tensors["final.norm"], eps) @ tensors["head"].T


def load_folder(folder: str, dtype=torch.float64):
    from safetensors import safe_open

    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        for k in f.keys():
            tensors[k] = f.get_tensor(k).to(dtype)
    return config, tensors
