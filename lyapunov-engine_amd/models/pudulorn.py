"""The Pudulorn architecture as a ModelSpec.

A pre-norm decoder (every norm multiplies by one plus its stored weight) with
two kinds of layer in any order:

  "latent_attention"  attention over one low-rank latent and one rotated key part per token, queries
                      out of a latent of their own, within a sliding window; a layer may read the
                      latents that an earlier one keeps (``kv_from``: its call names that layer's cache
                      buffer and writes nothing);
  "attention"         differential attention within chunks: two softmax maps a head over the same
                      values, normed queries and keys, a gate on every output value.

Rotations turn halves (i, i + dims / 2).  The feed-forward is dense with limited gate and up products, or a few
of many silu-gated experts weighted by their shares of the softmax over all, beside an expert that
every token uses through a gate of its own, or absent.  The output head is a matrix of its own.

Tensor names: ``embed``, ``l<i>.norm1`` / ``norm2``,
``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}`` or
``l<i>.mix.{q,k,v,q.norm,k.norm,lq1,lk1,lq2,lk2,g,o}``, ``l<i>.mlp.{gate,up,down}`` or
``l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down,sg}}``, ``final.norm``, ``head``.
"""
from __future__ import annotations

import math

from ..config.pudulorn_config import PudulornConfig
from ..config.registry import register_architecture
from ..config.specs import LayerCall, LayerSpec, ModelSpec, PartSpec

# No longest sequence is part of the design; position tables get as many rows as the engine's
# pool and model length allow (DecoderModel.materialize).
POSITIONS = 1 << 20

# The dense feed-forward's gate is g * sigmoid(1.702 g), and one is added to its up product: fixed by the design.
DENSE_SLOPE, DENSE_PLUS = 1.702, 1.0

LAYER_NAMES = {"norm1": "norm1", "mixer": "mix.", "norm2": "norm2", "ffn": "mlp.", "separator": ""}


def _rotation(m: dict):
    rot = m.get("rot")
    if not rot or not int(rot["dims"]):
        return None
    return PartSpec("rope", {"dim": int(rot["dims"]), "theta": float(rot["base"]), "max_position": POSITIONS, "precise": True})


def running_order(cfg: PudulornConfig) -> tuple:
    """Every layer once; one that reads another's latents names that layer's buffer."""
    return tuple(LayerCall(i, i if lc.kv_from is None else lc.kv_from, writes=lc.kv_from is None)
                 for i, lc in enumerate(cfg.layers))


def pudulorn_spec(cfg: PudulornConfig) -> ModelSpec:
    def norm():
        return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps, "tensor": "", "one_plus": True})

    layers, ignorable = [], []
    for i, lc in enumerate(cfg.layers):
        m = lc.mixer
        if lc.type == "latent_attention":
            mixer = PartSpec("latent_attention", {
                "hidden_size": cfg.width, "num_heads": int(m["heads"]), "dim": int(m["dim"]), "rot_dim": int(m["rot_dim"]),
                "vdim": int(m["vdim"]), "q_rank": int(m["q_rank"]), "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]),
                "eps": cfg.norm_eps, "position": _rotation(m) if int(m["rot_dim"]) else None, "use_sink": False,
                "pending": True, "window": lc.reach, "pairing": "halves", "own_kv": lc.kv_from is None})
        else:
            mixer = PartSpec("differential_attention", {
                "hidden_size": cfg.width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "dim": int(m["dim"]),
                "vdim": int(m["vdim"]), "scale": float(m["scale"]), "diff": float(m["diff"]), "eps": cfg.norm_eps,
                "chunk": lc.reach, "position": _rotation(m), "pairing": "halves"})
        ffn = None
        if lc.mlp is None:
            ignorable.append(f"l{i}.norm2")
        elif lc.mlp["kind"] == "dense":
            ffn = PartSpec("limited_glu", {"hidden_size": cfg.width, "intermediate_size": int(lc.mlp["ff"]),
                                           "limit": float(lc.mlp["limit"]), "gate_slope": DENSE_SLOPE, "plus": DENSE_PLUS})
        else:
            shared = lc.mlp.get("shared")
            ffn = PartSpec("routed_experts", {
                "hidden_size": cfg.width, "num_experts": int(lc.mlp["router"]["experts"]), "top": int(lc.mlp["router"]["top"]),
                "intermediate_size": int(lc.mlp["expert"]["ff"]), "limit": math.inf, "gate_slope": 1.0, "plus": 0.0,
                "router_bias": False, "scores": "all", "scale": float(lc.mlp["router"]["scale"]),
                "shared_size": int(shared["ff"]) if shared is not None else 0, "shared_limit": math.inf,
                "shared_gate": shared is not None, "pending": True})
        layers.append(LayerSpec(block="prenorm", mixer=mixer, ffn=ffn, norm1=norm(), norm2=norm(), names=LAYER_NAMES))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width, layers=tuple(layers), schedule=running_order(cfg),
        final_norm=norm(), tie_word_embeddings=False, max_position=POSITIONS,
        embed_prefix="embed", final_norm_prefix="final.norm", head_prefix="head", layer_prefix="l{i}.",
        embedding=PartSpec("lookup", {"tensor": ""}), head=PartSpec("linear", {"tensor": ""}),
        eos_token_ids=tuple(cfg.eos_token_id), ignorable_tensors=tuple(ignorable), init_std=0.05,
    )


register_architecture("Pudulorn", PudulornConfig, pudulorn_spec, replace=True)
