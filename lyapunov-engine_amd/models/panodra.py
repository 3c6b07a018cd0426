"""The Panodra architecture as a ModelSpec.

A pre-norm decoder whose norms bend every feature through a tanh
("dynamic_tanh").  The mixer is attention over low-rank latents with queries
straight from the layer's input; "latent_attention" has a learned sink in its
softmax and (where the file scales it) a rotation whose slow frequencies are
stretched, "latent_attention_2" an ordinary softmax.  The feed-forward is dense
with a squared relu, or a few of many silu-gated experts that a table picks by
the token's id, or absent.  A stretch of layers may run several times in a row:
every pass has a cache of its own and begins with a projection of the stream
beside the embedding's output.  The logits are products with the embedding's
matrix, scaled and capped.

Tensor names: ``embed``, ``loop.in`` [width, 2 width], ``l<i>.norm1`` /
``norm2`` (with ``.alpha`` and ``.b``), ``l<i>.mix.{q,dkv,dkv.norm,uk,uv,sink,o}``,
``l<i>.mlp.{up,down}`` or ``l<i>.mlp.{table,e<j>.{gate,up,down}}``, ``final.norm``.
"""
from __future__ import annotations

from ..config.panodra_config import PanodraConfig
from ..config.registry import register_architecture
from ..config.specs import LayerCall, LayerSpec, ModelSpec, PartSpec

# No longest sequence is part of the design; position tables get as many rows as the engine's
# pool and model length allow (DecoderModel.materialize).
POSITIONS = 1 << 20

LAYER_NAMES = {"norm1": "norm1", "mixer": "mix.", "norm2": "norm2", "ffn": "mlp.", "separator": ""}


def running_order(cfg: PanodraConfig) -> tuple:
    """Layers before the loop, the looped stretch once per pass (a cache buffer of its own per pass,
    the stream made anew before its first layer), the layers after it."""
    order = [(i, False) for i in range(cfg.loop_start)]
    for _ in range(cfg.loop_times if cfg.has_loop else 0):
        order += [(i, i == cfg.loop_start) for i in range(cfg.loop_start, cfg.loop_stop)]
    order += [(i, False) for i in range(cfg.loop_stop, len(cfg.layers))]
    return tuple(LayerCall(i, cache, enter=enter) for cache, (i, enter) in enumerate(order))


def _rotation(m: dict):
    if not int(m["rot_dim"]) or not int(m["rot"]["dims"]):
        return None
    scaling = m["rot"].get("scaling")
    if scaling is not None:
        scaling = {"rope_type": "yarn", **{k: float(scaling[k]) for k in ("factor", "original", "fast", "slow")}}
    return PartSpec("rope", {"dim": int(m["rot"]["dims"]), "theta": float(m["rot"]["base"]), "max_position": POSITIONS,
                             "scaling": scaling, "precise": True})


def panodra_spec(cfg: PanodraConfig) -> ModelSpec:
    def norm():
        return PartSpec("dynamic_tanh", {"size": cfg.width, "tensor": "", "names": {"bias": ".b", "alpha": ".alpha"}})

    layers, ignorable = [], []
    for i, lc in enumerate(cfg.layers):
        m = lc.mixer
        mixer = PartSpec("latent_attention", {
            "hidden_size": cfg.width, "num_heads": int(m["heads"]), "dim": int(m["dim"]), "rot_dim": int(m["rot_dim"]),
            "vdim": int(m["vdim"]), "q_rank": 0, "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]),
            "eps": cfg.norm_eps, "position": _rotation(m), "use_sink": lc.type == "latent_attention", "pending": True})
        ffn = None
        if lc.mlp is None:
            ignorable.append(f"l{i}.norm2*")
        elif lc.mlp["kind"] == "dense":
            ffn = PartSpec("dense", {"hidden_size": cfg.width, "intermediate_size": int(lc.mlp["ff"]), "activation": "relu2",
                                     "pending": True})
        else:
            ffn = PartSpec("table_experts", {
                "hidden_size": cfg.width, "num_experts": int(lc.mlp["router"]["experts"]), "top": int(lc.mlp["router"]["top"]),
                "intermediate_size": int(lc.mlp["expert"]["ff"]), "vocab_size": cfg.vocab})
        layers.append(LayerSpec(block="prenorm", mixer=mixer, ffn=ffn, norm1=norm(), norm2=norm(), names=LAYER_NAMES))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width, layers=tuple(layers), schedule=running_order(cfg),
        final_norm=norm(), tie_word_embeddings=True, max_position=POSITIONS,
        embed_prefix="embed", final_norm_prefix="final.norm", head_prefix="head", layer_prefix="l{i}.",
        embedding=PartSpec("lookup", {"tensor": ""}),
        head=PartSpec("linear", {"tensor": "", "scale": cfg.logit_scale, "cap": cfg.logit_softcap}),
        stream_entry=PartSpec("projected_pair", {"tensor": ""}) if cfg.has_loop else None,
        stream_entry_prefix="loop.in",
        eos_token_ids=tuple(cfg.eos_token_id), ignorable_tensors=tuple(ignorable), init_std=0.05,
    )


register_architecture("Panodra", PanodraConfig, panodra_spec, replace=True)
