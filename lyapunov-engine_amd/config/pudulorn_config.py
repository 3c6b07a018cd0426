"""Typed configuration of the Pudulorn decoder, read from config.json.

The file names its architecture in the singular (``"architecture": "Pudulorn"``)
and nests its constants: ``vocab``, ``width``, ``norm.eps`` and ``layers``, a
list whose entries give ``type`` (which mixer), ``mixer`` (its sizes and
constants) and ``mlp`` (``kind`` "dense" with ``ff`` and ``limit``, "moe" with
``expert.ff``, ``router.experts``, ``router.top``, ``router.scale`` and
optionally ``shared.ff``, or null for a layer without a feed-forward).

A "latent_attention" layer whose mixer has ``kv_from`` reads the latents of that
earlier layer.  Every size and constant comes from the file; a missing one is an
error, but ``mask`` may be absent or null (every earlier token is seen).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

from .faledra_config import _need
from .model_config import ConfigError
from .panodra_config import _positive

MIXER_TYPES = ("latent_attention", "attention")
MLP_KINDS = ("dense", "moe")


def _check_rotation(mixer: dict, width: int, where: str) -> None:
    _need(mixer, ("rot",), where)
    rot = mixer["rot"]
    _need(rot, ("base", "dims"), where + ".rot")
    dims = int(rot["dims"])
    if dims % 2 or not 0 <= dims <= width or not float(rot["base"]) > 0:
        raise ConfigError(f"{where}.rot: {dims} rotated dimensions of {width}, base {rot['base']}")


def _check_mask(mixer: dict, where: str) -> None:
    if mixer.get("mask") is not None:
        _need(mixer["mask"], ("size",), where + ".mask")
        _positive(mixer["mask"], ("size",), where + ".mask")


def _check_mlp(mlp: dict, where: str) -> None:
    _need(mlp, ("kind",), where)
    if mlp["kind"] == "dense":
        _need(mlp, ("ff", "limit"), where)
        _positive(mlp, ("ff",), where)
        if not float(mlp["limit"]) > 0:
            raise ConfigError(f"{where}.limit must be positive, got {mlp['limit']}")
    elif mlp["kind"] == "moe":
        _need(mlp, ("expert", "router"), where)
        _need(mlp["expert"], ("ff",), where + ".expert")
        _need(mlp["router"], ("experts", "top", "scale"), where + ".router")
        _positive(mlp["expert"], ("ff",), where + ".expert")
        if not 1 <= int(mlp["router"]["top"]) <= int(mlp["router"]["experts"]):
            raise ConfigError(f"{where}.router: {mlp['router']['top']} of {mlp['router']['experts']} experts")
        if mlp.get("shared") is not None:
            _need(mlp["shared"], ("ff",), where + ".shared")
            _positive(mlp["shared"], ("ff",), where + ".shared")
    else:
        raise ConfigError(f"{where}.kind {mlp['kind']!r} is not implemented (known: {list(MLP_KINDS)})")


@dataclass(frozen=True)
class PudulornLayer:
    type: str
    mixer: dict                      # the mixer's sizes and constants as the file gives them
    mlp: Optional[dict]

    @staticmethod
    def from_dict(d: dict, i: int) -> "PudulornLayer":
        where = f"layers[{i}]"
        _need(d, ("type", "mixer"), where)
        kind, mixer, mlp = d["type"], d["mixer"], d.get("mlp")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}: mixer type {kind!r} is not implemented (known: {list(MIXER_TYPES)})")
        at = where + ".mixer"
        if kind == "latent_attention":
            _need(mixer, ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale"), at)
            _positive(mixer, ("heads", "vdim", "q_rank", "kv_rank"), at)
            if int(mixer["dim"]) < 0 or int(mixer["rot_dim"]) < 0 or int(mixer["dim"]) + int(mixer["rot_dim"]) == 0:
                raise ConfigError(f"{at}: heads of {mixer['dim']} plain and {mixer['rot_dim']} rotated dimensions")
            if int(mixer["rot_dim"]) > 0:
                _check_rotation(mixer, int(mixer["rot_dim"]), at)
        else:
            _need(mixer, ("heads", "kv_heads", "dim", "vdim", "scale", "diff"), at)
            _positive(mixer, ("heads", "kv_heads", "dim", "vdim"), at)
            if int(mixer["heads"]) % int(mixer["kv_heads"]):
                raise ConfigError(f"{at}: {mixer['heads']} query heads over {mixer['kv_heads']} key/value heads")
            if mixer.get("rot") is not None:
                _check_rotation(mixer, int(mixer["dim"]), at)
        if not float(mixer["scale"]) > 0:
            raise ConfigError(f"{at}.scale must be positive, got {mixer['scale']}")
        _check_mask(mixer, at)
        if mlp is not None:
            _check_mlp(mlp, where + ".mlp")
        return PudulornLayer(kind, dict(mixer), dict(mlp) if mlp is not None else None)

    @property
    def kv_from(self) -> Optional[int]:
        """The layer whose latents this one reads; None: its own."""
        j = self.mixer.get("kv_from")
        return None if j is None else int(j)

    @property
    def reach(self) -> int:
        """The mask's size; 0: none."""
        return int(self.mixer["mask"]["size"]) if self.mixer.get("mask") is not None else 0

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": dict(self.mixer), "mlp": dict(self.mlp) if self.mlp is not None else None}


@dataclass(frozen=True)
class PudulornConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple                    # of PudulornLayer
    architectures: tuple = ("Pudulorn",)
    eos_token_id: tuple = ()
    extra: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict) -> "PudulornConfig":
        _need(d, ("vocab", "width", "norm", "layers"), "config.json")
        _need(d["norm"], ("eps",), "norm")
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("layers must be a list with at least one entry")
        layers = tuple(PudulornLayer.from_dict(l, i) for i, l in enumerate(d["layers"]))
        for i, lc in enumerate(layers):
            j = lc.kv_from
            if j is None:
                continue
            where = f"layers[{i}].mixer.kv_from"
            if lc.type != "latent_attention" or not 0 <= j < i or layers[j].type != "latent_attention" or \
                    layers[j].kv_from is not None:
                raise ConfigError(f"{where}: layer {j} is no earlier latent attention layer with latents of its own")
            mine, other = lc.mixer, layers[j].mixer
            rotation = (lambda m: (float(m["rot"]["base"]), int(m["rot"]["dims"])) if int(m["rot_dim"]) else None)
            if (int(mine["kv_rank"]), int(mine["rot_dim"]), rotation(mine)) != \
                    (int(other["kv_rank"]), int(other["rot_dim"]), rotation(other)):
                raise ConfigError(f"{where}: layer {j} keeps latents of other sizes or another rotation")
        known = {"architecture", "architectures", "vocab", "width", "norm", "layers", "eos_token_id"}
        eos = d.get("eos_token_id")
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=float(d["norm"]["eps"]), layers=layers,
                  eos_token_id=() if eos is None else tuple(int(t) for t in (eos if isinstance(eos, list) else [eos])),
                  extra={k: v for k, v in d.items() if k not in known})
        if cfg.vocab <= 0 or cfg.width <= 0 or not cfg.norm_eps > 0:
            raise ConfigError(f"vocab {cfg.vocab}, width {cfg.width}, norm.eps {cfg.norm_eps}")
        return cfg

    def to_dict(self) -> dict:
        d = {"architecture": "Pudulorn", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
             "layers": [l.to_dict() for l in self.layers]}
        if self.eos_token_id:
            d["eos_token_id"] = list(self.eos_token_id)
        return d


__all__ = ["PudulornConfig", "PudulornLayer"]
