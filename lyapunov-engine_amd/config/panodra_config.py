"""Typed configuration of the Panodra decoder, read from config.json.

The file names its architecture in the singular (``"architecture": "Panodra"``)
and nests its constants: ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` and
``logit_softcap`` (null or absent: 1, and no cap), ``loop`` (``start``, ``stop``,
``times``; absent or null: every layer runs once) and ``layers``, a list whose
entries give ``type`` (which mixer), ``mixer`` (its sizes and constants) and
``mlp`` (``kind`` "dense" with ``ff``, "moe" with ``expert.ff``,
``router.experts`` and ``router.top``, or null for a layer without a
feed-forward).  Every size and constant comes from the file; a missing one is an
error.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

from .faledra_config import _need
from .model_config import ConfigError

MIXER_TYPES = ("latent_attention", "latent_attention_2")
MLP_KINDS = ("dense", "moe")


def _positive(d: dict, keys, where: str) -> None:
    for k in keys:
        if int(d[k]) <= 0:
            raise ConfigError(f"{where}.{k} must be positive, got {d[k]}")


@dataclass(frozen=True)
class PanodraLayer:
    type: str
    mixer: dict                      # the mixer's sizes and constants as the file gives them
    mlp: Optional[dict]

    @staticmethod
    def from_dict(d: dict, i: int) -> "PanodraLayer":
        where = f"layers[{i}]"
        _need(d, ("type", "mixer"), where)
        kind, mixer, mlp = d["type"], d["mixer"], d.get("mlp")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}: mixer type {kind!r} is not implemented (known: {list(MIXER_TYPES)})")
        _need(mixer, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale"), where + ".mixer")
        _positive(mixer, ("heads", "vdim", "kv_rank"), where + ".mixer")
        if int(mixer["dim"]) < 0 or int(mixer["rot_dim"]) < 0 or int(mixer["dim"]) + int(mixer["rot_dim"]) == 0:
            raise ConfigError(f"{where}.mixer: heads of {mixer['dim']} plain and {mixer['rot_dim']} rotated dimensions")
        if int(mixer["rot_dim"]) > 0:
            _need(mixer, ("rot",), where + ".mixer")
            rot = mixer["rot"]
            _need(rot, ("base", "dims"), where + ".mixer.rot")
            dims = int(rot["dims"])
            if dims % 2 or not 0 <= dims <= int(mixer["rot_dim"]) or not float(rot["base"]) > 0:
                raise ConfigError(f"{where}.mixer.rot: {dims} rotated dimensions of {mixer['rot_dim']}, base {rot['base']}")
            if rot.get("scaling") is not None:
                sc = rot["scaling"]
                _need(sc, ("factor", "original", "fast", "slow"), where + ".mixer.rot.scaling")
                if not all(float(sc[k]) > 0 for k in ("factor", "original", "fast", "slow")) or float(rot["base"]) == 1:
                    raise ConfigError(f"{where}.mixer.rot.scaling: {sc}")
        if mlp is not None:
            _need(mlp, ("kind",), where + ".mlp")
            if mlp["kind"] == "dense":
                _need(mlp, ("ff",), where + ".mlp")
                _positive(mlp, ("ff",), where + ".mlp")
            elif mlp["kind"] == "moe":
                _need(mlp, ("expert", "router"), where + ".mlp")
                _need(mlp["expert"], ("ff",), where + ".mlp.expert")
                _need(mlp["router"], ("experts", "top"), where + ".mlp.router")
                _positive(mlp["expert"], ("ff",), where + ".mlp.expert")
                if not 1 <= int(mlp["router"]["top"]) <= int(mlp["router"]["experts"]):
                    raise ConfigError(f"{where}.mlp.router: {mlp['router']['top']} of {mlp['router']['experts']} experts")
            else:
                raise ConfigError(f"{where}.mlp.kind {mlp['kind']!r} is not implemented (known: {list(MLP_KINDS)})")
        return PanodraLayer(kind, dict(mixer), dict(mlp) if mlp is not None else None)

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": dict(self.mixer), "mlp": dict(self.mlp) if self.mlp is not None else None}


@dataclass(frozen=True)
class PanodraConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple                    # of PanodraLayer
    logit_scale: float = 1.0
    logit_softcap: float = 0.0       # 0: no cap
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1              # layers loop_start .. loop_stop - 1 run this many times in a row
    architectures: tuple = ("Panodra",)
    eos_token_id: tuple = ()
    extra: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict) -> "PanodraConfig":
        _need(d, ("vocab", "width", "norm", "layers"), "config.json")
        _need(d["norm"], ("eps",), "norm")
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("layers must be a list with at least one entry")
        layers = tuple(PanodraLayer.from_dict(l, i) for i, l in enumerate(d["layers"]))
        start = stop = 0
        times = 1
        if d.get("loop") is not None:
            _need(d["loop"], ("start", "stop", "times"), "loop")
            start, stop, times = int(d["loop"]["start"]), int(d["loop"]["stop"]), int(d["loop"]["times"])
            if not (0 <= start <= stop <= len(layers)) or times < 1:
                raise ConfigError(f"loop: layers {start} .. {stop - 1} of {len(layers)}, {times} times")
        known = {"architecture", "architectures", "vocab", "width", "norm", "layers", "loop", "logit_scale", "logit_softcap",
                 "eos_token_id"}
        eos = d.get("eos_token_id")
        scale, cap = d.get("logit_scale"), d.get("logit_softcap")
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=float(d["norm"]["eps"]), layers=layers,
                  logit_scale=1.0 if scale is None else float(scale), logit_softcap=0.0 if cap is None else float(cap),
                  loop_start=start, loop_stop=stop, loop_times=times,
                  eos_token_id=() if eos is None else tuple(int(t) for t in (eos if isinstance(eos, list) else [eos])),
                  extra={k: v for k, v in d.items() if k not in known})
        if cfg.vocab <= 0 or cfg.width <= 0 or not cfg.norm_eps > 0 or cfg.logit_softcap < 0:
            raise ConfigError(f"vocab {cfg.vocab}, width {cfg.width}, norm.eps {cfg.norm_eps}, logit_softcap {cfg.logit_softcap}")
        return cfg

    @property
    def has_loop(self) -> bool:
        return self.loop_stop > self.loop_start

    def to_dict(self) -> dict:
        d = {"architecture": "Panodra", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
             "logit_scale": self.logit_scale, "layers": [l.to_dict() for l in self.layers]}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        if self.has_loop:
            d["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.eos_token_id:
            d["eos_token_id"] = list(self.eos_token_id)
        return d


__all__ = ["PanodraConfig", "PanodraLayer"]
