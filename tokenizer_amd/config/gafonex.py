"""Configuration of the Gafonex decoder, from its config.json keys.

The file is nested: `layers` lists the layers in their order, each with its `type` (which mixer: "attention" or
"retention"), the mixer's sizes and constants under `mixer` and its feed-forward under `mlp` (null: the layer has
none); `norm.eps`, `norm.groups`, `logit_softcap`, `vocab` and `width` hold for the whole model.  Every size and
constant a model may choose is read from here; nothing is assumed equal between layers.
"""
from __future__ import annotations

import dataclasses
from typing import Any

from .base import ConfigError, ModelConfig
from .napadra import _number


def _rotation(where: str, rot: dict | None, head_dim: int) -> None:
    if rot is None:
        return
    dims = _number(where, rot, "dims", positive=False)
    if dims % 2 or not 0 <= dims <= head_dim:
        raise ConfigError(f"{where}.dims must be even and at most the head size {head_dim}, found {dims}")
    if not dims:
        return
    base = _number(where, rot, "base", float)
    scaling = rot.get("scaling")
    if scaling is not None:
        for key in ("factor", "original", "fast", "slow"):
            _number(f"{where}.scaling", scaling, key, float)
        if base == 1.0:
            raise ConfigError(f"{where}: a scaled rotation needs a base other than 1")


@dataclasses.dataclass(frozen=True)
class GafonexConfig(ModelConfig):
    vocab: int
    width: int
    norm: dict
    layers: list
    logit_softcap: float | None = None
    max_positions: int = 1 << 20      # positions are not bounded by the design: the bound is this engine's own

    MIXERS = ("attention", "retention")

    def validate(self) -> None:
        for key in ("vocab", "width", "max_positions"):
            if getattr(self, key) <= 0:
                raise ConfigError(f"{key} must be positive, found {getattr(self, key)}")
        _number("norm", self.norm, "eps", float, positive=False)
        groups = _number("norm", self.norm, "groups")
        if self.width % groups:
            raise ConfigError(f"norm.groups: a width of {self.width} does not fall into {groups} equal parts")
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ConfigError(f"logit_softcap must be positive, found {self.logit_softcap}")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config.json: `layers` must be a list with at least one layer")
        first = None                   # the first layer whose values later layers take in
        for index, layer in enumerate(self.layers):
            where = f"layers[{index}]"
            if not isinstance(layer, dict) or layer.get("type") not in self.MIXERS:
                raise ConfigError(f"config.json: {where}.type must be one of {', '.join(self.MIXERS)}")
            mixer = layer.get("mixer")
            for key in ("heads", "dim", "vdim"):
                _number(f"{where}.mixer", mixer, key)
            _rotation(f"{where}.mixer.rot", mixer.get("rot"), mixer["dim"])
            if layer["type"] == "attention":
                heads, kv_heads = mixer["heads"], _number(f"{where}.mixer", mixer, "kv_heads")
                if heads % kv_heads:
                    raise ConfigError(f"{where}: {heads} query heads is not a multiple of {kv_heads} kv heads")
                _number(f"{where}.mixer", mixer, "scale", float)
                if mixer.get("v_mix"):
                    if first is None:
                        first = index
                    other = self.layers[first]["mixer"]
                    if any(other[key] != mixer[key] for key in ("kv_heads", "vdim")):
                        raise ConfigError(f"{where} mixes in layer {first}'s values but has value heads of other number or size")
            else:
                decay = mixer.get("decay")
                if not isinstance(decay, list) or len(decay) != mixer["heads"]:
                    raise ConfigError(f"config.json: {where}.mixer.decay must list one number a head")
                for value in decay:
                    if isinstance(value, bool) or not isinstance(value, (int, float)) or not 0.0 <= value <= 1.0:
                        raise ConfigError(f"config.json: {where}.mixer.decay should lie between 0 and 1, found {value!r}")
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp.kind must be dense")
                _number(f"{where}.mlp", mlp, "ff")

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    @property
    def groups(self) -> int:
        return int(self.norm["groups"])

    def to_dict(self) -> dict[str, Any]:
        out = super().to_dict()
        out.pop("architectures")
        out.pop("max_positions")
        return {"architecture": self.architecture, **out}
