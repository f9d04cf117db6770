"""Configuration of the Zeridra decoder, from its config.json keys.

The file is nested: `layers` lists the layers in their order, each with its `type` (which mixer: "latent_attention",
attention over a cached latent with a window and a learned sink a head, or "attention", grouped heads whose values are
the keys and whose queries are scaled by their position), the mixer's sizes and constants under `mixer` and its
feed-forward under `mlp` (null: the layer has none; `kind` "moe").  A latent layer with `kv_from`: j reads the latents
that layer j keeps.  `embedding.scale`, `norm.eps`, `logit_scale`, `logit_softcap`, `vocab` and `width` hold for the
whole model.  Every size and constant a model may choose is read from here; nothing is assumed equal between layers
beyond what a layer must share with the one whose latents it reads.
"""
from __future__ import annotations

import dataclasses
from typing import Any

from .base import ConfigError, ModelConfig
from .napadra import _number


@dataclasses.dataclass(frozen=True)
class ZeridraConfig(ModelConfig):
    vocab: int
    width: int
    norm: dict
    layers: list
    embedding: dict | None = None
    logit_scale: float | None = None
    logit_softcap: float | None = None
    max_positions: int = 1 << 20      # positions are not bounded by the design: the bound is this engine's own

    MIXERS = ("latent_attention", "attention")

    def validate(self) -> None:
        for key in ("vocab", "width", "max_positions"):
            if getattr(self, key) <= 0:
                raise ConfigError(f"{key} must be positive, found {getattr(self, key)}")
        _number("norm", self.norm, "eps", float, positive=False)
        if self.embedding is not None:
            _number("embedding", self.embedding, "scale", float)
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ConfigError(f"logit_softcap must be positive, found {self.logit_softcap}")
        if self.logit_scale is not None and self.logit_scale == 0:
            raise ConfigError("logit_scale must not be 0")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config.json: `layers` must be a list with at least one layer")
        for index, layer in enumerate(self.layers):
            where = f"layers[{index}]"
            if not isinstance(layer, dict) or layer.get("type") not in self.MIXERS:
                raise ConfigError(f"config.json: {where}.type must be one of {', '.join(self.MIXERS)}")
            mixer = layer.get("mixer")
            for key in ("heads", "dim", "vdim"):
                _number(f"{where}.mixer", mixer, key)
            if _number(f"{where}.mixer", mixer, "scale", float, positive=False) == 0:
                raise ConfigError(f"config.json: {where}.mixer.scale must not be 0")
            if layer["type"] == "attention":
                self._check_attention(f"{where}.mixer", mixer)
            else:
                self._check_latent(f"{where}.mixer", mixer, index)
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
                    raise ConfigError(f"config.json: {where}.mlp.kind must be moe")
                _number(f"{where}.mlp.expert", mlp.get("expert"), "ff")
                experts = _number(f"{where}.mlp.router", mlp.get("router"), "experts")
                top = _number(f"{where}.mlp.router", mlp.get("router"), "top")
                if top > experts:
                    raise ConfigError(f"{where}.mlp.router: top {top} of {experts} experts")

    @staticmethod
    def _check_attention(where: str, mixer: dict) -> None:
        heads, kv_heads = mixer["heads"], _number(where, mixer, "kv_heads")
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} query heads is not a multiple of {kv_heads} kv heads")
        if mixer["vdim"] != mixer["dim"]:
            raise ConfigError(f"{where}: the values are the keys, so vdim {mixer['vdim']} must be dim {mixer['dim']}")
        if mixer.get("q_temp") is not None:
            _number(f"{where}.q_temp", mixer["q_temp"], "coef", float, positive=False)
            _number(f"{where}.q_temp", mixer["q_temp"], "every")

    def _check_latent(self, where: str, mixer: dict, index: int) -> None:
        for key in ("q_rank", "kv_rank"):
            _number(where, mixer, key)
        rot_dim = _number(where, mixer, "rot_dim")
        dims = _number(f"{where}.rot", mixer.get("rot"), "dims")
        base = _number(f"{where}.rot", mixer["rot"], "base", float)
        if dims != rot_dim or dims % 2:
            raise ConfigError(f"{where}: the rotation covers the whole rotated part, an even number of coordinates; found "
                              f"rot.dims {dims} and rot_dim {rot_dim}")
        if mixer.get("mask") is not None:
            _number(f"{where}.mask", mixer["mask"], "size")
        source = mixer.get("kv_from")
        if source is None:
            return
        if isinstance(source, bool) or not isinstance(source, int) or not 0 <= source < index \
                or self.layers[source]["type"] != "latent_attention":
            raise ConfigError(f"{where}.kv_from must name an earlier latent_attention layer, found {source!r}")
        other = self.layers[source]["mixer"]
        if other.get("kv_from") is not None:
            raise ConfigError(f"{where}.kv_from names layer {source}, which keeps no latents of its own")
        if any(other[key] != mixer[key] for key in ("kv_rank", "rot_dim")) or float(other["rot"]["base"]) != base:
            raise ConfigError(f"{where}.kv_from: layer {source}'s kv_rank, rot_dim and rotation differ")

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    @property
    def embedding_scale(self) -> float:
        return float(self.embedding["scale"]) if self.embedding else 1.0

    def latent_source(self, index: int) -> int:
        """The layer whose latents layer `index` reads (itself, unless it names another)."""
        source = self.layers[index]["mixer"].get("kv_from")
        return index if source is None else int(source)

    @staticmethod
    def reach(mixer: dict) -> int | None:
        """How many positions behind itself a query of a latent layer sees (None: all)."""
        mask = mixer.get("mask")
        return None if mask is None else int(mask["size"]) - 1

    def kept_reach(self, index: int) -> int | None:
        """How far back layer `index`'s latents are read by any layer that reads them (None: to the start)."""
        reaches = [self.reach(layer["mixer"]) for at, layer in enumerate(self.layers)
                   if layer["type"] == "latent_attention" and self.latent_source(at) == index]
        return None if any(reach is None for reach in reaches) else max(reaches)

    def to_dict(self) -> dict[str, Any]:
        out = super().to_dict()
        out.pop("architectures")
        out.pop("max_positions")
        return {"architecture": self.architecture, **out}
