"""Gafonex as a `ModelSpec`: a decoder whose sub-layers read the stream itself and are normalised behind,
x + ls1 * norm1(mixer(x)), then + ls2 * norm2(feed_forward(.)), with RMS norms over equal groups of coordinates and a
learned scale per coordinate; two mixers (attention whose heads' softmax weights are mixed with each other, with
normalised queries, keys and values, a rotation with slowed long waves, and values that take in the first such layer's;
a retention with one fixed decay per head and its state in the request's slot); a dense feed-forward gated by a ReLU;
capped logits.

Tensor names: `embed`, `head`, `final.norm`; layer i's start with `l<i>.`: `norm1`, `norm2`, `ls1`, `ls2`, `mix.*`
(attention: q, k, v, o, q.norm, k.norm, talk, vmix; retention: q, k, v, g, o) and `mlp.gate|up|down`.
"""
from __future__ import annotations

from ..config.gafonex import GafonexConfig
from ..config.registry import register_architecture
from ..parts.spec import FeedForwardSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec, ScheduleEntry

_ATTENTION_NAMES = (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("o_proj.weight", "o"),
                    ("q_norm", "q.norm"), ("k_norm", "k.norm"))
_FEED_FORWARD_NAMES = (("gate_proj.weight", "gate"), ("up_proj.weight", "up"), ("down_proj.weight", "down"))


def _position(rot: dict | None, head_dim: int, max_positions: int) -> PositionSpec:
    rot = rot or {"dims": 0}
    return PositionSpec("rope_partial", head_dim=head_dim, theta=float(rot.get("base", 1.0)), max_positions=max_positions,
                        options={"dims": int(rot["dims"]), "scaling": rot.get("scaling")})


def _attention(raw: dict, width: int, eps: float, max_positions: int, value_mix: str | None) -> MixerSpec:
    return MixerSpec("gqa_attention", hidden_size=width, n_heads=raw["heads"], n_kv_heads=raw["kv_heads"],
                     head_dim=raw["dim"], value_dim=raw["vdim"], scale=float(raw["scale"]), qk_norm="head", value_norm=True,
                     value_mix=value_mix, talking=True, eps=eps, position=_position(raw.get("rot"), raw["dim"], max_positions),
                     tensor_names=_ATTENTION_NAMES)


def _retention(raw: dict, width: int, eps: float, max_positions: int) -> MixerSpec:
    return MixerSpec("retention", hidden_size=width, n_heads=raw["heads"], head_dim=raw["dim"], value_dim=raw["vdim"],
                     decays=tuple(float(x) for x in raw["decay"]), eps=eps,
                     position=_position(raw.get("rot"), raw["dim"], max_positions))


def gafonex_spec(cfg: GafonexConfig) -> ModelSpec:
    width, eps = cfg.width, cfg.eps
    # The weight is the tensor the prefix names; every group of coordinates has a root mean square of its own.
    norm = NormSpec("rmsnorm", width, eps, options={"tensor_name": "", "groups": cfg.groups})
    layers, values_from = [], None
    for index, layer in enumerate(cfg.layers):
        prefix, raw = f"l{index}", layer["mixer"]
        if layer["type"] == "attention":
            value_mix = None
            if raw.get("v_mix"):
                value_mix = "give" if values_from is None else "take"
                values_from = index if values_from is None else values_from
            mixer = _attention(raw, width, eps, cfg.max_positions, value_mix)
        else:
            mixer = _retention(raw, width, eps, cfg.max_positions)
        mlp = layer.get("mlp")
        feed_forward = None if mlp is None else FeedForwardSpec(
            "gated_dense", hidden_size=width, intermediate_size=mlp["ff"], activation="relu", tensor_names=_FEED_FORWARD_NAMES)
        layers.append(LayerSpec(
            block="post_norm", mixer=mixer, feed_forward=feed_forward, mixer_norm=norm,
            feed_forward_norm=None if mlp is None else norm, mixer_prefix=f"{prefix}.mix",
            feed_forward_prefix=f"{prefix}.mlp", mixer_norm_prefix=f"{prefix}.norm1",
            feed_forward_norm_prefix=f"{prefix}.norm2", prefix=prefix, options={"width": width, "layer_scale": True}))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=width, max_positions=cfg.max_positions,
        embedding_name="embed", layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in range(len(layers))),
        final_norm=norm, final_norm_prefix="final.norm", tied_head=False, head_name="head",
        options={"head_cap": cfg.logit_softcap})


register_architecture("Gafonex", GafonexConfig, gafonex_spec)
