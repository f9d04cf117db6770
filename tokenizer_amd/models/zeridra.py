"""Zeridra as a `ModelSpec`: a decoder whose layers read ONE norm for a mixer and a routed feed-forward side by side,
x + (ls1 * mixer(h) + ls2 * feed_forward(h)) with h = norm1(x) and a learned scale per coordinate on each; two mixers
(attention over a cached latent with a window, a rotation of neighbouring coordinates and a learned sink a head, whose
latents a later such layer may read as its own; grouped heads without positions whose values are the keys, whose
queries are scaled by their position and whose softmax has one added to its denominator); gated experts chosen by their
sigmoid scores, which also weigh what an expert is handed; a scaled embedding; scaled and capped logits.

Tensor names: `embed`, `head`, `final.norm`; layer i's start with `l<i>.`: `norm1`, `ls1`, `ls2`, `mix.*` (attention:
q, k, o; latent: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, sink, o) and `mlp.*` (e<j>.gate|up|down, router).
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.zeridra import ZeridraConfig
from ..parts.spec import FeedForwardSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec, ScheduleEntry

_ATTENTION_NAMES = (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("o_proj.weight", "o"))


def _attention(raw: dict, width: int, eps: float) -> MixerSpec:
    temp = raw.get("q_temp") or {"coef": 0.0, "every": 1}
    return MixerSpec("gqa_attention", hidden_size=width, n_heads=raw["heads"], n_kv_heads=raw["kv_heads"],
                     head_dim=raw["dim"], value_dim=raw["dim"], scale=float(raw["scale"]), tied_values=True, fixed_sink=0.0,
                     eps=eps, position=PositionSpec("query_temperature", head_dim=raw["dim"],
                                                    options={"coef": float(temp["coef"]), "every": int(temp["every"])}),
                     tensor_names=_ATTENTION_NAMES)


def _latent(cfg: ZeridraConfig, index: int) -> MixerSpec:
    raw = cfg.layers[index]["mixer"]
    own = cfg.latent_source(index) == index
    return MixerSpec("latent_attention", hidden_size=cfg.width, n_heads=raw["heads"], n_kv_heads=1, head_dim=raw["dim"],
                     value_dim=raw["vdim"], scale=float(raw["scale"]), q_rank=raw["q_rank"], kv_rank=raw["kv_rank"],
                     rot_dim=int(raw["rot_dim"]), window=cfg.reach(raw), sink=True, own_kv=own, eps=cfg.eps,
                     options={"rot_base": float(raw["rot"]["base"]), "rot_pairs": "neighbours",
                              "kept_window": cfg.kept_reach(index) if own else None})


def zeridra_spec(cfg: ZeridraConfig) -> ModelSpec:
    width, eps = cfg.width, cfg.eps
    norm = NormSpec("rmsnorm", width, eps, options={"tensor_name": ""})     # the weight is the tensor the prefix names
    layers, schedule = [], []
    for index, layer in enumerate(cfg.layers):
        prefix, mlp, feed_forward = f"l{index}", layer.get("mlp"), None
        if mlp is not None:
            feed_forward = FeedForwardSpec("routed_experts", hidden_size=width, intermediate_size=mlp["expert"]["ff"],
                                           activation="silu", n_experts=mlp["router"]["experts"], top_k=mlp["router"]["top"],
                                           router="sigmoid", correction=False, renormalize=False, weigh_input=True)
        latent = layer["type"] == "latent_attention"
        layers.append(LayerSpec(
            block="parallel_scaled", mixer=_latent(cfg, index) if latent else _attention(layer["mixer"], width, eps),
            feed_forward=feed_forward, mixer_norm=norm, feed_forward_norm=None if mlp is None else norm,
            mixer_prefix=f"{prefix}.mix", feed_forward_prefix=f"{prefix}.mlp", mixer_norm_prefix=f"{prefix}.norm1",
            feed_forward_norm_prefix=f"{prefix}.norm1", prefix=prefix,
            options={"width": width, "layer_scale": True, "one_norm": True}))
        source = cfg.latent_source(index) if latent else index
        schedule.append(ScheduleEntry(index, cache_of=None if source == index else source))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=width, max_positions=cfg.max_positions,
        embedding_name="embed", layers=tuple(layers), schedule=tuple(schedule), final_norm=norm,
        final_norm_prefix="final.norm", tied_head=False, head_name="head", embedding_scale=cfg.embedding_scale,
        options={"head_scale": cfg.logit_scale, "head_cap": cfg.logit_softcap})


register_architecture("Zeridra", ZeridraConfig, zeridra_spec)
