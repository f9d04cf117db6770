"""Attention over a cached latent (multi-head latent attention) in its absorbed form."""
from __future__ import annotations

import torch

from .base import MIXERS, Mixer, Runtime
from .position import scaled_rates
from .spec import CacheNeed, MixerSpec, TensorSpec


@MIXERS.register("latent_attention")
class LatentAttention(Mixer):
    """Queries through a normalised latent, keys and values from one normalised latent a token that all heads share.

    With h the mixer's input, r = `kv_rank`, d = `head_dim`, e = `rot_dim`, dv = `value_dim`:
    c_q = norm(W_dq h) (weight `dq.norm`), q = W_uq c_q laid out head by head as [d plain | e rotated];
    W_dkv h has r + e rows: c = norm(first r) (weight `dkv.norm`), the last e (not normalised) are one key part that is
    rotated and shared by all heads; head i: k_i = W_uk,i c, v_i = W_uv,i c,
    score = (q_i,plain . k_i + rot(q_i,rot) . rot(k_rot)) * scale, causal softmax, o_i = sum of weights * v_i; the gate, if
    there is one (`head_gate`: sigmoid of one number a head; `element_gate`: of one number a coordinate of the joined
    heads, both projected from h by `g`), then W_o.  The rotation pairs coordinate j with j + e/2 (option `rot_pairs`
    "neighbours": coordinate 2j with 2j + 1) and turns pair j at position p by p * base^(-2j/e) (option `rot_base`;
    angles, sine and cosine in float32).

    Options, each on its own: `window` w (a key is visible when key + w >= query), `sink` (tensor `sink`, one number a
    head, joins the softmax's denominator as exp(sink): no key, no value, not scaled) and `own_kv` False (no W_dkv: the
    layer reads the rows [c | rot(k_rot)] that the layer it is pointed at keeps, with its own W_uk, W_uv and queries, and
    writes nothing).  Option `kept_window`: how far back any layer that reads these rows looks (None: to the start), which
    is what the cache keeps.

    Only c and the rotated key part are cached, and nothing is ever expanded from them: since
    q_i,plain . (W_uk,i c) = (W_uk,i^T q_i,plain) . c, a head's query is taken into the latent's space (a product per
    head with W_uk,i^T), the cache is read as ONE key head of r + e coordinates [c | rot(k_rot)] that all query heads
    share, the same rows serve as values, and a head's r leading output coordinates go through W_uv,i afterwards:
    sum_j w_j (W_uv,i c_j) = W_uv,i (sum_j w_j c_j).  So the paged attention kernels of the grouped-query mixer run it
    as they are (n_kv = 1, head size r + e), for prompts, portions and single tokens alike, and a token costs the
    cache r + e numbers a layer whatever the number of heads.  Scores and weights are float32 there.

    Tensors: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, sink, o (those of the options where they are set).
    """
    graph_safe = True

    def __init__(self, spec: MixerSpec, tensors: dict[str, torch.Tensor], runtime: Runtime):
        if spec.head_gate and spec.element_gate:
            raise ValueError("latent attention has a gate a head or a gate a coordinate, not both")
        self.spec, self.runtime = spec, runtime
        H, d, dv, r, e = spec.n_heads, spec.head_dim, spec.value_dim or spec.head_dim, spec.kv_rank, spec.rot_dim
        self.heads, self.d, self.dv, self.rank, self.rot, self.q_rank = H, d, dv, r, e, spec.q_rank
        self.key_dim = r + e                         # what a token's row of the cache holds
        self.eps, self.scale = float(spec.eps), float(spec.scale)
        if e % 2:
            raise ValueError(f"a rotation over {e} coordinates")
        self.window, self.own_kv, self.gated = spec.window, spec.own_kv, spec.head_gate or spec.element_gate
        pairs = spec.options.get("rot_pairs", "halves")
        if pairs not in ("halves", "neighbours"):
            raise ValueError(f"rot_pairs {pairs!r}: known are \"halves\" and \"neighbours\"")
        # (What the kernels take only where a layer has it.)
        self.turns = {"neighbours": True} if pairs == "neighbours" else {}
        self.more = {"tied_values": True}
        if spec.sink:
            self.more["sinks"] = tensors["sink"].to(torch.float32).contiguous()
        # One product for the down-projections and the gate; every part starts at a multiple of eight columns
        # (sixteen bytes in bfloat16), filled up with rows of zeros.
        parts, self.offsets, at = [], {}, 0
        for name in ("dq",) + (("dkv",) if self.own_kv else ()) + (("g",) if self.gated else ()):
            weight = tensors[name]
            self.offsets[name] = at
            fill = (-weight.shape[0]) % 8
            parts.append(weight if not fill else torch.cat([weight, weight.new_zeros((fill, weight.shape[1]))], dim=0))
            at += weight.shape[0] + fill
        self.w_in = torch.cat(parts, dim=0).contiguous()
        self.q_norm = tensors["dq.norm"].to(torch.float32).contiguous()
        self.kv_norm = tensors["dkv.norm"].to(torch.float32).contiguous() if self.own_kv else None
        self.w_uq = tensors["uq"]
        # W_uk,i^T as the matrix of a product out = x W^T: [H, r, d]; W_uv,i as it is: [H, dv, r].
        self.w_absorb = tensors["uk"].reshape(H, d, r).transpose(1, 2).contiguous()
        self.w_uv = tensors["uv"].reshape(H, dv, r).contiguous()
        self.w_o = tensors["o"]
        self.rates = scaled_rates(float(spec.options.get("rot_base", 1.0)), e, None).to(runtime.device).contiguous() if e else None

    @staticmethod
    def tensor_specs(spec: MixerSpec) -> dict[str, TensorSpec]:
        H, d, dv, hidden = spec.n_heads, spec.head_dim, spec.value_dim or spec.head_dim, spec.hidden_size
        gate_rows = H if spec.head_gate else H * dv
        out = {"dq": TensorSpec((spec.q_rank, hidden)), "dq.norm": TensorSpec((spec.q_rank,), init="ones", role="vector"),
               "uq": TensorSpec((H * (d + spec.rot_dim), spec.q_rank)),
               "uk": TensorSpec((H * d, spec.kv_rank)), "uv": TensorSpec((H * dv, spec.kv_rank)),
               "o": TensorSpec((hidden, H * dv))}
        if spec.own_kv:
            out["dkv"] = TensorSpec((spec.kv_rank + spec.rot_dim, hidden))
            out["dkv.norm"] = TensorSpec((spec.kv_rank,), init="ones", role="vector")
        if spec.head_gate or spec.element_gate:
            out["g"] = TensorSpec((gate_rows, hidden))
        if spec.sink:
            out["sink"] = TensorSpec((H,), role="vector", std=1.0)
        return out

    @staticmethod
    def cache_need(spec: MixerSpec) -> CacheNeed:
        # One key head of kv_rank + rot_dim coordinates; the same rows serve as values.
        if not spec.own_kv:
            return CacheNeed()                  # it reads the pages of the layer it is pointed at
        window = spec.options["kept_window"] if "kept_window" in spec.options else spec.window
        return CacheNeed(kind="full" if window is None else "window", n_kv_heads=1, head_dim=spec.kv_rank + spec.rot_dim,
                         window=window, tied_values=True)

    def forward(self, x, ctx, cache):
        ops, H, D = self.runtime.ops, self.heads, self.key_dim
        n_tokens = x.shape[0]
        rows = ops.linear(x, self.w_in)
        latent_q = torch.empty((n_tokens, self.q_rank), dtype=x.dtype, device=x.device)
        # Both latents' norms, the rotation of the shared key part and the store of [c | rot(k_rot)].
        ops.latent_store(rows, self.offsets["dq"], self.q_rank, self.q_norm, self.offsets.get("dkv", 0), self.rank, self.kv_norm,
                         self.rot, self.rates, self.eps, ctx.positions,
                         ctx.slots[cache.group] if cache.writes and self.own_kv else None, cache.k_pages, cache.v_pages, latent_q,
                         **self.turns)
        q = ops.linear(latent_q, self.w_uq)                                   # [T, H (d + e)]
        absorbed = torch.empty((n_tokens, H * D), dtype=x.dtype, device=x.device)
        ops.head_linear(q, 0, self.d + self.rot, self.w_absorb, absorbed, 0, D)
        if self.rot:
            ops.rotate_tails(q, H, self.d + self.rot, self.d, self.rot, self.rates, ctx.positions, absorbed, D, self.rank,
                             **self.turns)
        mixed = torch.empty((n_tokens, H * D), dtype=x.dtype, device=x.device)
        ops.paged_attention(absorbed, mixed, cache.k_pages, cache.v_pages, ctx.positions, ctx.entry_of_token,
                            ctx.block_tables[cache.group], H, 1, D, self.window, self.scale, max_position=ctx.max_position,
                            batch=ctx, **self.more)
        out = torch.empty((n_tokens, H * self.dv), dtype=x.dtype, device=x.device)
        ops.head_linear(mixed, 0, D, self.w_uv, out, 0, self.dv)
        if self.spec.head_gate:
            ops.sigmoid_head_gate(out, rows, self.offsets["g"], H, self.dv)
        elif self.gated:
            ops.sigmoid_head_gate(out, rows, self.offsets["g"], H * self.dv, 1)
        return ops.linear(out, self.w_o)
