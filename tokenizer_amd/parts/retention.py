"""Retention: a linear recurrence with one fixed decay per head and its state in the request's slot."""
from __future__ import annotations

import torch

from .base import MIXERS, POSITIONS, Mixer, Runtime
from .spec import CacheNeed, MixerSpec, PositionSpec, TensorSpec


@MIXERS.register("retention")
class Retention(Mixer):
    """With h the mixer's input and H = `n_heads`: q = W_q h, k = W_k h [H d], v = W_v h [H dv]; q and k turn by position
    (`position`, a rotation of the heads' leading coordinates), and k is multiplied by d^(-1/2).  Per head, with a fixed
    decay c (`decays`): S <- c S + k v^T, o = S^T q (no softmax, no divisor; a token sees its own write).  Each head's o is
    brought to unit RMS (`eps`, no weight), times silu(W_g h) [H dv], then W_o.  (The mixer of Sun et al., "Retentive
    Network: A Successor to Transformer for Large Language Models".)

    The layer's per-request state (float32, `CacheNeed.state_shape`) is S of every head, transposed: [H, dv, d] in one row
    a slot, read as zeros by a step that starts at position 0.  The rotation, the products with the state, the decays and
    the norm are float32 in every dtype.  Tensors: q, k, v, g, o.
    """
    graph_safe = True

    def __init__(self, spec: MixerSpec, tensors: dict[str, torch.Tensor], runtime: Runtime):
        self.spec, self.runtime = spec, runtime
        self.heads, self.d, self.dv = spec.n_heads, spec.head_dim, spec.value_dim or spec.head_dim
        if len(spec.decays) != self.heads:
            raise ValueError(f"{self.heads} heads need as many decays, found {len(spec.decays)}")
        self.eps = float(spec.eps)
        self.w_in = torch.cat([tensors[name] for name in ("q", "k", "v", "g")], dim=0).contiguous()
        self.w_o = tensors["o"]
        # A width of the joined product or of its input that is no multiple of eight is filled up (bfloat16 rows are read
        # sixteen bytes at a time).
        fill = (-self.w_in.shape[0]) % 8 if runtime.dtype == torch.bfloat16 else 0
        if fill:
            self.w_in = torch.cat([self.w_in, self.w_in.new_zeros((fill, self.w_in.shape[1]))], dim=0).contiguous()
        self.decays = torch.tensor(spec.decays, dtype=torch.float32, device=runtime.device)
        self.powers = runtime.ops.decay_powers(self.decays)
        position = spec.position or PositionSpec("rope_partial", head_dim=self.d, theta=1.0, options={"dims": 0})
        if position.kind != "rope_partial":
            raise ValueError(f"retention turns its queries and keys by the partial rotation, not {position.kind!r}")
        self.position = POSITIONS.get(position.kind)(position, runtime)

    @staticmethod
    def tensor_specs(spec: MixerSpec) -> dict[str, TensorSpec]:
        heads, d, dv, hidden = spec.n_heads, spec.head_dim, spec.value_dim or spec.head_dim, spec.hidden_size
        return {"q": TensorSpec((heads * d, hidden)), "k": TensorSpec((heads * d, hidden)),
                "v": TensorSpec((heads * dv, hidden)), "g": TensorSpec((heads * dv, hidden)),
                "o": TensorSpec((hidden, heads * dv))}

    @staticmethod
    def cache_need(spec: MixerSpec) -> CacheNeed:
        return CacheNeed(kind="none", state_shape=(spec.n_heads * (spec.value_dim or spec.head_dim) * spec.head_dim,))

    def forward(self, x, ctx, cache):
        ops = self.runtime.ops
        if cache.state is None:
            raise ValueError("the recurrent mixer needs its state in the request's slot")
        qkvg = ops.linear(x, self.w_in)
        mixed = torch.empty((x.shape[0], self.heads * self.dv), dtype=x.dtype, device=x.device)
        ops.retention(qkvg, self.position.angles(ctx), self.position.dims, self.decays, self.powers, cache.state, ctx.cu_q,
                      ctx.first_position, ctx.state_slots, mixed, self.heads, self.d, self.dv, self.eps,
                      single_rows=ctx.q_tiles.numel() == 0)
        return ops.linear(mixed, self.w_o)
