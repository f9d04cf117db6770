"""Interfaces of the parts a layer is put together from, and their registries.

A part is built from its spec, the tensors it asked for and a `Runtime`
(compute dtype, device, kernel library).  No part knows which model it is in.

Interfaces
----------
Norm            tensor_specs(spec) -> {local name: TensorSpec}
                apply(residual, delta, rows=None) -> normalised rows in the compute dtype.
                Optional: fold() -> NormFold, if the norm is x / sqrt(mean(x^2) + eps) * weight for some weight:
                a mixer or feed-forward may then take it into the prologue of its own product.
                `residual` is the float32 stream [T, H]; `delta` (or None) is added to it first and,
                unless `rows` picks a subset, the sum is stored back.  `delta` may also be a product still
                in parts (`kernels.PendingSum`, which the kernel library's `add_rmsnorm` takes as it is): a
                norm with kernels of its own calls `as_tensor(delta)` first.
PositionEncoding
                encode_and_store(qkv, geometry, ctx, cache, bias): adds the projection bias, encodes
                the query and key heads in place and writes keys and values of this step into `cache`.
                Optional: epilogue() -> StoreEpilogue, if the encoding is a rotation of half-split pairs by a
                table (or nothing at all): the fused projection then does it, and the store, in its epilogue.
Mixer           tensor_specs(spec), cache_need(spec) -> CacheNeed
                forward(x [T, H], ctx: StepContext, cache: LayerCache) -> [T, H] in the compute dtype.
                Optional: forward_normed(residual, delta, norm, ctx, cache) to fold the norm before it and the
                residual add after it into its own kernels (returns None when it added its output itself; what
                it returns is only ever handed to a norm as its delta, so it may be a product still in parts).
FeedForward     tensor_specs(spec); forward(x [T, H], ctx) -> [T, H]; optional forward_normed likewise.
Block           arranges two norms, a mixer and a feed-forward around the residual stream (either sub-layer may
                be absent: None for the part and its norm):
                forward(residual, delta, ctx, cache) -> delta still to be added.

Frame           what stands around the layers: `ModelSpec.frame` names it.  Static `expected_tensors(spec)` (every
                tensor name the model reads, with its `TensorSpec`) and `cache_needs(spec)` (one `CacheNeed` per
                layer); built from (spec, tensors, runtime); `graph_safe`; `forward(ctx, layer_caches)` -> float32
                logits [wanted, vocab].  The built-in "decoder" frame (`parts.model.DecoderModel`) is embedding,
                layers in schedule order, final norm, head, with `embed(ctx)` and `logits(residual, delta, ctx)` as
                the two places a subclass changes (a scaled embedding, a learned position table, a head bias, a cap
                on the logits); its constants beyond the spec's fields travel in `ModelSpec.options`.

Every part may also say `repeatable() -> Repeatable` (a block: `repeatable(cache)`): that on the device its forward
does nothing but call the kernel library, and that those calls depend on the part only through the constants and the
tensors it lists.  The model then records the calls of one such layer on a step's batch and makes them again for
the like layers after it, with their tensors' addresses put in place (`kernels.LaunchTape`), instead of running
their Python.  The promise is the class's own: a subclass does not inherit it and has to give it again.
"""
from __future__ import annotations

import dataclasses
from typing import Any

import torch

from .spec import CacheNeed, TensorSpec


@dataclasses.dataclass
class Runtime:
    dtype: torch.dtype
    device: torch.device
    ops: Any                      # tokenizer_amd.kernels.Ops (or a stand-in with the same methods)


class Registry:
    def __init__(self, what: str):
        self.what = what
        self._items: dict[str, type] = {}

    def register(self, kind: str, cls: type | None = None, replace: bool = False):
        def put(target: type) -> type:
            if kind in self._items and not replace:
                raise ValueError(f"{self.what} {kind!r} is already registered")
            self._items[kind] = target
            return target
        return put if cls is None else put(cls)

    def get(self, kind: str) -> type:
        try:
            return self._items[kind]
        except KeyError:
            raise KeyError(f"unknown {self.what} {kind!r}; registered: {', '.join(sorted(self._items))}") from None

    def kinds(self) -> list[str]:
        return sorted(self._items)


NORMS = Registry("norm")
POSITIONS = Registry("position encoding")
MIXERS = Registry("mixer")
FEED_FORWARDS = Registry("feed-forward")
BLOCKS = Registry("block")
FRAMES = Registry("model frame")


class Part:
    """Common base: a part names its tensors and is built from them.

    `graph_safe` says that the part's forward only launches device work whose shape depends on the
    batch's sizes, never on host-side values of the batch (positions, request ids): only then may a
    decode step be captured once and replayed.  Parts are taken not to be unless they say so.
    """
    graph_safe = False

    @staticmethod
    def tensor_specs(spec) -> dict[str, TensorSpec]:
        return {}


@dataclasses.dataclass
class NormFold:
    """A norm in the form the fused products take into their prologue: y = x / sqrt(mean(x^2) + eps) * weight,
    with `weight` float32 [H] on the device.  A norm of that form says so through `Norm.fold()`, whatever its
    class and however it derives the weight from its tensors.  (A norm over groups of coordinates is not of that form.)"""
    weight: torch.Tensor
    eps: float


@dataclasses.dataclass
class StoreEpilogue:
    """What the fused q/k/v projection can do behind its bias: rotate the half-split pairs of every query and
    key head by the row of `cos_sin` (float32 [positions, d]: cos half, then sin half) at the token's position,
    `cos_sin` None meaning no rotation, and write keys and values into their pages.  A position encoding that is
    of that form says so through `PositionEncoding.epilogue()`."""
    cos_sin: torch.Tensor | None


@dataclasses.dataclass(frozen=True)
class Repeatable:
    """What a part's library calls depend on: `constants` (hashable; parts whose constants are equal make the same
    calls) and `tensors` (their addresses are what differs from one such part to the next; None where a part has
    none, the same places in every like part)."""
    constants: tuple
    tensors: tuple


def repeatable_of(part, *args) -> Repeatable | None:
    """The part's `repeatable(*args)` if its own class gives that promise, else None."""
    if part is None:
        return Repeatable(("absent",), ())
    if "repeatable" not in vars(type(part)):
        return None
    return part.repeatable(*args)


class Norm(Part):
    def apply(self, residual: torch.Tensor, delta: torch.Tensor | None,
              rows: torch.Tensor | None = None) -> torch.Tensor:
        raise NotImplementedError

    def fold(self) -> NormFold | None:
        """The norm as a product's prologue can compute it, or None (the parts then call `apply`)."""
        return None


class PositionEncoding(Part):
    def encode_and_store(self, qkv, bias, n_q: int, n_kv: int, head_dim: int, ctx, cache) -> None:
        raise NotImplementedError

    def epilogue(self) -> StoreEpilogue | None:
        """The encoding as the fused projection's epilogue can apply it, or None (`encode_and_store` is called)."""
        return None


class Mixer(Part):
    @staticmethod
    def cache_need(spec) -> CacheNeed:
        return CacheNeed()

    def forward(self, x: torch.Tensor, ctx, cache) -> torch.Tensor:
        raise NotImplementedError

    def forward_normed(self, residual, delta, norm: Norm, ctx, cache):
        """The sub-layer from the residual stream on: add `delta`, normalise, mix.  Returns the output still
        to be added to the stream, or None if the part added it itself.  A part may override this to fold
        the norm and the add into its own kernels; this default keeps them apart."""
        return self.forward(norm.apply(residual, delta), ctx, cache)


class FeedForward(Part):
    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        raise NotImplementedError

    def forward_normed(self, residual, delta, norm: Norm, ctx):
        """As `Mixer.forward_normed`, for the feed-forward."""
        return self.forward(norm.apply(residual, delta), ctx)


class Block:
    graph_safe = False

    def forward(self, residual: torch.Tensor, delta: torch.Tensor | None, ctx, cache) -> torch.Tensor:
        raise NotImplementedError


class NormedDelta:
    """What a sub-layer that is normalised behind itself hands on: its output `rows` [T, H] (compute dtype) still to
    be brought to unit RMS, scaled by `weight` (float32 [H]) and added to the stream.  A norm of the form
    x / sqrt(mean(x^2) + eps) * w takes it as its delta and does all of that in its own kernel
    (`ops.norm_add_rmsnorm`); for anyone else `resolve()` gives the sum's term as a float32 tensor.

    `side` (or None): something that is still to be added behind this term and depends on the stream as it then
    stands (a block's per-layer token input): an object with `fused(residual, delta, weight, eps, out, rows)`, which
    does the add, its own addition and the next norm in one kernel or returns None, and `settle(residual, delta)`,
    which adds this term to the stream, works its own addition out step by step and returns it as a `NormedDelta`
    without a `side`.

    `groups`: the rows' coordinates form so many equal runs of neighbours, each brought to unit RMS on its own."""

    def __init__(self, ops, rows: torch.Tensor, weight: torch.Tensor, eps: float, side=None, groups: int = 1):
        self.ops, self.rows, self.weight, self.eps, self.side, self.groups = ops, rows, weight, float(eps), side, int(groups)

    def join(self, residual: torch.Tensor, weight, eps: float, out: torch.Tensor, rows=None, store_residual: bool = True,
             groups: int = 1) -> torch.Tensor:
        """The stream with this term added (stored back unless told not to), normalised by `weight` over `groups` groups
        (as it is where `weight` is None) into `out`."""
        more = {} if self.groups == 1 and groups == 1 else {"post_groups": self.groups, "groups": groups}
        return self.ops.norm_add_rmsnorm(residual, self.rows, self.weight, self.eps, weight, eps, out, rows,
                                         store_residual=store_residual, **more)

    def resolve(self) -> torch.Tensor:
        if self.side is not None:
            raise ValueError("a term with an addition behind it that reads the stream cannot stand alone: hand it to a norm")
        zero = torch.zeros((self.rows.shape[0], self.rows.shape[1]), dtype=torch.float32, device=self.rows.device)
        return self.join(zero, None, 0.0, torch.empty_like(zero), store_residual=False)


class SumDelta:
    """What a layer whose two sub-layers read the same normalised rows hands on: their outputs `first` and `second`
    [T, H] (compute dtype), still to be added to each other and to the stream, x + (first + second) in float32.  A norm
    of the form x / sqrt(mean(x^2) + eps) * w takes it as its delta and does the two additions and the norm in one
    kernel (`ops.add_pair_rmsnorm`); for anyone else `resolve()` gives the sum as a float32 tensor."""

    def __init__(self, ops, first: torch.Tensor, second: torch.Tensor):
        self.ops, self.first, self.second = ops, first, second

    def resolve(self) -> torch.Tensor:
        zero = torch.zeros(self.first.shape, dtype=torch.float32, device=self.first.device)
        rows = torch.empty(self.first.shape, dtype=self.first.dtype, device=self.first.device)
        self.ops.add_pair_rmsnorm(zero, self.first, self.second, None, 0.0, rows)
        return zero


class ScaledSum:
    """What a layer hands on whose sub-layers' outputs are still to be weighted and added: `terms`, each (rows [T, H] in
    the compute dtype, a factor, a scale float32 [H] or None), standing for x + sum(factor * scale * rows) in float32.
    A norm of the form x / sqrt(mean(x^2) + eps) * w takes it as its delta and does the additions and the norm in one
    kernel (`ops.add_terms_rmsnorm`); for anyone else `resolve()` gives the sum as a float32 tensor."""
    MAX_TERMS = 4

    def __init__(self, ops, terms=()):
        self.ops, self.terms = ops, tuple(terms)

    @classmethod
    def of(cls, ops, value) -> "ScaledSum":
        """A sub-layer's output as a sum: one itself, or a tensor as its one term (a product still in parts stays one where
        the kernel library's `add_terms_rmsnorm` adds them up)."""
        if isinstance(value, cls):
            return value
        kept = hasattr(value, "partial") and getattr(ops, "takes_pending_terms", False)
        return cls(ops, () if value is None else ((value if kept else as_tensor(value), 1.0, None),))

    def scaled_by(self, scale, factor: float = 1.0) -> "ScaledSum":
        """Every term times `factor` and, coordinate by coordinate, `scale` (float32 [H] or None)."""
        def both(old):
            return scale if old is None else old if scale is None else (old * scale).contiguous()
        return ScaledSum(self.ops, tuple((rows, f * float(factor), both(s)) for rows, f, s in self.terms))

    def plus(self, other: "ScaledSum") -> "ScaledSum":
        out = ScaledSum(self.ops, self.terms + other.terms)
        if len(out.terms) > self.MAX_TERMS:
            raise ValueError(f"a sum of more than {self.MAX_TERMS} terms")
        return out

    def resolve(self) -> torch.Tensor:
        rows = as_tensor(self.terms[0][0])
        zero = torch.zeros(rows.shape, dtype=torch.float32, device=rows.device)
        self.ops.add_terms_rmsnorm(zero, self.terms, None, 0.0, torch.empty_like(rows))
        return zero


def as_tensor(delta):
    """The delta as a tensor: a product still in parts has them added now."""
    resolve = getattr(delta, "resolve", None)
    return resolve() if resolve is not None and not isinstance(delta, torch.Tensor) else delta


def can_fuse_decode(ops, residual, dtype) -> bool:
    """Whether the kernel library offers its fused decode products for these rows of the residual stream
    (few bfloat16 rows of a width whose normalised copy fits in LDS); a library without them says no."""
    check = getattr(ops, "can_fuse_decode", None)
    return bool(check and check(residual.shape[0], dtype, residual.shape[1]))
