"""Device memory of the cache: pages of keys and values per group, and per-request state slots."""
from __future__ import annotations

import torch

from .manager import CacheManager

_STATE_DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16, "int32": torch.int32}


class CachePools:
    """For group g: `pages[g]` of shape [layers in g, num_pages, n_kv, page_size * (d + dv)] elements in the
    compute dtype, a layer's keys first and then its values (d: a key head's size, dv: a value head's, which
    is d unless the mixer says otherwise).  Inside a page keys are laid out [page_size, d] and values
    transposed, [dv, page_size] (the layout the matrix-core attention kernels read).  A group whose values are its keys
    (`CacheNeed.tied_values`) has key pages alone.  For a layer with
    fixed-size state: `states[layer]` of shape [max_requests, *state_shape]; for a layer whose block keeps
    state of its own: `block_states[layer]`, float32 [max_requests, *block_state_shape]."""

    def __init__(self, manager: CacheManager, needs, dtype: torch.dtype, device):
        self.manager = manager
        self.pages = []
        for group in manager.groups:
            need = group.need
            per_layer = manager.num_pages * need.n_kv_heads * manager.page_size * max(need.head_dim, need.v_dim)
            if per_layer >= 2 ** 31:
                # The attention kernels count a layer's keys (and its values) with 32 bits.
                raise ValueError(f"{manager.num_pages} pages of {manager.page_size} tokens are {per_layer} key elements "
                                 f"a layer; the kernels address fewer than 2^31 (at most "
                                 f"{(2 ** 31 - 1) // (need.n_kv_heads * manager.page_size * max(need.head_dim, need.v_dim))} pages here)")
            self.pages.append(torch.zeros((len(group.layers), manager.num_pages * manager.page_size
                                           * (need.n_kv_heads * need.head_dim
                                              + (0 if need.tied_values else need.v_heads * need.v_dim))),
                                          dtype=dtype, device=device))
        self.states, self.block_states = {}, {}
        for layer, need in enumerate(needs):
            if need.state_shape is not None:
                self.states[layer] = torch.zeros((manager.max_requests, *need.state_shape),
                                                 dtype=_STATE_DTYPES[need.state_dtype], device=device)
            if need.block_state_shape is not None:
                self.block_states[layer] = torch.zeros((manager.max_requests, *need.block_state_shape),
                                                       dtype=torch.float32, device=device)

    def layer_pages(self, layer: int):
        """(keys [num_pages, n_kv, page_size, d], values [num_pages, n_v, dv, page_size]) of one layer (n_v = n_kv
        unless the need names fewer value heads; None where the values are the keys), or (None, None)."""
        group = self.manager.group_of_layer[layer]
        if group is None:
            return None, None
        need = self.manager.groups[group].need
        index = self.manager.groups[group].layers.index(layer)
        pages, page_size = self.pages[group], self.manager.page_size
        shape = (self.manager.num_pages, need.n_kv_heads)
        keys = shape[0] * shape[1] * page_size * need.head_dim
        if need.tied_values:
            return pages[index].view(*shape, page_size, need.head_dim), None
        return (pages[index, :keys].view(*shape, page_size, need.head_dim),
                pages[index, keys:].view(shape[0], need.v_heads, need.v_dim, page_size))

    def keep_states(self) -> list:
        """Copies of every state tensor (for a run whose effect on them is to be undone)."""
        return [(t, t.clone()) for t in list(self.states.values()) + list(self.block_states.values())]

    @staticmethod
    def put_states_back(kept: list) -> None:
        for tensor, copy in kept:
            tensor.copy_(copy)

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.pages) + \
            sum(t.numel() * t.element_size() for t in list(self.states.values()) + list(self.block_states.values()))

    def poison(self, value: float = float("nan")) -> None:
        """Fill every page and state row with a value that shows if a kernel reads what no request wrote."""
        for tensor in self.pages + list(self.states.values()) + list(self.block_states.values()):
            tensor.fill_(value)
