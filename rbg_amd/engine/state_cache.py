"""Cache of models whose layers keep different things of a sequence.

Two kinds of memory per sequence, both carved at start-up:

* pages: attention layers that cache one low-rank latent per token, or keys and
  values of a layer's own head counts and sizes.  Page accounting, block tables
  and slot mapping are PagedKVCache's; the pool is one allocation with views per
  layer: latents [pages, page_size, rank], keys and values [pages, heads,
  page_size, size].  A layer that reads another's pages has none of its own.
* one state slot: fixed-size tensors that a token rewrites in place (the past
  inputs of a short convolution, a recurrence's matrix).  Slot 0 is scratch for
  the padding rows of captured decode batches, like page 0.

A slot is handed out dirty: the kernels take a sequence's state as zero at
position 0 instead of reading it.  Pages of a model with state cannot be shared
by prompt prefix (the state at the page's end is not kept), so it has no prefix
cache.  A model without state has pages only: no slots limit its sequences.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from .config import EngineConfig
from .kv_cache import OutOfPages, PagedKVCache


@dataclass
class LayerCacheSpec:
    """What one layer keeps for a sequence."""
    latent_rank: int = 0            # row per token in the paged pool, 0: none
    # (heads, key size, value size) of keys and values in the paged pool
    kv: Optional[Tuple[int, int, int]] = None
    # name -> (shape without the slot dim, dtype)
    state: Dict[str, Tuple[Tuple[int, ...], torch.dtype]] = \
        field(default_factory=dict)

    def paged_shapes(self) -> List[Tuple[int, int]]:
        """(heads, size) of each paged tensor; a latent has one head."""
        out = [(1, self.latent_rank)] if self.latent_rank else []
        if self.kv is not None:
            heads, dim, vdim = self.kv
            out += [(heads, dim), (heads, vdim)]
        return out

    def row_elements(self) -> int:
        """Paged elements per token."""
        return sum(heads * size for heads, size in self.paged_shapes())


class StateCache(PagedKVCache):
    def __init__(self, cfg: EngineConfig, device: torch.device,
                 specs: List[LayerCacheSpec], dtype: torch.dtype,
                 num_pages: Optional[int] = None):
        self.specs = specs
        self.dtype = dtype
        self.has_state = any(s.state for s in specs)
        self.num_slots = ((cfg.state_slots or cfg.max_batch_size) + 1
                          if self.has_state else 1)
        super().__init__(cfg, device, num_pages, num_layers=len(specs))
        if self.has_state:
            self.prefix = None
        self._free_slots: List[int] = list(range(self.num_slots - 1, 0, -1))

    def _page_bytes(self) -> int:
        rows = sum(s.row_elements() for s in self.specs) * self.cfg.page_size
        return max(1, rows * self.dtype.itemsize)

    def _fixed_bytes(self) -> int:
        return self.num_slots * sum(
            math.prod(shape) * dt.itemsize for spec in self.specs
            for shape, dt in spec.state.values())

    def _size_pool(self, device: torch.device) -> int:
        pages = super()._size_pool(device)
        # a model without paged layers has pages of no size: bound their number
        return min(pages, 1 << 22)

    def _alloc_storage(self, device: torch.device) -> None:
        rows = self.num_pages * self.page_size
        total = sum(s.row_elements() for s in self.specs) * rows
        self.kv = torch.zeros(total, dtype=self.dtype, device=device)
        self._pages: List[List[torch.Tensor]] = []  # [pages, heads, rows, size]
        self.states: List[Dict[str, torch.Tensor]] = []
        at = 0
        for spec in self.specs:
            views = []
            for heads, size in spec.paged_shapes():
                n = rows * heads * size
                views.append(self.kv[at:at + n].view(
                    self.num_pages, heads, self.page_size, size))
                at += n
            self._pages.append(views)
            self.states.append({
                name: torch.zeros((self.num_slots,) + tuple(shape),
                                  dtype=dt, device=device)
                for name, (shape, dt) in spec.state.items()})

    # -- views ------------------------------------------------------------------

    def latents(self, layer: int) -> torch.Tensor:
        assert self.specs[layer].latent_rank, f"layer {layer}: no latents"
        return self._pages[layer][0].squeeze(1)

    def kv_pages(self, layer: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """Keys and values, [pages, heads, page_size, size] each."""
        assert self.specs[layer].kv is not None, f"layer {layer}: no keys"
        return self._pages[layer][-2], self._pages[layer][-1]

    def state(self, layer: int, name: str) -> torch.Tensor:
        return self.states[layer][name]

    # -- slots ------------------------------------------------------------------

    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    def has_room(self, num_pages: int) -> bool:
        return (bool(self._free_slots) or not self.has_state) and \
            super().has_room(num_pages)

    def alloc_slot(self) -> int:
        if not self.has_state:
            return 0
        with self._lock:
            if not self._free_slots:
                raise OutOfPages("no free state slot")
            return self._free_slots.pop()

    def free_slot(self, slot: int) -> None:
        with self._lock:
            self._free_slots.append(slot)

    # -- migration: a layer's pages, then the slot's state, as bytes -----------

    def export_pages(self, pages: List[int], slot: int = 0) -> torch.Tensor:
        idx = torch.tensor(pages, dtype=torch.int64, device=self.kv.device)
        parts = []
        for views, states in zip(self._pages, self.states):
            parts.extend(view.index_select(0, idx) for view in views)
            parts.extend(t[slot] for t in states.values())
        return torch.cat([p.contiguous().view(-1).view(torch.uint8)
                          for p in parts])

    def _export_bytes(self, num_pages: int) -> int:
        n = 0
        for spec in self.specs:
            n += (spec.row_elements() * self.page_size * num_pages *
                  self.dtype.itemsize)
            n += sum(math.prod(shape) * dt.itemsize
                     for shape, dt in spec.state.values())
        return n

    def export_shape(self, num_pages: int):
        return (self._export_bytes(num_pages),), torch.uint8

    def import_pages(self, pages: List[int], buf: torch.Tensor,
                     slot: int = 0) -> None:
        assert buf.numel() == self._export_bytes(len(pages))
        idx = torch.tensor(pages, dtype=torch.int64, device=self.kv.device)
        buf = buf.to(self.kv.device)
        at = 0

        def take(shape, dtype):
            nonlocal at
            n = math.prod(shape) * dtype.itemsize
            # clone: a view as a wider dtype needs its alignment
            part = buf[at:at + n].clone().view(dtype).view(shape)
            at += n
            return part
        for views, states in zip(self._pages, self.states):
            for view in views:
                view.index_copy_(0, idx, take((len(pages),) + view.shape[1:],
                                              view.dtype))
            for t in states.values():
                t[slot].copy_(take(t.shape[1:], t.dtype))
