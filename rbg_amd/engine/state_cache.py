"""Cache of models whose layers keep latents or recurrent state.

Two kinds of memory per sequence, both carved at start-up:

* pages of latents: attention layers that cache one low-rank row per token.
  Page accounting, block tables and slot mapping are PagedKVCache's; the pool
  is one allocation with a view [pages, page_size, rank] per layer (the ranks
  may differ between layers).
* one state slot: fixed-size tensors that a token rewrites in place (the past
  inputs of a short convolution, a recurrence's matrix).  Slot 0 is scratch for
  the padding rows of captured decode batches, like page 0.

A slot is handed out dirty: the kernels take a sequence's state as zero at
position 0 instead of reading it.  Pages of such a model cannot be shared by
prompt prefix (the state at the page's end is not kept), so there is no prefix
cache.
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
    # name -> (shape without the slot dim, dtype)
    state: Dict[str, Tuple[Tuple[int, ...], torch.dtype]] = \
        field(default_factory=dict)


class StateCache(PagedKVCache):
    def __init__(self, cfg: EngineConfig, device: torch.device,
                 specs: List[LayerCacheSpec], dtype: torch.dtype,
                 num_pages: Optional[int] = None):
        self.specs = specs
        self.dtype = dtype
        self.num_slots = (cfg.state_slots or cfg.max_batch_size) + 1
        super().__init__(cfg, device, num_pages, num_layers=len(specs))
        self.prefix = None
        self._free_slots: List[int] = list(range(self.num_slots - 1, 0, -1))

    def _page_bytes(self) -> int:
        rows = sum(s.latent_rank for s in self.specs) * self.cfg.page_size
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
        total = sum(s.latent_rank for s in self.specs) * rows
        self.kv = torch.zeros(total, dtype=self.dtype, device=device)
        self._latents: List[Optional[torch.Tensor]] = []
        self.states: List[Dict[str, torch.Tensor]] = []
        at = 0
        for spec in self.specs:
            view = None
            if spec.latent_rank:
                n = rows * spec.latent_rank
                view = self.kv[at:at + n].view(
                    self.num_pages, self.page_size, spec.latent_rank)
                at += n
            self._latents.append(view)
            self.states.append({
                name: torch.zeros((self.num_slots,) + tuple(shape),
                                  dtype=dt, device=device)
                for name, (shape, dt) in spec.state.items()})

    # -- views ------------------------------------------------------------------

    def latents(self, layer: int) -> torch.Tensor:
        view = self._latents[layer]
        assert view is not None, f"layer {layer} caches no latents"
        return view

    def state(self, layer: int, name: str) -> torch.Tensor:
        return self.states[layer][name]

    # -- slots ------------------------------------------------------------------

    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    def has_room(self, num_pages: int) -> bool:
        return bool(self._free_slots) and super().has_room(num_pages)

    def alloc_slot(self) -> int:
        with self._lock:
            if not self._free_slots:
                raise OutOfPages("no free state slot")
            return self._free_slots.pop()

    def free_slot(self, slot: int) -> None:
        with self._lock:
            self._free_slots.append(slot)

    # -- migration: latents of the pages, then the slot's state, as bytes -----------

    def export_pages(self, pages: List[int], slot: int = 0) -> torch.Tensor:
        idx = torch.tensor(pages, dtype=torch.int64, device=self.kv.device)
        parts = []
        for view, states in zip(self._latents, self.states):
            if view is not None:
                parts.append(view.index_select(0, idx))
            parts.extend(t[slot] for t in states.values())
        return torch.cat([p.contiguous().view(-1).view(torch.uint8)
                          for p in parts])

    def _export_bytes(self, num_pages: int) -> int:
        n = 0
        for spec in self.specs:
            n += (spec.latent_rank * self.page_size * num_pages *
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
        for view, states in zip(self._latents, self.states):
            if view is not None:
                view.index_copy_(0, idx, take((len(pages),) + view.shape[1:],
                                              view.dtype))
            for t in states.values():
                t[slot].copy_(take(t.shape[1:], t.dtype))
