"""What one forward step feeds the kernels.

``ForwardBatch`` is the device side; ``VarlenLayout`` the host's description of
a step that brings several tokens per sequence, from which layers derive what
their kind needs (convolution tiles, the keys inside a window) once per step
and distinct window, not once per layer.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import numpy as np
import torch


@dataclass
class ForwardBatch:
    """Everything the kernels need for one step; built by the model runner."""
    mode: str                       # "prefill" (varlen rows) | "decode"
    positions: torch.Tensor         # [T] int32
    slot_mapping: torch.Tensor      # [T] int32 (KV write slots)
    # prefill
    cu_seqlens: Optional[torch.Tensor] = None   # [B+1] int32 (q rows)
    cu_seqlens_k: Optional[torch.Tensor] = None  # [B+1] int32 (total KV)
    kv_gather_slots: Optional[torch.Tensor] = None  # [Tkv] int32 — prefix
    #   caching / chunked prefill: gather the FULL [past; new] K/V from the
    #   paged pool (the new tokens' rows were just written by rope_store_kv)
    # decode (and the leading decode rows of a mixed step)
    block_tables: Optional[torch.Tensor] = None  # [S, max_pages] int32
    context_lens: Optional[torch.Tensor] = None  # [S] int32
    decode_num_splits: int = 0      # 0 = pick host-side (sync-free in graphs)
    # models that look at pairs of tokens: [T] int64, -1 before the first
    prev_tokens: Optional[torch.Tensor] = None
    # models with per-sequence state
    starts: Optional[torch.Tensor] = None       # [B] int32 first row's position
    state_slots: Optional[torch.Tensor] = None  # [B] int32
    cu_prefill: Optional[torch.Tensor] = None   # cu_seqlens after those rows
    num_decode: int = 0             # leading one-token sequences with a past
    layout: Optional["VarlenLayout"] = None


@dataclass
class WindowView:
    """The keys that a step's prefill rows can see through one window.

    Per sequence they are the rows [max(0, start - window + 1), end) of its
    positions, laid out one sequence after another.  ``slots`` gathers them
    from the paged pool; None when they are exactly this step's new rows."""
    slots: Optional[torch.Tensor]   # [keys] int64
    row_info: torch.Tensor          # [rows, 2] int32: first key row of the
    #                                 sequence, the query's offset among them
    seq_info: torch.Tensor          # [seqs, 4] int32: first query row, rows,
    #                                 first key row, first query's offset
    blocks: torch.Tensor            # [n, 2] int32: (sequence, first query)
    #                                 of every 128 query rows


@dataclass
class PagedView:
    """The prefill rows of a step whose keys are read from the pages."""
    tables: torch.Tensor            # [seqs, pages] int32
    seq_info: torch.Tensor          # [seqs, 3] int32: first query row, rows,
    #                                 position of the first
    row_info: torch.Tensor          # [rows, 2] int32: (sequence, position)
    blocks: torch.Tensor            # [n, 2] int32: (sequence, first query)
    #                                 of every QUERY_BLOCK query rows


QUERY_BLOCK = 128       # query rows per workgroup of the prompt attentions


def table_array(tables) -> np.ndarray:
    """Block tables as one array [n, pages], padded with the scratch page."""
    # numpy staging: batch composition churns every step under continuous
    # serving, so the rebuild is on the step critical path
    out = np.zeros((len(tables), max(len(t.pages) for t in tables)),
                   dtype=np.int32)
    for i, t in enumerate(tables):
        out[i, :len(t.pages)] = t.pages
    return out


class VarlenLayout:
    """Sequences of a varlen step in row order: decode rows first."""

    def __init__(self, starts: List[int], ends: List[int], tables: List,
                 num_decode: int, page_size: int, device: torch.device):
        self.starts, self.ends = starts, ends
        self.tables = tables            # BlockTable per sequence
        self.num_decode = num_decode
        self.page_size = page_size
        self.device = device
        self._views: Dict[int, WindowView] = {}
        self._paged: Optional[PagedView] = None
        self._tiles: Dict[object, torch.Tensor] = {}

    def _dev(self, a: np.ndarray) -> torch.Tensor:
        return torch.from_numpy(np.ascontiguousarray(a)).to(self.device)

    def tiles(self, tile: int) -> torch.Tensor:
        """[n, 2] int32 (sequence, first token) of `tile`-token pieces."""
        if tile not in self._tiles:
            out = [(b, t) for b, (s, e) in enumerate(zip(self.starts,
                                                         self.ends))
                   for t in range(0, e - s, tile)]
            self._tiles[tile] = self._dev(np.array(out, dtype=np.int32))
        return self._tiles[tile]

    def prefill_tiles(self, tile: int) -> torch.Tensor:
        """Like tiles(), over the sequences after the decode rows, with
        sequence numbers counted from there."""
        key = ("prefill", tile)
        if key not in self._tiles:
            out = [(b, t) for b in range(len(self.starts) - self.num_decode)
                   for t in range(0, self.ends[b + self.num_decode] -
                                  self.starts[b + self.num_decode], tile)]
            self._tiles[key] = self._dev(
                np.array(out, dtype=np.int32).reshape(-1, 2))
        return self._tiles[key]

    def prefill_tile_cu(self, tile: int) -> torch.Tensor:
        """[seqs + 1] int32: where each sequence's prefill_tiles begin."""
        key = ("cu", tile)
        if key not in self._tiles:
            n = [0] + [(e - s + tile - 1) // tile
                       for s, e in zip(self.starts[self.num_decode:],
                                       self.ends[self.num_decode:])]
            self._tiles[key] = self._dev(np.cumsum(n).astype(np.int32))
        return self._tiles[key]

    def window_view(self, window: int) -> WindowView:
        """Of the prefill sequences; rows are counted after the decode rows."""
        if window in self._views:
            return self._views[window]
        ps = self.page_size
        slots, info, seqs = [], [], []
        base = row = 0
        past = False
        for s, e, table in list(zip(self.starts, self.ends,
                                    self.tables))[self.num_decode:]:
            k0 = max(0, s - window + 1) if window > 0 else 0
            past |= k0 < s
            pos = np.arange(k0, e)
            pages = np.asarray(table.pages, dtype=np.int64)
            slots.append(pages[pos // ps] * ps + pos % ps)
            off = np.arange(s - k0, e - k0)
            info.append(np.stack([np.full_like(off, base), off], axis=1))
            seqs.append((row, e - s, base, s - k0))
            base += e - k0
            row += e - s
        view = WindowView(
            slots=self._dev(np.concatenate(slots)) if past else None,
            row_info=self._dev(np.concatenate(info).astype(np.int32)),
            seq_info=self._dev(np.array(seqs, dtype=np.int32)),
            blocks=self.prefill_tiles(QUERY_BLOCK))
        self._views[window] = view
        return view

    def paged_view(self) -> PagedView:
        """Of the prefill sequences; rows are counted after the decode rows."""
        if self._paged is None:
            nd = self.num_decode
            starts, ends = self.starts[nd:], self.ends[nd:]
            info, rows, row = [], [], 0
            for b, (s, e) in enumerate(zip(starts, ends)):
                info.append((row, e - s, s))
                pos = np.arange(s, e)
                rows.append(np.stack([np.full_like(pos, b), pos], axis=1))
                row += e - s
            self._paged = PagedView(
                tables=self._dev(table_array(self.tables[nd:])),
                seq_info=self._dev(np.array(info, dtype=np.int32)),
                row_info=self._dev(np.concatenate(rows).astype(np.int32)),
                blocks=self.prefill_tiles(QUERY_BLOCK))
        return self._paged
