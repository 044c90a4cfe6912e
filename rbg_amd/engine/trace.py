"""Trace replay: given token ids, step by step, through an engine's runner.

``TraceSession`` admits a request at its first entry, feeds each step's tokens
as one batch from the cache and state that earlier steps left, and gives back
what a finished request held.  Nothing is sampled.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional

import torch

from .config import EngineConfig, ModelConfig
from .kv_cache import BlockTable
from .model_runner import ModelRunner
from .sequence import Sequence


class TraceSession:
    def __init__(self, model: ModelConfig, max_tokens: int,
                 max_requests: int = 4, device: str = "cuda",
                 page_size: int = 16, enforce_eager: Optional[bool] = None):
        pages = (max_tokens + page_size - 1) // page_size
        eager = device != "cuda" if enforce_eager is None else enforce_eager
        self.runner = ModelRunner(EngineConfig(
            model=model, device=device, page_size=page_size,
            max_batch_size=max_requests, state_slots=max_requests,
            max_seq_len=pages * page_size,
            # one page more: page 0 is scratch
            kv_pool_tokens=(pages + 1) * page_size,
            enable_prefix_cache=False, enforce_eager=eager))
        self.live: Dict[Any, Sequence] = {}

    def step(self, entries: List[Dict[str, Any]], end: List[Any]
             ) -> torch.Tensor:
        """Runs one step; logits [wanted, vocab] in entry order, on the host."""
        vocab = self.runner.cfg.model.vocab_size
        chunks, want = [], []
        for e in entries:
            tokens, w = list(e["tokens"]), list(e.get("want", []))
            if not tokens or min(tokens) < 0 or max(tokens) >= vocab:
                raise ValueError(f"request {e['id']!r}: tokens missing or "
                                 f"outside [0, {vocab})")
            if any(p < 0 or p >= len(tokens) for p in w):
                raise ValueError(f"request {e['id']!r}: 'want' outside")
            seq = self.live.get(e["id"])
            if seq is None:
                seq = Sequence([])
                seq.block_table = BlockTable(self.runner.cache)
                self.live[e["id"]] = seq
            start = seq.num_prompt_tokens
            seq.prompt_tokens.extend(tokens)
            seq.block_table.ensure(seq.num_prompt_tokens)
            chunks.append((seq, start, tokens))
            want.append(w)
        out = torch.empty(0, vocab)
        if chunks:
            out = self.runner.feed(chunks, want).float().cpu()
        for rid in end:
            self.live.pop(rid).block_table.release()
        return out
