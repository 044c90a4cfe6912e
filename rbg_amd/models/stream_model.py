"""What decoders over a 32-bit residual stream share: embedding and head,
pipeline stages, weight loading and in-place refresh.

A layer is called as ``layer(x, pending, batch, cache)``: it first adds what
the layer before left pending to the stream x (in place, inside its own norm
kernel) and returns what it leaves itself.  Subclasses say how layers and
embeddings are built and what "pending" means.  The surface is that of
LlamaForCausalLM (engine/model_runner.py drives both).
"""
from __future__ import annotations

from typing import Any, Optional, Set

import torch
import torch.nn as nn

from ..engine.batch import ForwardBatch
from ..engine.config import EngineConfig, ModelConfig
from ..engine.state_cache import StateCache
from .llama import PPContext, TPContext
from .mixers import param
from .weights import WeightSource, open_weights

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


class StreamForCausalLM(nn.Module):
    stateful = True             # sequences hold a state slot
    varlen = True               # portions come with a VarlenLayout
    mixed_steps = True          # portions and decoded tokens together
    needs_prev = False          # step batches carry each token's predecessor

    def __init__(self, cfg: ModelConfig, device: torch.device,
                 tp: Optional[TPContext] = None, base_seed: int = 1234,
                 pp: Optional[PPContext] = None):
        super().__init__()
        self.cfg, self.device = cfg, device
        self.tp = tp or TPContext()
        self.pp = pp or PPContext()
        self.dtype = DTYPES[cfg.dtype]
        self.stream_dtype = torch.float32
        src = open_weights(cfg.weights_path, base_seed, device)
        L = cfg.num_layers
        assert L % self.pp.size == 0, "PP degree must divide layer count"
        per = L // self.pp.size
        self.layer_start = self.pp.stage * per
        self.layer_end = self.layer_start + per
        self.embed = self.final_norm = self.lm_head = None
        w = cfg.hidden_size
        if self.pp.first:
            self.embed = param(src.take("embed", (cfg.vocab_size, w),
                                        "linear"), self.dtype)
            self.load_embeddings(src)
        self.layers = nn.ModuleList([
            self.build_layer(i, src)
            for i in range(self.layer_start, self.layer_end)])
        if self.pp.last:
            self.final_norm = self.load_norm(src, "final.norm")
            self.lm_head = param(src.take("head", (cfg.vocab_size, w)),
                                 self.dtype)
        if self.pp.size == 1:
            src.finish(optional=self.spare_tensors())

    # -- what a family defines ----------------------------------------------

    def load_embeddings(self, src: WeightSource) -> None:
        """Tensors of the embedding besides ``embed``."""

    def load_norm(self, src: WeightSource, name: str) -> nn.Parameter:
        return param(src.take(name, (self.cfg.hidden_size,), "ones"),
                     torch.float32)

    def build_layer(self, index: int, src: WeightSource) -> nn.Module:
        raise NotImplementedError

    def spare_tensors(self) -> Set[str]:
        """Tensors that a file may hold though the model does not use them."""
        return set()

    def embed_rows(self, tokens: torch.Tensor,
                   batch: ForwardBatch) -> torch.Tensor:
        raise NotImplementedError

    def add(self, x: torch.Tensor, pending: Any) -> torch.Tensor:
        """The stream with what is pending."""
        raise NotImplementedError

    def final(self, x: torch.Tensor, pending: Any) -> torch.Tensor:
        """The last norm of the stream with what is pending."""
        raise NotImplementedError

    # -- surface ------------------------------------------------------------

    @property
    def num_local_layers(self) -> int:
        return self.layer_end - self.layer_start

    def make_cache(self, cfg: EngineConfig) -> StateCache:
        return StateCache(cfg, self.device,
                          [layer.cache_spec() for layer in self.layers],
                          self.dtype)

    @property
    def stream_width(self) -> int:
        """Columns of what one pipeline stage hands to the next."""
        return self.cfg.hidden_size

    def decode_splits(self, batch_size: int, max_seq_len: int) -> int:
        return 0                        # per layer, from its sizes

    @torch.inference_mode()
    def forward(self, tokens: torch.Tensor, batch: ForwardBatch,
                cache: StateCache,
                hidden: Optional[torch.Tensor] = None) -> torch.Tensor:
        """First PP stage embeds `tokens`, later stages take the stream from
        the one before; the last returns normed rows ready for logits()."""
        if self.pp.first:
            x = self.embed_rows(tokens, batch)
        else:
            assert hidden is not None, "non-first PP stage needs hidden"
            x = hidden
        pending = None
        for layer in self.layers:
            pending = layer(x, pending, batch, cache)
        if not self.pp.last:
            return self.add(x, pending)
        return self.final(x, pending)

    @torch.inference_mode()
    def logits(self, hidden: torch.Tensor,
               gather_idx: Optional[torch.Tensor] = None) -> torch.Tensor:
        if gather_idx is not None:
            hidden = hidden[gather_idx.long()]
        return torch.nn.functional.linear(hidden, self.lm_head).float()

    def reload_weights(self, seed: int) -> None:
        """In-place refresh from the weights' file, or from a new seed when
        the model is random (the cache and captured graphs keep their
        addresses)."""
        fresh = type(self)(self.cfg, self.device, self.tp, base_seed=seed,
                           pp=self.pp)
        with torch.no_grad():
            for p, q in zip(self.parameters(), fresh.parameters()):
                p.copy_(q)
        del fresh
        if self.device.type == "cuda":
            torch.cuda.empty_cache()
        if self.tp.size > 1:
            torch.distributed.barrier(group=self.tp.group)
