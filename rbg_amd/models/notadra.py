"""Notadra: a decoder of soft-capped attention with a sink and of sparse
feed-forwards, normed before and after each, over an f32 residual stream.

    x <- x + norm1b(attention(norm1(x))),  x <- x + norm2b(experts(norm2(x)))

Every norm weight is stored as its distance from one.  Tokens are embedded by
their own row plus a hashed row for (previous token, token).  A layer may attend
to an earlier layer's keys and values instead of its own.  On the GPU a layer is:

  sandwich_norm   x += norm2b(last experts, weighed and summed); norm1 of x
  GEMM, rope      queries, keys, values; biases, rotation, paged store
  attention       prompt rows and decoded rows, both from the pages
  GEMM            W_o
  sandwich_norm   x += norm1b(it); norm2 of x
  router, route   logits, choice, rows in expert order
  2 grouped GEMMs W_up with the squared relu, W_down
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, NamedTuple, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.batch import ForwardBatch
from ..engine.config import EngineConfig, ModelConfig
from ..engine.state_cache import StateCache
from .llama import TPContext
from .mixers import PagedAttention, SparseExperts, param
from .rotary import assign_tables
from .stream_model import StreamForCausalLM
from .weights import WeightSource


@dataclass
class NotadraConfig(ModelConfig):
    architecture: str = "Notadra"
    max_position: int = 1 << 30     # the engine's limit sizes the angle tables
    layers: List[Dict[str, Any]] = field(default_factory=list)
    bigram: Dict[str, int] = field(default_factory=dict)
    logit_scale: float = 1.0

    @staticmethod
    def from_json(d: Dict[str, Any], name: str = "notadra",
                  weights_path: str = "") -> "NotadraConfig":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            m, src = layer["mixer"], layer["mixer"].get("kv_from")
            if src is None:
                continue
            if not 0 <= src < i:
                raise ValueError(f"layer {i}: kv_from {src} is not before it")
            other = layers[src]["mixer"]
            if other.get("kv_from") is not None or any(
                    m[k] != other[k] for k in ("kv_heads", "dim", "vdim")):
                raise ValueError(f"layer {i}: cannot use layer {src}'s keys")
        bigram = d["embedding"]["bigram"]
        return NotadraConfig(
            name=name, weights_path=weights_path, layers=layers,
            hidden_size=int(d["width"]), vocab_size=int(d["vocab"]),
            num_layers=len(layers), rms_eps=float(d["norm"]["eps"]),
            bigram={k: int(bigram[k])
                    for k in ("buckets", "mul_prev", "mul_cur")},
            logit_scale=float(d["logit_scale"]))

    @staticmethod
    def stacked(name: str, width: int, vocab: int, layers: int, heads: int,
                kv_heads: int, dim: int, vdim: int, rot_dims: int, ff: int,
                experts: int, top: int, groups: int, keep: int,
                shared: int = 0, buckets: int = 0) -> "NotadraConfig":
        """A configuration of equal layers, e.g. for presets and benchmarks;
        the last ``shared`` use the keys of the one before them."""
        out = []
        for i in range(layers):
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim, "scale": dim ** -0.5, "softcap": 30.0,
                     "rot": {"dims": rot_dims, "base": 500000.0,
                             "scaling": {"factor": 4.0, "original": 4096,
                                         "fast": 32.0, "slow": 1.0}}}
            if i >= layers - shared:
                mixer["kv_from"] = layers - shared - 1
            out.append({"type": "attention", "mixer": mixer, "mlp": {
                "kind": "moe", "expert": {"ff": ff},
                "router": {"experts": experts, "top": top,
                           "groups": {"count": groups, "keep": keep}}}})
        return NotadraConfig.from_json({
            "width": width, "vocab": vocab, "layers": out,
            "norm": {"eps": 1e-6}, "logit_scale": 1.0,
            "embedding": {"bigram": {"buckets": buckets or vocab,
                                     "mul_prev": 1000003, "mul_cur": 7919}},
        }, name=name)


def preset(name: str) -> Optional[NotadraConfig]:
    if name == "tiny-notadra":          # CPU test shape
        return NotadraConfig.stacked(
            name, width=96, vocab=512, layers=4, heads=4, kv_heads=2, dim=24,
            vdim=16, rot_dims=12, ff=40, experts=8, top=2, groups=4, keep=2,
            shared=1)
    if name == "notadra-30b-a3b":       # widths of current sparse models
        return NotadraConfig.stacked(
            name, width=2048, vocab=151936, layers=48, heads=32, kv_heads=4,
            dim=128, vdim=128, rot_dims=64, ff=1152, experts=128, top=8,
            groups=8, keep=4, shared=8)
    return None


class Pending(NamedTuple):
    """A branch that the stream has yet to take: rows (of tokens, or of chosen
    experts with their routing) and the weight of the norm they go through."""
    rows: torch.Tensor
    route: Optional[ops.Routing]
    weight: torch.Tensor


def load_norm(src: WeightSource, name: str, width: int) -> nn.Parameter:
    return param(1.0 + src.take(name, (width,), "zeros").float(),
                 torch.float32)


class NotadraLayer(nn.Module):
    def __init__(self, cfg: NotadraConfig, index: int, first: int,
                 tp: TPContext, src: WeightSource, dtype: torch.dtype):
        super().__init__()
        spec, w, p = cfg.layers[index], cfg.hidden_size, f"l{index}."
        self.tp, self.dtype, self.eps = tp, dtype, cfg.rms_eps
        self.norm1 = load_norm(src, p + "norm1", w)
        self.norm1b = load_norm(src, p + "norm1b", w)
        self.mixer = PagedAttention(spec["mixer"], w, src, p + "mix.", tp,
                                    dtype, sink=True)
        kv = self.mixer.kv_from
        # index into this stage's cache
        self.kv_layer = (index if kv is None else kv) - first
        if self.kv_layer < 0:
            raise ValueError(f"layer {index} uses the keys of layer {kv}, "
                             "which is on another pipeline stage")
        self.mlp = self.norm2 = self.norm2b = None
        if spec.get("mlp") is not None:
            self.norm2 = load_norm(src, p + "norm2", w)
            self.norm2b = load_norm(src, p + "norm2b", w)
            self.mlp = SparseExperts(spec["mlp"], w, src, p + "mlp.", tp,
                                     dtype)

    def cache_spec(self):
        return self.mixer.cache_spec()

    def forward(self, x: torch.Tensor, pending: Optional[Pending],
                batch: ForwardBatch, cache: StateCache) -> Pending:
        h = ops.sandwich_norm(x, pending, self.norm1, self.eps, self.dtype)
        y = self.tp.all_reduce(self.mixer(h, batch, cache, self.kv_layer))
        pending = Pending(y, None, self.norm1b)
        if self.mlp is None:
            return pending
        h = ops.sandwich_norm(x, pending, self.norm2, self.eps, self.dtype)
        y, route = self.mlp(h)
        if self.tp.size > 1:
            # the sum over the shards comes before the norm
            y, route = self.tp.all_reduce(ops.moe_combine(y, route)), None
        return Pending(y, route, self.norm2b)


class NotadraForCausalLM(StreamForCausalLM):
    stateful = False            # its tokens and pages are all a sequence has
    needs_prev = True           # the embedding looks at pairs of tokens

    def load_embeddings(self, src: WeightSource) -> None:
        self.bigram = param(src.take("bigram", (
            self.cfg.bigram["buckets"] + 1, self.cfg.hidden_size)), self.dtype)

    def load_norm(self, src: WeightSource, name: str) -> nn.Parameter:
        return load_norm(src, name, self.cfg.hidden_size)

    def build_layer(self, index: int, src: WeightSource) -> NotadraLayer:
        return NotadraLayer(self.cfg, index, self.layer_start, self.tp, src,
                            self.dtype)

    def spare_tensors(self):
        return {f"l{i}.{n}" for i in range(self.cfg.num_layers)
                for n in ("norm2", "norm2b")}

    def make_cache(self, cfg: EngineConfig) -> StateCache:
        assign_tables((layer.mixer for layer in self.layers), cfg.max_seq_len,
                      self.device)
        return super().make_cache(cfg)

    def embed_rows(self, tokens: torch.Tensor,
                   batch: ForwardBatch) -> torch.Tensor:
        return ops.embed_pairs(tokens, batch.prev_tokens, self.embed,
                               self.bigram, self.cfg.bigram["mul_prev"],
                               self.cfg.bigram["mul_cur"])

    def add(self, x: torch.Tensor, pending: Pending) -> torch.Tensor:
        ops.sandwich_norm(x, pending, None, self.cfg.rms_eps, self.dtype)
        return x

    def final(self, x: torch.Tensor, pending: Pending) -> torch.Tensor:
        return ops.sandwich_norm(x, pending, self.final_norm,
                                 self.cfg.rms_eps, self.dtype)

    @torch.inference_mode()
    def logits(self, hidden: torch.Tensor,
               gather_idx: Optional[torch.Tensor] = None) -> torch.Tensor:
        return super().logits(hidden, gather_idx).mul_(self.cfg.logit_scale)
