"""Gogalix: a decoder of gated delta rules and windowed differential attention,
each beside a feed-forward that reads the same norm, over an f32 residual
stream.

    h = norm1(x),  x <- x + ls1 * sigmoid(rg1 h) * mixer(h)
                          + ls2 * sigmoid(rg2 h) * ff(h)

Norm weights are single numbers.  A mixer is a delta rule with one decay per head
or per key channel, behind a short convolution, or differential attention without
positions, which may use an earlier layer's keys and values.  A feed-forward is
dense, or a mixture of experts with a softmax over the chosen.  On the GPU a
layer is:

  gate_norm     x += the last layer's two branches, scaled and gated; norm1 of x
  GEMM          everything that reads h: the mixer's inputs, both gates, the
                dense feed-forward's gate and up
  mixer         models/mixers.py; GEMM W_o
  ff            gated linear unit and GEMM W_down, or router and experts
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.batch import ForwardBatch
from ..engine.config import ModelConfig
from ..engine.state_cache import StateCache
from .llama import TPContext
from .mixers import (DifferentialAttention, FusedProjection, GatedDeltaRule,
                     GatedSilu, GluExperts, param)
from .stream_model import StreamForCausalLM
from .weights import WeightSource


@dataclass
class GogalixConfig(ModelConfig):
    architecture: str = "Gogalix"
    max_position: int = 1 << 30         # nothing in the design is positional
    layers: List[Dict[str, Any]] = field(default_factory=list)
    embed_scale: float = 1.0
    low_rank: int = 64                  # of random weights; files bring theirs

    @staticmethod
    def from_json(d: Dict[str, Any], name: str = "gogalix",
                  weights_path: str = "") -> "GogalixConfig":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] not in ("delta", "channel_delta", "attention"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp.get("kind") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward kind "
                                 f"{mlp.get('kind')!r}")
            m, src = layer["mixer"], layer["mixer"].get("kv_from")
            if src is None:
                continue
            if not 0 <= src < i:
                raise ValueError(f"layer {i}: kv_from {src} is not before it")
            other = layers[src]["mixer"]
            if (layers[src]["type"] != "attention" or
                    other.get("kv_from") is not None or any(
                        m[k] != other[k] for k in ("kv_heads", "dim",
                                                   "vdim"))):
                raise ValueError(f"layer {i}: cannot use layer {src}'s keys")
        return GogalixConfig(
            name=name, weights_path=weights_path, layers=layers,
            hidden_size=int(d["width"]), vocab_size=int(d["vocab"]),
            num_layers=len(layers), rms_eps=float(d["norm"]["eps"]),
            embed_scale=float(d["embedding"]["scale"]))

    @staticmethod
    def stacked(name: str, width: int, vocab: int, pattern: str, heads: int,
                kv_heads: int, dim: int, vdim: int, window: int, ff: int,
                delta_heads: int, delta_kv_heads: int, delta_dim: int,
                delta_vdim: int, taps: int = 4, experts: int = 0,
                top: int = 0, expert_ff: int = 0, low_rank: int = 64,
                diff: float = 0.4) -> "GogalixConfig":
        """A configuration from a layer pattern, e.g. for presets and
        benchmarks: 'd' and 'c' are delta rules (a decay per head or per
        channel), 'a' is attention, 's' attention with the keys of the last
        'a'; a capital has experts instead of a dense feed-forward."""
        layers: List[Dict[str, Any]] = []
        last = None
        for i, kind in enumerate(pattern):
            low = kind.lower()
            if low in "dc":
                layer = {"type": "delta" if low == "d" else "channel_delta",
                         "mixer": {"heads": delta_heads,
                                   "kv_heads": delta_kv_heads,
                                   "dim": delta_dim, "vdim": delta_vdim,
                                   "conv": taps}}
            else:
                layer = {"type": "attention",
                         "mixer": {"heads": heads, "kv_heads": kv_heads,
                                   "dim": dim, "vdim": vdim, "diff": diff,
                                   "mask": {"size": window},
                                   "scale": dim ** -0.5}}
                if low == "s":
                    layer["mixer"]["kv_from"] = last
                else:
                    last = i
            if kind.islower():
                layer["mlp"] = {"kind": "dense", "ff": ff}
            else:
                layer["mlp"] = {"kind": "moe", "expert": {"ff": expert_ff},
                                "router": {"experts": experts, "top": top}}
            layers.append(layer)
        cfg = GogalixConfig.from_json({
            "width": width, "vocab": vocab, "layers": layers,
            "norm": {"eps": 1e-6}, "embedding": {"scale": 2.0}}, name=name)
        cfg.low_rank = low_rank
        return cfg


def preset(name: str) -> Optional[GogalixConfig]:
    if name == "tiny-gogalix":          # CPU test shape
        return GogalixConfig.stacked(
            name, width=96, vocab=512, pattern="caDs", heads=4, kv_heads=2,
            dim=12, vdim=24, window=20, ff=160, delta_heads=4,
            delta_kv_heads=2, delta_dim=24, delta_vdim=16, taps=3, experts=6,
            top=2, expert_ff=40, low_rank=8)
    if name == "gogalix-8b":            # widths and depth of llama-3-8b
        return GogalixConfig.stacked(
            name, width=4096, vocab=128256, pattern="caDs" * 8, heads=16,
            kv_heads=4, dim=128, vdim=256, window=4096, ff=14336,
            delta_heads=32, delta_kv_heads=16, delta_dim=128, delta_vdim=128,
            experts=64, top=8, expert_ff=1792, low_rank=128)
    return None


class GogalixLayer(nn.Module):
    def __init__(self, cfg: GogalixConfig, index: int, first: int,
                 tp: TPContext, src: WeightSource, dtype: torch.dtype):
        super().__init__()
        spec, w, p = cfg.layers[index], cfg.hidden_size, f"l{index}."
        self.local = self.kv_layer = index - first  # into this stage's cache
        self.tp, self.dtype, self.eps = tp, dtype, cfg.rms_eps
        f32 = torch.float32
        self.norm1 = load_norm(src, p + "norm1")
        if spec["type"] == "attention":
            self.mixer = DifferentialAttention(spec["mixer"], w, self.eps, src,
                                               p + "mix.", tp, dtype)
            if self.mixer.kv_from is not None:
                self.kv_layer = self.mixer.kv_from - first
                if self.kv_layer < 0:
                    raise ValueError(
                        f"layer {index} uses the keys of layer "
                        f"{self.mixer.kv_from}, which is on another pipeline "
                        "stage")
        else:
            self.mixer = GatedDeltaRule(
                spec["mixer"], w, self.eps, src, p + "mix.", tp, dtype,
                spec["type"] == "channel_delta", cfg.low_rank)
        self.mlp = None
        if spec.get("mlp") is not None:
            kind = GatedSilu if spec["mlp"]["kind"] == "dense" else GluExperts
            self.mlp = kind(spec["mlp"], w, src, p + "mlp.", tp, dtype)
        # per branch: a scale, and a gate that reads the layer's input
        scales, biases, parts = [], [], list(self.mixer.parts)
        for n in ("1", "2")[:2 if self.mlp is not None else 1]:
            scales.append(src.take(p + "ls" + n, (w,), "ones"))
            biases.append(src.take(p + f"rg{n}.b", (w,), "zeros"))
            parts.append(("rg" + n, src.take(p + "rg" + n, (w, w))))
        self.scale = param(torch.stack(scales), f32)
        self.gate_bias = param(torch.stack(biases), f32)
        if self.mlp is not None:
            parts += self.mlp.parts
            self.mlp.parts = []
        self.mixer.parts = []
        self.proj = FusedProjection(parts, dtype)

    def cache_spec(self):
        return self.mixer.cache_spec()

    def forward(self, x: torch.Tensor,
                pending: Optional[List[ops.Branch]], batch: ForwardBatch,
                cache: StateCache) -> List[ops.Branch]:
        h = ops.gate_norm(x, pending or [], self.norm1, self.eps, self.dtype)
        y = self.proj(h)
        m = self.tp.all_reduce(self.mixer(y, self.proj, batch, cache,
                                          self.kv_layer))
        left = [ops.Branch(m, self.proj.slice(y, "rg1"), self.gate_bias[0],
                           self.scale[0])]
        if self.mlp is not None:
            f, route = self.mlp(h, y, self.proj)
            if self.tp.size > 1:
                if route is not None:
                    f, route = ops.moe_combine(f, route), None
                f = self.tp.all_reduce(f)
            left.append(ops.Branch(f, self.proj.slice(y, "rg2"),
                                   self.gate_bias[1], self.scale[1],
                                   self.mlp.bias, route))
        return left


def load_norm(src: WeightSource, name: str) -> nn.Parameter:
    """A norm's one number, as a vector of one element."""
    return param(src.take(name, (), "ones").view(1), torch.float32)


class GogalixForCausalLM(StreamForCausalLM):
    def load_norm(self, src: WeightSource, name: str) -> nn.Parameter:
        return load_norm(src, name)

    def build_layer(self, index: int, src: WeightSource) -> GogalixLayer:
        return GogalixLayer(self.cfg, index, self.layer_start, self.tp, src,
                            self.dtype)

    def spare_tensors(self):
        """Of branches that a layer does not have."""
        return {f"l{i}.{n}" for i in range(self.cfg.num_layers)
                for n in ("ls2", "rg2", "rg2.b")}

    def embed_rows(self, tokens: torch.Tensor,
                   batch: ForwardBatch) -> torch.Tensor:
        return ops.embed_stream(tokens, self.embed, self.cfg.embed_scale)

    def add(self, x: torch.Tensor,
            pending: List[ops.Branch]) -> torch.Tensor:
        ops.gate_norm(x, pending, None, self.cfg.rms_eps, self.dtype)
        return x

    def final(self, x: torch.Tensor,
              pending: List[ops.Branch]) -> torch.Tensor:
        return ops.gate_norm(x, pending, self.final_norm, self.cfg.rms_eps,
                             self.dtype)
