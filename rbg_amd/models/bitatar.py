"""Bitatar: a decoder of generalized-delta and windowed latent-attention
layers over an f32 residual stream.

A layer adds mixer(norm1(x)) + ff(norm2(x)) to the stream, both of the same x;
the norms are grouped RMS norms, and the mixer's input first goes through a
short causal convolution with a residual.  On the GPU a layer is:

  stream_norm   x += last layer's sum; norm1 and norm2 of x (in decode also
                the convolution, with the history in the sequence's slot)
  GEMM + mixer  models/mixers.py, into columns [0, m) of the output operand
  GEMM + gelu   into columns [m, m + ff)
  GEMM          [W_o | W_down], which sums both branches; one all-reduce
                under tensor parallelism
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
from .mixers import GatedGelu, GeneralDelta, LatentAttention, param
from .stream_model import StreamForCausalLM
from .weights import WeightSource


@dataclass
class BitatarConfig(ModelConfig):
    architecture: str = "Bitatar"
    max_position: int = 1 << 30         # nothing in the design is positional
    layers: List[Dict[str, Any]] = field(default_factory=list)
    norm_groups: int = 1
    embed_scale: float = 1.0
    conv_taps: int = 1
    decay_rank: int = 64                # of random weights; files bring theirs

    @staticmethod
    def from_json(d: Dict[str, Any], name: str = "bitatar",
                  weights_path: str = "") -> "BitatarConfig":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] not in ("general_delta", "latent_attention"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        return BitatarConfig(
            name=name, weights_path=weights_path, layers=layers,
            hidden_size=int(d["width"]), vocab_size=int(d["vocab"]),
            num_layers=len(layers), rms_eps=float(d["norm"]["eps"]),
            norm_groups=int(d["norm"]["groups"]),
            embed_scale=float(d["embedding"]["scale"]),
            conv_taps=int(d["canon"]["taps"]))

    @staticmethod
    def stacked(name: str, width: int, vocab: int, pattern: str, heads: int,
                dim: int, kv_rank: int, vdim: int, window: int, ff: int,
                groups: int, taps: int, delta_heads: int,
                delta_dim: int) -> "BitatarConfig":
        """A configuration from a layer pattern of 'd' (delta) and 'a'
        (latent attention), e.g. for presets and benchmarks."""
        layers = []
        for kind in pattern:
            if kind == "d":
                layer = {"type": "general_delta",
                         "mixer": {"heads": delta_heads, "dim": delta_dim}}
            else:
                layer = {"type": "latent_attention",
                         "mixer": {"heads": heads, "dim": dim,
                                   "kv_rank": kv_rank, "vdim": vdim,
                                   "mask": {"size": window},
                                   "scale": dim ** -0.5}}
            layer["mlp"] = {"kind": "dense", "ff": ff}
            layers.append(layer)
        return BitatarConfig.from_json({
            "width": width, "vocab": vocab, "layers": layers,
            "norm": {"eps": 1e-5, "groups": groups},
            "embedding": {"scale": width ** 0.5},
            "canon": {"taps": taps}}, name=name)


def preset(name: str) -> Optional[BitatarConfig]:
    if name == "tiny-bitatar":          # CPU test shape
        return BitatarConfig.stacked(
            name, width=96, vocab=512, pattern="dada", heads=3, dim=16,
            kv_rank=24, vdim=24, window=20, ff=160, groups=3, taps=3,
            delta_heads=2, delta_dim=24)
    if name == "bitatar-8b":            # widths and depth of llama-3-8b
        return BitatarConfig.stacked(
            name, width=4096, vocab=128256, pattern="daa" * 10 + "da",
            heads=32, dim=128, kv_rank=512, vdim=128, window=4096, ff=14336,
            groups=8, taps=4, delta_heads=32, delta_dim=128)
    return None


class BitatarLayer(nn.Module):
    def __init__(self, cfg: BitatarConfig, spec: Dict[str, Any],
                 index: int, local: int, tp: TPContext, src: WeightSource,
                 dtype: torch.dtype):
        super().__init__()
        self.local = local              # index into this stage's cache
        self.tp, self.dtype = tp, dtype
        self.groups, self.eps = cfg.norm_groups, cfg.rms_eps
        w, p = cfg.hidden_size, f"l{index}."
        f32 = torch.float32
        self.norm1 = param(src.take(p + "norm1", (w,), "ones"), f32)
        self.mlp = self.norm2 = None
        if spec.get("mlp") is not None:
            self.norm2 = param(src.take(p + "norm2", (w,), "ones"), f32)
            self.mlp = GatedGelu(spec["mlp"], w, src, p + "mlp.", tp, dtype)
        # [taps, width]: a tap is one contiguous row
        self.conv_w = param(src.take(p + "canon1", (w, cfg.conv_taps),
                                     "conv").T, f32)
        if spec["type"] == "general_delta":
            self.mixer = GeneralDelta(spec["mixer"], w, self.eps, src,
                                      p + "mix.", tp, dtype, cfg.decay_rank)
        else:
            self.mixer = LatentAttention(spec["mixer"], w, self.eps, src,
                                         p + "mix.", tp, dtype)
        outs = [self.mixer.w_out] + ([self.mlp.w_out] if self.mlp else [])
        self.w_out = param(torch.cat(outs, dim=1), dtype)
        self.mixer.w_out = None
        if self.mlp:
            self.mlp.w_out = None
        self.width, self.taps = w, cfg.conv_taps

    def cache_spec(self):
        spec = self.mixer.cache_spec()
        if self.taps > 1:
            spec.state["conv"] = ((self.taps - 1, self.width), self.dtype)
        return spec

    def forward(self, x: torch.Tensor, delta: Optional[torch.Tensor],
                batch: ForwardBatch, cache: StateCache) -> torch.Tensor:
        """Adds ``delta`` to the stream x in place; returns the sum that the
        next layer adds."""
        if self.taps > 1:
            conv_state = cache.state(self.local, "conv")
        else:
            conv_state = x.new_empty((cache.num_slots, 0, self.width),
                                     dtype=self.dtype)
        if batch.mode == "decode":
            h, n2 = ops.stream_norm_conv(
                x, delta, self.norm1, self.norm2, self.groups, self.eps,
                self.dtype, self.conv_w, conv_state, batch.state_slots,
                batch.positions)
        else:
            n1, n2 = ops.stream_norm(x, delta, self.norm1, self.norm2,
                                     self.groups, self.eps, self.dtype)
            tile = max(ops.CONV_TILE, self.taps)
            h = ops.causal_conv(n1, self.conv_w, conv_state,
                                batch.layout.tiles(tile), batch.cu_seqlens,
                                batch.starts, batch.state_slots)
        act = h.new_empty((h.shape[0], self.w_out.shape[1]))
        m = self.mixer.out_dim
        self.mixer(h, act[:, :m], batch, cache, self.local)
        if self.mlp is not None:
            self.mlp(n2, act[:, m:])
        return self.tp.all_reduce(ops.linear(act, self.w_out))


class BitatarForCausalLM(StreamForCausalLM):
    def build_layer(self, index: int, src: WeightSource) -> BitatarLayer:
        return BitatarLayer(self.cfg, self.cfg.layers[index], index,
                            index - self.layer_start, self.tp, src,
                            self.dtype)

    def spare_tensors(self):
        return {f"l{i}.norm2" for i in range(self.cfg.num_layers)}

    def embed_rows(self, tokens: torch.Tensor,
                   batch: ForwardBatch) -> torch.Tensor:
        return ops.embed_stream(tokens, self.embed, self.cfg.embed_scale)

    def add(self, x: torch.Tensor, pending: torch.Tensor) -> torch.Tensor:
        return x + pending.float()

    def final(self, x: torch.Tensor, pending: torch.Tensor) -> torch.Tensor:
        return ops.stream_norm(x, pending, self.final_norm, None,
                               self.cfg.norm_groups, self.cfg.rms_eps,
                               self.dtype)[0]
