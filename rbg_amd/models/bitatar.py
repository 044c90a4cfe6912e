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
from ..engine.config import EngineConfig, ModelConfig
from ..engine.state_cache import StateCache
from .llama import PPContext, TPContext
from .mixers import GatedGelu, GeneralDelta, LatentAttention, param
from .weights import WeightSource, open_weights

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


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


class BitatarForCausalLM(nn.Module):
    """Same surface as LlamaForCausalLM (engine/model_runner.py drives it)."""

    stateful = True                     # step batches carry slots and starts
    mixed_steps = True                  # portions and decoded tokens together

    def __init__(self, cfg: BitatarConfig, device: torch.device,
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
        self.layers = nn.ModuleList([
            BitatarLayer(cfg, cfg.layers[i], i, i - self.layer_start, self.tp,
                         src, self.dtype)
            for i in range(self.layer_start, self.layer_end)])
        if self.pp.last:
            self.final_norm = param(src.take("final.norm", (w,), "ones"),
                                    torch.float32)
            self.lm_head = param(src.take("head", (cfg.vocab_size, w)),
                                 self.dtype)
        if self.pp.size == 1:
            src.finish(optional={f"l{i}.norm2" for i in range(L)})

    @property
    def num_local_layers(self) -> int:
        return self.layer_end - self.layer_start

    def make_cache(self, cfg: EngineConfig) -> StateCache:
        return StateCache(cfg, self.device,
                          [layer.cache_spec() for layer in self.layers],
                          self.dtype)

    def decode_splits(self, batch_size: int, max_seq_len: int) -> int:
        return 0                        # per layer, from its window

    @torch.inference_mode()
    def forward(self, tokens: torch.Tensor, batch: ForwardBatch,
                cache: StateCache,
                hidden: Optional[torch.Tensor] = None) -> torch.Tensor:
        """First PP stage embeds `tokens`, later stages take the stream from
        the one before; the last returns normed rows ready for logits()."""
        if self.pp.first:
            x = ops.embed_stream(tokens, self.embed, self.cfg.embed_scale)
        else:
            assert hidden is not None, "non-first PP stage needs hidden"
            x = hidden
        delta = None
        for layer in self.layers:
            delta = layer(x, delta, batch, cache)
        if not self.pp.last:
            return x + delta.float()
        return ops.stream_norm(x, delta, self.final_norm, None,
                               self.cfg.norm_groups, self.cfg.rms_eps,
                               self.dtype)[0]

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
        fresh = BitatarForCausalLM(self.cfg, self.device, self.tp,
                                   base_seed=seed, pp=self.pp)
        with torch.no_grad():
            for p, q in zip(self.parameters(), fresh.parameters()):
                p.copy_(q)
        del fresh
        if self.device.type == "cuda":
            torch.cuda.empty_cache()
        if self.tp.size > 1:
            torch.distributed.barrier(group=self.tp.group)
