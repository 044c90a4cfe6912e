"""Danipel: a decoder of latent attentions and of dense or expert feed-forwards
between hyper-connected f32 residual streams, under dynamic tanh norms.

There are several streams x_1 .. x_S, at first all the token's embedding.  A
sublayer (mixer, then feed-forward) reads a weighed sum of them and writes to all:

    y = sublayer(norm(sum_s in[s] x_s)),  norm(u) = tanh(alpha u) * w + b
    x_t <- sum_s mix[s, t] x_s + m * out[t] * y

and the head reads their sum.  The two kinds of latent attention differ in how
rotated pairs lie, in a sink, and in a latent for the queries.  Experts are clamped
gated units; some of the router's experts return their input.  On the GPU a layer
is:

  hyper_norm    the streams take the last sublayer's rows (or weighed expert rows);
                norm of what the mixer reads
  GEMM          queries (or their latent) and the key/value latent
  mixer         models/mixers.py LatentAttention; GEMM W_o
  hyper_norm    the same, for the feed-forward
  ff            gated GEMMs, or router, choice and grouped GEMMs
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
from .llama import TPContext
from .mixers import ClampedExperts, GatedGelu, LatentAttention, param
from .rotary import assign_tables
from .stream_model import StreamForCausalLM
from .weights import WeightSource

# what tells the two mixers apart
MIXERS: Dict[str, Dict[str, Any]] = {
    "latent_attention": {"rotary": "interleaved", "sink": True},
    "latent_attention_2": {"rotary": "halves", "q_latent": True},
}


@dataclass
class DanipelConfig(ModelConfig):
    architecture: str = "Danipel"
    max_position: int = 1 << 30     # the engine's limit sizes the angle tables
    layers: List[Dict[str, Any]] = field(default_factory=list)
    embed_scale: float = 1.0
    streams: int = 1
    residual_mult: float = 1.0

    @staticmethod
    def from_json(d: Dict[str, Any], name: str = "danipel",
                  weights_path: str = "") -> "DanipelConfig":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp.get("kind") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward kind "
                                 f"{mlp.get('kind')!r}")
        if int(d["streams"]) < 1:
            raise ValueError(f"{d['streams']} streams")
        return DanipelConfig(
            name=name, weights_path=weights_path, layers=layers,
            hidden_size=int(d["width"]), vocab_size=int(d["vocab"]),
            num_layers=len(layers), rms_eps=float(d["norm"]["eps"]),
            embed_scale=float(d["embedding"]["scale"]),
            streams=int(d["streams"]),
            residual_mult=float(d["residual_mult"]))

    @staticmethod
    def stacked(name: str, width: int, vocab: int, pattern: str, heads: int,
                dim: int, rot_dim: int, vdim: int, kv_rank: int, q_rank: int,
                ff: int, streams: int = 4, experts: int = 0, identity: int = 0,
                top: int = 0, expert_ff: int = 0,
                shared_ff: int = 0) -> "DanipelConfig":
        """A configuration from a layer pattern, e.g. for presets and
        benchmarks: 'a' has queries straight from the stream, 'b' queries from
        a latent; a capital has experts instead of a dense feed-forward."""
        layers = []
        for kind in pattern:
            mixer: Dict[str, Any] = {
                "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                "kv_rank": kv_rank, "scale": (dim + rot_dim) ** -0.5,
                "rot": {"dims": rot_dim, "base": 500000.0}}
            if kind.lower() == "a":
                mixer["rot"]["scaling"] = {"factor": 4.0, "original": 4096,
                                           "fast": 32.0, "slow": 1.0}
                layer = {"type": "latent_attention", "mixer": mixer}
            else:
                mixer["q_rank"] = q_rank
                layer = {"type": "latent_attention_2", "mixer": mixer}
            if kind.islower():
                layer["mlp"] = {"kind": "dense", "ff": ff}
            else:
                layer["mlp"] = {
                    "kind": "moe", "expert": {"ff": expert_ff, "limit": 7.0},
                    "router": {"experts": experts, "identity": identity,
                               "top": top, "scale": 2.0}}
                if shared_ff:
                    layer["mlp"]["shared"] = {"ff": shared_ff, "limit": 7.0}
            layers.append(layer)
        return DanipelConfig.from_json({
            "width": width, "vocab": vocab, "layers": layers,
            "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "streams": streams, "residual_mult": 0.5}, name=name)


def preset(name: str) -> Optional[DanipelConfig]:
    if name == "tiny-danipel":          # CPU test shape
        return DanipelConfig.stacked(
            name, width=96, vocab=512, pattern="aBAb", heads=4, dim=16,
            rot_dim=8, vdim=24, kv_rank=40, q_rank=32, ff=160, streams=3,
            experts=6, identity=2, top=2, expert_ff=40, shared_ff=48)
    if name == "danipel-16b-a3b":       # widths of current latent-attention models
        return DanipelConfig.stacked(
            name, width=2048, vocab=102400, pattern="aBAB" * 7, heads=16,
            dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536, ff=10944,
            streams=4, experts=64, identity=8, top=6, expert_ff=1408,
            shared_ff=2816)
    return None


class TanhNorm(nn.Module):
    def __init__(self, src: WeightSource, name: str, width: int):
        super().__init__()
        f32 = torch.float32
        self.alpha = param(src.take(name + ".alpha", (), "ones").view(1), f32)
        self.w = param(src.take(name, (width,), "ones"), f32)
        self.b = param(src.take(name + ".b", (width,), "zeros"), f32)

    def op(self) -> ops.TanhNorm:
        return ops.TanhNorm(self.alpha, self.w, self.b)


class HyperConnection(nn.Module):
    """How one sublayer reads the streams and is written to them."""

    def __init__(self, src: WeightSource, prefix: str, streams: int):
        super().__init__()
        n, f32 = streams, torch.float32
        self.read = param(src.take(prefix + "in", (n,)), f32)
        out = src.take(prefix + "out", (n,)).float()
        mix = src.take(prefix + "mix", (n, n), "eye").float()
        self.conn = param(torch.cat([mix.reshape(-1), out]), f32)


class DanipelLayer(nn.Module):
    def __init__(self, cfg: DanipelConfig, index: int, local: int,
                 tp: TPContext, src: WeightSource, dtype: torch.dtype):
        super().__init__()
        spec, w, p = cfg.layers[index], cfg.hidden_size, f"l{index}."
        self.local = local              # index into this stage's cache
        self.tp, self.dtype = tp, dtype
        self.streams, self.mult = cfg.streams, cfg.residual_mult
        self.norm1 = TanhNorm(src, p + "norm1", w)
        self.hc1 = HyperConnection(src, p + "hc1.", self.streams)
        self.mixer = LatentAttention(
            spec["mixer"], w, cfg.rms_eps, src, p + "mix.", tp, dtype,
            gated=False, **MIXERS[spec["type"]])
        self.w_o = param(self.mixer.w_out, dtype)
        self.mixer.w_out = None
        self.mlp = self.w_down = None
        if spec.get("mlp") is None:
            return
        self.norm2 = TanhNorm(src, p + "norm2", w)
        self.hc2 = HyperConnection(src, p + "hc2.", self.streams)
        if spec["mlp"]["kind"] == "dense":
            self.mlp = GatedGelu(spec["mlp"], w, src, p + "mlp.", tp, dtype)
            self.w_down = param(self.mlp.w_out, dtype)
            self.mlp.w_out = None
        else:
            self.mlp = ClampedExperts(spec["mlp"], w, src, p + "mlp.", tp,
                                      dtype)

    def cache_spec(self):
        return self.mixer.cache_spec()

    def _read(self, x: torch.Tensor, pending: Optional[ops.Stir],
              hc: HyperConnection, norm: TanhNorm) -> torch.Tensor:
        return ops.hyper_norm(x, self.streams, pending, hc.read, norm.op(),
                              self.dtype)

    def forward(self, x: torch.Tensor, pending: Optional[ops.Stir],
                batch: ForwardBatch, cache: StateCache) -> ops.Stir:
        h = self._read(x, pending, self.hc1, self.norm1)
        act = h.new_empty((h.shape[0], self.mixer.out_dim))
        self.mixer(h, act, batch, cache, self.local)
        y = self.tp.all_reduce(ops.linear(act, self.w_o))
        pending = ops.Stir(self.hc1.conn, self.mult, y)
        if self.mlp is None:
            return pending
        h = self._read(x, pending, self.hc2, self.norm2)
        if self.w_down is not None:
            act = h.new_empty((h.shape[0], self.mlp.out_dim))
            self.mlp(h, act)
            y = self.tp.all_reduce(ops.linear(act, self.w_down))
            return ops.Stir(self.hc2.conn, self.mult, y)
        shared, y, route = self.mlp(h)
        if self.tp.size > 1:
            # the shards' sum, without the experts that are whole everywhere
            y = ops.moe_combine(y, route)
            shared = self.tp.all_reduce(y if shared is None else y + shared)
            y = None
        return ops.Stir(self.hc2.conn, self.mult, shared, y, route,
                        h if self.mlp.identity else None)


class DanipelForCausalLM(StreamForCausalLM):
    stateful = False            # its tokens and pages are all a sequence has

    def load_norm(self, src: WeightSource, name: str) -> TanhNorm:
        self.every = param(torch.ones(self.cfg.streams, device=self.device),
                           torch.float32)
        return TanhNorm(src, name, self.cfg.hidden_size)

    def build_layer(self, index: int, src: WeightSource) -> DanipelLayer:
        return DanipelLayer(self.cfg, index, index - self.layer_start, self.tp,
                            src, self.dtype)

    def spare_tensors(self):
        """Of feed-forwards that a layer does not have."""
        return {f"l{i}.{n}" for i in range(self.cfg.num_layers)
                for n in ("norm2", "norm2.alpha", "norm2.b", "hc2.in",
                          "hc2.out", "hc2.mix")}

    @property
    def stream_width(self) -> int:
        return self.cfg.streams * self.cfg.hidden_size

    def make_cache(self, cfg: EngineConfig) -> StateCache:
        assign_tables((layer.mixer for layer in self.layers), cfg.max_seq_len,
                      self.device)
        return super().make_cache(cfg)

    def embed_rows(self, tokens: torch.Tensor,
                   batch: ForwardBatch) -> torch.Tensor:
        return ops.embed_stream(tokens, self.embed, self.cfg.embed_scale,
                                self.cfg.streams)

    def add(self, x: torch.Tensor, pending: ops.Stir) -> torch.Tensor:
        ops.hyper_norm(x, self.cfg.streams, pending, None, None, self.dtype)
        return x

    def final(self, x: torch.Tensor, pending: ops.Stir) -> torch.Tensor:
        return ops.hyper_norm(x, self.cfg.streams, pending, self.every,
                              self.final_norm.op(), self.dtype)
