"""Token mixers and feed-forwards of models with an f32 residual stream.

Each part loads its tensors, declares what it keeps for a sequence
(``cache_spec``) and computes from the layer's normed input into a column slice
of the layer's output operand: the layer concatenates the parts' products and
applies all their output projections as ONE GEMM, which also adds them up.
The parts that read the same input are one GEMM too (``FusedProjection``).

Work split: library GEMMs for the projections, one hand-written kernel each
for the recurrence (with decay, gates, unit keys and head norm inside) and for
the attention (with window, softmax and, in prefill, the output gate inside).
Tensor parallelism shards heads and feed-forward columns.

Parts of a design that norms or gates each branch before adding it
(``PagedAttention``, ``SparseExperts``, and those after them) apply their own
output projection instead.  ``GatedDeltaRule``, ``DifferentialAttention`` and
``GatedSilu`` leave the input projection to the layer as ``parts``: where every
sublayer reads one norm, a layer has a single input GEMM.
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from .. import ops
from ..engine.batch import ForwardBatch
from ..engine.state_cache import LayerCacheSpec, StateCache
from .weights import WeightSource


def param(t: torch.Tensor, dtype: torch.dtype) -> nn.Parameter:
    return nn.Parameter(t.to(dtype).contiguous(), requires_grad=False)


def shard(t: torch.Tensor, tp, dim: int = 0) -> torch.Tensor:
    return t if tp.size == 1 else t.chunk(tp.size, dim=dim)[tp.rank]


class FusedProjection(nn.Module):
    """Several projections of one input as one GEMM.  Segments start at
    multiples of 8 columns (zero rows between), so that every slice of the
    result can be read 16 bytes at a time."""

    def __init__(self, parts: List[Tuple[str, torch.Tensor]],
                 dtype: torch.dtype):
        super().__init__()
        rows, at = [], 0
        self.cols: Dict[str, Tuple[int, int]] = {}
        for name, w in parts:
            self.cols[name] = (at, w.shape[0])
            rows.append(w)
            pad = -w.shape[0] % 8
            if pad:
                rows.append(w.new_zeros(pad, w.shape[1]))
            at += w.shape[0] + pad
        self.weight = param(torch.cat(rows), dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.linear(x, self.weight)

    def offset(self, name: str) -> int:
        return self.cols[name][0]

    def slice(self, y: torch.Tensor, name: str) -> torch.Tensor:
        at, n = self.cols[name]
        return y[:, at:at + n]


Parts = List[Tuple[str, torch.Tensor]]


def pad8(t: torch.Tensor, dim: int = 0) -> torch.Tensor:
    """t with zeros up to a multiple of 8 along ``dim``."""
    n = -t.shape[dim] % 8
    if not n:
        return t
    shape = list(t.shape)
    shape[dim] = n
    return torch.cat([t, t.new_zeros(shape)], dim=dim)


class GeneralDelta(nn.Module):
    """Generalized delta rule with per-channel decay and removal rate."""

    decay_scale = math.exp(-0.5)    # w = exp(-decay_scale * sigmoid(.))
    unit_eps = 1e-6                 # inside the root of the key's norm

    def __init__(self, spec: Dict[str, Any], width: int, eps: float,
                 src: WeightSource, prefix: str, tp, dtype: torch.dtype,
                 decay_rank: int):
        super().__init__()
        heads, dim = int(spec["heads"]), int(spec["dim"])
        assert heads % tp.size == 0, "TP degree must divide head counts"
        self.heads, self.dim, self.eps, self.dtype = \
            heads // tp.size, dim, eps, dtype
        full = heads * dim
        rank = src.shape(prefix + "w1", (decay_rank, width))[0]

        def lin(name, shape):
            return src.take(prefix + name, shape)
        parts = [(n, shard(lin(n, (full, width)), tp))
                 for n in ("r", "k", "v", "a", "g")]
        parts.append(("w1", lin("w1", (rank, width))))
        self.proj = FusedProjection(parts, dtype)
        self.offs = [self.proj.offset(n)
                     for n in ("r", "k", "v", "a", "g", "w1")]
        self.w2 = param(shard(lin("w2", (full, rank)), tp), dtype)
        f32 = torch.float32
        self.w0 = param(shard(src.take(prefix + "w0", (full,), "normal"), tp),
                        f32)
        self.a_bias = param(shard(src.take(prefix + "a.b", (full,), "normal"),
                                  tp), f32)
        self.norm = param(shard(src.take(prefix + "norm", (full,), "ones"),
                                tp), f32)
        self.w_out = shard(lin("o", (width, full)), tp, dim=1)
        self.out_dim = self.heads * dim

    def cache_spec(self) -> LayerCacheSpec:
        return LayerCacheSpec(state={
            "delta": ((self.heads, self.dim, self.dim), torch.float32)})

    def forward(self, h: torch.Tensor, out: torch.Tensor, batch: ForwardBatch,
                cache: StateCache, layer: int) -> None:
        y = self.proj(h)
        state = cache.state(layer, "delta")

        def run(rows, z, seqs, cu, chunks=None):
            ops.delta_rule(y[rows], z, self.w2, self.w0, self.a_bias,
                           self.norm, state, batch.state_slots[seqs], cu,
                           batch.starts[seqs], out[rows], self.offs,
                           self.decay_scale, self.unit_eps, self.eps, chunks)
        every = slice(None)
        if batch.mode == "decode":
            run(every, None, every, None)
            return
        nd = batch.num_decode
        if nd:
            run(slice(0, nd), None, slice(0, nd), None)
        if nd == y.shape[0]:
            return
        low = ops.tanh_rows(self.proj.slice(y[nd:], "w1"))
        z = ops.linear(low, self.w2)
        layout = batch.layout
        run(slice(nd, None), z, slice(nd, None), batch.cu_prefill,
            (layout.prefill_tiles(ops.DELTA_CHUNK),
             layout.prefill_tile_cu(ops.DELTA_CHUNK)))


class LatentAttention(nn.Module):
    """Softmax attention over a cached low-rank latent, through a sliding window,
    with an output gate (``gated``).

    With ``rotary`` ("interleaved" or "halves", how pairs lie) the spec's
    rot_dim last dims of a head's query meet one rotated key part that all
    heads share and that is cached behind the latent.  ``q_latent``: queries
    come from a normed latent of their own.  ``sink``: a learned logit per head
    that has no key and no value.

    Prefill expands the visible latents to per-head keys and values; decode
    folds the key expansion into the query and the value expansion into the
    output, so that it streams only the latents."""

    def __init__(self, spec: Dict[str, Any], width: int, eps: float,
                 src: WeightSource, prefix: str, tp, dtype: torch.dtype,
                 gated: bool = True, rotary: Optional[str] = None,
                 q_latent: bool = False, sink: bool = False):
        super().__init__()
        heads = int(spec["heads"])
        assert heads % tp.size == 0, "TP degree must divide head counts"
        self.heads = heads // tp.size
        self.dim, self.vdim = int(spec["dim"]), int(spec["vdim"])
        self.rank = int(spec["kv_rank"])
        self.scale = float(spec["scale"])
        self.rot = self.cos_sin = None  # the table is set with the cache
        self.rot_dim = 0
        if rotary is not None:
            self.rot, self.rot_dim = spec["rot"], int(spec["rot_dim"])
            if int(self.rot["dims"]) != self.rot_dim:
                raise ValueError(f"{self.rot['dims']} rotated dimensions in a "
                                 f"part of {self.rot_dim}")
        self.interleaved = rotary == "interleaved"
        mask = spec.get("mask") or {}
        self.window = int(mask.get("size") or 0)     # 0: everything before
        self.eps, self.dtype = eps, dtype
        f32 = torch.float32
        qk, vo = heads * (self.dim + self.rot_dim), heads * self.vdim

        def lin(name, shape):
            return src.take(prefix + name, shape)
        self.uq: Optional[nn.Parameter] = None
        if q_latent:
            q_rank = int(spec["q_rank"])
            parts = [("dq", lin("dq", (q_rank, width)))]
            self.uq = param(shard(lin("uq", (qk, q_rank)), tp), dtype)
            self.q_norm = param(src.take(prefix + "dq.norm", (q_rank,),
                                         "ones"), f32)
        else:
            parts = [("q", shard(lin("q", (qk, width)), tp))]
        parts.append(("dkv", lin("dkv", (self.rank + self.rot_dim, width))))
        self.gated = gated
        if gated:
            parts.append(("g", shard(lin("g", (vo, width)), tp)))
        self.proj = FusedProjection(parts, dtype)
        self.c_norm = param(src.take(prefix + "dkv.norm", (self.rank,),
                                     "ones"), f32)
        uk = shard(lin("uk", (heads * self.dim, self.rank)), tp)
        uv = shard(lin("uv", (vo, self.rank)), tp)
        # prefill: one expansion GEMM.  decode: per-head maps [n, k]
        self.expand = FusedProjection([("k", uk), ("v", uv)], dtype)
        self.uk_t = param(uk.reshape(self.heads, self.dim, self.rank)
                          .transpose(1, 2), dtype)
        self.uv = param(uv.reshape(self.heads, self.vdim, self.rank), dtype)
        self.sink: Optional[nn.Parameter] = None
        if sink:
            self.sink = param(shard(src.take(prefix + "sink", (heads,),
                                             "normal"), tp), f32)
        self.w_out = shard(lin("o", (width, vo)), tp, dim=1)
        self.out_dim = self.heads * self.vdim

    def cache_spec(self) -> LayerCacheSpec:
        return LayerCacheSpec(latent_rank=self.rank + self.rot_dim)

    def forward(self, h: torch.Tensor, out: torch.Tensor, batch: ForwardBatch,
                cache: StateCache, layer: int) -> None:
        y = self.proj(h)
        latents = cache.latents(layer)
        rot = None
        if self.rot is not None:
            rot = ops.Rotary(self.cos_sin, batch.positions, self.interleaved)
        low = self.proj.slice(y, "dkv")
        if self.uq is None:
            c = ops.latent_store(low, self.c_norm, latents,
                                 batch.slot_mapping, self.eps, rot)
            q = self.proj.slice(y, "q")
        else:
            c, cq = ops.latent_store(
                low, self.c_norm, latents, batch.slot_mapping, self.eps, rot,
                second=(self.proj.slice(y, "dq"), self.q_norm))
            q = ops.linear(cq, self.uq)
        q = q.unflatten(1, (self.heads, self.dim + self.rot_dim))
        g = self.proj.slice(y, "g") if self.gated else None
        nd = y.shape[0] if batch.mode == "decode" else batch.num_decode

        def run(step, part, *args):
            step(q[part], None if g is None else g[part],
                 None if rot is None else rot.rows(part), out[part], batch,
                 latents, *args)
        if nd:
            run(self._decode, slice(0, nd))
        if nd < y.shape[0]:
            run(self._prefill, slice(nd, None), c[nd:])

    def _prefill(self, q, g, rot, out, batch, latents, c) -> None:
        view = batch.layout.window_view(self.window)
        if view.slots is not None:
            c = latents.view(-1, latents.shape[-1])[view.slots]
        kv = self.expand(c[:, :self.rank])
        k = self.expand.slice(kv, "k").unflatten(1, (self.heads, self.dim))
        v = self.expand.slice(kv, "v").unflatten(1, (self.heads, self.vdim))
        shared = None
        if rot is not None:
            ops.rotate_rows(q[..., self.dim:], rot)
            shared = c[:, self.rank:]
        ops.window_attention(q, k, v, g, out, view, self.scale, self.window,
                             shared, self.sink)

    def _decode(self, q, g, rot, out, batch, latents) -> None:
        if rot is None:
            q = ops.head_linear(q, self.uk_t).unflatten(
                1, (self.heads, self.rank))
        else:
            q = ops.head_linear(q[..., :self.dim], self.uk_t,
                                tail=q[..., self.dim:], rot=rot)
        o = ops.latent_decode(q, latents, batch.block_tables,
                              batch.context_lens, self.scale, self.window,
                              self.rank, self.sink)
        ops.head_linear(o, self.uv, gate=g, out=out)


class GatedGelu(nn.Module):
    """down(gelu_tanh(gate x) * up x); the layer applies ``down``."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        if spec.get("kind") != "dense":
            raise ValueError(f"unknown feed-forward kind {spec.get('kind')!r}")
        ff = int(spec["ff"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        gate = shard(src.take(prefix + "gate", (ff, width)), tp)
        up = shard(src.take(prefix + "up", (ff, width)), tp)
        self.gate_up = param(torch.cat([gate, up]), dtype)
        self.w_out = shard(src.take(prefix + "down", (width, ff)), tp, dim=1)
        self.out_dim = ff // tp.size

    def forward(self, x: torch.Tensor, out: torch.Tensor) -> None:
        ops.gelu_mul(ops.linear(x, self.gate_up), out)


class PagedAttention(nn.Module):
    """Causal softmax attention over paged keys and values of any sizes:
    grouped heads, biases, partial rotary positions, scores squashed by a soft
    cap, a silent key of score zero (a sink), and, with ``kv_from``, another
    layer's keys and values.

    One GEMM projects queries (and keys and values); one kernel adds the
    biases, rotates, and writes keys and values to the pages; the attention
    kernels read pages only, so that a layer's own tokens and another layer's
    are found in the same place."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype, sink: bool):
        super().__init__()
        heads, kv_heads = int(spec["heads"]), int(spec["kv_heads"])
        if heads % kv_heads:
            raise ValueError(f"{heads} heads over {kv_heads} key heads")
        assert heads % tp.size == 0 and kv_heads % tp.size == 0, \
            "TP degree must divide head counts"
        self.heads, self.kv_heads = heads // tp.size, kv_heads // tp.size
        self.dim, self.vdim = int(spec["dim"]), int(spec["vdim"])
        self.scale = float(spec["scale"])
        self.softcap = float(spec.get("softcap") or 0.0)    # 0: none
        self.sink = sink
        self.rot = spec["rot"]
        if int(self.rot["dims"]) > self.dim:
            raise ValueError("more rotated dimensions than a head has")
        self.kv_from: Optional[int] = spec.get("kv_from")   # global layer
        self.cos_sin: Optional[torch.Tensor] = None         # set with the cache
        outs = {"q": heads * self.dim}
        if self.kv_from is None:
            outs.update(k=kv_heads * self.dim, v=kv_heads * self.vdim)
        parts, biases = [], []
        for name, n in outs.items():
            parts.append((name, shard(src.take(prefix + name, (n, width)),
                                      tp)))
            bias = shard(src.take(prefix + name + ".b", (n,)), tp)
            biases += [bias, bias.new_zeros(-bias.numel() % 8)]
        self.proj = FusedProjection(parts, dtype)
        self.bias = param(torch.cat(biases), torch.float32)
        self.w_out = param(shard(src.take(prefix + "o",
                                          (width, heads * self.vdim)),
                                 tp, dim=1), dtype)

    def cache_spec(self) -> LayerCacheSpec:
        if self.kv_from is not None:
            return LayerCacheSpec()
        return LayerCacheSpec(kv=(self.kv_heads, self.dim, self.vdim))

    def forward(self, h: torch.Tensor, batch: ForwardBatch, cache: StateCache,
                kv_layer: int) -> torch.Tensor:
        y = self.proj(h)
        k, v = cache.kv_pages(kv_layer)
        offs = [self.proj.offset(n) for n in self.proj.cols]
        ops.rope_store_paged(y, self.bias, self.cos_sin, batch.positions,
                             batch.slot_mapping, self.heads, self.dim, k, v,
                             offs)
        q = self.proj.slice(y, "q").unflatten(1, (self.heads, self.dim))
        out = y.new_empty((y.shape[0], self.heads * self.vdim))
        score = (self.scale, self.softcap, self.sink)
        nd = y.shape[0] if batch.mode == "decode" else batch.num_decode
        if nd:
            ops.paged_decode(q[:nd], k, v, batch.block_tables,
                             batch.context_lens, out[:nd], *score)
        if nd < y.shape[0]:
            ops.paged_prefill(q[nd:], k, v, batch.layout.paged_view(),
                              out[nd:], *score)
        return ops.linear(out, self.w_out)


class SparseExperts(nn.Module):
    """Mixture of small feed-forwards down(relu(up x)^2): sigmoid router
    scores, a correction that only the choice sees, a choice limited to the
    best groups of neighbouring experts, unnormalized weights.

    Tensor parallelism shards every expert's inner columns."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        if spec.get("kind") != "moe":
            raise ValueError(f"unknown feed-forward kind {spec.get('kind')!r}")
        r, ff = spec["router"], int(spec["expert"]["ff"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        n, self.top = int(r["experts"]), int(r["top"])
        groups = r.get("groups") or {}
        self.groups = int(groups.get("count", 1))
        self.keep = int(groups.get("keep", self.groups))
        if n % self.groups or not 1 <= self.keep <= self.groups or not \
                1 <= self.top <= self.keep * (n // self.groups):
            raise ValueError(f"router: {n} experts, {self.groups} groups, "
                             f"{self.keep} kept, {self.top} chosen")

        def stack(name, shape, dim):
            return param(torch.stack([
                shard(src.take(f"{prefix}e{e}.{name}", shape), tp, dim)
                for e in range(n)]), dtype)
        self.up = stack("up", (ff, width), 0)
        self.down = stack("down", (width, ff), 1)
        self.router = param(src.take(prefix + "router", (n, width)), dtype)
        self.correction = param(src.take(prefix + "correction", (n,)),
                                torch.float32)

    def forward(self, x: torch.Tensor):
        """Outputs of the chosen experts, one row per (token, choice) in
        expert order, and the routing that weighs and finds them."""
        logits = ops.router_logits(x, self.router)
        route = ops.moe_route(logits, self.correction, self.groups, self.keep,
                              self.top, ops.expert_tile(x, self.up, self.top))
        h = ops.expert_linear(x, self.up, route, gather=True, relu2=True)
        return ops.expert_linear(h, self.down, route), route


class GatedDeltaRule(nn.Module):
    """Gated delta rule behind a short convolution, with one decay per head or
    (``per_channel``) one per head and key channel from a low-rank map, grouped
    query/key heads, a head norm and an output gate (silu, or a sigmoid of a
    low-rank map)."""

    unit_eps = 1e-6                 # inside the root of q's and k's norms

    def __init__(self, spec: Dict[str, Any], width: int, eps: float,
                 src: WeightSource, prefix: str, tp, dtype: torch.dtype,
                 per_channel: bool, rank: int):
        super().__init__()
        heads, kv_heads = int(spec["heads"]), int(spec["kv_heads"])
        if heads % kv_heads:
            raise ValueError(f"{heads} heads over {kv_heads} key heads")
        assert heads % tp.size == 0 and kv_heads % tp.size == 0, \
            "TP degree must divide head counts"
        self.heads, self.kv_heads = heads // tp.size, kv_heads // tp.size
        self.dim, self.vdim = int(spec["dim"]), int(spec["vdim"])
        self.taps, self.eps, self.dtype = int(spec["conv"]), eps, dtype
        self.per_channel = per_channel
        qk, vo, f32 = kv_heads * self.dim, heads * self.vdim, torch.float32

        def take(name, shape, init="linear"):
            return src.take(prefix + name, shape, init)

        def mine(t, dim=0):
            return shard(t, tp, dim)
        self.parts: Parts = []
        conv = []
        for name, n in (("q", qk), ("k", qk), ("v", vo)):
            self.parts.append((name, mine(take(name, (n, width)))))
            # [taps, channels]; zero columns where the projection has zero rows
            conv.append(pad8(mine(take(name + ".conv", (n, self.taps),
                                       "conv"))).T)
        self.conv_w = param(torch.cat(conv, dim=1), f32)
        self.parts.append(("b", mine(take("b", (heads, width)))))
        self.low: Optional[nn.Parameter] = None
        if per_channel:
            # both low-rank maps' second halves as one block-diagonal matrix
            names = (("a1", "a2", heads * self.dim), ("g1", "g2", vo))
            second = []
            for one, two, n in names:
                r = src.shape(prefix + one, (rank, width))[0]
                self.parts.append((one, take(one, (r, width))))
                second.append(pad8(pad8(mine(take(two, (n, r)))), 1))
            self.low = param(torch.block_diag(*second), dtype)
            self.gate_at = second[0].shape[0]
        else:
            self.parts.append(("a", mine(take("a", (heads, width)))))
            self.parts.append(("g", mine(take("g", (vo, width)))))
        bias = heads * self.dim if per_channel else heads
        self.a_log = param(mine(take("A_log", (heads,), "normal")), f32)
        self.dt_bias = param(mine(take("dt_bias", (bias,), "rate")), f32)
        self.norm = param(take("norm", (self.vdim,), "ones"), f32)
        self.w_out = param(mine(take("o", (width, vo)), 1), dtype)

    def cache_spec(self) -> LayerCacheSpec:
        state = {"delta": ((self.heads, self.dim, self.vdim), torch.float32)}
        if self.taps > 1:
            state["conv"] = ((self.taps, self.conv_w.shape[1]), self.dtype)
        return LayerCacheSpec(state=state)

    def forward(self, y: torch.Tensor, proj: FusedProjection,
                batch: ForwardBatch, cache: StateCache,
                layer: int) -> torch.Tensor:
        width = self.conv_w.shape[1]
        at = proj.offset("q")
        offs = [proj.offset(n) - at for n in ("q", "k", "v")]
        qkv, beta = y[:, at:at + width], proj.slice(y, "b")
        if self.per_channel:
            lo = proj.offset("a1")
            z = ops.linear(y[:, lo:lo + self.low.shape[1]], self.low)
            decay = z[:, :self.dt_bias.numel()]
            gate = z[:, self.gate_at:self.gate_at + self.heads * self.vdim]
        else:
            decay, gate = proj.slice(y, "a"), proj.slice(y, "g")
        p = ops.GatedDelta(self.a_log, self.dt_bias, self.norm, self.kv_heads,
                           not self.per_channel, self.dim ** -0.5,
                           self.unit_eps, self.eps)
        state = cache.state(layer, "delta")
        # one tap looks at nothing past: the ring is never read
        ring = (cache.state(layer, "conv") if self.taps > 1 else
                y.new_empty((cache.num_slots, 1, width)))
        out = y.new_empty((y.shape[0], self.heads * self.vdim))
        nd = y.shape[0] if batch.mode == "decode" else batch.num_decode
        if nd:
            ops.gated_delta(p, qkv[:nd], offs, beta[:nd], decay[:nd],
                            gate[:nd], state, batch.state_slots[:nd], None,
                            batch.starts[:nd], out[:nd],
                            conv=(self.conv_w, ring))
        if nd < y.shape[0]:
            slots, starts = batch.state_slots[nd:], batch.starts[nd:]
            layout, cu = batch.layout, batch.cu_prefill
            c = ops.short_conv(
                qkv[nd:], self.conv_w, ring,
                layout.prefill_tiles(max(ops.CONV_TILE, self.taps)), cu,
                starts, slots)
            ops.gated_delta(p, c, offs, beta[nd:], decay[nd:], gate[nd:],
                            state, slots, cu, starts, out[nd:],
                            chunks=(layout.prefill_tiles(ops.DELTA_CHUNK),
                                    layout.prefill_tile_cu(ops.DELTA_CHUNK)))
        return ops.linear(out, self.w_out)


class DifferentialAttention(nn.Module):
    """Attention of two maps over paged keys and values, without positions,
    through a sliding window; a head's output is the maps' weighed difference
    over its root mean square.  With ``kv_from`` the keys and values are
    another layer's."""

    def __init__(self, spec: Dict[str, Any], width: int, eps: float,
                 src: WeightSource, prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        heads, kv_heads = int(spec["heads"]), int(spec["kv_heads"])
        if heads % kv_heads:
            raise ValueError(f"{heads} heads over {kv_heads} key heads")
        assert heads % tp.size == 0 and kv_heads % tp.size == 0, \
            "TP degree must divide head counts"
        self.heads, self.kv_heads = heads // tp.size, kv_heads // tp.size
        self.dim, self.vdim = int(spec["dim"]), int(spec["vdim"])
        self.scale, self.eps = float(spec["scale"]), eps
        mask = spec.get("mask") or {}
        self.window = int(mask.get("size") or 0)     # 0: everything before
        self.kv_from: Optional[int] = spec.get("kv_from")   # global layer
        outs = {"q": heads * 2 * self.dim}
        if self.kv_from is None:
            outs.update(k=kv_heads * 2 * self.dim, v=kv_heads * self.vdim)
        self.parts: Parts = [
            (name, shard(src.take(prefix + name, (n, width)), tp))
            for name, n in outs.items()]
        self.diff = float(spec["diff"])
        lq1, lk1, lq2, lk2 = (src.take(prefix + n, (self.dim,)).float()
                              for n in ("lq1", "lk1", "lq2", "lk2"))
        lam = (lq1 * lk1).sum().exp() - (lq2 * lk2).sum().exp() + self.diff
        self.lam = param(lam.view(1), torch.float32)
        self.w_out = param(shard(src.take(prefix + "o",
                                          (width, heads * self.vdim)),
                                 tp, dim=1), dtype)

    def cache_spec(self) -> LayerCacheSpec:
        if self.kv_from is not None:
            return LayerCacheSpec()
        return LayerCacheSpec(kv=(self.kv_heads, 2 * self.dim, self.vdim))

    def forward(self, y: torch.Tensor, proj: FusedProjection,
                batch: ForwardBatch, cache: StateCache,
                kv_layer: int) -> torch.Tensor:
        k, v = cache.kv_pages(kv_layer)
        if self.kv_from is None:
            ops.rope_store_paged(
                y, None, None, batch.positions, batch.slot_mapping,
                self.heads, 2 * self.dim, k, v,
                [proj.offset(n) for n in ("q", "k", "v")])
        q = proj.slice(y, "q").unflatten(1, (self.heads, 2 * self.dim))
        out = y.new_empty((y.shape[0], self.heads * self.vdim))
        kw = dict(window=self.window, diff=ops.Difference(
            self.lam, 1.0 - self.diff, self.eps))
        nd = y.shape[0] if batch.mode == "decode" else batch.num_decode
        if nd:
            ops.paged_decode(q[:nd], k, v, batch.block_tables,
                             batch.context_lens, out[:nd], self.scale, 0.0,
                             False, **kw)
        if nd < y.shape[0]:
            ops.paged_prefill(q[nd:], k, v, batch.layout.paged_view(),
                              out[nd:], self.scale, 0.0, False, **kw)
        return ops.linear(out, self.w_out)


class GatedSilu(nn.Module):
    """down(silu(gate x) * up x), all with biases; the last one is left to the
    kernel that adds the branch (``bias``)."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        ff = int(spec["ff"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        f32 = torch.float32
        self.parts: Parts = [
            (n, shard(src.take(prefix + n, (ff, width)), tp))
            for n in ("gate", "up")]
        self.gate_b, self.up_b = (
            param(shard(src.take(prefix + n + ".b", (ff,), "zeros"), tp), f32)
            for n in ("gate", "up"))
        self.down = param(shard(src.take(prefix + "down", (width, ff)), tp,
                                dim=1), dtype)
        self.bias = param(src.take(prefix + "down.b", (width,), "zeros"), f32)

    def forward(self, h: torch.Tensor, y: torch.Tensor,
                proj: FusedProjection):
        act = y.new_empty((y.shape[0], self.down.shape[1]))
        ops.silu_glu(proj.slice(y, "gate"), proj.slice(y, "up"), self.gate_b,
                     self.up_b, act)
        return ops.linear(act, self.down), None


def glu_stack(prefixes: List[str], ff: int, width: int, src: WeightSource, tp,
              dtype: torch.dtype) -> Tuple[nn.Parameter, nn.Parameter]:
    """Gated feed-forwards of equal size as ops.expert_linear takes them: gate
    and up interleaved, and down."""
    def take(name, shape, dim):
        # columns up to a multiple of 8: a gate of zero meets zeros in down
        return pad8(shard(src.take(name, shape), tp, dim), dim)
    up = [ops.interleave_glu(take(p + "gate", (ff, width), 0),
                             take(p + "up", (ff, width), 0))
          for p in prefixes]
    down = [take(p + "down", (width, ff), 1) for p in prefixes]
    return param(torch.stack(up), dtype), param(torch.stack(down), dtype)


class GluExperts(nn.Module):
    """Mixture of small gated feed-forwards down(silu(gate x) * up x); the
    largest router logits are chosen and weighed by their softmax.

    Tensor parallelism shards every expert's inner columns."""

    bias = None
    parts: Parts = []

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        r, ff = spec["router"], int(spec["expert"]["ff"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        n, self.top = int(r["experts"]), int(r["top"])
        if not 1 <= self.top <= n:
            raise ValueError(f"router: {n} experts, {self.top} chosen")

        self.up, self.down = glu_stack(
            [f"{prefix}e{e}." for e in range(n)], ff, width, src, tp, dtype)
        self.router = param(src.take(prefix + "router", (n, width)), dtype)
        self.router_b = param(src.take(prefix + "router.b", (n,), "zeros"),
                              torch.float32)

    def forward(self, h: torch.Tensor, y: torch.Tensor,
                proj: FusedProjection):
        """Outputs of the chosen experts, one row per (token, choice) in
        expert order, and the routing that weighs and finds them."""
        logits = ops.router_logits(h, self.router)
        route = ops.moe_route(logits, self.router_b, 1, 1, self.top,
                              ops.expert_tile(h, self.up, self.top),
                              softmax=True)
        a = ops.expert_linear(h, self.up, route, gather=True, swiglu=True)
        return ops.expert_linear(a, self.down, route), route


class ClampedGlu(nn.Module):
    """down(g * sigmoid(1.702 g) * (u + 1)), g = min(gate x, limit) and u = up x
    within +-limit."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        ff, self.limit = int(spec["ff"]), float(spec["limit"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        self.proj = FusedProjection(
            [(n, pad8(shard(src.take(prefix + n, (ff, width)), tp)))
             for n in ("gate", "up")], dtype)
        self.down = param(pad8(shard(src.take(prefix + "down", (width, ff)),
                                     tp, dim=1), 1), dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        y = self.proj(x)
        act = y.new_empty((y.shape[0], self.down.shape[1]))
        ops.clamped_glu(self.proj.slice(y, "gate"), self.proj.slice(y, "up"),
                        self.limit, act)
        return ops.linear(act, self.down)


class ClampedExperts(nn.Module):
    """Mixture of clamped gated feed-forwards (ClampedGlu): scores are a softmax
    over all experts, the choice adds a correction to them, weights are the
    chosen ones' shares of their scores times a constant.  The last
    ``identity`` experts of the router have no weights and return their input;
    a ``shared`` expert runs for every token.

    Tensor parallelism shards every expert's inner columns."""

    def __init__(self, spec: Dict[str, Any], width: int, src: WeightSource,
                 prefix: str, tp, dtype: torch.dtype):
        super().__init__()
        r, ff = spec["router"], int(spec["expert"]["ff"])
        assert ff % tp.size == 0, "TP degree must divide the feed-forward"
        n, self.top = int(r["experts"]), int(r["top"])
        self.identity = int(r.get("identity") or 0)
        every = n + self.identity
        if n < 1 or not 1 <= self.top <= every:
            raise ValueError(f"router: {n} experts and {self.identity} "
                             f"identity experts, {self.top} chosen")
        self.share = float(r["scale"])
        self.limit = float(spec["expert"]["limit"])
        self.up, self.down = glu_stack(
            [f"{prefix}e{e}." for e in range(n)], ff, width, src, tp, dtype)
        self.router = param(src.take(prefix + "router", (every, width)), dtype)
        self.correction = param(src.take(prefix + "correction", (every,),
                                         "zeros"), torch.float32)
        self.shared: Optional[ClampedGlu] = None
        if spec.get("shared"):
            self.shared = ClampedGlu(spec["shared"], width, src,
                                     prefix + "shared.", tp, dtype)
        # pairs that get a row, per choice
        self.rows_per_choice = n / every

    def forward(self, h: torch.Tensor):
        """The shared expert's rows (or None), the chosen experts' outputs, one
        row per (token, choice) in expert order, and the routing that weighs
        and finds them."""
        logits = ops.router_logits(h, self.router)
        route = ops.moe_route(
            logits, self.correction, 1, 1, self.top,
            ops.expert_tile(h, self.up, self.top * self.rows_per_choice),
            share=self.share, identity=self.identity)
        a = ops.expert_linear(h, self.up, route, gather=True, swiglu=True,
                              limit=self.limit)
        y = ops.expert_linear(a, self.down, route)
        return None if self.shared is None else self.shared(h), y, route
