"""Gogalix's side of engine/model_bench.py: sizes, and its kernels beside the
like kernels of the other families.

The closest family is Bitatar (a delta rule and windowed attention beside a
dense feed-forward, on an f32 stream); equal size means its width, layers, mixer
and feed-forward widths.  A differential head is two maps of 128 over values of
256, so there are half as many.  The form with experts chooses as many
feed-forward columns per token.
"""
from __future__ import annotations

from typing import Any, Dict, List

import torch

from ..models.gogalix import GogalixConfig
from .config import ModelConfig
from .model_bench import SIZES, VOCAB, _row, _time, pair

DIM, VDIM, TAPS, LOW_RANK = 128, 256, 4, 128
EXPERTS, TOP = 64, 8


def gogalix_set(size: str) -> List[ModelConfig]:
    w, ff, heads, kvh, layers, _, window, dh, dd = SIZES[size]

    def make(name: str, pattern: str) -> GogalixConfig:
        return GogalixConfig.stacked(
            name, width=w, vocab=VOCAB, pattern=(pattern * layers)[:layers],
            heads=heads // 2, kv_heads=kvh // 2, dim=DIM, vdim=VDIM,
            window=window, ff=ff, delta_heads=dh, delta_kv_heads=dh // 2,
            delta_dim=dd, delta_vdim=dd, taps=TAPS, experts=EXPERTS, top=TOP,
            expert_ff=ff // TOP, low_rank=LOW_RANK)
    return [make(f"gogalix-{size}", "casdas"),
            make(f"gogalix-{size}-experts", "CASDAS"), pair(size)[0]]


def gogalix_kernels(size: str, batches=(1, 8, 32, 128), ctx: int = 2048,
                    prompts: int = 4) -> List[Dict[str, Any]]:
    """Rooflines: bytes that must move, or the operations the algorithm has to
    do (causal halves and windows counted, the recurrence at the f32 rate)."""
    import math

    from .. import ops
    from ..models.rotary import rotary_table
    from .batch import VarlenLayout
    w, ff, heads, kvh, _, _, window, dh, dd = SIZES[size]
    H, G, dkv, eff = heads // 2, kvh // 2, dh // 2, ff // TOP
    dev, bf = torch.device("cuda"), torch.bfloat16
    out: List[Dict[str, Any]] = []
    ps = 16
    gen = torch.Generator(device=dev).manual_seed(3)

    def rnd(*shape, dtype=bf):
        return torch.randn(*shape, device=dev, dtype=torch.float32,
                           generator=gen).to(dtype)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)

    def copies(nbytes: int) -> int:
        return max(1, min(12, int(600e6 // max(nbytes, 1)) + 1))
    f32 = torch.float32
    hd, qk = dh * dd, dkv * dd
    ones, one = torch.ones(w, device=dev), torch.ones(1, device=dev)
    bias = rnd(w, dtype=f32)
    lam = ops.Difference(torch.tensor([0.4], device=dev), 0.6, 1e-6)
    conv_w = rnd(TAPS, 2 * qk + hd, dtype=f32) * 0.3
    offs = [0, qk, 2 * qk]
    rules = {
        kind: ops.GatedDelta(
            rnd(dh, dtype=f32) * 0.5, rnd(n, dtype=f32) - 3.0,
            torch.ones(dd, device=dev), dkv, kind == "head", dd ** -0.5, 1e-6,
            1e-6)
        for kind, n in (("channel", hd), ("head", dh))}
    # Bitatar's rule
    boffs = [hd * i for i in range(6)]
    bargs = (rnd(hd, 64), rnd(hd, dtype=f32), rnd(hd, dtype=f32),
             torch.ones(hd, device=dev))
    ups = [rnd(EXPERTS, 2 * eff, w) for _ in range(2)]
    downs = [rnd(EXPERTS, w, eff) for _ in range(2)]
    router, rb = rnd(EXPERTS, w) / w ** 0.5, torch.zeros(EXPERTS, device=dev)
    table = rotary_table({"dims": DIM // 2, "base": 5e5}, ctx + 64, dev)

    def both(T: int, tag: str) -> None:
        """Kernels that see rows of tokens, whatever the step is."""
        x, y, f, z = rnd(T, w, dtype=f32), rnd(T, w), rnd(T, w), rnd(T, 2 * w)
        left = [ops.Branch(y, z[:, :w], bias, ones),
                ops.Branch(f, z[:, w:], bias, ones, bias)]
        us = _time(lambda i: ops.gate_norm(x, left, one, 1e-6, bf))
        out.append(_row(f"gate_norm {tag}", us, T * w * 18))
        us = _time(lambda i: ops.sandwich_norm(x, (y, None, ones), ones, 1e-6,
                                               bf))
        out.append(_row(f"notadra sandwich_norm {tag}", us, T * w * 12))
        h = ops.gate_norm(x, [], one, 1e-6, bf)
        logits = ops.router_logits(h, router)
        tile = ops.expert_tile(h, ups[0], TOP)
        us = _time(lambda i: ops.moe_route(logits, rb, 1, 1, TOP, tile,
                                           softmax=True))
        out.append(_row(f"moe_route softmax {tag}", us,
                        T * (EXPERTS * 4 + TOP * 16)))
        us = _time(lambda i: ops.moe_route(logits, rb, 8, 4, TOP, tile))
        out.append(_row(f"notadra moe_route {tag}", us,
                        T * (EXPERTS * 4 + TOP * 16)))
        route = ops.moe_route(logits, rb, 1, 1, TOP, tile, softmax=True)
        used = len(set(route.tiles[:int(route.count), 0].tolist()))
        P = T * TOP
        us = _time(lambda i: ops.expert_linear(h, ups[i % 2], route,
                                               gather=True, swiglu=True))
        out.append(_row(f"expert gate/up {tag}", us,
                        used * 2 * eff * w * 2 + T * w * 2 + P * eff * 2,
                        bf16=4 * P * eff * w))
        us = _time(lambda i: ops.expert_linear(h, ups[i % 2], route,
                                               gather=True, relu2=True))
        out.append(_row(f"notadra expert up {tag}", us,
                        used * 2 * eff * w * 2 + T * w * 2 + P * eff * 4,
                        bf16=4 * P * eff * w))
        a = ops.expert_linear(h, ups[0], route, gather=True, swiglu=True)
        us = _time(lambda i: ops.expert_linear(a, downs[i % 2], route))
        out.append(_row(f"expert down {tag}", us,
                        used * eff * w * 2 + P * (w + eff) * 2,
                        bf16=2 * P * eff * w))
        e = ops.expert_linear(a, downs[0], route)
        mixed = [left[0], ops.Branch(e, z[:, w:], bias, ones, None, route)]
        us = _time(lambda i: ops.gate_norm(x, mixed, one, 1e-6, bf))
        out.append(_row(f"gate_norm of experts {tag}", us,
                        T * w * (16 + 2 * TOP)))
        us = _time(lambda i: ops.sandwich_norm(x, (e, route, ones), ones, 1e-6,
                                               bf))
        out.append(_row(f"notadra sandwich_norm of experts {tag}", us,
                        T * w * (10 + 2 * TOP)))
        gu, act = rnd(T, 2 * ff), rnd(T, ff)
        fb = rnd(ff, dtype=f32)
        us = _time(lambda i: ops.silu_glu(gu[:, :ff], gu[:, ff:], fb, fb, act))
        out.append(_row(f"silu_glu {tag}", us, T * ff * 6))
        us = _time(lambda i: ops.gelu_mul(gu, act))
        out.append(_row(f"bitatar gelu_mul {tag}", us, T * ff * 6))
        pages = T // ps + 2
        qn, kn, vn = H * 2 * DIM, G * 2 * DIM, G * VDIM
        kp, vp = rnd(pages, G, ps, 2 * DIM), rnd(pages, G, ps, VDIM)
        pos = i32([i % ctx for i in range(T)])
        slots = torch.arange(ps, T + ps, device=dev, dtype=torch.int32)
        qkv = rnd(T, qn + kn + vn)
        us = _time(lambda i: ops.rope_store_paged(
            qkv, None, None, pos, slots, H, 2 * DIM, kp, vp,
            [0, qn, qn + kn]))
        out.append(_row(f"paged store {tag}", us, T * (kn + vn) * 4))
        nb = torch.zeros(qkv.shape[1], device=dev)
        us = _time(lambda i: ops.rope_store_paged(
            qkv, nb, table, pos, slots, H, 2 * DIM, kp, vp,
            [0, qn, qn + kn]))
        out.append(_row(f"notadra rope_store_paged {tag}", us,
                        T * (qn + kn + vn) * 4))

    for b in batches:
        tag = f"B={b}"
        pages = b * ctx // ps + 1
        bt = (torch.arange(b * (ctx // ps), device=dev, dtype=torch.int32)
              .view(b, -1) + 1)
        cl = i32([ctx] * b)
        keys = min(window, ctx)
        row = G * (2 * DIM + VDIM) * 2
        n = copies(pages * ps * row)
        kv = [(rnd(pages, G, ps, 2 * DIM), rnd(pages, G, ps, VDIM))
              for _ in range(n)]
        q, o = rnd(b, H, 2 * DIM), rnd(b, H * VDIM)
        us = _time(lambda i: ops.paged_decode(
            q, *kv[i % n], bt, cl, o, 0.09, 0.0, False, window=window,
            diff=lam))
        out.append(_row(f"difference decode {tag}", us,
                        b * keys * row + b * H * (2 * DIM + VDIM) * 2))
        del kv
        kn = kvh * DIM
        n = copies(pages * ps * kn * 4)
        kv = [(rnd(pages, kvh, ps, DIM), rnd(pages, kvh, ps, DIM))
              for _ in range(n)]
        q, o = rnd(b, heads, DIM), rnd(b, heads * DIM)
        us = _time(lambda i: ops.paged_decode(q, *kv[i % n], bt, cl, o, 0.05,
                                              30.0, True))
        out.append(_row(f"notadra paged_decode {tag}", us,
                        b * ctx * kn * 4 + 2 * b * heads * DIM * 2))
        del kv
        slots = i32(range(1, b + 1))
        sbytes = b * dh * dd * dd * 8
        n = copies(sbytes)
        st = [torch.randn(b + 1, dh, dd, dd, device=dev) for _ in range(n)]
        qkv = rnd(b, 2 * qk + hd)
        ring = rnd(b + 1, TAPS, 2 * qk + hd)
        beta, gate, o = rnd(b, dh), rnd(b, hd), rnd(b, hd)
        for kind, rule in rules.items():
            z = rnd(b, rule.dt_bias.numel())
            us = _time(lambda i: ops.gated_delta(
                rule, qkv, offs, beta, z, gate, st[i % n], slots, None, cl, o,
                conv=(conv_w, ring)))
            out.append(_row(f"gated_step {kind} {tag}", us, sbytes +
                            b * (2 * qk + hd) * 2 * (TAPS + 1) +
                            b * (2 * hd + z.shape[1]) * 2))
        proj = rnd(b, hd * 5 + 64)
        us = _time(lambda i: ops.delta_rule(
            proj, None, *bargs, st[i % n], slots, None, cl, o, boffs,
            math.exp(-0.5), 1e-6, 1e-5))
        out.append(_row(f"bitatar delta_step {tag}", us, sbytes +
                        bargs[0].numel() * 2 + b * hd * 12))
        del st
        both(b, tag)
    T, tag = prompts * ctx, f"{prompts}x{ctx}"
    per = ctx // ps

    class Table:
        def __init__(self, i):
            self.pages = list(range(1 + i * per, 1 + (i + 1) * per))
    lay = VarlenLayout([0] * prompts, [ctx] * prompts,
                       [Table(i) for i in range(prompts)], 0, ps, dev)
    view = lay.paged_view()
    pairs = prompts * sum(min(i + 1, window) for i in range(ctx))
    q, o = rnd(T, H, 2 * DIM), rnd(T, H * VDIM)
    kp, vp = rnd(T // ps + 1, G, ps, 2 * DIM), rnd(T // ps + 1, G, ps, VDIM)
    us = _time(lambda i: ops.paged_prefill(q, kp, vp, view, o, 0.09, 0.0,
                                           False, window=window, diff=lam))
    out.append(_row(f"difference prefill {tag}", us,
                    T * (H + G) * (2 * DIM + VDIM) * 2,
                    bf16=pairs * H * 4 * (DIM + VDIM)))
    q, o = rnd(T, heads, DIM), rnd(T, heads * DIM)
    kp, vp = rnd(T // ps + 1, kvh, ps, DIM), rnd(T // ps + 1, kvh, ps, DIM)
    for name, cap in (("notadra paged_prefill", 30.0),
                      ("paged_prefill without cap", 0.0)):
        us = _time(lambda i: ops.paged_prefill(q, kp, vp, view, o, 0.05, cap,
                                               True))
        out.append(_row(f"{name} {tag}", us,
                        T * (2 * heads + 2 * kvh) * DIM * 2,
                        bf16=prompts * ctx * (ctx + 1) // 2 * heads * 4 * DIM))
    g = rnd(T, heads * DIM)
    k, v = rnd(T, heads, DIM), rnd(T, heads, DIM)
    us = _time(lambda i: ops.window_attention(q, k, v, g, o,
                                              lay.window_view(window), 0.05,
                                              window))
    out.append(_row(f"bitatar window_attention {tag}", us,
                    T * heads * DIM * 10, bf16=pairs * heads * 4 * DIM))
    del k, v
    cu = i32([i * ctx for i in range(prompts + 1)])
    slots, starts = i32(range(1, prompts + 1)), i32([0] * prompts)
    wide = rnd(T, 2 * qk + hd + w)
    ring = rnd(prompts + 1, TAPS, 2 * qk + hd)
    tiles = lay.prefill_tiles(ops.CONV_TILE)
    x = wide[:, :2 * qk + hd]
    us = _time(lambda i: ops.short_conv(x, conv_w, ring, tiles, cu, starts,
                                        slots))
    out.append(_row(f"short_conv {tag}", us, T * (2 * qk + hd) * 4))
    d, hist = rnd(T, w), rnd(prompts + 1, 3, w)
    cw = rnd(4, w, dtype=f32)
    us = _time(lambda i: ops.causal_conv(d, cw, hist, tiles, cu, starts,
                                         slots))
    out.append(_row(f"bitatar causal_conv {tag}", us, T * w * 4))
    qkv = ops.short_conv(x, conv_w, ring, tiles, cu, starts, slots)
    beta, gate, o = rnd(T, dh), rnd(T, hd), rnd(T, hd)
    st = torch.zeros(prompts + 1, dh, dd, dd, device=dev)
    chunks = (lay.prefill_tiles(ops.DELTA_CHUNK),
              lay.prefill_tile_cu(ops.DELTA_CHUNK))
    for kind, rule in rules.items():
        z = rnd(T, rule.dt_bias.numel())
        us = _time(lambda i: ops.gated_delta(
            rule, qkv, offs, beta, z, gate, st, slots, cu, starts, o,
            chunks=chunks), 4)
        out.append(_row(f"gated_chunk {kind} (3 kernels) {tag}", us,
                        T * (2 * qk + 3 * hd + z.shape[1]) * 2,
                        f32=T * dh * 7 * dd * dd))
    proj, z = rnd(T, hd * 5 + 64), rnd(T, hd)
    us = _time(lambda i: ops.delta_rule(
        proj, z, *bargs, st, slots, cu, starts, o, boffs, math.exp(-0.5),
        1e-6, 1e-5, chunks), 4)
    out.append(_row(f"bitatar delta_chunk (3 kernels) {tag}", us, T * hd * 14,
                    f32=T * dh * 8 * dd * dd))
    del proj, wide, qkv
    both(T, tag)
    return out
