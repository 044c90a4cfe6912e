"""Danipel's side of engine/model_bench.py: sizes, and its kernels beside the like
kernels of the other families.

The closest family with dense feed-forwards is Bitatar (latent attention on an f32
stream), with experts Gogalix; equal size means their width, layers, heads and
feed-forward columns per token.
"""
from __future__ import annotations

from typing import Any, Dict, List

import torch

from ..models.danipel import DanipelConfig
from .config import ModelConfig
from .gogalix_bench import EXPERTS, TOP, gogalix_set
from .model_bench import SIZES, VOCAB, _row, _time, pair

DIM, ROT, VDIM, STREAMS, IDENTITY = 128, 64, 128, 4, 8


def q_rank(size: str) -> int:
    return 3 * SIZES[size][0] // 8


def danipel_set(size: str) -> List[ModelConfig]:
    w, ff, heads, _, layers, rank, _, _, _ = SIZES[size]

    def make(name: str, pattern: str) -> DanipelConfig:
        return DanipelConfig.stacked(
            name, width=w, vocab=VOCAB, pattern=(pattern * layers)[:layers],
            heads=heads, dim=DIM, rot_dim=ROT, vdim=VDIM, kv_rank=rank,
            q_rank=q_rank(size), ff=ff, streams=STREAMS, experts=EXPERTS,
            identity=IDENTITY, top=TOP, expert_ff=ff // TOP,
            shared_ff=ff // TOP)
    return [make(f"danipel-{size}", "ab"), pair(size)[0],
            make(f"danipel-{size}-experts", "AB"), gogalix_set(size)[1]]


def danipel_kernels(size: str, batches=(1, 8, 32, 128), ctx: int = 2048,
                    prompts: int = 4) -> List[Dict[str, Any]]:
    """Rooflines: bytes that must move, or the operations the algorithm has to
    do (causal halves counted once)."""
    from .. import ops
    from ..models.rotary import rotary_table
    from .batch import VarlenLayout
    w, ff, heads, kvh, _, rank, _, _, _ = SIZES[size]
    H, S, eff, qr, ps = heads, STREAMS, ff // TOP, q_rank(size), 16
    dev, bf, f32 = torch.device("cuda"), torch.bfloat16, torch.float32
    out: List[Dict[str, Any]] = []
    gen = torch.Generator(device=dev).manual_seed(3)

    def rnd(*shape, dtype=bf):
        return torch.randn(*shape, device=dev, dtype=f32,
                           generator=gen).to(dtype)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)

    def copies(nbytes: int) -> int:
        return max(1, min(12, int(600e6 // max(nbytes, 1)) + 1))

    def add(name: str, fn, nbytes: float = 0.0, bf16: float = 0.0) -> None:
        out.append(_row(name, _time(fn), nbytes, bf16=bf16))
    ones, one = torch.ones(w, device=dev), torch.ones(1, device=dev)
    norm = ops.TanhNorm(one, ones, rnd(w, dtype=f32))
    read, conn = rnd(S, dtype=f32), rnd(S * S + S, dtype=f32)
    cn, qnorm = torch.ones(rank, device=dev), torch.ones(qr, device=dev)
    sink = rnd(H, dtype=f32)
    table = rotary_table({"dims": ROT, "base": 5e5}, ctx + 64, dev)
    every = EXPERTS + IDENTITY
    ups = [rnd(EXPERTS, 2 * eff, w) for _ in range(2)]
    downs = [rnd(EXPERTS, w, eff) for _ in range(2)]
    router, corr = rnd(every, w) / w ** 0.5, torch.zeros(every, device=dev)
    emb = rnd(VOCAB, w)

    def both(T: int, tag: str) -> None:
        """Kernels that see rows of tokens, whatever the step is."""
        x, x1, y, z = rnd(T, S * w, dtype=f32), rnd(T, w, dtype=f32), \
            rnd(T, w), rnd(T, w)
        stir = ops.Stir(conn, 0.5, y)
        add(f"hyper_norm {tag}", lambda i: ops.hyper_norm(
            x, S, stir, read, norm, bf), T * w * (S * 8 + 4))
        add(f"bitatar stream_norm {tag}", lambda i: ops.stream_norm(
            x1, y, ones, None, 8, 1e-5, bf), T * w * 12)
        h = ops.hyper_norm(x, S, None, read, norm, bf)
        logits = ops.router_logits(h, router)
        few = logits[:, :EXPERTS].contiguous()
        per = TOP * EXPERTS / every
        tile = ops.expert_tile(h, ups[0], per)

        def share():
            return ops.moe_route(logits, corr, 1, 1, TOP, tile, share=2.0,
                                 identity=IDENTITY)
        add(f"moe_route shares {tag}", lambda i: share(),
            T * (every * 4 + TOP * 16))
        add(f"gogalix moe_route {tag}", lambda i: ops.moe_route(
            few, corr[:EXPERTS], 1, 1, TOP, tile, softmax=True),
            T * (EXPERTS * 4 + TOP * 16))
        route = share()
        tiles = route.tiles[:int(route.count)]
        used = len(set(tiles[:, 0].tolist()))
        P = int(tiles[:, 2].sum())
        nbytes = used * 2 * eff * w * 2 + T * w * 2 + P * eff * 2
        add(f"expert gate/up clamped {tag}", lambda i: ops.expert_linear(
            h, ups[i % 2], route, gather=True, swiglu=True, limit=7.0),
            nbytes, 4 * P * eff * w)
        add(f"gogalix expert gate/up {tag}", lambda i: ops.expert_linear(
            h, ups[i % 2], route, gather=True, swiglu=True), nbytes,
            4 * P * eff * w)
        a = ops.expert_linear(h, ups[0], route, gather=True, swiglu=True,
                              limit=7.0)
        add(f"expert down {tag}", lambda i: ops.expert_linear(
            a, downs[i % 2], route), used * eff * w * 2 + P * (w + eff) * 2,
            2 * P * eff * w)
        e = ops.expert_linear(a, downs[0], route)
        mixed = ops.Stir(conn, 0.5, z, e, route, h)
        add(f"hyper_norm of experts {tag}", lambda i: ops.hyper_norm(
            x, S, mixed, read, norm, bf),
            T * w * (S * 8 + 6) + P * w * 2)
        # as many rows of experts as above
        plain = ops.moe_route(few, corr[:EXPERTS], 1, 1, TOP, tile,
                              softmax=True)
        wide = rnd(T, 2 * w)
        left = [ops.Branch(y, wide[:, :w], ones, ones),
                ops.Branch(e, wide[:, w:], ones, ones, None, plain)]
        add(f"gogalix gate_norm of experts {tag}", lambda i: ops.gate_norm(
            x1, left, one, 1e-6, bf), T * w * (16 + 2 * TOP))
        gu, act = rnd(T, 2 * ff), rnd(T, ff)
        add(f"clamped_glu {tag}", lambda i: ops.clamped_glu(
            gu[:, :ff], gu[:, ff:], 7.0, act), T * ff * 6)
        add(f"bitatar gelu_mul {tag}", lambda i: ops.gelu_mul(gu, act),
            T * ff * 6)
        pos = i32([i % ctx for i in range(T)])
        rot, rot2 = (ops.Rotary(table, pos, il) for il in (True, False))
        slots = torch.arange(ps, T + ps, device=dev, dtype=torch.int32)
        low, lq = rnd(T, rank + ROT), rnd(T, qr)
        cache = rnd(T // ps + 2, ps, rank + ROT)
        add(f"latent_store {tag}", lambda i: ops.latent_store(
            low, cn, cache, slots, 1e-6, rot), T * (rank + ROT) * 6)
        add(f"latent_store and query latent {tag}",
            lambda i: ops.latent_store(low, cn, cache, slots, 1e-6, rot2,
                                       second=(lq, qnorm)),
            T * ((rank + ROT) * 6 + qr * 4))
        bl, bc = rnd(T, rank), rnd(T // ps + 2, ps, rank)
        add(f"bitatar latent_store {tag}", lambda i: ops.latent_store(
            bl, cn, bc, slots, 1e-6), T * rank * 6)
        tok = torch.arange(T, device=dev) % 997
        add(f"embed_stream x{S} {tag}", lambda i: ops.embed_stream(
            tok, emb, 1.0, S), T * w * (2 + 4 * S))
        add(f"bitatar embed_stream {tag}", lambda i: ops.embed_stream(
            tok, emb, 1.0), T * w * 6)

    for b in batches:
        tag = f"B={b}"
        pages = b * ctx // ps + 1
        bt = (torch.arange(b * (ctx // ps), device=dev, dtype=torch.int32)
              .view(b, -1) + 1)
        cl = i32([ctx] * b)
        for name, d, kw in (("latent_decode", rank + ROT,
                             {"rank": rank, "sink": sink}),
                            ("bitatar latent_decode", rank, {})):
            n = copies(pages * ps * d * 2)
            lat = [rnd(pages, ps, d) for _ in range(n)]
            q = rnd(b, H, d)
            add(f"{name} {tag}", lambda i: ops.latent_decode(
                q, lat[i % n], bt, cl, 0.05, 0, **kw),
                b * ctx * d * 2 + b * H * (d + rank) * 2,
                b * H * ctx * (d + rank) * 2)
            del lat
        q, uk = rnd(b, H, DIM + ROT), rnd(H, rank, DIM)
        qb = q[..., :DIM].contiguous()
        rot = ops.Rotary(table, i32([7] * b), True)
        nbytes = uk.numel() * 2 + b * H * (DIM + rank) * 2
        add(f"head_linear and rotation {tag}", lambda i: ops.head_linear(
            q[..., :DIM], uk, tail=q[..., DIM:], rot=rot),
            nbytes + b * H * ROT * 4)
        add(f"bitatar head_linear {tag}", lambda i: ops.head_linear(qb, uk),
            nbytes)
        both(b, tag)
    T, tag = prompts * ctx, f"{prompts}x{ctx}"
    per = ctx // ps

    class Table:
        def __init__(self, i):
            self.pages = list(range(1 + i * per, 1 + (i + 1) * per))
    view = VarlenLayout([0] * prompts, [ctx] * prompts,
                        [Table(i) for i in range(prompts)], 0, ps,
                        dev).window_view(0)
    pairs = prompts * ctx * (ctx + 1) // 2
    q, o = rnd(T, H, DIM + ROT), rnd(T, H * VDIM)
    kv, shared = rnd(T, H * (DIM + VDIM)), rnd(T, rank + ROT)[:, rank:]
    k, v = (kv[:, i * H * DIM:(i + 1) * H * DIM].unflatten(1, (H, DIM))
            for i in range(2))
    add(f"attention with shared key part {tag}",
        lambda i: ops.window_attention(q, k, v, None, o, view, 0.05, 0, shared,
                                       sink),
        T * H * (DIM + ROT + DIM + 2 * VDIM) * 2 + T * ROT * 2,
        pairs * H * 2 * (DIM + ROT + VDIM))
    qb = q[..., :DIM].contiguous()
    add(f"bitatar window_attention {tag}", lambda i: ops.window_attention(
        qb, k, v, None, o, view, 0.05, 0), T * H * (2 * DIM + 2 * VDIM) * 2,
        pairs * H * 2 * (DIM + VDIM))
    pos = i32([i % ctx for i in range(T)])
    for il, name in ((True, "interleaved"), (False, "halves")):
        rot = ops.Rotary(table, pos, il)
        add(f"rotate_rows {name} {tag}", lambda i: ops.rotate_rows(
            q[..., DIM:], rot), T * H * ROT * 4)
    qn, kn = H * DIM, kvh * DIM
    kp, vp = rnd(T // ps + 2, kvh, ps, DIM), rnd(T // ps + 2, kvh, ps, DIM)
    slots = torch.arange(ps, T + ps, device=dev, dtype=torch.int32)
    qkv, bias = rnd(T, qn + 2 * kn), torch.zeros(qn + 2 * kn, device=dev)
    add(f"notadra rope_store_paged {tag}", lambda i: ops.rope_store_paged(
        qkv, bias, table, pos, slots, H, DIM, kp, vp, [0, qn, qn + kn]),
        T * (qn + 2 * kn) * 4)
    both(T, tag)
    return out
