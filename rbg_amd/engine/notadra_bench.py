"""Notadra's side of engine/model_bench.py: sizes, and its kernels beside the
like kernels of Llama.

Equal size means equal attention shapes and as many feed-forward weights per
token: the chosen experts' two matrices against Llama's three.
"""
from __future__ import annotations

from typing import Any, Dict, List

import torch

from ..models.notadra import NotadraConfig
from .config import ModelConfig
from .model_bench import VOCAB, _row, _time

# name -> (width, heads, kv heads, layers, experts, chosen, expert ff, Llama ff)
NOTADRA_SIZES = {
    "2k": (2048, 16, 4, 6, 64, 6, 1408, 5632),
    "4k": (4096, 32, 8, 6, 64, 8, 2688, 14336),
}
DIM, GROUPS, KEEP = 128, 8, 4


def notadra_pair(size: str) -> List[ModelConfig]:
    w, heads, kvh, layers, n, top, ff, llama_ff = NOTADRA_SIZES[size]
    return [
        NotadraConfig.stacked(
            f"notadra-{size}", width=w, vocab=VOCAB, layers=layers,
            heads=heads, kv_heads=kvh, dim=DIM, vdim=DIM, rot_dims=DIM // 2,
            ff=ff, experts=n, top=top, groups=GROUPS, keep=KEEP),
        ModelConfig(name=f"llama-{size}", hidden_size=w,
                    intermediate_size=llama_ff, num_layers=layers,
                    num_heads=heads, num_kv_heads=kvh, vocab_size=VOCAB)]


def notadra_kernels(size: str, batches=(1, 8, 32, 128), ctx: int = 2048,
                    prompts: int = 4) -> List[Dict[str, Any]]:
    """Rooflines: bytes that must move (the weights of experts that are chosen
    at all, once), or the operations the algorithm has to do."""
    from .. import ops
    from ..models.rotary import rotary_table
    from .batch import VarlenLayout
    w, heads, kvh, _, E, top, ff, lff = NOTADRA_SIZES[size]
    dev, bf = torch.device("cuda"), torch.bfloat16
    out: List[Dict[str, Any]] = []
    ps, qn, kn = 16, heads * DIM, kvh * DIM
    gen = torch.Generator(device=dev).manual_seed(3)

    def rnd(*shape, dtype=bf):
        return torch.randn(*shape, device=dev, dtype=torch.float32,
                           generator=gen).to(dtype)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)

    def copies(nbytes: int) -> int:
        return max(1, min(12, int(600e6 // max(nbytes, 1)) + 1))
    ones = torch.ones(w, device=dev)
    wn = rnd(w)
    table = rotary_table({"dims": DIM // 2, "base": 5e5}, ctx + 64, dev)
    lt = ops.build_cos_sin_table(DIM, ctx + 64, device=dev)
    bias = torch.zeros(qn + 2 * kn, device=dev)
    # several sets of expert and dense weights, so that caches do not hold them
    ups = [rnd(E, ff, w) for _ in range(2)]
    downs = [rnd(E, w, ff) for _ in range(2)]
    router, corr = rnd(E, w) / w ** 0.5, torch.zeros(E, device=dev)
    gus = [rnd(2 * lff, w) for _ in range(4)]
    lds = [rnd(w, lff) for _ in range(4)]

    def both(T: int, tag: str) -> None:
        """Kernels that see rows of tokens, whatever the step is."""
        x, y = rnd(T, w, dtype=torch.float32), rnd(T, w)
        us = _time(lambda i: ops.sandwich_norm(x, (y, None, ones), ones, 1e-6,
                                               bf))
        out.append(_row(f"sandwich_norm {tag}", us, T * w * 12))
        r = rnd(T, w)
        us = _time(lambda i: ops.fused_add_rmsnorm(y, r, wn, 1e-5))
        out.append(_row(f"llama fused_add_rmsnorm {tag}", us, T * w * 8))
        h = ops.sandwich_norm(x, None, ones, 1e-6, bf)
        logits = ops.router_logits(h, router)
        us = _time(lambda i: ops.router_logits(h, router))
        out.append(_row(f"router_logits {tag}", us,
                        T * (w * 2 + E * 4) + E * w * 2,
                        bf16=2 * T * w * E))
        us = _time(lambda i: ops.linear(h, router))
        out.append(_row(f"llama linear of that shape {tag}", us,
                        T * (w * 2 + E * 2) + E * w * 2, bf16=2 * T * w * E))
        tile = ops.expert_tile(h, ups[0], top)
        route = ops.moe_route(logits, corr, GROUPS, KEEP, top, tile)
        us = _time(lambda i: ops.moe_route(logits, corr, GROUPS, KEEP, top,
                                           tile))
        out.append(_row(f"moe_route {tag}", us, T * (E * 4 + top * 16)))
        used = len(set(route.tiles[:int(route.count), 0].tolist()))
        P = T * top
        us = _time(lambda i: ops.expert_linear(h, ups[i % 2], route,
                                               gather=True, relu2=True))
        out.append(_row(f"expert up {tag}", us,
                        used * ff * w * 2 + T * w * 2 + P * ff * 2,
                        bf16=2 * P * ff * w))
        us = _time(lambda i: ops.linear(h, gus[i % 4]))
        out.append(_row(f"llama gate/up {tag}", us,
                        lff * w * 4 + T * w * 2 + T * lff * 4,
                        bf16=4 * T * lff * w))
        a = ops.expert_linear(h, ups[0], route, gather=True, relu2=True)
        us = _time(lambda i: ops.expert_linear(a, downs[i % 2], route))
        out.append(_row(f"expert down {tag}", us,
                        used * ff * w * 2 + P * (w + ff) * 2,
                        bf16=2 * P * ff * w))
        g = rnd(T, lff)
        us = _time(lambda i: ops.linear(g, lds[i % 4]))
        out.append(_row(f"llama down {tag}", us,
                        lff * w * 2 + T * (w + lff) * 2,
                        bf16=2 * T * lff * w))
        y = ops.expert_linear(a, downs[0], route)
        us = _time(lambda i: ops.sandwich_norm(x, (y, route, ones), ones, 1e-6,
                                               bf))
        out.append(_row(f"sandwich_norm of experts {tag}", us,
                        T * w * (10 + 2 * top)))
        pages = T // ps + 2
        kp, vp = rnd(pages, kvh, ps, DIM), rnd(pages, kvh, ps, DIM)
        pos = i32([i % ctx for i in range(T)])
        slots = torch.arange(ps, T + ps, device=dev, dtype=torch.int32)
        qkv = rnd(T, qn + 2 * kn)
        us = _time(lambda i: ops.rope_store_paged(
            qkv, bias, table, pos, slots, heads, DIM, kp, vp,
            [0, qn, qn + kn]))
        out.append(_row(f"rope_store_paged {tag}", us, T * (qn + 2 * kn) * 4))
        us = _time(lambda i: ops.rope_store_kv(
            qkv[:, :qn], qkv[:, qn:qn + kn], qkv[:, qn + kn:], kp, vp, lt, pos,
            slots))
        # its keys and queries rotate in place and the keys are stored too
        out.append(_row(f"llama rope_store_kv {tag}", us,
                        T * (qn + 2 * kn) * 4 + T * kn * 2))
        tok = torch.arange(T, device=dev) % 997
        emb, pairs = rnd(VOCAB, w), rnd(VOCAB + 1, w)
        us = _time(lambda i: ops.embed_pairs(tok, tok, emb, pairs, 31, 7))
        out.append(_row(f"embed_pairs {tag}", us, T * w * 8))
        us = _time(lambda i: emb[tok])
        out.append(_row(f"llama embedding {tag}", us, T * w * 4))

    for b in batches:
        tag = f"B={b}"
        pages = b * ctx // ps + 1
        bt = (torch.arange(b * (ctx // ps), device=dev, dtype=torch.int32)
              .view(b, -1) + 1)
        cl = i32([ctx] * b)
        n = copies(pages * ps * kn * 4)
        kv = [(rnd(pages, kvh, ps, DIM), rnd(pages, kvh, ps, DIM))
              for _ in range(n)]
        q, o = rnd(b, heads, DIM), rnd(b, qn)
        nbytes = b * ctx * kn * 4 + 2 * b * qn * 2
        us = _time(lambda i: ops.paged_decode(q, *kv[i % n], bt, cl, o, 0.05,
                                              30.0, True))
        out.append(_row(f"paged_decode {tag}", us, nbytes))
        sp = ops.pick_decode_splits(b, kvh, ctx + 128)
        us = _time(lambda i: ops.decode_attention(q, *kv[i % n], bt, cl, 0.05,
                                                  num_splits=sp))
        out.append(_row(f"llama decode_attention {tag}", us, nbytes))
        del kv
        both(b, tag)
    T, tag = prompts * ctx, f"{prompts}x{ctx}"
    pages = list(range(1, T // ps + 1))
    per = ctx // ps

    class Table:
        def __init__(self, i):
            self.pages = pages[i * per:(i + 1) * per]
    view = VarlenLayout([0] * prompts, [ctx] * prompts,
                        [Table(i) for i in range(prompts)], 0, ps,
                        dev).paged_view()
    q, o = rnd(T, heads, DIM), rnd(T, qn)
    kp, vp = rnd(T // ps + 1, kvh, ps, DIM), rnd(T // ps + 1, kvh, ps, DIM)
    flops = prompts * ctx * (ctx + 1) // 2 * heads * 4 * DIM
    us = _time(lambda i: ops.paged_prefill(q, kp, vp, view, o, 0.05, 30.0,
                                           True))
    out.append(_row(f"paged_prefill {tag}", us, T * (2 * qn + 2 * kn) * 2,
                    bf16=flops))
    cu = i32([i * ctx for i in range(prompts + 1)])
    bi, sl = ops.reference.prefill_block_info(cu.cpu(), qtile=128)
    bi, sl = bi.to(dev), sl.to(dev)
    k, v = rnd(T, kvh, DIM), rnd(T, kvh, DIM)
    us = _time(lambda i: ops._require_hip().prefill_attention(
        q, k, v, bi, sl, 0.05, ops.PREFILL_SWZ))
    out.append(_row(f"llama prefill_attention {tag}", us,
                    T * (2 * qn + 2 * kn) * 2, bf16=flops))
    both(T, tag)
    return out
