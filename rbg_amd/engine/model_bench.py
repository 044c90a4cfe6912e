"""Prefill and decode throughput of one model family beside another.

Random weights, a few layers of a real model's widths, one GPU, bf16.  Each
workload runs through the engine (scheduler, cache, captured decode steps), so
the numbers are those of serving.  ``bench.py --compare <family>`` prints them.
"""
from __future__ import annotations

import time
from typing import Any, Dict, List, Optional

import torch

from ..models.bitatar import BitatarConfig
from .config import EngineConfig, ModelConfig
from .engine import LLMEngine
from .sequence import SamplingParams

VOCAB = 32768

# name -> (width, ff, heads, kv heads, layers, kv_rank, window, delta heads,
# delta dim); head size 128 in both families
SIZES = {
    "2k": (2048, 5632, 16, 4, 6, 256, 1024, 32, 64),
    "4k": (4096, 14336, 32, 8, 6, 512, 4096, 32, 128),
}


def pair(size: str, family: str = "bitatar") -> List[ModelConfig]:
    """The family's model and the one of equal size it is compared to."""
    if family == "notadra":
        from .notadra_bench import notadra_pair
        return notadra_pair(size)
    if family == "gogalix":
        from .gogalix_bench import gogalix_set
        return gogalix_set(size)
    if family == "danipel":
        from .danipel_bench import danipel_set
        return danipel_set(size)
    w, ff, heads, kvh, layers, rank, window, dh, dd = SIZES[size]
    return [
        BitatarConfig.stacked(
            f"bitatar-{size}", width=w, vocab=VOCAB,
            pattern=("daa" * layers)[:layers], heads=heads, dim=128,
            kv_rank=rank, vdim=128, window=window, ff=ff, groups=8, taps=4,
            delta_heads=dh, delta_dim=dd),
        ModelConfig(name=f"llama-{size}", hidden_size=w, intermediate_size=ff,
                    num_layers=layers, num_heads=heads, num_kv_heads=kvh,
                    vocab_size=VOCAB),
    ]


def _sync(device: str) -> float:
    if device == "cuda":
        torch.cuda.synchronize()
    return time.monotonic()


def run_one(model: ModelConfig, device: str, batch: int, prompt: int,
            steps: int, warmup: int, eager: bool = False) -> Dict[str, Any]:
    eng = LLMEngine(EngineConfig(
        model=model, device=device, max_batch_size=max(batch, 4),
        max_seq_len=prompt + steps + warmup + 64, max_prefill_tokens=8192,
        kv_pool_tokens=(batch + 1) * (prompt + steps + warmup + 128),
        enable_prefix_cache=False, enforce_eager=eager or device != "cuda"))
    gen = torch.Generator().manual_seed(5)
    prompts = torch.randint(0, model.vocab_size, (batch, prompt),
                            generator=gen).tolist()
    # a full step warms kernels and libraries up, then the timed prefill
    eng.generate(prompts[:max(1, eng.cfg.max_prefill_tokens // prompt)],
                 SamplingParams(max_new_tokens=1))
    for p in prompts:
        eng.add_request(p, SamplingParams(max_new_tokens=steps + warmup + 32))
    t0 = _sync(device)
    while eng.scheduler.waiting:
        eng.step()
    prefill_s = _sync(device) - t0
    for _ in range(warmup):
        eng.step()
    t0 = _sync(device)
    for _ in range(steps):
        mode = eng.step()
        assert mode == "decode", mode
    decode_s = _sync(device) - t0
    out = {"model": model.name, "batch": batch, "prompt": prompt,
           "prefill_tok_s": round(batch * prompt / prefill_s, 1),
           "decode_tok_s": round(batch * steps / decode_s, 1),
           "decode_ms_per_step": round(decode_s / steps * 1e3, 3)}
    del eng
    if device == "cuda":
        torch.cuda.empty_cache()
    return out


def run_compare(device: str, steps: int, warmup: int,
                sizes: Optional[List[str]] = None,
                batches=(1, 32), prompt: int = 2048,
                eager: bool = False,
                family: str = "bitatar") -> List[Dict[str, Any]]:
    return [run_one(model, device, b, prompt, steps, warmup, eager)
            for size in (sizes or SIZES) for b in batches
            for model in pair(size, family)]


# -- kernels against their rooflines -------------------------------------------

HBM_TB_S, BF16_TF, F32_TF = 8.0, 2500.0, 157.0


def _time(fn, n: int = 12) -> float:
    """Mean microseconds on the GPU of fn(0), fn(1), ... in one graph."""
    for i in range(3):
        fn(i)
    torch.cuda.synchronize()
    a, b = (torch.cuda.Event(enable_timing=True) for _ in range(2))
    # a captured graph keeps launch gaps out of short kernels' times
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for i in range(n):
            fn(i)
    g.replay()
    torch.cuda.synchronize()
    a.record()
    g.replay()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) * 1e3 / n


def _row(name: str, us: float, nbytes: float = 0.0, bf16: float = 0.0,
         f32: float = 0.0) -> Dict[str, Any]:
    bound = max(nbytes / HBM_TB_S / 1e6, bf16 / BF16_TF / 1e6,
                f32 / F32_TF / 1e6)
    return {"kernel": name, "us": round(us, 1),
            "roofline_us": round(bound, 1),
            "times_roofline": round(us / bound, 2)}


def run_kernels(size: str, batches=(1, 8, 32, 128), ctx: int = 2048,
                prompts: int = 4,
                family: str = "bitatar") -> List[Dict[str, Any]]:
    """The mixers' kernels and the like kernels of Llama, one layer's shapes
    of ``size``; decode inputs rotate through buffers larger than the caches.
    Rooflines: bytes that must move, or the operations the algorithm has to
    do (causal halves counted once, the 32-bit recurrence at the f32 rate)."""
    if family == "notadra":
        from .notadra_bench import notadra_kernels
        return notadra_kernels(size, batches, ctx, prompts)
    if family == "gogalix":
        from .gogalix_bench import gogalix_kernels
        return gogalix_kernels(size, batches, ctx, prompts)
    if family == "danipel":
        from .danipel_bench import danipel_kernels
        return danipel_kernels(size, batches, ctx, prompts)
    import math

    from .. import ops
    from .batch import VarlenLayout
    w, ff, heads, kvh, _, rank, window, dh, dd = SIZES[size]
    dev, bf = torch.device("cuda"), torch.bfloat16
    out: List[Dict[str, Any]] = []

    def rnd(*shape, dtype=bf):
        return torch.randn(*shape, device=dev, dtype=torch.float32).to(dtype)

    def copies(nbytes: int) -> int:
        return max(1, min(12, int(600e6 // max(nbytes, 1)) + 1))

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)
    ps = 16
    ones, conv_w = torch.ones(w, device=dev), torch.randn(4, w, device=dev)
    hd = dh * dd
    offs = [hd * i for i in range(6)]
    dargs = (rnd(hd, 64), torch.randn(hd, device=dev),
             torch.randn(hd, device=dev), torch.ones(hd, device=dev))
    for b in batches:
        tag = f"B={b}"
        pages = b * ctx // ps + 1
        bt = (torch.arange(b * (ctx // ps), device=dev, dtype=torch.int32)
              .view(b, -1) + 1)
        cl = i32([ctx] * b)
        keys = min(window, ctx)
        n = copies(pages * ps * rank * 2)
        lat = [rnd(pages, ps, rank) for _ in range(n)]
        q = rnd(b, heads, rank)
        us = _time(lambda i: ops.latent_decode(q, lat[i % n], bt, cl, 0.05,
                                               window))
        out.append(_row(f"latent_decode {tag}", us,
                        b * keys * rank * 2 + 2 * b * heads * rank * 2,
                        bf16=b * heads * keys * rank * 4))
        del lat
        n = copies(pages * ps * kvh * 128 * 4)
        kv = [(rnd(pages, kvh, ps, 128), rnd(pages, kvh, ps, 128))
              for _ in range(n)]
        q = rnd(b, heads, 128)
        sp = ops.pick_decode_splits(b, kvh, ctx + 128)
        us = _time(lambda i: ops.decode_attention(q, *kv[i % n], bt, cl, 0.05,
                                                  num_splits=sp))
        out.append(_row(f"llama decode_attention {tag}", us,
                        b * ctx * kvh * 128 * 4 + 2 * b * heads * 128 * 2))
        del kv
        q, uk = rnd(b, heads, 128), rnd(heads, rank, 128)
        us = _time(lambda i: ops.head_linear(q, uk))
        out.append(_row(f"head_linear {tag}", us, uk.numel() * 2 +
                        b * heads * (128 + rank) * 2))
        slots = i32(range(1, b + 1))
        sbytes = b * dh * dd * dd * 8
        n = copies(sbytes)
        st = [torch.randn(b + 1, dh, dd, dd, device=dev) for _ in range(n)]
        proj = rnd(b, hd * 5 + 64)
        o = rnd(b, hd)
        us = _time(lambda i: ops.delta_rule(
            proj, None, *dargs, st[i % n], slots, None, cl, o, offs,
            math.exp(-0.5), 1e-6, 1e-5))
        out.append(_row(f"delta_step {tag}", us, sbytes + dargs[0].numel() * 2
                        + b * hd * 12))
        del st
        x, d = rnd(b, w, dtype=torch.float32), rnd(b, w)
        hist = rnd(b + 1, 3, w)
        us = _time(lambda i: ops.stream_norm_conv(
            x, d, ones, ones, 8, 1e-5, bf, conv_w, hist, slots, cl))
        out.append(_row(f"stream_norm_conv {tag}", us,
                        b * w * (8 + 2 + 4 + 12) + w * 4 * 6))
        r, wn = rnd(b, w), rnd(w)
        us = _time(lambda i: ops.fused_add_rmsnorm(d, r, wn, 1e-5))
        out.append(_row(f"llama fused_add_rmsnorm {tag}", us, b * w * 8))
        gu, act = rnd(b, 2 * ff), rnd(b, ff)
        us = _time(lambda i: ops.gelu_mul(gu, act))
        out.append(_row(f"gelu_mul {tag}", us, b * ff * 6))
        us = _time(lambda i: ops.silu_mul(gu))
        out.append(_row(f"llama silu_mul {tag}", us, b * ff * 6))
    # prefill: `prompts` prompts of ctx tokens
    T = prompts * ctx

    class Table:
        pages = list(range(1, ctx // ps + 1))
    lay = VarlenLayout([0] * prompts, [ctx] * prompts, [Table()] * prompts, 0,
                       ps, dev)
    cu = i32([i * ctx for i in range(prompts + 1)])
    q, k, v, g = (rnd(T, heads, 128) for _ in range(4))
    act = rnd(T, heads * 128)
    view = lay.window_view(window)
    pairs = prompts * sum(min(i + 1, window) for i in range(ctx))
    tag = f"{prompts}x{ctx}"
    us = _time(lambda i: ops.window_attention(
        q, k, v, g.flatten(1), act, view, 0.05, window))
    out.append(_row(f"window_attention {tag}", us, T * heads * 128 * 10,
                    bf16=pairs * heads * 4 * 128))
    bi, sl = ops.reference.prefill_block_info(cu.cpu(), qtile=128)
    bi, sl = bi.to(dev), sl.to(dev)
    kk, vv = k[:, :kvh].contiguous(), v[:, :kvh].contiguous()
    us = _time(lambda i: ops._require_hip().prefill_attention(
        q, kk, vv, bi, sl, 0.05, ops.PREFILL_SWZ))
    out.append(_row(f"llama prefill_attention {tag}", us, T * heads * 128 * 6,
                    bf16=prompts * ctx * (ctx + 1) // 2 * heads * 4 * 128))
    proj, z, o = rnd(T, hd * 5 + 64), rnd(T, hd), rnd(T, hd)
    st = torch.zeros(prompts + 1, dh, dd, dd, device=dev)
    slots, starts = i32(range(1, prompts + 1)), i32([0] * prompts)
    chunks = (lay.prefill_tiles(ops.DELTA_CHUNK),
              lay.prefill_tile_cu(ops.DELTA_CHUNK))
    us = _time(lambda i: ops.delta_rule(
        proj, z, *dargs, st, slots, cu, starts, o, offs, math.exp(-0.5), 1e-6,
        1e-5, chunks), 4)
    out.append(_row(f"delta_chunk (3 kernels) {tag}", us, T * hd * 14,
                    f32=T * dh * 8 * dd * dd))
    x, d = rnd(T, w, dtype=torch.float32), rnd(T, w)
    us = _time(lambda i: ops.stream_norm(x, d, ones, ones, 8, 1e-5, bf))
    out.append(_row(f"stream_norm {tag}", us, T * w * 14))
    hist = rnd(prompts + 1, 3, w)
    tiles = lay.tiles(ops.CONV_TILE)
    us = _time(lambda i: ops.causal_conv(d, conv_w, hist, tiles, cu, starts,
                                         slots))
    out.append(_row(f"causal_conv {tag}", us, T * w * 4))
    r, wn = rnd(T, w), rnd(w)
    us = _time(lambda i: ops.fused_add_rmsnorm(d, r, wn, 1e-5))
    out.append(_row(f"llama fused_add_rmsnorm {tag}", us, T * w * 8))
    gu, act = rnd(T, 2 * ff), rnd(T, ff)
    us = _time(lambda i: ops.gelu_mul(gu, act))
    out.append(_row(f"gelu_mul {tag}", us, T * ff * 6))
    us = _time(lambda i: ops.silu_mul(gu))
    out.append(_row(f"llama silu_mul {tag}", us, T * ff * 6))
    x = rnd(T, rank + 8)
    cache = rnd(T // ps + 1, ps, rank)
    sl = torch.arange(ps, T + ps, device=dev, dtype=torch.int32)
    us = _time(lambda i: ops.latent_store(
        x[:, :rank], torch.ones(rank, device=dev), cache, sl, 1e-5))
    out.append(_row(f"latent_store {tag}", us, T * rank * 6))
    return out
