"""Prefill and decode throughput of one model family beside another.

Random weights, a few layers of a real model's widths, one GPU, bf16.  Each
workload runs through the engine (scheduler, cache, captured decode steps), so
the numbers are those of serving.  ``bench.py --compare bitatar`` prints them.
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


def pair(size: str) -> List[ModelConfig]:
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
    # one prompt warms kernels and libraries up, then the timed prefill
    eng.generate(prompts[:1], SamplingParams(max_new_tokens=1))
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
                eager: bool = False) -> List[Dict[str, Any]]:
    return [run_one(model, device, b, prompt, steps, warmup, eager)
            for size in (sizes or SIZES) for b in batches
            for model in pair(size)]
