"""In-tree build of the HIP extensions (gfx950) and their freshness stamps.

Each extension carries a stamp: a hash over its sources and headers
at build time.  A process on a GPU box refuses an extension whose sources have
changed since (ops/__init__.py), and ``ensure`` builds a missing or stale one,
so that a fresh checkout compiles only what its model runs on.
"""
from __future__ import annotations

import fcntl
import glob
import hashlib
import os
import shutil
import subprocess
import sys
from typing import Iterable, Optional

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(
    os.path.abspath(__file__))))
OPS_DIR = os.path.join(ROOT, "rbg_amd", "ops")
HIP_DIR = os.path.join(OPS_DIR, "hip")

# Canonical sources, listed explicitly: a glob would also pick up hipify
# build artifacts (*_hip.hip) that torch's cpp_extension emits next to
# the originals, risking duplicate extern-C symbols from drifted copies.
HIP_SOURCES = {
    # bf16 attention/norm/GEMM kernels, KV push, xGMI all-reduce
    "_hip_ops": [
        "attn_decode.hip",
        "attn_prefill.hip",
        "mfma_probe.hip",
        "rmsnorm.hip",
        "rope_kv.hip",
        "silu_mul.hip",
        "skinny_gemm.hip",
        "kv_peer_copy.hip",
        "allreduce.hip",
        "bindings.cpp",
    ],
    # f32-stream norms, gates and the generalized delta rule
    "_hip_mix": [
        "embed.hip",
        "stream_norm.hip",
        "gated_act.hip",
        "delta_rule.hip",
        "delta_chunk.hip",
        "skinny_gemm.hip",
        "mix_bindings.cpp",
    ],
    # latent attention
    "_hip_latent": [
        "latent_attn.hip",
        "latent_decode.hip",
        "window_attn.hip",
        "head_linear.hip",
        "latent_bindings.cpp",
    ],
    # mixtures of experts
    "_hip_experts": [
        "moe_route.hip",
        "moe_gemm.hip",
        "moe_combine.hip",
        "expert_bindings.cpp",
    ],
    # sandwich norms, paged attention of any sizes
    "_hip_moe": [
        "sandwich_norm.hip",
        "rope_paged.hip",
        "paged_attn.hip",
        "skinny_gemm.hip",
        "moe_bindings.cpp",
    ],
    # hyper-connections, tanh norms, gated linear units
    "_hip_hyper": [
        "embed.hip",
        "hyper_norm.hip",
        "gated_act.hip",
        "skinny_gemm.hip",
        "hyper_bindings.cpp",
    ],
    # gated delta rule, short convolution, gated norms and linear units
    "_hip_gated": [
        "embed.hip",
        "gate_norm.hip",
        "gated_act.hip",
        "short_conv.hip",
        "gated_delta.hip",
        "gated_delta_chunk.hip",
        "skinny_gemm.hip",
        "gated_bindings.cpp",
    ],
}

HIP_HEADERS = {
    "_hip_ops": ["common.h", "gemm_bindings.h"],
    "_hip_mix": ["act.h", "act_kinds.h", "bind_util.h", "common.h",
                 "delta_scan.h", "embed_bindings.h", "gemm_bindings.h",
                 "glu_bindings.h", "mfma_util.h", "mix_args.h", "vec_io.h"],
    "_hip_latent": ["bind_util.h", "common.h", "latent_args.h", "lds_stream.h",
                    "mfma_util.h", "rotary.h", "vec_io.h"],
    "_hip_experts": ["act.h", "act_kinds.h", "bind_util.h", "common.h",
                     "expert_args.h", "expert_rows.h", "lds_stream.h",
                     "mfma_util.h", "vec_io.h"],
    "_hip_moe": ["bind_util.h", "common.h", "expert_rows.h", "gemm_bindings.h",
                 "mfma_util.h", "moe_args.h", "vec_io.h"],
    "_hip_hyper": ["act.h", "act_kinds.h", "bind_util.h", "common.h",
                   "embed_bindings.h", "expert_rows.h", "gemm_bindings.h",
                   "glu_bindings.h", "hyper_args.h", "vec_io.h"],
    "_hip_gated": ["act.h", "act_kinds.h", "bind_util.h", "common.h",
                   "delta_scan.h", "embed_bindings.h", "expert_rows.h",
                   "gated_args.h", "gated_delta.h", "gemm_bindings.h",
                   "glu_bindings.h", "mfma_util.h", "vec_io.h"],
}

# model architecture -> the extensions with its kernels (default: _hip_ops)
EXTENSIONS_OF = {"Bitatar": ("_hip_mix", "_hip_latent"),
                 "Notadra": ("_hip_moe", "_hip_experts"),
                 "Gogalix": ("_hip_gated", "_hip_moe", "_hip_experts"),
                 "Danipel": ("_hip_hyper", "_hip_latent", "_hip_experts")}


def source_hash(name: str) -> str:
    h = hashlib.sha256()
    for f in sorted(HIP_SOURCES[name] + HIP_HEADERS[name]):
        with open(os.path.join(HIP_DIR, f), "rb") as fh:
            h.update(f.encode() + b"\0" + fh.read() + b"\0")
    return h.hexdigest()


def stamp_path(name: str) -> str:
    return os.path.join(OPS_DIR, f"{name}.srchash")


def is_stale(name: str) -> bool:
    """The stamp disagrees with the sources (no stamp: cannot tell)."""
    try:
        with open(stamp_path(name)) as f:
            recorded = f.read().strip()
    except FileNotFoundError:
        return False
    return bool(recorded) and recorded != source_hash(name)


def is_built(name: str) -> bool:
    return bool(glob.glob(os.path.join(OPS_DIR, f"{name}.*.so")))


def build(names: Optional[Iterable[str]] = None, clean: bool = False) -> None:
    """Compile extensions in-tree; ``clean`` recompiles every object."""
    names = list(names or HIP_SOURCES)
    if clean:
        shutil.rmtree(os.path.join(ROOT, "build"), ignore_errors=True)
    env = dict(os.environ, PYTORCH_ROCM_ARCH="gfx950",
               RBG_BUILD_EXT=",".join(names))
    # compiler output goes to stderr: a caller's stdout may be a protocol
    subprocess.run([sys.executable, "setup.py", "build_ext", "--inplace"],
                   cwd=ROOT, env=env, check=True, stdout=sys.stderr)
    for name in names:
        with open(stamp_path(name), "w") as f:
            f.write(source_hash(name))


def ensure(*names: str) -> None:
    """Build extensions that are missing or stale (one builder at a time)."""
    def due():
        return [n for n in names if not is_built(n) or is_stale(n)]
    if not due():
        return
    with open(os.path.join(ROOT, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if due():
            build(due())
