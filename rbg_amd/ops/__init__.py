"""rbg_amd.ops — dispatch layer over the CDNA4 HIP kernels.

On a GPU the compiled in-tree extension (_hip_ops, built by setup.py for
gfx950) is MANDATORY: a missing extension raises instead of silently running
an eager fallback, so GPU tests always exercise the native path.  On CPU
(unit tests, GPU-less CI) the fp32 torch references in ops.reference serve
as the implementation.
"""
from __future__ import annotations

import importlib
from dataclasses import dataclass
from typing import Any, Dict, Optional

import torch

from ..utils import hip_build
from . import reference

# Extension modules by name, loaded as far as they are built; a process needs
# those that its model runs on (utils/hip_build.py EXTENSIONS_OF).
EXTENSIONS: Dict[str, Any] = {}
_errors: Dict[str, Exception] = {}
for _name in hip_build.HIP_SOURCES:
    try:
        EXTENSIONS[_name] = importlib.import_module("." + _name, __name__)
    except Exception as e:  # noqa: BLE001
        _errors[_name] = e

_hip = EXTENSIONS.get("_hip_ops")
HAVE_HIP = _hip is not None


def _check_stale() -> None:
    """Fail loudly on a GPU box if a shipped .so predates its kernel sources
    (stale-binary guard; the stamps are written by utils/hip_build.py)."""
    for name in EXTENSIONS:
        if hip_build.is_stale(name):
            raise RuntimeError(
                f"rbg_amd HIP extension {name} is STALE: kernel sources "
                "changed after the last build.  Rebuild in-tree: "
                "PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext "
                "--inplace")


if EXTENSIONS and torch.cuda.is_available():
    _check_stale()


def require(*names: str):
    """The first of these extensions that is built."""
    for name in names:
        if name in EXTENSIONS:
            return EXTENSIONS[name]
    errors = "; ".join(f"{n}: {_errors[n]!r}" for n in names)
    raise RuntimeError(
        f"rbg_amd HIP extension {' or '.join(names)} is not built but a GPU "
        "tensor was passed.  Build it in-tree: PYTORCH_ROCM_ARCH=gfx950 "
        f"python setup.py build_ext --inplace (import error: {errors})")


def _require_hip():
    return _hip if _hip is not None else require("_hip_ops")


def _require_mix():
    return require("_hip_mix")


def _require_latent():
    return require("_hip_latent")


def _require_moe():
    return require("_hip_moe")


def _require_hyper():
    return require("_hip_hyper")


def _require_experts():
    return require("_hip_experts")


def _require_gated():
    return require("_hip_gated")


def _on_gpu(t: torch.Tensor) -> bool:
    return t.is_cuda


SKINNY_GEMM = int(__import__("os").environ.get("RBG_SKINNY_GEMM", "1"))


def linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """Projection GEMM with decode-shape dispatch: for M <= 128 rows the
    hand-written split-K streaming kernel (hip/skinny_gemm.hip) replaces
    hipBLASLt, which leaves 2-5x on narrow-N skinny shapes
    (profiles/gemm_ab_b128.json).  Prefill-sized M goes to the library."""
    # measured policy (profiles/sg_micro7_b*.json): the custom kernel wins
    # on narrow-N shapes (o/down, N<=4096) at any decode batch, on mid-N
    # (qkv, 6144) only up to M=64, and never on wide-N (gate_up 28672,
    # where hipBLASLt already streams at ~6 TB/s).  Between them, for a few
    # rows, hipBLASLt takes up to 2.7 times as long (18432 x 2048: 58 us
    # against 22) and is nowhere ahead by more than a tenth
    if (SKINNY_GEMM and _on_gpu(x) and x.dim() == 2 and
            x.dtype == torch.bfloat16 and x.shape[0] <= 128 and
            w.shape[0] % 32 == 0 and x.shape[1] % 512 == 0 and
            (w.shape[0] <= 4608 or
             (x.shape[0] <= 64 and w.shape[0] <= 8192) or
             (x.shape[0] <= 16 and w.shape[0] <= 24576 and
              x.shape[1] <= 4096))):
        # one of these is there whatever the model
        return require("_hip_ops", "_hip_mix", "_hip_gated", "_hip_moe",
                       "_hip_hyper").skinny_gemm(
            x if x.is_contiguous() else x.contiguous(), w)
    return torch.nn.functional.linear(x, w)


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    if _on_gpu(x):
        return _require_hip().rmsnorm(x, weight, eps)
    return reference.rmsnorm(x, weight, eps)


def fused_add_rmsnorm(x: torch.Tensor, residual: torch.Tensor,
                      weight: torch.Tensor, eps: float) -> None:
    if _on_gpu(x):
        _require_hip().fused_add_rmsnorm(x, residual, weight, eps)
        return
    reference.fused_add_rmsnorm(x, residual, weight, eps)


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    if _on_gpu(x):
        return _require_hip().silu_mul(x)
    return reference.silu_mul(x)


def rope_store_kv(q, k, v, key_cache, value_cache, cos_sin, positions,
                  slot_mapping) -> None:
    if _on_gpu(q):
        _require_hip().rope_store_kv(q, k, v, key_cache, value_cache,
                                     cos_sin, positions, slot_mapping)
        return
    reference.rope_store_kv(q, k, v, key_cache, value_cache, cos_sin,
                            positions, slot_mapping)


def pick_decode_splits(num_seqs: int, num_kv_heads: int,
                       max_context: int, variant: int = -1) -> int:
    """Fill the chip: MI355X has 256 CUs / 8 XCDs; measured optimum is
    ~1024 workgroups for BOTH kernels (profiles/decode_breakdown r59
    sweep: V4 B128 peaks at splits=2 = 1024 WGs, B64 at splits=4 = 1024).
    The MFMA kernel packs 2 sequences per WG, so its base WG count is
    half the dot2 kernel's at equal splits."""
    if variant < 0:
        variant = DECODE_VARIANT
    if variant >= 4:
        # v4/v5 pack 2 seqs per WG; v6 runs 1 seq per (2-wave) WG
        per_wg = 2 if variant in (4, 5) else 1
        base = num_kv_heads * ((num_seqs + per_wg - 1) // per_wg)
        by_ctx = max(1, max_context // 32)      # >= one page pair per split
    else:
        base = num_seqs * num_kv_heads
        by_ctx = max(1, max_context // 256)
    if base >= 1024:
        return 1
    want = max(1, 1024 // max(base, 1))
    return int(min(want, by_ctx, 16))


DECODE_VARIANT = int(__import__("os").environ.get("RBG_DECODE_VARIANT", "4"))  # MFMA page-pair decode: 5.6 TB/s vs 4.0 dot2 (B128, within-probe)
PREFILL_SWZ = int(__import__("os").environ.get("RBG_PREFILL_SWZ", "6"))  # 8-wave + K/V double-buffer (305 TF/s vs 252 @ swz=4, within-probe)


def decode_attention(q, key_cache, value_cache, block_tables, context_lens,
                     scale: float, num_splits: int = 0,
                     variant: int = -1) -> torch.Tensor:
    if _on_gpu(q):
        if num_splits <= 0:
            max_ctx = int(context_lens.max().item()) if context_lens.numel() else 1
            num_splits = pick_decode_splits(q.shape[0], key_cache.shape[1],
                                            max_ctx)
        if variant < 0:
            variant = DECODE_VARIANT
        return _require_hip().decode_attention(
            q, key_cache, value_cache, block_tables, context_lens, scale,
            num_splits, variant)
    return reference.decode_attention(q, key_cache, value_cache, block_tables,
                                      context_lens, scale)


def prefill_attention(q, k, v, cu_seqlens, scale: float,
                      cu_seqlens_k=None) -> torch.Tensor:
    if _on_gpu(q):
        # bit 2 = 8-wave 16x16 blocks; bit 3 = 4-wave 32x32 blocks
        qtile = 128 if (PREFILL_SWZ & 12) else 64
        block_info, seq_lens = reference.prefill_block_info(
            cu_seqlens.cpu(), qtile=qtile,
            cu_seqlens_k=None if cu_seqlens_k is None else cu_seqlens_k.cpu())
        return _require_hip().prefill_attention(
            q, k, v, block_info.to(q.device), seq_lens.to(q.device), scale,
            PREFILL_SWZ)
    return reference.prefill_attention(q, k, v, cu_seqlens, scale,
                                       cu_seqlens_k)


build_cos_sin_table = reference.build_cos_sin_table


# -- f32 residual stream ----------------------------------------------------


def embed_stream(tokens, table, scale: float, copies: int = 1) -> torch.Tensor:
    """f32 stream [T, W] = table[tokens] * scale; [T, copies * W] of equal
    streams."""
    if _on_gpu(table):
        # linked into every extension of designs that scale
        return require("_hip_mix", "_hip_gated", "_hip_hyper").embed_stream(
            tokens, table, scale, copies)
    return reference.embed_stream(tokens, table, scale, copies)


def stream_norm(x, delta, w1, w2, groups: int, eps: float, dtype):
    """x += delta (in place, f32); returns the grouped RMS norms of x under
    w1 and w2 (None without w2) in ``dtype``."""
    if _on_gpu(x):
        out = _require_mix().stream_norm(x, delta, w1, w2, groups, eps,
                                         dtype == torch.float32, None, None,
                                         None, None)
        return out[0], (out[1] if w2 is not None else None)
    return reference.stream_norm(x, delta, w1, w2, groups, eps, dtype)


def stream_norm_conv(x, delta, w1, w2, groups: int, eps: float, dtype,
                     conv_w, conv_state, slots, positions):
    """Decode form of stream_norm + causal_conv, one token per sequence: the
    first result is convolved with its slot's history, which moves on."""
    if _on_gpu(x):
        out = _require_mix().stream_norm(x, delta, w1, w2, groups, eps,
                                         dtype == torch.float32, conv_w,
                                         conv_state, slots, positions)
        return out[0], (out[1] if w2 is not None else None)
    n1, n2 = reference.stream_norm(x, delta, w1, w2, groups, eps, dtype)
    cu = torch.arange(n1.shape[0] + 1, dtype=torch.int32)
    return reference.causal_conv(n1, conv_w, conv_state, cu, positions,
                                 slots), n2


CONV_TILE = 16


def causal_conv(x, conv_w, conv_state, tiles, cu_seqlens, starts, slots):
    """x + causal depthwise convolution over varlen sequences; conv_w is
    [taps, W], conv_state [slots, taps-1, W] (advanced in place)."""
    if _on_gpu(x):
        return _require_mix().causal_conv(x, conv_w, conv_state, tiles,
                                          cu_seqlens, starts, slots,
                                          max(CONV_TILE, conv_w.shape[0]))
    return reference.causal_conv(x, conv_w, conv_state, cu_seqlens, starts,
                                 slots)


# -- gates ------------------------------------------------------------------


def gelu_mul(x, out) -> None:
    """out (may be a column slice) = gelu_tanh(x[:, :F]) * x[:, F:]."""
    if _on_gpu(x):
        require("_hip_mix", "_hip_hyper").gelu_mul(x, out)
        return
    reference.gelu_mul(x, out)


def clamped_glu(gate, up, limit: float, out) -> None:
    """out = g sigmoid(1.702 g) (u + 1), g = min(gate, limit), u = up within
    +-limit; gate and up are column slices of one buffer."""
    if _on_gpu(gate):
        _require_hyper().clamped_glu(gate, up, limit, out)
        return
    reference.clamped_glu(gate, up, limit, out)


def tanh_rows(x) -> torch.Tensor:
    if _on_gpu(x):
        return _require_mix().tanh_rows(x)
    return torch.tanh(x.float()).to(x.dtype)


# -- generalized delta rule ---------------------------------------------------


DELTA_CHUNK = 16        # tokens per chunk of the prompt kernels


def delta_rule(proj, z, w2, w0, a_bias, norm_w, state, slots, cu_seqlens,
               starts, out, offs, decay_scale: float, unit_eps: float,
               norm_eps: float, chunks=None) -> None:
    """Gated delta rule over varlen rows (cu_seqlens None: one row per
    sequence), with the head norm and the output gate; ``offs`` are the
    columns of r, k, v, a, g and the low-rank decay input in ``proj``.  The
    decay logit is ``z``, or W2 tanh(low) formed in the kernel when None.
    With ``chunks`` = (tiles, chunk_cu) of DELTA_CHUNK tokens and a ``z``, the
    rows go through the matrix cores a chunk at a time."""
    if _on_gpu(proj):
        mix = _require_mix()
        args = (proj, z, w2, w0, a_bias, norm_w, state, slots, cu_seqlens,
                starts, out, offs, decay_scale, unit_eps, norm_eps)
        # the chunk form scales by e^(DELTA_CHUNK * decay_scale)
        if (chunks is not None and z is not None and state.shape[-1] <= 128
                and decay_scale * DELTA_CHUNK <= 60.0):
            mix.delta_chunk(*args, *chunks)
        else:
            mix.delta_step(*args)
        return
    reference.delta_rule(proj, z, w2, w0, a_bias, norm_w, state, slots,
                         cu_seqlens, starts, out, offs, decay_scale, unit_eps,
                         norm_eps)


# -- latent attention -----------------------------------------------------------


@dataclass
class Rotary:
    """Rotary positions of a step's rows: table [positions, dims] = [cos | sin]
    (models/rotary.py); pairs are neighbours (interleaved) or half the dims
    apart."""
    table: torch.Tensor
    positions: torch.Tensor     # [T] int32
    interleaved: bool

    def rows(self, part: slice) -> "Rotary":
        return Rotary(self.table, self.positions[part], self.interleaved)

    @property
    def dims(self) -> int:
        return self.table.shape[1]


def _rotary(rot: Optional[Rotary]):
    return (None, None, False) if rot is None else (rot.table, rot.positions,
                                                    rot.interleaved)


def latent_store(x, w, cache, slots, eps: float,
                 rot: Optional[Rotary] = None, second=None):
    """c = rms_norm(x) * w, written to the paged latents; returns c.  With
    ``rot`` x's last columns are no latent but a key part: rotated, it follows
    in the cache and in c.  ``second`` = (x2, w2), another latent of the same
    rows: its norm is returned beside c."""
    if _on_gpu(x):
        out = _require_latent().latent_store(x, w, cache, slots, eps,
                                             *_rotary(rot),
                                             *(second or (None, None)))
    else:
        out = reference.latent_store(x, w, cache, slots, eps, rot, second)
    return out[0] if second is None else out


def rotate_rows(x, rot: Rotary) -> None:
    """Rotates x [T, H, rot.dims] in place."""
    if _on_gpu(x):
        _require_latent().rotate_rows(x, *_rotary(rot))
        return
    x.copy_(reference.rotate(x, rot))


def window_attention(q, k, v, gate, out, view, scale: float, window: int,
                     shared=None, sink=None) -> None:
    """Causal attention over the last ``window`` positions (0: all), q/k
    [T, H, D], v [T, H, Dv]; ``view`` locates each query among the keys
    (engine/batch.py WindowView).  out = o * sigmoid(gate).  ``shared`` [T, D2]
    are the last dims of every head's key (k then has the others); ``sink`` [H]
    f32 is a logit per head without key and value."""
    if _on_gpu(q):
        _require_latent().window_attention(q, k, v, gate, out, view.row_info,
                                           view.seq_info, view.blocks, scale,
                                           window, shared, sink)
        return
    reference.window_attention(q, k, v, gate, out, view.row_info, scale,
                               window, shared, sink)


def pick_latent_splits(num_seqs: int, num_heads: int, max_keys: int) -> int:
    """Key splits of latent_decode: two workgroups per CU, one for small
    batches (the splits' sums cost more than they hide there), at least one
    64-key step each.  Depends on sizes only, so a captured decode step keeps
    its value."""
    base = num_seqs * ((num_heads + 15) // 16)
    want = 512 if base >= 64 else 256
    steps = (max_keys + 63) // 64
    return int(max(1, min((want + base - 1) // base, steps, 64)))


def latent_decode(q, cache, block_tables, context_lens, scale: float,
                  window: int, rank: int = 0, sink=None) -> torch.Tensor:
    """q [S, H, D] absorbed queries against the paged latents [.., D], whose
    first ``rank`` columns (0: all) are the value; returns [S, H, rank].
    ``sink`` as in window_attention."""
    rank = rank or q.shape[2]
    if _on_gpu(q):
        keys = block_tables.shape[1] * cache.shape[1]
        splits = pick_latent_splits(q.shape[0], q.shape[1],
                                    min(keys, window) if window else keys)
        return _require_latent().latent_decode(q, cache, block_tables,
                                               context_lens, scale, window,
                                               splits, rank, sink)
    return reference.latent_decode(q, cache, block_tables, context_lens,
                                   scale, window, rank, sink)


def head_linear(x, w, gate=None, out=None, tail=None,
                rot: Optional[Rotary] = None) -> torch.Tensor:
    """out[s, h, j] = sum_k x[s, h, k] w[h, j, k], times sigmoid(gate); ``out``
    [S, H * n] may be a column slice.  With ``tail`` [S, H, rot.dims] each head
    of out ends in its rotation: out [S, H, n + dims]."""
    heads, n = w.shape[0], w.shape[1]
    full = n + (rot.dims if rot is not None else 0)
    if out is None:
        out = x.new_empty((x.shape[0], heads * full))
    o = out.unflatten(1, (heads, full))
    if _on_gpu(x):
        _require_latent().head_linear(x, w, gate, o, tail, *_rotary(rot))
    else:
        reference.head_linear(x, w, gate, o[..., :n])
        if rot is not None:
            o[..., n:] = reference.rotate(tail, rot)
    return out if rot is None else o


# -- sandwich norms, paged attention, sparse experts ---------------------------


@dataclass
class Routing:
    """Which experts a step's tokens go to: T * top (token, choice) pairs,
    stored in expert order and cut into tiles of one expert each."""
    top: int
    tile: int                   # most rows of a tile
    weights: torch.Tensor       # [T, top] f32
    inv: torch.Tensor           # [T * top] int32: a pair's row
    rows: torch.Tensor          # [T * top] int32: a row's token
    tiles: torch.Tensor         # [n, 3] int32: expert, first row, rows
    count: Optional[torch.Tensor] = None    # GPU: how many tiles are used


def embed_pairs(tokens, prev, table, pairs, mul_prev: int,
                mul_cur: int) -> torch.Tensor:
    """f32 stream: table[token] + pairs[(prev * mul_prev + token * mul_cur) mod
    buckets], the last row of ``pairs`` where prev is -1."""
    if _on_gpu(table):
        return _require_moe().embed_pairs(tokens, prev, table, pairs, mul_prev,
                                          mul_cur)
    return reference.embed_pairs(tokens, prev, table, pairs, mul_prev, mul_cur)


def sandwich_norm(x, pending, w, eps: float, dtype):
    """x += RMS norm of what is pending under its weight (in place, f32; None:
    nothing); returns the RMS norm of x under w in ``dtype`` (None without w).
    ``pending`` = (rows, routing or None, weight); rows with a routing are
    weighed and summed first."""
    rows = route = wb = None
    if pending is not None:
        rows, route, wb = pending
    if _on_gpu(x):
        return _require_moe().sandwich_norm(
            x, rows, route.inv if route else None,
            route.weights if route else None, wb, w, eps,
            dtype == torch.float32)
    return reference.sandwich_norm(x, rows, route, wb, w, eps, dtype)


def moe_combine(y, route) -> torch.Tensor:
    """Weighed sums of each token's expert rows, in y's dtype."""
    if _on_gpu(y):
        return _require_experts().moe_combine(y, route.inv, route.weights)
    return reference.moe_combine(y, route).to(y.dtype)


def rope_store_paged(proj, bias, cos_sin, positions, slots, heads: int,
                     dim: int, k, v, offs) -> None:
    """Adds the biases (None: none) of a fused projection, rotates the leading
    dimensions of its queries (in place) and keys by cos_sin [positions, dims]
    = [cos | sin] (None: not), and writes keys and values to the pages [pages,
    kv heads, page_size, size].  ``offs`` are the columns of q, k, v; of q
    alone when the keys are another layer's."""
    if _on_gpu(proj):
        _require_moe().rope_store_paged(proj, bias, cos_sin, positions, slots,
                                        heads, dim, k, v, offs)
        return
    reference.rope_store_paged(proj, bias, cos_sin, positions, slots, heads,
                               dim, k, v, offs)


@dataclass
class Difference:
    """Differential heads: a head's query and key are two, whose softmaxes o1
    and o2 over the same values become (o1 - lam o2) / rms * scale."""
    lam: torch.Tensor           # [1] f32
    scale: float
    eps: float                  # inside the root


def _difference(diff: Optional[Difference]):
    return (None, 1.0, 0.0) if diff is None else (diff.lam, diff.scale,
                                                  diff.eps)


def paged_prefill(q, k, v, view, out, scale: float, softcap: float,
                  sink: bool, window: int = 0,
                  diff: Optional[Difference] = None) -> None:
    """Causal attention of portions [R, H, D] over the pages; ``view`` is the
    step's engine/batch.py PagedView.  Scores are scale * q.k, then softcap *
    tanh(score / softcap) (0: as they are); ``sink`` adds a key of score 0 and
    no value; ``window`` is how many keys a row sees, itself included (0: all
    before it).  With ``diff`` q and k hold two maps of half the size."""
    if _on_gpu(q):
        _require_moe().paged_prefill(q, k, v, view.tables, view.seq_info,
                                     view.row_info, view.blocks, out, scale,
                                     softcap, sink, window,
                                     *_difference(diff))
        return
    reference.paged_rows(q, k, v, view.tables, view.row_info, out, scale,
                         softcap, sink, window, diff)


def pick_paged_splits(num_seqs: int, kv_heads: int, max_keys: int) -> int:
    """Key splits of paged_decode: two workgroups per CU, at least one
    128-key step each.  Depends on sizes only, so that a captured decode step
    keeps its value."""
    base = max(1, num_seqs * kv_heads)
    steps = (max_keys + 127) // 128
    return int(max(1, min((512 + base - 1) // base, steps, 64)))


def paged_decode(q, k, v, tables, context_lens, out, scale: float,
                 softcap: float, sink: bool, splits: int = 0, window: int = 0,
                 diff: Optional[Difference] = None) -> None:
    """One query row per sequence, [S, H, D]; scores as in paged_prefill."""
    if _on_gpu(q):
        if splits <= 0:
            keys = tables.shape[1] * k.shape[2]
            # a window may begin anywhere in its first step
            splits = pick_paged_splits(
                q.shape[0], k.shape[1],
                min(keys, window + 127) if window else keys)
        _require_moe().paged_decode(q, k, v, tables, context_lens, out, scale,
                                    softcap, sink, window,
                                    *_difference(diff), splits)
        return
    info = torch.stack([torch.arange(q.shape[0], dtype=torch.int32),
                        context_lens - 1], dim=1)
    reference.paged_rows(q, k, v, tables, info, out, scale, softcap, sink,
                         window, diff)


def router_logits(x, w) -> torch.Tensor:
    """x W^T in 32-bit, [T, experts] f32."""
    if _on_gpu(x):
        return _require_experts().router_logits(x, w)
    return x.float() @ w.float().T


def expert_tile(x, w, top: float) -> int:
    """Rows per tile that suit x [T, K] through experts w [E, N, K], ``top`` of
    them a token on average."""
    pairs = x.shape[0] * top
    rows = pairs / w.shape[0]                   # per expert, on average
    if (not _on_gpu(x) or x.dtype == torch.float32 or w.shape[1] % 8 or
            w.shape[2] % 8 or
            # the chip would not be full of 64-column pieces
            pairs * ((w.shape[1] + 63) // 64) < 256):
        return 16
    return 32 if rows <= 20 else 64 if rows <= 40 else 128


def moe_route(logits, correction, groups: int, keep: int, top: int,
              tile: int, softmax: bool = False, share: Optional[float] = None,
              identity: int = 0) -> Routing:
    """Chooses the ``top`` experts of each token by sigmoid(logit) + correction
    among the ``keep`` groups with the largest sums of their two best, and lays
    the pairs out by expert.  Weights are the sigmoids.  ``softmax``: the
    choice is by logit + correction, the weights are the softmax of the
    chosen.  ``share``: the scores are the softmax of all, the weights the
    chosen ones' shares of their scores times ``share``.  The last ``identity``
    experts return their input: their pairs are weighed but get no row."""
    if _on_gpu(logits):
        mod = _require_experts()
        mode = (mod.ROUTE_SHARE if share is not None else
                mod.ROUTE_CHOSEN if softmax else mod.ROUTE_SIGMOID)
        weights, inv, rows, tiles, count = mod.moe_route(
            logits, correction, groups, keep, top, tile, mode, identity,
            1.0 if share is None else share)
        return Routing(top, tile, weights, inv, rows, tiles, count)
    ids, weights = reference.moe_choose(logits, correction, groups, keep, top,
                                        softmax, share)
    return Routing(top, tile, weights, *reference.moe_tiles(
        ids, logits.shape[1] - identity, tile))


def interleave_glu(gate, up) -> torch.Tensor:
    """Rows of two matrices [.., F, K] (F even) as expert_linear's ``swiglu``
    reads them: two of the gate, two of the up matrix, and so on."""
    f, k = gate.shape[-2:]
    pair = [t.unflatten(-2, (f // 2, 2)) for t in (gate, up)]
    return torch.cat(pair, dim=-2).flatten(-3, -2)


def expert_linear(x, w, route, gather: bool = False, relu2: bool = False,
                  swiglu: bool = False,
                  limit: Optional[float] = None) -> torch.Tensor:
    """Rows in expert order times their expert's w [E, N, K]; ``gather`` takes
    x's rows by token, ``relu2`` applies max(0, .)^2, ``swiglu`` takes w's rows
    as interleave_glu lays them and gives silu(gate) * up, [.., N / 2]; with
    ``limit`` it is clamped_glu."""
    if _on_gpu(x):
        mod = _require_experts()
        act = (mod.EXPERT_RELU2 if relu2 else mod.EXPERT_NONE if not swiglu
               else mod.EXPERT_SILU_GLU if limit is None else
               mod.EXPERT_CLAMPED_GLU)
        return mod.expert_linear(
            x, w, route.rows if gather else None, route.tiles, route.count,
            route.rows.numel(), route.tile, act, limit or 0.0)
    return reference.expert_linear(x, w, route, gather, relu2, swiglu, limit)


# -- hyper-connections -----------------------------------------------------------


@dataclass
class TanhNorm:
    """Dynamic tanh: tanh(alpha * x) * w + b, no statistics of the row."""
    alpha: torch.Tensor         # [1] f32
    w: torch.Tensor             # [W] f32
    b: torch.Tensor             # [W] f32


@dataclass
class Stir:
    """A sublayer's output on its way into the streams: x_t becomes
    sum_s mix[s, t] x_s + mult * out[t] * y, y = rows plus, with a routing, the
    weighed sum of the token's expert rows (``self_rows``: of experts that
    return their input)."""
    conn: torch.Tensor          # [S * S + S] f32 = mix[from, to] | out
    mult: float
    rows: Optional[torch.Tensor] = None         # [T, W]
    experts: Optional[torch.Tensor] = None      # [T * top, W]
    route: Optional[Routing] = None
    self_rows: Optional[torch.Tensor] = None    # [T, W]


def hyper_norm(x, streams: int, stir: Optional[Stir], read,
               norm: Optional[TanhNorm], dtype):
    """x [T, streams * W] f32 takes what is pending (in place); returns the
    norm of sum_s read[s] x_s in ``dtype`` (None without a norm)."""
    if _on_gpu(x):
        s = stir or Stir(None, 1.0)
        n = norm or TanhNorm(None, None, None)
        return _require_hyper().hyper_norm(
            x, streams, s.conn, s.rows, s.experts,
            s.route.inv if s.route else None,
            s.route.weights if s.route else None, s.self_rows, s.mult, read,
            n.w, n.b, n.alpha, dtype == torch.float32)
    return reference.hyper_norm(x, streams, stir, read, norm, dtype)


# -- gated branches, gated delta rule -------------------------------------------


@dataclass
class Branch:
    """What a layer leaves to be added to the stream: (rows + bias) * scale *
    sigmoid(logits + gate_bias), rows of tokens or (with a routing) of their
    chosen experts, weighed and summed."""
    rows: torch.Tensor          # [T, W], or expert rows
    logits: torch.Tensor        # [T, W]
    gate_bias: torch.Tensor     # [W] f32
    scale: torch.Tensor         # [W] f32
    bias: Optional[torch.Tensor] = None         # [W] f32
    route: Optional[Routing] = None


def gate_norm(x, branches, w, eps: float, dtype):
    """x += the branches (in place, f32; at most two); returns the RMS norm of
    x under w, one number or one per coordinate, in ``dtype`` (None without
    w)."""
    if _on_gpu(x):
        return _require_gated().gate_norm(
            x, [(b.rows, b.route.inv if b.route else None,
                 b.route.weights if b.route else None, b.logits, b.gate_bias,
                 b.scale, b.bias) for b in branches], w, eps,
            dtype == torch.float32)
    return reference.gate_norm(x, branches, w, eps, dtype)


def silu_glu(gate, up, gate_bias, up_bias, out) -> None:
    """out = silu(gate + gate_bias) * (up + up_bias); gate and up are column
    slices of one buffer, the biases may be None."""
    if _on_gpu(gate):
        _require_gated().silu_glu(gate, up, gate_bias, up_bias, out)
        return
    reference.silu_glu(gate, up, gate_bias, up_bias, out)


def short_conv(x, conv_w, ring, tiles, cu_seqlens, starts, slots):
    """silu of the causal depthwise convolution of varlen rows (a column
    slice); conv_w [taps, W], the last tap the current token's; ring [slots,
    taps, W] holds a sequence's last inputs, position p's at p % taps."""
    if _on_gpu(x):
        return _require_gated().short_conv(x, conv_w, ring, tiles, cu_seqlens,
                                           starts, slots,
                                           max(CONV_TILE, conv_w.shape[0]))
    return reference.short_conv(x, conv_w, ring, cu_seqlens, starts, slots)


@dataclass
class GatedDelta:
    """Constants of a gated delta rule (gated_delta)."""
    a_log: torch.Tensor         # [H] f32
    dt_bias: torch.Tensor       # [H] f32, or [H*D]: a decay per key channel
    norm: torch.Tensor          # [E] f32
    kv_heads: int
    silu: bool                  # output gate: silu, else sigmoid
    q_scale: float
    unit_eps: float             # inside the root of q's and k's norms
    norm_eps: float             # inside the root of the head norm's


def gated_delta(p: GatedDelta, qkv, offs, beta, decay, gate, state, slots,
                cu_seqlens, starts, out, conv=None, chunks=None) -> None:
    """Gated delta rule over varlen rows (cu_seqlens None: one row per
    sequence) with the head norm and the output gate.  ``offs`` are the columns
    of q, k [kv_heads, D], v [H, E] in ``qkv``; state [slots, H, D, E].
    Per token, with unit q (times q_scale) and k, g = exp(-exp(a_log) *
    softplus(decay + dt_bias)):
      S <- g S;  u = sigmoid(beta) (v - S^T k);  S <- S + k u^T;  o = S^T q.
    ``conv`` = (conv_w, ring): decode rows, whose q, k, v are first convolved
    as by short_conv, over the columns from q's on.  With ``chunks`` = (tiles,
    chunk_cu) of DELTA_CHUNK tokens the rows go through the matrix cores."""
    if _on_gpu(qkv):
        mod = _require_gated()
        args = (qkv, beta, decay, gate, p.a_log, p.dt_bias, p.norm, state,
                slots, cu_seqlens, starts, out, offs, p.kv_heads, p.silu,
                p.q_scale, p.unit_eps, p.norm_eps)
        if chunks is not None and state.shape[2] <= mod.CHUNK_MAX_DIM:
            assert mod.CHUNK == DELTA_CHUNK
            mod.gated_chunk(*args, *chunks)
        else:
            mod.gated_step(*args, *(conv or (None, None)))
        return
    if conv is not None:
        n = slots.numel()
        width = conv[0].shape[1]
        x = reference.short_conv(
            qkv[:, offs[0]:offs[0] + width], *conv,
            torch.arange(n + 1, dtype=torch.int32), starts, slots)
        qkv, offs = x, [o - offs[0] for o in offs]
    reference.gated_delta(p, qkv, offs, beta, decay, gate, state, slots,
                          cu_seqlens, starts, out)
