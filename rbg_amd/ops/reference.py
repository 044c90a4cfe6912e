"""Pure-PyTorch fp32 reference implementations of every HIP op.

Two jobs (SURVEY §4 test strategy): (a) the numerics oracle the GPU kernels
are compared against in tests/test_ops_gpu.py, and (b) the CPU execution
path that lets the whole engine run (tiny configs) in GPU-less CI.  These
are NOT a production fallback — on a GPU the HIP extension is mandatory and
its absence raises (ops/__init__.py).
"""
from __future__ import annotations

from typing import Optional, Tuple

import torch


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    xf = x.float()
    inv = torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return (xf * inv * weight.float()).to(x.dtype)


def fused_add_rmsnorm(x: torch.Tensor, residual: torch.Tensor,
                      weight: torch.Tensor, eps: float) -> None:
    """In-place contract of the HIP kernel: residual += x; x = rmsnorm(residual)."""
    summed = (residual.float() + x.float())
    residual.copy_(summed.to(residual.dtype))
    x.copy_(rmsnorm(residual, weight, eps))


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    gate, up = x.float().chunk(2, dim=-1)
    return (torch.nn.functional.silu(gate) * up).to(x.dtype)


def build_cos_sin_table(head_dim: int, max_positions: int,
                        theta: float = 500000.0,
                        device="cpu") -> torch.Tensor:
    """[max_pos, head_dim] fp32 = [cos(half) | sin(half)] — host-precomputed
    (guide Appendix B: no on-device trig in the RoPE kernel)."""
    half = head_dim // 2
    inv_freq = 1.0 / (theta ** (torch.arange(0, half, dtype=torch.float64,
                                             device=device) / half))
    pos = torch.arange(max_positions, dtype=torch.float64, device=device)
    freqs = torch.outer(pos, inv_freq)
    return torch.cat([freqs.cos(), freqs.sin()], dim=-1).float().contiguous()


def apply_rope(x: torch.Tensor, positions: torch.Tensor,
               cos_sin: torch.Tensor) -> torch.Tensor:
    """x [T, H, D]; rotate-half (Llama/NeoX) in fp32."""
    T, H, D = x.shape
    half = D // 2
    cs = cos_sin[positions.long()]            # [T, D]
    cos = cs[:, :half].unsqueeze(1)           # [T,1,half]
    sin = cs[:, half:].unsqueeze(1)
    xf = x.float()
    x1, x2 = xf[..., :half], xf[..., half:]
    out = torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1)
    return out.to(x.dtype)


def rope_store_kv(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                  key_cache: torch.Tensor, value_cache: torch.Tensor,
                  cos_sin: torch.Tensor, positions: torch.Tensor,
                  slot_mapping: torch.Tensor) -> None:
    """Mutates q,k in place (rotated) and scatters k,v into the paged caches.
    Cache layout: [pages, kv_heads, page_size, head_dim]."""
    T = q.shape[0]
    head_dim = key_cache.shape[3]
    kvh = key_cache.shape[1]
    page_size = key_cache.shape[2]
    qh = q.numel() // (T * head_dim)
    q3 = q.view(T, qh, head_dim)
    k3 = k.view(T, kvh, head_dim)
    v3 = v.view(T, kvh, head_dim)
    q3.copy_(apply_rope(q3, positions, cos_sin))
    k3.copy_(apply_rope(k3, positions, cos_sin))
    slots = slot_mapping.long()
    valid = slots >= 0
    pages = torch.div(slots[valid], page_size, rounding_mode="floor")
    offs = slots[valid] % page_size
    key_cache[pages, :, offs] = k3[valid]
    value_cache[pages, :, offs] = v3[valid]


def decode_attention(q: torch.Tensor, key_cache: torch.Tensor,
                     value_cache: torch.Tensor, block_tables: torch.Tensor,
                     context_lens: torch.Tensor, scale: float) -> torch.Tensor:
    """q [S, QH, D] one token per sequence; paged KV."""
    S, QH, D = q.shape
    kvh = key_cache.shape[1]
    page_size = key_cache.shape[2]
    qpg = QH // kvh
    out = torch.empty_like(q)
    for s in range(S):
        ctx = int(context_lens[s])
        npages = (ctx + page_size - 1) // page_size
        pages = block_tables[s, :npages].long()
        k = key_cache[pages].permute(1, 0, 2, 3).reshape(kvh, -1, D)[:, :ctx]
        v = value_cache[pages].permute(1, 0, 2, 3).reshape(kvh, -1, D)[:, :ctx]
        qs = q[s].float().view(kvh, qpg, D)
        attn = torch.einsum("hgd,hkd->hgk", qs, k.float()) * scale
        p = torch.softmax(attn, dim=-1)
        o = torch.einsum("hgk,hkd->hgd", p, v.float())
        out[s] = o.reshape(QH, D).to(q.dtype)
    return out


def prefill_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                      cu_seqlens: torch.Tensor, scale: float,
                      cu_seqlens_k: Optional[torch.Tensor] = None
                      ) -> torch.Tensor:
    """Varlen causal attention; q [Tq,QH,D], k/v [Tkv,KVH,D].  With
    cu_seqlens_k, each sequence's q rows are its LAST (Lq) positions of the
    Lk-token KV (prefix caching / chunked prefill)."""
    Tq, QH, D = q.shape
    kvh = k.shape[1]
    qpg = QH // kvh
    out = torch.empty_like(q)
    cu = cu_seqlens.long().tolist()
    cuk = (cu_seqlens_k.long().tolist()
           if cu_seqlens_k is not None else cu)
    for b in range(len(cu) - 1):
        s, e = cu[b], cu[b + 1]
        sk, ek = cuk[b], cuk[b + 1]
        Lq, Lk = e - s, ek - sk
        off = Lk - Lq
        qs = q[s:e].float().view(Lq, kvh, qpg, D)
        ks = k[sk:ek].float()
        vs = v[sk:ek].float()
        attn = torch.einsum("qhgd,khd->hgqk", qs, ks) * scale
        qpos = torch.arange(off, Lk, device=q.device).unsqueeze(1)
        kpos = torch.arange(Lk, device=q.device).unsqueeze(0)
        attn.masked_fill_(kpos > qpos, float("-inf"))
        p = torch.softmax(attn, dim=-1)
        o = torch.einsum("hgqk,khd->qhgd", p, vs)
        out[s:e] = o.reshape(Lq, QH, D).to(q.dtype)
    return out


def prefill_block_info(cu_seqlens: torch.Tensor, qtile: int = 64,
                       cu_seqlens_k: Optional[torch.Tensor] = None
                       ) -> Tuple[torch.Tensor, torch.Tensor]:
    """Host-side block map for the prefill kernel: per block
    (q_start_row, q_block_index, kv_start_row, q_offset) plus the block's
    total KV length."""
    infos = []
    lens = []
    cu = cu_seqlens.tolist()
    cuk = cu_seqlens_k.tolist() if cu_seqlens_k is not None else cu
    for b in range(len(cu) - 1):
        qs, qe = cu[b], cu[b + 1]
        ks, ke = cuk[b], cuk[b + 1]
        Lq, Lk = qe - qs, ke - ks
        off = Lk - Lq
        for qb in range((Lq + qtile - 1) // qtile):
            infos.append((qs, qb, ks, off))
            lens.append(Lk)
    device = cu_seqlens.device
    return (torch.tensor(infos, dtype=torch.int32, device=device).view(-1, 4),
            torch.tensor(lens, dtype=torch.int32, device=device))


# -- f32 residual stream, delta rule, latent attention ------------------------


def embed_stream(tokens, table, scale, copies=1):
    return (table[tokens.long()].float() * scale).repeat(1, copies)


def stream_norm(x, delta, w1, w2, groups, eps, dtype):
    if delta is not None:
        x += delta.float()
    g = x.view(x.shape[0], groups, -1)
    y = (g / torch.sqrt(g.pow(2).mean(-1, keepdim=True) + eps)).view_as(x)
    return ((y * w1).to(dtype),
            (y * w2).to(dtype) if w2 is not None else None)


def causal_conv(x, conv_w, conv_state, cu_seqlens, starts, slots):
    taps = conv_w.shape[0]
    out = torch.empty_like(x)
    cu = cu_seqlens.tolist()
    for b, slot in enumerate(slots.tolist()):
        rows = x[cu[b]:cu[b + 1]].float()
        hist = conv_state[slot].float()
        if int(starts[b]) == 0:
            hist = torch.zeros_like(hist)
        ext = torch.cat([hist, rows])
        y = rows.clone()
        for j in range(taps):
            y += conv_w[j] * ext[j:j + rows.shape[0]]
        out[cu[b]:cu[b + 1]] = y.to(x.dtype)
        conv_state[slot] = ext[ext.shape[0] - (taps - 1):].to(x.dtype)
    return out


def gelu_mul(x, out):
    gate, up = x.float().chunk(2, dim=-1)
    act = torch.nn.functional.gelu(gate, approximate="tanh")
    out.copy_((act * up).to(x.dtype))


def clamped_glu_act(g, u, limit):
    g = g.clamp(max=limit)
    return g * torch.sigmoid(1.702 * g) * (u.clamp(-limit, limit) + 1)


def clamped_glu(gate, up, limit, out):
    out.copy_(clamped_glu_act(gate.float(), up.float(), limit).to(out.dtype))


def delta_rule(proj, z, w2, w0, a_bias, norm_w, state, slots, cu_seqlens,
               starts, out, offs, decay_scale, unit_eps, norm_eps):
    H, D = state.shape[1:3]
    r, k, v, a, g = (proj[:, o:o + H * D].float().view(-1, H, D)
                     for o in offs[:5])
    if z is None:
        low = torch.tanh(proj[:, offs[5]:offs[5] + w2.shape[1]].float())
        z = torch.nn.functional.linear(low.to(proj.dtype), w2)
    w = torch.exp(-decay_scale * torch.sigmoid(z.float() + w0)).view(-1, H, D)
    a = torch.sigmoid(a + a_bias.view(H, D))
    u = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + unit_eps)
    B = slots.numel()
    cu = (cu_seqlens.tolist() if cu_seqlens is not None
          else list(range(B + 1)))
    for b, slot in enumerate(slots.tolist()):
        S = state[slot]
        if int(starts[b]) == 0:
            S.zero_()
        for t in range(cu[b], cu[b + 1]):
            proj_u = torch.einsum("hk,hkv->hv", u[t], S)
            S.mul_(w[t].unsqueeze(-1))
            S.sub_((a[t] * u[t]).unsqueeze(-1) * proj_u.unsqueeze(1))
            S.add_(k[t].unsqueeze(-1) * v[t].unsqueeze(1))
            o = torch.einsum("hk,hkv->hv", r[t], S)
            o = o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + norm_eps)
            o = o.reshape(-1) * norm_w * torch.sigmoid(g[t].reshape(-1))
            out[t] = o.to(out.dtype)


def rotate(x, rot):
    """x [T, .., dims] by its rows' positions, in f32."""
    half = rot.dims // 2
    cs = rot.table[rot.positions.long()]
    cs = cs.view(cs.shape[0], *[1] * (x.dim() - 2), rot.dims)
    cos, sin = cs[..., :half], cs[..., half:]
    xf = x.float()
    if rot.interleaved:
        u, v = xf[..., ::2], xf[..., 1::2]
        y = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1)
        return y.flatten(-2).to(x.dtype)
    u, v = xf[..., :half], xf[..., half:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin],
                     dim=-1).to(x.dtype)


def latent_store(x, w, cache, slots, eps, rot=None, second=None):
    n = w.numel()
    c = _rms(x[:, :n].float(), w, eps).to(x.dtype)
    if rot is not None:
        c = torch.cat([c, rotate(x[:, n:], rot)], dim=1)
    cache.view(-1, cache.shape[-1])[slots.long()] = c
    if second is None:
        return [c]
    return [c, _rms(second[0].float(), second[1], eps).to(x.dtype)]


def window_attention(q, k, v, gate, out, row_info, scale, window, shared=None,
                     sink=None):
    T, H, _ = q.shape
    if shared is not None:
        k = torch.cat([k, shared.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    for t, (base, pos) in enumerate(row_info.tolist()):
        lo = max(0, pos - window + 1) if window > 0 else 0
        ks = k[base + lo:base + pos + 1].float()
        s = torch.einsum("hd,khd->hk", q[t].float(), ks) * scale
        o = torch.einsum("hk,khd->hd", _softmax(s, sink),
                         v[base + lo:base + pos + 1].float()).reshape(-1)
        if gate is not None:
            o = o * torch.sigmoid(gate[t].float())
        out[t] = o.to(out.dtype)


def _softmax(s, sink):
    """Over the last dim of s [H, keys], with a logit per head that counts in
    the sum alone."""
    if sink is None:
        return torch.softmax(s, dim=-1)
    return torch.softmax(torch.cat([s, sink.view(-1, 1)], dim=-1),
                         dim=-1)[:, :-1]


def latent_decode(q, cache, block_tables, context_lens, scale, window, rank,
                  sink=None):
    S, H, D = q.shape
    out = q.new_empty((S, H, rank))
    ps = cache.shape[1]
    flat = cache.view(-1, D)
    for s in range(S):
        ctx = int(context_lens[s])
        lo = max(0, ctx - window) if window > 0 else 0
        j = torch.arange(lo, ctx)
        c = flat[block_tables[s].long()[j // ps] * ps + j % ps].float()
        p = _softmax(q[s].float() @ c.T * scale, sink)
        out[s] = (p @ c[:, :rank]).to(q.dtype)
    return out


def head_linear(x, w, gate, out):
    y = torch.einsum("shk,hjk->shj", x.float(), w.float())
    if gate is not None:
        y = y * torch.sigmoid(gate.float()).view(y.shape)
    out.copy_(y.to(out.dtype))


# -- sandwich norms, paged attention, sparse experts ---------------------------


def embed_pairs(tokens, prev, table, pairs, mul_prev, mul_cur):
    buckets = pairs.shape[0] - 1
    row = (prev * mul_prev + tokens * mul_cur) % buckets
    row = torch.where(prev < 0, torch.full_like(row, buckets), row)
    return table[tokens].float() + pairs[row].float()


def _rms(x, w, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w


def moe_combine(y, route):
    """f32 sums of each token's weighed expert rows (a pair without a row
    counts nothing)."""
    inv = route.inv.long()
    # rows that no pair has are never written
    rows = y.float()[inv.clamp(min=0)].masked_fill((inv < 0).unsqueeze(1), 0)
    rows = rows.view(-1, route.top, y.shape[1])
    return (rows * route.weights.unsqueeze(-1)).sum(1)


def sandwich_norm(x, rows, route, wb, w, eps, dtype):
    if rows is not None:
        y = rows.float() if route is None else moe_combine(rows, route)
        x += _rms(y, wb, eps)
    return None if w is None else _rms(x, w, eps).to(dtype)


def rope_store_paged(proj, bias, cos_sin, positions, slots, heads, dim, k, v,
                     offs):
    y = proj.float() if bias is None else proj.float() + bias
    half = 0 if cos_sin is None else cos_sin.shape[1] // 2
    if half:
        cs = cos_sin[positions.long()].unsqueeze(1)
        cos, sin = cs[..., :half], cs[..., half:]

    def turn(at, n):
        t = y[:, at:at + n * dim].view(-1, n, dim)
        if not half:
            return t
        a, b = t[..., :half], t[..., half:2 * half]
        return torch.cat([a * cos - b * sin, b * cos + a * sin,
                          t[..., 2 * half:]], dim=-1)
    if half or bias is not None:
        proj[:, offs[0]:offs[0] + heads * dim] = \
            turn(offs[0], heads).flatten(1).to(proj.dtype)
    if len(offs) == 1:
        return
    ps, kvh, vdim = k.shape[2], k.shape[1], v.shape[3]
    pages, at = slots.long() // ps, slots.long() % ps
    k[pages, :, at] = turn(offs[1], kvh).to(k.dtype)
    v[pages, :, at] = y[:, offs[2]:offs[2] + kvh * vdim].view(
        -1, kvh, vdim).to(v.dtype)


def paged_rows(q, k, v, tables, row_info, out, scale, softcap, sink, window=0,
               diff=None):
    """Each row of q [R, H, D] against the keys of its sequence up to its
    position; row_info [R, 2] = (row of tables, position)."""
    ps, kvh = k.shape[2], k.shape[1]
    per, maps = q.shape[1] // kvh, 1 if diff is None else 2
    for r, (seq, pos) in enumerate(row_info.tolist()):
        j = torch.arange(max(0, pos + 1 - window) if window else 0, pos + 1)
        pages, at = tables[seq].long()[j // ps], j % ps
        ks = k[pages, :, at].float().view(len(j), kvh, maps, -1)
        qs = q[r].float().view(kvh, per, maps, -1)
        s = torch.einsum("gpmd,kgmd->gpmk", qs, ks) * scale
        if softcap > 0:
            s = softcap * torch.tanh(s / softcap)
        if sink:                                    # a key without a value
            s = torch.cat([s, torch.zeros_like(s[..., :1])], dim=-1)
        p = torch.softmax(s, dim=-1)[..., :len(j)]
        o = torch.einsum("gpmk,kgd->gpmd", p, v[pages, :, at].float())
        if diff is None:
            o = o[:, :, 0]
        else:
            o = _rms(o[:, :, 0] - diff.lam * o[:, :, 1], diff.scale, diff.eps)
        out[r] = o.reshape(-1).to(out.dtype)


def moe_choose(logits, correction, groups, keep, top, softmax=False,
               share=None):
    """(experts, weights) of each token, [T, top]."""
    T, E = logits.shape
    s = (torch.softmax(logits, dim=-1) if share is not None else
         logits if softmax else torch.sigmoid(logits))
    choice = (s + correction).view(T, groups, E // groups)
    best = choice.topk(min(2, E // groups), dim=-1).values.sum(-1)
    kept = torch.zeros(T, groups, dtype=torch.bool)
    kept.scatter_(1, best.topk(keep, dim=-1).indices, True)
    choice = choice.masked_fill(~kept.unsqueeze(-1), float("-inf"))
    chosen = choice.view(T, E).topk(top, dim=-1)
    if softmax:
        return chosen.indices, torch.softmax(chosen.values, dim=-1)
    w = s.gather(1, chosen.indices)
    if share is not None:
        w = w / (w.sum(-1, keepdim=True) + 1e-20) * share
    return chosen.indices, w


def moe_tiles(ids, experts, tile):
    """Pairs in expert order: (inverse permutation, their tokens, tiles [n, 3]
    = (expert, first row, rows)).  Pairs of experts from ``experts`` on have no
    row: -1."""
    flat = ids.reshape(-1)
    order = torch.sort(flat, stable=True).indices
    inv = torch.empty_like(order)
    inv[order] = torch.arange(order.numel())
    tiles, at = [], 0
    inv[flat >= experts] = -1
    counts = torch.bincount(flat, minlength=experts).tolist()
    for e, n in enumerate(counts[:experts]):
        tiles += [(e, at + i, min(tile, n - i)) for i in range(0, n, tile)]
        at += n
    return (inv.int(), (order // ids.shape[1]).int(),
            torch.tensor(tiles, dtype=torch.int32).view(-1, 3))


def expert_linear(x, w, route, gather, relu2, swiglu=False, limit=None):
    out = x.new_empty((route.rows.numel(), w.shape[1] // (2 if swiglu else 1)))
    for e, at, n in route.tiles.tolist():
        rows = x[route.rows[at:at + n].long()] if gather else x[at:at + n]
        y = rows.float() @ w[e].float().T
        if relu2:
            y = torch.relu(y).pow(2)
        elif swiglu:                    # columns gate, gate, up, up
            y = y.unflatten(1, (-1, 2, 2))
            g, u = y[:, :, 0], y[:, :, 1]
            y = (torch.nn.functional.silu(g) * u if limit is None else
                 clamped_glu_act(g, u, limit)).flatten(1)
        out[at:at + n] = y.to(x.dtype)
    return out


# -- hyper-connections -----------------------------------------------------------


def hyper_norm(x, streams, stir, read, norm, dtype):
    xs = x.view(x.shape[0], streams, -1)
    if stir is not None:
        y = 0.0 if stir.rows is None else stir.rows.float()
        if stir.route is not None:
            if stir.experts is not None:
                y = y + moe_combine(stir.experts, stir.route)
            if stir.self_rows is not None:
                none = (stir.route.inv < 0).view(-1, stir.route.top)
                y = y + (stir.route.weights * none).sum(
                    1, keepdim=True) * stir.self_rows.float()
        mix = stir.conn[:streams * streams].view(streams, streams)
        out = stir.conn[streams * streams:] * stir.mult
        new = torch.einsum("st,nsw->ntw", mix, xs)
        xs.copy_(new + out.view(1, -1, 1) * y.unsqueeze(1))
    if norm is None:
        return None
    u = torch.einsum("s,nsw->nw", read, xs)
    return (torch.tanh(norm.alpha * u) * norm.w + norm.b).to(dtype)


# -- gated branches, gated delta rule -------------------------------------------


def gate_norm(x, branches, w, eps, dtype):
    for b in branches:
        y = b.rows.float() if b.route is None else moe_combine(b.rows, b.route)
        if b.bias is not None:
            y = y + b.bias
        x += y * b.scale * torch.sigmoid(b.logits.float() + b.gate_bias)
    return None if w is None else _rms(x, w, eps).to(dtype)


def silu_glu(gate, up, gate_bias, up_bias, out):
    g, u = gate.float(), up.float()
    if gate_bias is not None:
        g, u = g + gate_bias, u + up_bias
    out.copy_((torch.nn.functional.silu(g) * u).to(out.dtype))


def short_conv(x, conv_w, ring, cu_seqlens, starts, slots):
    taps = conv_w.shape[0]
    out = x.new_empty(x.shape)
    cu = cu_seqlens.tolist()
    for b, slot in enumerate(slots.tolist()):
        start, rows = int(starts[b]), x[cu[b]:cu[b + 1]].float()
        hist = [ring[slot, p % taps].float() if p >= 0 else
                torch.zeros_like(conv_w[0])
                for p in range(start - taps + 1, start)]
        ext = torch.cat([torch.stack(hist), rows]) if hist else rows
        y = sum(conv_w[j] * ext[j:j + rows.shape[0]] for j in range(taps))
        out[cu[b]:cu[b + 1]] = torch.nn.functional.silu(y).to(x.dtype)
        for t in range(max(0, rows.shape[0] - taps + 1), rows.shape[0]):
            ring[slot, (start + t) % taps] = rows[t].to(ring.dtype)
    return out


def gated_delta(p, qkv, offs, beta, decay, gate, state, slots, cu_seqlens,
                starts, out):
    H, D, E = state.shape[1:]
    G = p.kv_heads

    def heads(at, n, size):
        return qkv[:, at:at + n * size].float().view(-1, n, size)

    def unit(t):
        t = t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) + p.unit_eps)
        return t.repeat_interleave(H // G, dim=1)
    q = unit(heads(offs[0], G, D)) * p.q_scale
    k = unit(heads(offs[1], G, D))
    v = heads(offs[2], H, E)
    per = p.dt_bias.numel() // H        # 1, or D
    rate = torch.exp(p.a_log).view(H, 1)
    g = torch.exp(-rate * torch.nn.functional.softplus(
        decay.float() + p.dt_bias, threshold=30).view(-1, H, per))
    beta = torch.sigmoid(beta.float()).unsqueeze(-1)
    z = gate.float()
    z = torch.nn.functional.silu(z) if p.silu else torch.sigmoid(z)
    cu = (cu_seqlens.tolist() if cu_seqlens is not None
          else list(range(slots.numel() + 1)))
    for b, slot in enumerate(slots.tolist()):
        S = state[slot]
        if int(starts[b]) == 0:
            S.zero_()
        for t in range(cu[b], cu[b + 1]):
            S.mul_(g[t].unsqueeze(-1))
            u = beta[t] * (v[t] - torch.einsum("hkv,hk->hv", S, k[t]))
            S.add_(k[t].unsqueeze(-1) * u.unsqueeze(1))
            o = _rms(torch.einsum("hkv,hk->hv", S, q[t]), p.norm, p.norm_eps)
            out[t] = (o.reshape(-1) * z[t]).to(out.dtype)
