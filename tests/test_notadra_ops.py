"""Notadra's mechanisms one by one against the plain oracle: on the CPU the
reference path, on the GPU (marked) every HIP kernel in f32 and bf16, at sizes
that take the vector, the matrix-core and the any-size forms."""
import math

import pytest
import torch

import rbg_amd.ops as ops
from rbg_amd.models.rotary import rotary_table, rotation
from tests import notadra_oracle as oracle
from tests.test_bitatar_ops import (BF16, F32, WHERE, Table, close, i32,
                                    layout, put, rnd, seen)


def score_of(q, k, v, scale, softcap):
    return oracle.sink_attention(q, k, v, scale, softcap)


# -- embedding and norms -------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width", [40, 33])
def test_embed_pairs(where, width):
    cfg = {"buckets": 23, "mul_prev": 1000003, "mul_cur": 17}
    table, pairs = rnd(61, width), rnd(24, width, seed=1)
    toks = [60, 0, 60, 60, 7]
    tok = torch.tensor(toks, device=where[0])
    prev = torch.tensor([-1] + toks[:-1], device=where[0])
    x = ops.embed_pairs(tok, prev, put(table, where), put(pairs, where),
                        cfg["mul_prev"], cfg["mul_cur"])
    assert x.dtype == F32
    want = oracle.embedding(toks, seen(table, where), seen(pairs, where), cfg)
    close(x, want, where, 1e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width", [48, 256, 2056, 5120, 37, 1030])
def test_sandwich_norm(where, width):
    T, eps = 5, 3e-3                    # an eps that shows
    x, y = rnd(T, width, seed=1, scale=0.1), rnd(T, width, seed=2, scale=0.1)
    wb, w = 0.3 * rnd(width, seed=3), 0.3 * rnd(width, seed=4)
    xs = put(x, where, F32)
    b1, w1 = put(1 + wb, where, F32), put(1 + w, where, F32)
    h = ops.sandwich_norm(xs, (put(y, where), None, b1), w1, eps, where[1])
    want = x.float().double() + oracle.norm(seen(y, where), wb, eps)
    close(xs, want, where, 2e-6)        # the stream is f32 in every mode
    assert h.dtype == where[1]
    close(h, oracle.norm(want, w, eps), where)
    # nothing pending; and no second norm
    h2 = ops.sandwich_norm(xs, None, w1, eps, where[1])
    close(xs, want, where, 2e-6)
    close(h2, oracle.norm(want, w, eps), where)
    assert ops.sandwich_norm(xs, (put(y, where), None, b1), None, eps,
                             where[1]) is None
    close(xs, want + oracle.norm(seen(y, where), wb, eps), where, 2e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width,top", [(64, 3), (35, 1), (2048, 8)])
def test_weighed_experts_in_the_norm(where, width, top):
    T, E, eps = 6, 12, 1e-4
    logits = rnd(T, E, seed=5, scale=2.0).float()
    route = ops.moe_route(put(logits, where, F32),
                          put(rnd(E, seed=6), where, F32), 3, 2, top, 16)
    y = rnd(T * top, width, seed=7)
    yd = put(y, where)
    picked = seen(y, where)[route.inv.cpu().long()].view(T, top, width)
    total = (picked * route.weights.double().cpu().unsqueeze(-1)).sum(1)
    close(ops.moe_combine(yd, route), total, where)
    x, wb, w = (rnd(*s, seed=8 + i) for i, s in enumerate(
        [(T, width), (width,), (width,)]))
    xs = put(x, where, F32)
    h = ops.sandwich_norm(xs, (yd, route, put(1 + wb, where, F32)),
                          put(1 + w, where, F32), eps, where[1])
    want = x.float().double() + oracle.norm(total, wb, eps)
    close(xs, want, where, 2e-6)
    close(h, oracle.norm(want, w, eps), where)


# -- rotary positions ------------------------------------------------------------

ROTS = [
    {"dims": 8, "base": 1000.0, "scaling": {"factor": 4.0, "original": 64,
                                            "fast": 8.0, "slow": 1.0}},
    # the ramp's ends meet, and both clamps
    {"dims": 16, "base": 10.0, "scaling": {"factor": 2.5, "original": 4096,
                                           "fast": 700.0, "slow": 690.0}},
    {"dims": 64, "base": 5e5, "scaling": {"factor": 40.0, "original": 32,
                                          "fast": 32.0, "slow": 0.01}},
    {"dims": 2, "base": 7.0, "scaling": {"factor": 1.0, "original": 10,
                                         "fast": 4.0, "slow": 1.0}},
    {"dims": 12, "base": 1e4}]


@pytest.mark.parametrize("rot", ROTS)
def test_rotary_table(rot):
    freqs, mult = oracle.frequencies(rot)
    f, m = rotation(rot)
    assert m == pytest.approx(mult) and len(f) == len(freqs)
    assert torch.allclose(f, torch.tensor(freqs, dtype=torch.float64))
    table = rotary_table(rot, 5000, torch.device("cpu"))
    for p in (0, 1, 77, 4999):
        for i, fr in enumerate(freqs):
            assert table[p, i].item() == pytest.approx(
                math.cos(p * fr) * mult, abs=1e-6)
            assert table[p, len(freqs) + i].item() == pytest.approx(
                math.sin(p * fr) * mult, abs=1e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,DV,dims", [
    (4, 2, 32, 16, 16), (2, 1, 64, 80, 64), (3, 3, 24, 8, 16),
    (2, 2, 10, 7, 6), (6, 2, 16, 24, 8)])
@pytest.mark.parametrize("own", [True, False])
def test_rope_store(where, H, G, D, DV, dims, own):
    """Biases, partial rotation and the paged store; every other row of the
    pages stays as it was.  Without keys of its own a layer stores nothing."""
    T, ps, first = 5, 16, 13
    rot = dict(ROTS[0], dims=dims)
    sizes = [H * D] + ([G * D, G * DV] if own else [])
    offs, at = [], 0
    for n in sizes:
        offs.append(at)
        at += n + -n % 8
    y, bias = rnd(T, at), rnd(at, seed=1)
    k = torch.full((4, G, ps, D), 9.0, device=where[0], dtype=where[1])
    v = torch.full((4, G, ps, DV), 9.0, device=where[0], dtype=where[1])
    slots = [17, 40, 16, 63, 31]
    pos = list(range(first, first + T))
    yd = put(y, where)
    table = rotary_table(rot, 64, torch.device(where[0]))
    ops.rope_store_paged(yd, put(bias, where, F32), table, i32(pos, where),
                         i32(slots, where), H, D, k, v, offs)
    want = seen(y, where) + bias.float().double()
    q = oracle.rotate(want[:, :H * D].view(T, H, D), rot, first)
    close(yd[:, :H * D], q.reshape(T, -1), where)
    kept = [s for s in range(64) if not own or s not in slots]
    flat_k, flat_v = (t.permute(0, 2, 1, 3).reshape(64, G, -1) for t in (k, v))
    assert (flat_k[kept] == 9.0).all() and (flat_v[kept] == 9.0).all()
    if own:
        wk = want[:, offs[1]:offs[1] + G * D].view(T, G, D)
        close(flat_k[slots], oracle.rotate(wk, rot, first), where)
        close(flat_v[slots],
              want[:, offs[2]:offs[2] + G * DV].view(T, G, DV), where)


# -- attention -----------------------------------------------------------------

#            H   G   D    DV
ATTN_SIZES = [(4, 2, 32, 32), (3, 3, 8, 16), (8, 1, 64, 80), (2, 2, 128, 128),
              (20, 1, 64, 96), (2, 1, 256, 256), (4, 4, 96, 40),
              (2, 1, 20, 36), (34, 2, 16, 8)]


def pages_of(k, v, where, lens, page_size=16, seed=3):
    """Keys and values [tokens, G, .] of several sequences in shuffled pages
    whose other rows are poisoned; (k pages, v pages, tables)."""
    n = [(t + page_size - 1) // page_size for t in lens]
    order = (torch.randperm(sum(n) + 3, generator=torch.Generator()
                            .manual_seed(seed)) + 1).tolist()
    kp = torch.full((sum(n) + 4, k.shape[1], page_size, k.shape[2]), 3e4,
                    dtype=torch.float64)
    vp = torch.full((sum(n) + 4, v.shape[1], page_size, v.shape[2]), 3e4,
                    dtype=torch.float64)
    tables, at = [], 0
    for t, m in zip(lens, n):
        pages, order = order[:m], order[m:]
        tables.append(Table(pages))
        for i in range(t):
            kp[pages[i // page_size], :, i % page_size] = k[at + i]
            vp[pages[i // page_size], :, i % page_size] = v[at + i]
        at += t
    return put(kp, where), put(vp, where), tables


def attn_case(H, G, D, DV, n, scale, seed=0):
    """Every seventh query singles one key out, far back or at a page's edge;
    others find no key at all, and the sink takes them."""
    q, k, v = rnd(n, H, D, seed=seed), rnd(n, G, D, seed=seed + 1), \
        rnd(n, G, DV, seed=seed + 2)
    for i in range(0, n, 7):
        j = [0, i // 2, i, max(0, i - 1), i // 16 * 16,
             max(0, i // 16 * 16 - 1)][i // 7 % 6]
        for h in range(H):
            key = k[j, h // (H // G)]
            q[i, h] = key * 14 / scale / (key * key).sum()
    mean = k.mean(1)
    for i in range(3, n, 7):
        q[i] = -mean[max(0, i - 1)] * 9 / scale / \
            (mean[max(0, i - 1)] ** 2).sum()
    return q, k, v


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,DV", ATTN_SIZES)
@pytest.mark.parametrize("softcap", [6.0, 50.0, 300.0])
def test_paged_prefill_portions(where, H, G, D, DV, softcap):
    """Portions cut anywhere, over keys in shuffled pages."""
    n, scale = 150, 0.7 / math.sqrt(D)
    q, k, v = (seen(t, where) for t in attn_case(H, G, D, DV, n, scale, D))
    want = score_of(q, k, v, scale, softcap).reshape(n, -1)
    kp, vp, tables = pages_of(k, v, where, [n])
    at = 0
    for m in [70, 2, 3, 75]:
        lay = layout([at], [at + m], where, tables=tables)
        buf = torch.zeros(m, H * DV + 8, device=where[0], dtype=where[1])
        # rows of q are a slice of something wider
        qd = put(torch.nn.functional.pad(q[at:at + m].reshape(m, -1), (0, 8)),
                 where)[:, :H * D].unflatten(1, (H, D))
        ops.paged_prefill(qd, kp, vp, lay.paged_view(), buf[:, :H * DV], scale,
                          softcap, True)
        close(buf[:, :H * DV], want[at:at + m], where)
        assert (buf[:, H * DV:] == 0).all()
        at += m


@pytest.mark.parametrize("where", WHERE)
def test_paged_prefill_batch_after_decode_rows(where):
    """Unequal sequences in one launch; the layout skips the decode rows."""
    H, G, D, DV, scale, cap = 4, 2, 32, 48, 0.2, 9.0
    starts, ends = [7, 0, 40, 15], [8, 130, 42, 64]
    parts = [attn_case(H, G, D, DV, e, scale, seed=e) for e in ends]
    parts = [tuple(seen(t, where) for t in p) for p in parts]
    kp, vp, tables = pages_of(torch.cat([p[1] for p in parts]),
                              torch.cat([p[2] for p in parts]), where, ends)
    lay = layout(starts, ends, where, num_decode=1, tables=tables)
    q = torch.cat([p[0][s:] for p, s in zip(parts[1:], starts[1:])])
    out = torch.zeros(q.shape[0], H * DV, device=where[0], dtype=where[1])
    ops.paged_prefill(put(q, where), kp, vp, lay.paged_view(), out, scale, cap,
                      True)
    at = 0
    for (qs, ks, vs), s in zip(parts[1:], starts[1:]):
        want = score_of(qs, ks, vs, scale, cap)[s:]
        close(out[at:at + len(want)], want.flatten(1), where)
        at += len(want)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,DV", ATTN_SIZES)
def test_paged_decode(where, H, G, D, DV):
    """Contexts around page and step borders, the last rows of pages
    poisoned."""
    scale = 0.7 / math.sqrt(D)
    ctxs = [1, 15, 16, 17, 31, 32, 33, 127, 128, 129, 161, 290]
    parts = [tuple(seen(t, where)
                   for t in attn_case(H, G, D, DV, c, scale, seed=c))
             for c in ctxs]
    kp, vp, tables = pages_of(torch.cat([p[1] for p in parts]),
                              torch.cat([p[2] for p in parts]), where, ctxs)
    wide = max(len(t.pages) for t in tables)
    bt = i32([t.pages + [0] * (wide - len(t.pages)) for t in tables], where)
    picks = [(c - 1) // 7 * 7 for c in ctxs]    # a query with a key of its own
    q = torch.stack([p[0][i] for p, i in zip(parts, picks)])
    for splits, cap in ((0, 12.0), (1, 50.0), (3, 300.0)):
        out = torch.zeros(len(ctxs), H * DV, device=where[0], dtype=where[1])
        ops.paged_decode(put(q, where), kp, vp, bt, i32(ctxs, where), out,
                         scale, cap, True, splits)
        for b, (c, i) in enumerate(zip(ctxs, picks)):
            qs = torch.zeros(c, H, D, dtype=torch.float64)
            qs[c - 1] = parts[b][0][i]
            want = score_of(qs, parts[b][1], parts[b][2], scale, cap)[-1]
            close(out[b], want.flatten(), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sink,cap", [(False, 0.0), (True, 0.0), (False, 5.0)])
def test_score_options_and_page_sizes(where, sink, cap):
    """Without a cap, without a sink; larger pages, and pages that the
    matrix-core forms do not take."""
    H, G, D, DV, n, scale = 4, 2, 32, 32, 70, 0.3
    q, k, v = (seen(t, where) for t in attn_case(H, G, D, DV, n, scale))
    want = torch.zeros(n, H, DV, dtype=torch.float64)
    for i in range(n):
        for h in range(H):
            s = k[:i + 1, h // 2] @ q[i, h] * scale
            s = cap * torch.tanh(s / cap) if cap else s
            m = max(s.max().item(), 0)
            e = torch.exp(s - m)
            want[i, h] = e @ v[:i + 1, h // 2] / (
                e.sum() + (math.exp(-m) if sink else 0))
    for ps in (16, 64, 24):
        kp, vp, tables = pages_of(k, v, where, [n], page_size=ps)
        lay = layout([0], [n], where, page_size=ps, tables=tables)
        out = torch.zeros(n, H * DV, device=where[0], dtype=where[1])
        ops.paged_prefill(put(q, where), kp, vp, lay.paged_view(), out, scale,
                          cap, sink)
        close(out, want.flatten(1), where)
        one = torch.zeros(1, H * DV, device=where[0], dtype=where[1])
        ops.paged_decode(put(q[n - 1:], where), kp, vp,
                         i32([tables[0].pages], where), i32([n], where), one,
                         scale, cap, sink)
        close(one, want[n - 1:].flatten(1), where)


# -- experts -------------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("T,E,K", [(1, 16, 48), (5, 8, 264), (70, 20, 64),
                                   (600, 33, 128), (3, 7, 37),
                                   (1000, 130, 200)])
def test_router_logits(where, T, E, K):
    x, w = rnd(T, K), rnd(E, K, seed=1)
    out = ops.router_logits(put(x, where), put(w, where))
    assert out.dtype == F32             # and sums in 32-bit
    close(out, seen(x, where) @ seen(w, where).T, where, 3e-6)


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("T,E,count,keep,top", [
    (7, 16, 4, 3, 3), (1, 8, 8, 2, 2), (9, 12, 3, 1, 4), (80, 8, 1, 1, 1),
    (5, 6, 2, 2, 6), (300, 128, 8, 4, 8), (65, 96, 96, 70, 5),
    (40, 520, 4, 2, 3)])
@pytest.mark.parametrize("tile", [16, 128])
def test_route(where, T, E, count, keep, top, tile):
    """Choice and layout.  Corrections of both signs: a left-out group must
    not win against negative choice scores."""
    logits = rnd(T, E, seed=E + T, scale=1.5).float()
    corr = (rnd(E, seed=2, scale=0.5) - 0.9).float()
    r = ops.moe_route(put(logits, where, F32), put(corr, where, F32), count,
                      keep, top, tile)
    spec = {"top": top, "groups": {"count": count, "keep": keep}}
    rows, inv = r.rows.cpu().tolist(), r.inv.cpu().view(T, top).tolist()
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    tiles = r.tiles[:n].cpu().tolist()
    owner = {}
    for e, at, m in tiles:
        assert 0 < m <= tile
        for i in range(at, at + m):
            assert i not in owner
            owner[i] = e
    assert len(owner) == T * top and sorted(sum(inv, [])) == sorted(owner)
    for t in range(T):
        want = oracle.route(logits[t].double(), corr.double(), spec)
        got = {owner[i]: w for i, w in zip(inv[t], r.weights[t].tolist())}
        assert sorted(got) == sorted(e for e, _ in want)
        for e, w in want:
            assert got[e] == pytest.approx(w.item(), rel=1e-5)
        assert all(rows[i] == t for i in inv[t])


@pytest.mark.gpu
def test_route_places_everyone_whatever_the_scores():
    """Equal scores, infinities and NaNs still fill every place once."""
    where = ("cuda", F32)
    T, E, top = 70, 24, 4
    logits = torch.zeros(T, E)
    logits[1] = float("nan")
    logits[2, ::2] = float("inf")
    logits[3] = -float("inf")
    for n in (10, T):
        r = ops.moe_route(put(logits[:n], where), put(torch.zeros(E), where),
                          6, 2, top, 16)
        assert sorted(r.inv.tolist()) == list(range(n * top))
        tiles = r.tiles[:int(r.count)].tolist()
        assert sum(m for _, _, m in tiles) == n * top
        assert all(0 <= e < E for e, _, _ in tiles)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("T,E,top,N,K", [
    (1, 16, 3, 24, 48), (3, 4, 2, 40, 136), (20, 8, 2, 96, 256),
    (150, 4, 2, 136, 72), (400, 4, 3, 264, 200), (5, 6, 2, 13, 21),
    (130, 3, 3, 8, 8)])
@pytest.mark.parametrize("tile", [16, 32, 64, 128])
def test_expert_linear(where, T, E, top, N, K, tile):
    """Gathered rows with the squared relu, then rows in expert order."""
    if tile > 16 and (where[1] == F32 or N % 8 or K % 8):
        pytest.skip("these sizes have one form")
    logits = rnd(T, E, seed=3, scale=3.0).float()
    logits[:, E - 1] -= 2.0             # unequal experts, perhaps an empty one
    r = ops.moe_route(put(logits, where, F32),
                      put(torch.zeros(E), where, F32), 1, 1, top, tile)
    x, up = rnd(T, K), rnd(E, N, K, seed=1, scale=1 / math.sqrt(K))
    down = rnd(E, K, N, seed=2, scale=1 / math.sqrt(N))
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    owner = torch.zeros(T * top, dtype=torch.long)
    for e, at, m in r.tiles[:n].tolist():
        owner[at:at + m] = e
    h = ops.expert_linear(put(x, where), put(up, where), r, gather=True,
                          relu2=True)
    xs = seen(x, where)[r.rows.cpu().long()]
    ups, downs = seen(up, where), seen(down, where)
    want = torch.relu(torch.stack([ups[e] @ v for e, v in zip(owner, xs)])) ** 2
    close(h, want, where)
    y = ops.expert_linear(h, put(down, where), r)
    hs = h.double().cpu()
    close(y, torch.stack([downs[e] @ v for e, v in zip(owner, hs)]), where)


def test_tile_choice():
    w = torch.zeros(64, 32, 32)
    assert ops.expert_tile(torch.zeros(4, 32), w, 8) == 16


@pytest.mark.gpu
def test_tile_choice_by_load():
    w = torch.zeros(64, 256, 32, device="cuda", dtype=BF16)
    x = torch.zeros(8192, 32, device="cuda", dtype=BF16)
    assert ops.expert_tile(x[:1], w, 8) == 16
    assert ops.expert_tile(x[:128], w, 8) == 32
    assert ops.expert_tile(x[:256], w, 8) == 64
    assert ops.expert_tile(x, w, 8) == 128
    assert ops.expert_tile(x.float(), w.float(), 8) == 16
    odd = torch.zeros(64, 31, 32, device="cuda", dtype=BF16)
    assert ops.expert_tile(x, odd, 8) == 16
