"""Danipel's mechanisms one by one against the plain oracle: on the CPU the
reference path, on the GPU (marked) every HIP kernel in f32 and bf16, at sizes
that take the vector, the matrix-core and the any-size forms."""
import math

import pytest
import torch

import rbg_amd.ops as ops
from rbg_amd.models.rotary import rotary_table, rotation
from tests import danipel_oracle as oracle
from tests.test_bitatar_ops import (BF16, F32, WHERE, close, i32, layout, put,
                                    rnd, seen)

PLAIN = {"dims": 12, "base": 900.0}
YARN = {"dims": 32, "base": 1e4,
        "scaling": {"factor": 6.0, "original": 300, "fast": 8.0, "slow": 1.0}}
STEEP = {"dims": 6, "base": 50.0,       # the ramp's ends meet the clamps
         "scaling": {"factor": 3.0, "original": 20, "fast": 90.0,
                     "slow": 0.01}}


# -- streams -----------------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W,copies", [(40, 3), (33, 1), (33, 5)])
def test_embed_into_every_stream(where, W, copies):
    table = rnd(19, W)
    tok = torch.tensor([3, 18, 0, 3], device=where[0])
    x = ops.embed_stream(tok, put(table, where), 0.7, copies)
    assert x.dtype == F32 and x.shape == (4, copies * W)
    want = seen(table, where)[tok.cpu()] * 0.7
    for c in range(copies):
        close(x[:, c * W:(c + 1) * W], want, where, 1e-6)


def tanh_norm(W, where, seed=3):
    alpha, w, b = torch.tensor([0.8]), rnd(W, seed=seed), rnd(W, seed=seed + 1)
    own = [t.float().double() for t in (alpha, w, b)]
    return ops.TanhNorm(*(put(t, where, F32) for t in (alpha, w, b))), \
        lambda u: oracle.tanh_norm(u, *own)


def route_of(T, E, top, identity, where, seed=5):
    return ops.moe_route(put(rnd(T, E, seed=seed, scale=2.0), where, F32),
                         put(rnd(E, seed=seed + 1, scale=0.1), where, F32), 1,
                         1, top, 16, share=1.3, identity=identity)


def weighed(route, y, h):
    """Expert rows by routing; h for pairs without a row."""
    out = torch.zeros_like(h)
    inv = route.inv.cpu().view(-1, route.top).tolist()
    for t, row in enumerate(inv):
        for k, at in enumerate(row):
            out[t] += route.weights[t, k].double().cpu() * (
                h[t] if at < 0 else y[at])
    return out


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("S,W,T", [(1, 48, 5), (2, 256, 3), (3, 37, 5),
                                   (3, 104, 7), (4, 2048, 3), (5, 40, 4),
                                   (9, 33, 3), (4, 1024, 2100)])
def test_hyper_norm(where, S, W, T):
    """What is pending reaches every stream from the old ones, mix[from, to];
    then a norm of what is read, with and without either."""
    mult, read = 0.45, rnd(S, seed=1)
    mix, out = rnd(S, S, seed=2), rnd(S, seed=7)
    norm, norm_of = tanh_norm(W, where)
    x = rnd(T, S * W, seed=8)
    xs = put(x, where, F32)
    rd = put(read, where, F32)
    want = x.float().double().view(T, S, W).transpose(0, 1)
    read, mix, out = (t.float().double() for t in (read, mix, out))
    h = ops.hyper_norm(xs, S, None, rd, norm, where[1])
    assert h.dtype == where[1]
    close(h, norm_of(oracle.gather(want, read)), where)
    y = rnd(T, W, seed=9)
    conn = put(torch.cat([mix.reshape(-1), out]), where, F32)
    stir = ops.Stir(conn, mult, put(y, where))
    h = ops.hyper_norm(xs, S, stir, rd, norm, where[1])
    want = oracle.scatter(want, mix, out, seen(y, where), mult)
    close(xs.view(T, S, W).transpose(0, 1), want, where, 2e-6)
    close(h, norm_of(oracle.gather(want, read)), where)
    assert ops.hyper_norm(xs, S, stir, None, None, where[1]) is None
    want = oracle.scatter(want, mix, out, seen(y, where), mult)
    close(xs.view(T, S, W).transpose(0, 1), want, where, 3e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("S,W,top,identity", [
    (3, 64, 3, 2), (2, 35, 1, 5), (4, 2048, 6, 1), (6, 24, 2, 3), (1, 40, 2,
                                                                   0)])
def test_experts_into_the_streams(where, S, W, top, identity):
    """Weighed expert rows, the token's own row for experts without weights,
    and a shared expert's rows; each alone too."""
    T, E = 6, 8
    route = route_of(T, E, top, identity, where)
    assert (route.inv >= 0).any() and ((route.inv < 0).any() or not identity)
    y, h, z = rnd(T * top, W, seed=1), rnd(T, W, seed=2), rnd(T, W, seed=3)
    mix, out = rnd(S, S, seed=4), rnd(S, seed=5)
    conn = put(torch.cat([mix.reshape(-1), out]), where, F32)
    mix, out = mix.float().double(), out.float().double()
    norm, norm_of = tanh_norm(W, where)
    read = put(torch.ones(S), where, F32)
    none = torch.zeros(T, W, dtype=torch.float64)
    ys, hs, zs = (seen(t, where) for t in (y, h, z))
    for stir, add in (
            (ops.Stir(conn, 0.5, put(z, where), put(y, where), route,
                      put(h, where)), weighed(route, ys, hs) + zs),
            (ops.Stir(conn, 0.5, None, put(y, where), route, None),
             weighed(route, ys, none)),
            (ops.Stir(conn, 0.5, put(z, where), None, route, put(h, where)),
             weighed(route, torch.zeros_like(ys), hs) + zs)):
        x = rnd(T, S * W, seed=6)
        xs = put(x, where, F32)
        got = ops.hyper_norm(xs, S, stir, read, norm, where[1])
        want = oracle.scatter(
            x.float().double().view(T, S, W).transpose(0, 1), mix, out, add,
            0.5)
        close(xs.view(T, S, W).transpose(0, 1), want, where, 3e-6)
        close(got, norm_of(want.sum(0)), where)
    close(ops.moe_combine(put(y, where), route), weighed(route, ys, none),
          where)


@pytest.mark.parametrize("where", WHERE)
def test_only_experts_without_rows(where):
    """Nothing is read of expert rows that nobody wrote."""
    T, W, S = 3, 40, 2
    route = ops.moe_route(put(torch.tensor([[0.0, 9.0, 8.0]] * T), where, F32),
                          put(torch.zeros(3), where, F32), 1, 1, 2, 16,
                          share=1.0, identity=2)
    assert (route.inv < 0).all()
    y = torch.full((2 * T, W), float("nan"), device=where[0], dtype=where[1])
    h = rnd(T, W)
    x = torch.zeros(T, S * W, device=where[0])
    conn = put(torch.cat([torch.eye(S).reshape(-1), torch.ones(S)]), where,
               F32)
    ops.hyper_norm(x, S, ops.Stir(conn, 1.0, None, y, route, put(h, where)),
                   None, None, where[1])
    close(x, seen(h, where).repeat(1, S), where, 1e-6)
    assert ops.moe_combine(y, route).abs().max() == 0


# -- rotation ----------------------------------------------------------------------


@pytest.mark.parametrize("rot", [PLAIN, YARN, STEEP])
def test_frequencies(rot):
    got, mult = rotation(rot)
    want, m = oracle.frequencies(rot)
    assert mult == pytest.approx(m, rel=1e-12)
    assert got.tolist() == pytest.approx(want, rel=1e-12)
    table = rotary_table(rot, 500, torch.device("cpu"))
    a = torch.outer(torch.arange(500).double(),
                    torch.tensor(want, dtype=torch.float64))
    assert (table[:, :rot["dims"] // 2] - a.cos() * m).abs().max() < 2e-7
    assert (table[:, rot["dims"] // 2:] - a.sin() * m).abs().max() < 2e-7


def rotary(rot, where, positions, interleaved):
    return ops.Rotary(rotary_table(rot, 400, torch.device(where[0])),
                      i32(positions, where), interleaved)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("rot,H,before", [(PLAIN, 3, 5), (YARN, 2, 16),
                                          (STEEP, 1, 0),
                                          ({"dims": 64, "base": 5e5}, 5, 128)])
def test_rotate_rows(where, interleaved, rot, H, before):
    """The last dims of every head, in place, the others untouched."""
    D, T, first = rot["dims"], 9, 290
    x = rnd(T, H, before + D)
    xs = put(x, where)
    keep = xs[..., :before].clone()
    ops.rotate_rows(xs[..., before:], rotary(
        rot, where, list(range(first, first + T)), interleaved))
    want = oracle.rotate(seen(x, where)[..., before:], rot, interleaved, first)
    close(xs[..., before:], want, where)
    assert torch.equal(xs[..., :before], keep)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("rank,rot,q_rank", [(24, YARN, 0), (37, PLAIN, 19),
                                             (512, YARN, 1536), (8, STEEP, 40)])
def test_latent_store_with_a_rotated_part(where, interleaved, rank, rot,
                                          q_rank):
    T, eps = 5, 2e-3                    # an eps that shows
    D, slots = rot["dims"], [17, 40, 16, 63, 31]
    pos = [0, 1, 399, 17, 16]
    seg = -(rank + D) % 8 + rank + D
    y, w = rnd(T, seg + q_rank + -q_rank % 8, scale=0.05), 1 + 0.2 * rnd(rank)
    w2 = 1 + 0.2 * rnd(q_rank, seed=3)
    cache = torch.zeros(4, 16, rank + D, device=where[0], dtype=where[1])
    yd, ys = put(y, where), seen(y, where)
    second = (yd[:, seg:seg + q_rank], put(w2, where, F32)) if q_rank else None
    got = ops.latent_store(yd[:, :rank + D], put(w, where, F32), cache,
                           i32(slots, where), eps,
                           rotary(rot, where, pos, interleaved), second)
    c = got[0] if q_rank else got
    close(c[:, :rank], oracle.rms(ys[:, :rank], eps) * w, where)
    for t, p in enumerate(pos):
        want = oracle.rotate(ys[t:t + 1, rank:rank + D], rot, interleaved, p)
        close(c[t:t + 1, rank:], want, where)
    flat = cache.view(-1, rank + D)
    assert torch.equal(flat[slots], c)
    assert (flat.abs().sum(-1) > 0).sum() == T
    if q_rank:
        close(got[1], oracle.rms(ys[:, seg:seg + q_rank], eps) * w2, where)


# -- attention ---------------------------------------------------------------------


def stand_out(q, k, rows, pick, size=12.0):
    """Makes one key score far above the rest for some query rows."""
    for i in rows:
        key = k[pick(i)]
        q[i] = key * size / (key * key).sum(-1, keepdim=True)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sink", [True, False])
@pytest.mark.parametrize("H,D,D2,DV", [
    (2, 24, 8, 32), (3, 5, 6, 7), (2, 128, 64, 128), (1, 64, 32, 96),
    (1, 200, 56, 256), (4, 32, 16, 32), (2, 16, 12, 24)])
def test_attention_with_a_shared_key_part(where, sink, H, D, D2, DV):
    """Portions cut anywhere over the keys so far.  For some rows a far key, the
    first, or one beside a page's border stands out; for others the sink."""
    n, scale = 150, 0.7
    q, k = rnd(n, H, D + D2, seed=D), rnd(n, H, D, seed=1)
    k2, v = rnd(n, D2, seed=2), rnd(n, H, DV, seed=3)
    full = torch.cat([k, k2.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    for first, pick in ((20, lambda i: 0), (21, lambda i: i // 16 * 16),
                        (22, lambda i: i // 16 * 16 - 1), (23, lambda i: i),
                        (24, lambda i: 3)):
        stand_out(q, full, range(first, n, 10), pick, 12 / scale)
    s = rnd(H, seed=4) + 4.0 if sink else None
    if sink:
        q[25::10] *= 0.05               # only the sink is left of these
    q, k, k2, v = (seen(t, where) for t in (q, k, k2, v))
    full = torch.cat([k, k2.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    want = oracle.causal_attention(q, full, v, scale,
                                   s.float().double() if sink else None)
    want = want.reshape(n, -1)
    at = 0
    # the shared part as the cache has it: behind other columns
    wide = put(torch.cat([torch.zeros(n, 8, dtype=k2.dtype), k2], dim=1),
               where)
    for m in [70, 2, 3, 75]:
        lay = layout([at], [at + m], where)
        out = torch.zeros(m, H * DV, device=where[0], dtype=where[1])
        ops.window_attention(put(q[at:at + m], where),
                             put(k[:at + m], where), put(v[:at + m], where),
                             None, out, lay.window_view(0), scale, 0,
                             wide[:at + m, 8:],
                             put(s, where, F32) if sink else None)
        close(out, want[at:at + m], where)
        at += m


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,D,D2,DV", [(2, 128, 64, 128), (1, 64, 64, 64),
                                       (3, 64, 0, 128), (1, 40, 8, 24)])
def test_long_portions(where, H, D, D2, DV):
    """Several query blocks and many key tiles, after a past that ends inside
    a tile; a key of another tile stands out."""
    n, past, scale = 463, 150, 0.5
    q, k = rnd(n, H, D + D2, seed=D), rnd(n, H, D, seed=1)
    k2, v = rnd(n, max(D2, 8), seed=2)[:, :D2], rnd(n, H, DV, seed=3)
    full = torch.cat([k, k2.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    for first, pick in ((150, lambda i: 0), (151, lambda i: i - 64),
                        (152, lambda i: i // 64 * 64 - 1), (153, lambda i: i),
                        (154, lambda i: i // 64 * 64)):
        stand_out(q, full, range(first, n, 9), pick, 12 / scale)
    s = rnd(H, seed=4) + 2.0
    q, k, k2, v = (seen(t, where) for t in (q, k, k2, v))
    full = torch.cat([k, k2.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    want = oracle.causal_attention(q, full, v, scale, s.float().double())
    lay = layout([past], [n], where)
    out = torch.zeros(n - past, H * DV, device=where[0], dtype=where[1])
    ops.window_attention(put(q[past:], where), put(k, where), put(v, where),
                         None, out, lay.window_view(0), scale, 0,
                         put(k2, where) if D2 else None, put(s, where, F32))
    close(out, want.reshape(n, -1)[past:], where)


@pytest.mark.parametrize("where", WHERE)
def test_attention_batch_with_sinks(where):
    """Unequal prompts together; a sink that takes nearly everything counts
    once for each."""
    H, D, D2, DV, lens = 2, 32, 16, 48, [5, 130, 1, 64]
    q, k = rnd(200, H, D + D2), rnd(200, H, D, seed=1)
    k2, v = rnd(200, D2, seed=2), rnd(200, H, DV, seed=3)
    s = torch.tensor([7.0, -3.0])
    lay = layout([0] * 4, lens, where)
    out = torch.zeros(200, H * DV, device=where[0], dtype=where[1])
    ops.window_attention(put(q, where), put(k, where), put(v, where), None,
                         out, lay.window_view(0), 0.3, 0, put(k2, where),
                         put(s, where, F32))
    q, k, k2, v = (seen(t, where) for t in (q, k, k2, v))
    full = torch.cat([k, k2.unsqueeze(1).expand(-1, H, -1)], dim=-1)
    at = 0
    for n in lens:
        r = slice(at, at + n)
        want = oracle.causal_attention(q[r], full[r], v[r], 0.3, s.double())
        close(out[r], want.reshape(n, -1), where)
        at += n


def paged(cache, ctxs, where, ps):
    pages = torch.randperm(cache.shape[0] - 1,
                           generator=torch.Generator().manual_seed(3))
    tables, at = [], 0
    for c in ctxs:
        n = (c + ps - 1) // ps
        tables.append((pages[at:at + n] + 1).tolist())
        at += n
    width = max(len(t) for t in tables)
    return tables, i32([t + [0] * (width - len(t)) for t in tables], where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sink", [True, False])
@pytest.mark.parametrize("H,rank,D2", [
    (3, 24, 8), (17, 64, 16), (2, 37, 6), (16, 136, 64), (5, 256, 64),
    (17, 512, 64), (4, 96, 16), (2, 64, 200), (1, 512, 128)])
def test_latent_decode_with_a_rotated_part(where, sink, H, rank, D2):
    """Shuffled pages, contexts around page borders; the first key, the last
    or one at a page's border stands out, or the sink does."""
    ps, D = 16, rank + D2
    scale = 1.0 / math.sqrt(D)
    ctxs = [1, 15, 16, 17, 40, 161, 250, 251]
    cache = rnd(70, ps, D, seed=rank)
    cache[0] = 0
    tables, bt = paged(cache, ctxs, where, ps)
    q = rnd(len(ctxs), H, D, seed=1)
    for b, (t, c, far) in enumerate(zip(tables, ctxs, [0, 0, 15, 16, 15, 0,
                                                       249, 31])):
        key = cache[t].reshape(-1, D)[far]
        q[b] = key * 14 / scale / (key * key).sum()
    s = rnd(H, seed=4) + 12.0 if sink else None
    q, cache = seen(q, where), seen(cache, where)
    o = ops.latent_decode(put(q, where), put(cache, where), bt,
                          i32(ctxs, where), scale, 0, rank,
                          put(s, where, F32) if sink else None)
    assert o.shape == (len(ctxs), H, rank)
    for b, c in enumerate(ctxs):
        keys = cache[tables[b]].reshape(-1, D)[:c]
        # the last row of the causal form; earlier queries do not matter
        rows = torch.cat([torch.zeros(c - 1, H, D, dtype=q.dtype), q[b:b + 1]])
        want = oracle.causal_attention(
            rows, keys.unsqueeze(1).expand(-1, H, -1),
            keys[:, :rank].unsqueeze(1).expand(-1, H, -1), scale,
            s.float().double() if sink else None)[-1]
        close(o[b], want, where)


@pytest.mark.gpu
@pytest.mark.parametrize("splits", [1, 2, 3, 64])
def test_a_sink_counts_once_over_splits(splits):
    where = ("cuda", BF16)
    H, rank, D2, ps = 4, 64, 32, 16
    D = rank + D2
    cache = seen(rnd(30, ps, D), where)
    q = seen(rnd(2, H, D, seed=1), where)
    s = torch.tensor([3.0, 6.0, -2.0, 0.0])
    bt = i32([list(range(1, 11)), list(range(11, 21))], where)
    o = ops._require_latent().latent_decode(
        put(q, where), put(cache, where), bt, i32([150, 3], where), 0.1, 0,
        splits, rank, put(s, where, F32))
    for b, c in enumerate([150, 3]):
        keys = cache[1 + 10 * b:11 + 10 * b].reshape(-1, D)[:c]
        x = torch.cat([q[b] @ keys.T * 0.1, s.double().view(-1, 1)], dim=1)
        close(o[b], torch.softmax(x, dim=-1)[:, :-1] @ keys[:, :rank], where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("S,H,n,k,rot", [
    (1, 2, 24, 40, PLAIN), (5, 3, 17, 33, STEEP), (20, 2, 130, 64, YARN),
    (70, 1, 64, 128, YARN), (33, 2, 48, 16, PLAIN)])
def test_absorbed_query_with_its_rotated_part(where, interleaved, S, H, n, k,
                                              rot):
    """A head's mapped columns, then its rotated ones, from one query."""
    D = rot["dims"]
    q, w = rnd(S, H, k + D), rnd(H, n, k, seed=1, scale=1 / math.sqrt(k))
    qd, qs = put(q, where), seen(q, where)
    pos = [(7 * i) % 390 for i in range(S)]
    got = ops.head_linear(qd[..., :k], put(w, where), tail=qd[..., k:],
                          rot=rotary(rot, where, pos, interleaved))
    assert got.shape == (S, H, n + D)
    want = torch.einsum("shk,hjk->shj", qs[..., :k], seen(w, where))
    close(got[..., :n], want, where)
    for s, p in enumerate(pos):
        close(got[s:s + 1, :, n:],
              oracle.rotate(qs[s:s + 1, :, k:], rot, interleaved, p), where)


# -- feed-forwards -----------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("F", [40, 33])
@pytest.mark.parametrize("limit", [0.5, 2.0])
def test_clamped_glu(where, F, limit):
    seg = F + -F % 8
    y = rnd(6, 2 * seg + 8, scale=2.0)          # many beyond the limits
    yd, ys = put(y, where), seen(y, where)
    out = torch.zeros(6, F, device=where[0], dtype=where[1])
    ops.clamped_glu(yd[:, 8:8 + F], yd[:, 8 + seg:8 + seg + F], limit, out)
    close(out, oracle.clamped_glu(ys[:, 8:8 + F],
                                  ys[:, 8 + seg:8 + seg + F], limit), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("F", [40, 33])
def test_gelu_glu(where, F):
    x = rnd(6, 2 * F, scale=2.0)
    out = torch.zeros(6, F, device=where[0], dtype=where[1])
    ops.gelu_mul(put(x, where), out)
    xs = seen(x, where)
    close(out, oracle.gelu_tanh(xs[:, :F]) * xs[:, F:], where)


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("T,E,identity,top,tile", [
    (1, 6, 2, 2, 16), (3, 3, 1, 3, 16), (9, 12, 4, 3, 16), (40, 72, 8, 6, 16),
    (700, 20, 5, 4, 32), (5, 4, 0, 1, 16), (70, 9, 8, 5, 64)])
def test_route_by_shares(where, T, E, identity, top, tile):
    """Choice by corrected scores, weights without the correction; experts
    without weights get no rows."""
    logits = rnd(T, E, seed=E + T, scale=1.5).float()
    corr = rnd(E, seed=2, scale=0.1).float()
    r = ops.moe_route(put(logits, where, F32), put(corr, where, F32), 1, 1,
                      top, tile, share=1.7, identity=identity)
    inv = r.inv.cpu().view(T, top).tolist()
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    owner = {}
    for e, at, m in r.tiles[:n].cpu().tolist():
        assert 0 < m <= tile and e < E - identity
        for i in range(at, at + m):
            assert i not in owner
            owner[i] = e
    rows = r.rows.cpu().tolist()
    placed = sorted(i for row in inv for i in row if i >= 0)
    assert placed == sorted(owner) == list(range(len(owner)))
    for t in range(T):
        want = oracle.route(logits[t].double(), corr.double(), top, 1.7)
        got = {owner[i]: w for i, w in zip(inv[t], r.weights[t].tolist())
               if i >= 0}
        assert sorted(got) == sorted(e for e, _ in want if e < E - identity)
        for e, w in want:
            if e < E - identity:
                assert got[e] == pytest.approx(w.item(), rel=2e-5)
        rest = sum(w for i, w in zip(inv[t], r.weights[t].tolist()) if i < 0)
        assert rest == pytest.approx(
            sum(w.item() for e, w in want if e >= E - identity), rel=2e-5)
        assert all(rows[i] == t for i in inv[t] if i >= 0)


@pytest.mark.gpu
def test_route_by_shares_whatever_the_scores():
    """Equal scores, infinities and NaNs still fill every place once."""
    where = ("cuda", F32)
    T, E, identity, top = 70, 24, 6, 4
    logits = torch.zeros(T, E)
    logits[1] = float("nan")
    logits[2, ::2] = float("inf")
    logits[3] = -float("inf")
    for n in (3, 10, T):
        r = ops.moe_route(put(logits[:n], where), put(torch.zeros(E), where),
                          1, 1, top, 16, share=1.0, identity=identity)
        placed = [i for i in r.inv.tolist() if i >= 0]
        assert sorted(placed) == list(range(len(placed)))
        tiles = r.tiles[:int(r.count)].tolist()
        assert sum(m for _, _, m in tiles) == len(placed)
        assert all(0 <= e < E - identity for e, _, _ in tiles)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("T,E,identity,top,F,K,tile", [
    (7, 5, 2, 2, 24, 40, 16), (3, 4, 1, 3, 14, 33, 16), (40, 5, 1, 2, 48, 64,
                                                         32),
    (90, 6, 2, 2, 40, 72, 64), (200, 5, 2, 3, 96, 136, 128)])
def test_clamped_experts(where, T, E, identity, top, F, K, tile):
    if tile > 16 and (where[1] == F32 or 2 * F % 8 or K % 8):
        pytest.skip("these sizes have one form")
    real, limit = E - identity, 0.8
    r = ops.moe_route(put(rnd(T, E, seed=3, scale=2.0), where, F32),
                      put(torch.zeros(E), where, F32), 1, 1, top, tile,
                      share=1.0, identity=identity)
    x = rnd(T, K)
    gate, up = (rnd(real, F, K, seed=s, scale=2 / math.sqrt(K))
                for s in (1, 2))
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    h = ops.expert_linear(put(x, where), put(ops.interleave_glu(gate, up),
                                             where), r, gather=True,
                          swiglu=True, limit=limit)
    assert h.shape == (T * top, F)
    g, u, xs = seen(gate, where), seen(up, where), seen(x, where)
    rows, got, want = r.rows.cpu().tolist(), [], []
    for e, at, m in r.tiles[:n].cpu().tolist():
        got.append(h[at:at + m])
        t = xs[rows[at:at + m]]
        want.append(oracle.clamped_glu(t @ g[e].T, t @ u[e].T, limit))
    close(torch.cat(got), torch.cat(want), where)
