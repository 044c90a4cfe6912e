"""Bitatar's mechanisms one by one against the plain oracle: on the CPU the
reference path, on the GPU (marked) every HIP kernel in f32 and bf16, at sizes
that take the vector, the matrix-core and the any-size forms."""
import math

import pytest
import torch

import rbg_amd.ops as ops
from rbg_amd.engine.batch import VarlenLayout
from tests import bitatar_oracle as oracle

GPU = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
WHERE = [pytest.param(("cpu", F32), id="cpu-f32"),
         pytest.param(("cuda", F32), id="gpu-f32", marks=GPU),
         pytest.param(("cuda", BF16), id="gpu-bf16", marks=GPU)]
TOL = {F32: 2e-5, BF16: 2e-2}


def rnd(*shape, seed=0, scale=1.0):
    gen = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=gen, dtype=torch.float64) * scale


def put(x, where, dtype=None):
    return x.to(device=where[0], dtype=dtype or where[1]).contiguous()


def i32(x, where):
    return torch.tensor(x, dtype=torch.int32, device=where[0])


def close(got, want, where, tol=None):
    want = want.double()
    err = (got.double().cpu() - want).abs().max() / want.abs().max()
    assert err.item() < (tol or TOL[where[1]]), err.item()


def seen(x, where):
    """The float64 value of what the kernel will read."""
    return x.to(where[1]).double()


class Table:
    def __init__(self, pages):
        self.pages = pages


def layout(starts, ends, where, page_size=16, num_decode=0, tables=None):
    if tables is None:
        tables, at = [], 1
        for e in ends:
            n = (e + page_size - 1) // page_size
            tables.append(Table(list(range(at, at + n))[::-1]))
            at += n
    return VarlenLayout(starts, ends, tables, num_decode, page_size,
                        torch.device(where[0]))


# -- residual stream ---------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width,groups", [(48, 3), (256, 1), (520, 5),
                                          (42, 7), (1024, 32)])
def test_stream_norm(where, width, groups):
    T, eps = 5, 3e-3                    # an eps that shows
    x, d = rnd(T, width, seed=1, scale=0.1), rnd(T, width, seed=2, scale=0.1)
    w1, w2 = 1 + 0.3 * rnd(width, seed=3), 1 + 0.3 * rnd(width, seed=4)
    xs = put(x, where, F32)
    n1, n2 = ops.stream_norm(xs, put(d, where), put(w1, where, F32),
                             put(w2, where, F32), groups, eps, where[1])
    want = x.float().double() + seen(d, where)
    close(xs, want, where, 1e-6)        # the stream is f32 in every mode
    close(n1, oracle.group_norm(want, w1, groups, eps), where)
    close(n2, oracle.group_norm(want, w2, groups, eps), where)
    n1, n2 = ops.stream_norm(xs, None, put(w1, where, F32), None, groups, eps,
                             where[1])
    assert n2 is None
    close(n1, oracle.group_norm(want, w1, groups, eps), where)


@pytest.mark.parametrize("where", WHERE)
def test_embed_stream(where):
    for width in (40, 33):
        table = rnd(19, width)
        tok = torch.tensor([3, 18, 0, 3], device=where[0])
        x = ops.embed_stream(tok, put(table, where), 5.25)
        assert x.dtype == F32
        close(x, seen(table, where)[tok.cpu()] * 5.25, where, 1e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width,taps", [(64, 4), (50, 2), (32, 7), (16, 1)])
def test_conv_portions_and_decode(where, width, taps):
    """Portions down to one token, then the decode form, on dirty slots."""
    n = [29, 11]
    xs = [seen(rnd(t, width, seed=t), where) for t in n]
    w = rnd(width, taps, seed=9, scale=0.5)
    wt = put(w.T, where, F32)
    want = [oracle.conv_residual(x, w.float().double()) for x in xs]
    state = torch.full((4, taps - 1, width), 7.0, device=where[0],
                       dtype=where[1])
    slots = i32([3, 1], where)
    at = [0, 0]
    for portion in [(17, 2), (1, 1), (2, 3)]:
        ends = [a + p for a, p in zip(at, portion)]
        lay = layout(at, ends, where)
        rows = torch.cat([x[a:e] for x, a, e in zip(xs, at, ends)])
        cu = i32([0, portion[0], sum(portion)], where)
        h = ops.causal_conv(put(rows, where), wt, state,
                            lay.tiles(max(ops.CONV_TILE, taps)), cu,
                            i32(at, where), slots)
        close(h, torch.cat([y[a:e] for y, a, e in zip(want, at, ends)]), where)
        at = ends
    # decode: norm with unit weight and one group, so feed its input
    for _ in range(4):
        x = torch.stack([xs[b][at[b]] for b in range(2)])
        inv = 1 / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-5)
        ones = torch.ones(width, device=where[0])
        stream = put(x, where, F32)
        h, n2 = ops.stream_norm_conv(
            stream, None, ones, ones, 1, 1e-5, where[1], wt, state, slots,
            i32(at, where))
        normed = (x * inv).to(where[1]).double()
        close(n2, normed, where)
        # histories hold earlier inputs: compare against the same sequence
        for b in range(2):
            xs[b][at[b]] = normed[b]
            y = oracle.conv_residual(xs[b][:at[b] + 1], w.float().double())
            close(h[b], y[-1], where)
            at[b] += 1


@pytest.mark.parametrize("where", WHERE)
def test_decode_conv_at_position_zero_ignores_the_slot(where):
    w = rnd(24, 3, seed=1)
    state = torch.full((2, 2, 24), 9.0, device=where[0], dtype=where[1])
    ones = torch.ones(24, device=where[0])
    x = rnd(1, 24, seed=2)
    h, _ = ops.stream_norm_conv(put(x, where, F32), None, ones, None, 1, 1e-5,
                                where[1], put(w.T, where, F32), state,
                                i32([1], where), i32([0], where))
    normed = oracle.rms_norm(x, torch.ones(24).double(), 1e-5)
    close(h, oracle.conv_residual(normed.to(where[1]).double(), w), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("ff,pad", [(40, 8), (33, 3)])
def test_gates(where, ff, pad):
    x = rnd(6, 2 * ff, scale=2.0)
    buf = torch.zeros(6, pad + ff, device=where[0], dtype=where[1])
    ops.gelu_mul(put(x, where), buf[:, pad:])
    xs = seen(x, where)
    close(buf[:, pad:], oracle.gelu_tanh(xs[:, :ff]) * xs[:, ff:], where)
    assert buf[:, :pad].abs().max() == 0
    y = put(x, where)
    close(ops.tanh_rows(y[:, 2:2 + ff]), torch.tanh(xs[:, 2:2 + ff]), where)


# -- delta rule ----------------------------------------------------------------


def delta_case(where, heads, dim, rank, T, seed=0, strong=False):
    """Inputs in a fused projection with gaps, and the oracle's rows."""
    HD = heads * dim
    seg = HD + 8 - HD % 8
    offs = [seg * i for i in range(5)] + [seg * 5]
    proj = rnd(T, seg * 5 + rank + 3, seed=seed)
    proj = torch.nn.functional.pad(proj, (0, -proj.shape[1] % 8))
    w0, ab = rnd(HD, seed=seed + 1), rnd(HD, seed=seed + 2)
    if strong:      # fast decay and full removal: old state must really go
        w0, ab = w0 + 4.0, ab + 4.0
    nw = 1 + 0.2 * rnd(HD, seed=seed + 3)
    w2 = rnd(HD, rank, seed=seed + 4, scale=1 / math.sqrt(rank))
    p = seen(proj, where)
    r, k, v, a, g = (p[:, o:o + HD].reshape(T, heads, dim) for o in offs[:5])
    low = torch.tanh(p[:, offs[5]:offs[5] + rank]).to(where[1]).double()
    z = (low @ seen(w2, where).T)
    w = torch.exp(-math.exp(-0.5) * torch.sigmoid(
        z.view(T, heads, dim) + w0.view(heads, dim)))
    av = torch.sigmoid(a + ab.view(heads, dim))
    return dict(proj=put(proj, where), w2=put(w2, where),
                w0=put(w0, where, F32), ab=put(ab, where, F32),
                nw=put(nw, where, F32), offs=offs, z=z,
                rows=(r, w, k, v, av), g=g.reshape(T, HD), norm=nw)


def delta_want(case, eps):
    o, S = oracle.delta_recurrence(*case["rows"])
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return (o.reshape(o.shape[0], -1) * case["norm"] *
            torch.sigmoid(case["g"])), S


DELTA_SIZES = [(2, 64, 16), (3, 12, 9), (1, 128, 8), (2, 40, 24), (1, 33, 5),
               (1, 160, 8)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("heads,dim,rank", DELTA_SIZES)
@pytest.mark.parametrize("strong", [False, True])
def test_delta_rule_portions(where, heads, dim, rank, strong):
    """Portions of 2..37 tokens through the chunk form, single tokens through
    the step form, on a slot full of somebody else's state."""
    T, eps, HD = 61, 1e-5, heads * dim
    c = delta_case(where, heads, dim, rank, T, seed=dim, strong=strong)
    want, S = delta_want(c, eps)
    state = torch.full((3, heads, dim, dim), 5.0, device=where[0])
    slots = i32([2], where)
    buf = torch.zeros(T, HD + 8, device=where[0], dtype=where[1])
    z16 = put(c["z"], where)
    at = 0
    for n in [37, 1, 2, 1, 5, 15]:
        out = buf[at:at + n, :HD]
        lay = layout([at], [at + n], where)
        chunks = None if n == 1 else (lay.prefill_tiles(ops.DELTA_CHUNK),
                                      lay.prefill_tile_cu(ops.DELTA_CHUNK))
        ops.delta_rule(c["proj"][at:at + n],
                       None if n == 1 else z16[at:at + n], c["w2"], c["w0"],
                       c["ab"], c["nw"], state, slots, i32([0, n], where)
                       if n > 1 else None, i32([at], where), out, c["offs"],
                       math.exp(-0.5), 1e-6, eps, chunks)
        at += n
    assert at == T
    close(buf[:, :HD], want, where)
    # the state is f32 in every mode (its inputs are not)
    close(state[2], S, where, 2e-5 if where[1] == F32 else 1e-2)
    assert (state[1] == 5.0).all()


@pytest.mark.parametrize("where", WHERE)
def test_delta_rule_batch(where):
    """Unequal sequences in one launch, each on its own slot."""
    heads, dim, rank, eps = 2, 24, 8, 1e-5
    lens = [3, 16, 33, 1]
    cases = [delta_case(where, heads, dim, rank, n, seed=40 + n)
             for n in lens]
    # one set of weights: the first case's
    for c, n in zip(cases[1:], lens[1:]):
        d = delta_case(where, heads, dim, rank, n, seed=40 + n)
        r, _, k, v, _ = d["rows"]
        p = d["proj"].double().cpu()
        z = torch.tanh(p[:, c["offs"][5]:c["offs"][5] + rank]).to(
            where[1]).double() @ cases[0]["w2"].double().cpu().T
        w0, ab = (cases[0][x].double().cpu().view(heads, dim)
                  for x in ("w0", "ab"))
        a = p[:, c["offs"][3]:c["offs"][3] + heads * dim].view(n, heads, dim)
        c["rows"] = (r, torch.exp(-math.exp(-0.5) * torch.sigmoid(
            z.view(n, heads, dim) + w0)), k, v, torch.sigmoid(a + ab))
        c["z"], c["norm"] = z, cases[0]["norm"]
    proj = torch.cat([c["proj"] for c in cases])
    z = put(torch.cat([c["z"] for c in cases]), where)
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    lay = layout([0] * 4, lens, where)
    out = torch.zeros(cu[-1], heads * dim, device=where[0], dtype=where[1])
    state = torch.zeros(6, heads, dim, dim, device=where[0])
    c0 = cases[0]
    ops.delta_rule(proj, z, c0["w2"], c0["w0"], c0["ab"], c0["nw"], state,
                   i32([5, 2, 4, 1], where), i32(cu, where),
                   i32([0] * 4, where), out, c0["offs"], math.exp(-0.5), 1e-6,
                   eps, (lay.prefill_tiles(ops.DELTA_CHUNK),
                         lay.prefill_tile_cu(ops.DELTA_CHUNK)))
    for c, a, b in zip(cases, cu, cu[1:]):
        close(out[a:b], delta_want(c, eps)[0], where)


# -- latent attention ------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("rank", [24, 64, 37])
def test_latent_store(where, rank):
    x, w = rnd(5, rank + 11, scale=0.05), 1 + 0.2 * rnd(rank, seed=2)
    cache = torch.zeros(4, 16, rank, device=where[0], dtype=where[1])
    slots = [17, 40, 16, 63, 31]
    xd = put(torch.nn.functional.pad(x, (0, -x.shape[1] % 8)), where)
    c = ops.latent_store(xd[:, 8:8 + rank], put(w, where, F32), cache,
                         i32(slots, where), 2e-3)
    want = oracle.rms_norm(seen(x, where)[:, 8:8 + rank], w, 2e-3)
    close(c, want, where)
    flat = cache.view(-1, rank)
    assert torch.equal(flat[slots], c)
    assert (flat.abs().sum(-1) > 0).sum() == 5


ATTN_SIZES = [(2, 32, 32), (3, 8, 16), (2, 64, 128), (1, 128, 64),
              (1, 256, 256), (1, 96, 40), (2, 20, 36)]


def attn_case(where, H, D, DV, n, seed=0):
    q = rnd(n, H, D, seed=seed)
    k = rnd(n, H, D, seed=seed + 1)
    v = rnd(n, H, DV, seed=seed + 2)
    return q, k, v


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,D,DV", ATTN_SIZES)
@pytest.mark.parametrize("window", [1, 2, 19, 64, 65])
def test_window_attention_portions(where, H, D, DV, window):
    """Portions cut anywhere, keys laid out as the layout gathers them; one
    key per query stands out, at the window's last place or one before it."""
    n, scale = 150, 1.0 / math.sqrt(D)
    q, k, v = attn_case(where, H, D, DV, n, seed=D + window)
    g = rnd(n, H * DV, seed=5)
    for i in range(40, n, 7):           # alternate: just inside, just outside
        j = i - window + (1 if i % 2 else 0)
        if j >= 0:
            unit = k[j] / k[j].norm(dim=-1, keepdim=True)
            q[i] = unit * 12 * math.sqrt(D) / k[j].norm(dim=-1, keepdim=True)
    q, k, v, g = (seen(t, where) for t in (q, k, v, g))
    want = oracle.window_attention(q, k, v, scale, window)
    want = want.reshape(n, -1) * torch.sigmoid(g)
    at = 0
    for m in [70, 2, 3, 75]:
        lay = layout([at], [at + m], where)
        view = lay.window_view(window)
        lo = max(0, at - window + 1)
        out = torch.zeros(m, H * DV, device=where[0], dtype=where[1])
        ops.window_attention(put(q[at:at + m], where),
                             put(k[lo:at + m], where),
                             put(v[lo:at + m], where),
                             put(g[at:at + m], where), out, view, scale,
                             window)
        close(out, want[at:at + m], where)
        at += m


@pytest.mark.parametrize("where", WHERE)
def test_window_attention_batch_and_no_window(where):
    H, D, DV, lens = 2, 32, 48, [5, 130, 1, 64]
    parts = [attn_case(where, H, D, DV, n, seed=n) for n in lens]
    q, k, v = (torch.cat([p[i] for p in parts]) for i in range(3))
    for window in (0, 33):
        lay = layout([0] * 4, lens, where)
        out = torch.zeros(sum(lens), H * DV, device=where[0], dtype=where[1])
        ops.window_attention(put(q, where), put(k, where), put(v, where), None,
                             out, lay.window_view(window), 0.2, window)
        at = 0
        for (a, b, c), n in zip(parts, lens):
            want = oracle.window_attention(
                seen(a, where), seen(b, where), seen(c, where), 0.2,
                window or n)
            close(out[at:at + n], want.reshape(n, -1), where)
            at += n


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,rank,window", [(3, 24, 21), (18, 64, 32),
                                           (2, 37, 7), (16, 136, 0),
                                           (5, 256, 48), (17, 512, 100)])
def test_latent_decode(where, H, rank, window):
    """Shuffled pages, contexts around page borders, a key that stands out
    just inside or just outside the window (or at a page's border)."""
    ps, scale = 16, 1.0 / math.sqrt(rank)
    ctxs = [1, 15, 16, 17, window or 40, (window or 40) + 1, 161, 250]
    pages = torch.randperm(199, generator=torch.Generator().manual_seed(3))
    cache = rnd(200, ps, rank, seed=rank)
    cache[0] = 0
    tables, at = [], 0
    for c in ctxs:
        n = (c + ps - 1) // ps
        tables.append((pages[at:at + n] + 1).tolist())
        at += n
    width = max(len(t) for t in tables)
    bt = i32([t + [0] * (width - len(t)) for t in tables], where)
    q = rnd(len(ctxs), H, rank, seed=1)
    rows = [cache[t].reshape(-1, rank)[:c] for t, c in zip(tables, ctxs)]
    for b, c in enumerate(ctxs):
        far = c - (window or c) - (b % 2)       # inside, or one outside
        if far >= 0:
            key = rows[b][far]
            q[b] = key * 14 / scale / (key * key).sum()
    q, cache = seen(q, where), seen(cache, where)
    o = ops.latent_decode(put(q, where), put(cache, where), bt,
                          i32(ctxs, where), scale, window)
    for b, c in enumerate(ctxs):
        keys = cache[tables[b]].reshape(-1, rank)[:c]
        keys = keys[max(0, c - window):] if window else keys
        p = torch.softmax(q[b] @ keys.T * scale, dim=-1)
        close(o[b], p @ keys, where)


@pytest.mark.gpu
@pytest.mark.parametrize("splits", [1, 3, 64])
def test_latent_decode_splits(splits):
    """More splits than chunks, and one."""
    where = ("cuda", BF16)
    H, rank, ps, window = 4, 64, 16, 90
    cache = seen(rnd(30, ps, rank), where)
    q = seen(rnd(2, H, rank, seed=1), where)
    bt = i32([list(range(1, 11)), list(range(11, 21))], where)
    o = ops._require_latent().latent_decode(
        put(q, where), put(cache, where), bt, i32([150, 3], where), 0.1,
        window, splits, rank, None)
    for b, c in enumerate([150, 3]):
        keys = cache[1 + 10 * b:11 + 10 * b].reshape(-1, rank)
        keys = keys[max(0, c - window):c]
        p = torch.softmax(q[b] @ keys.T * 0.1, dim=-1)
        close(o[b], p @ keys, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("S,H,n,k", [(1, 2, 24, 40), (5, 3, 17, 33),
                                     (20, 2, 130, 64), (70, 1, 64, 128)])
def test_head_linear(where, S, H, n, k):
    x, w = rnd(S, H, k), rnd(H, n, k, seed=1, scale=1 / math.sqrt(k))
    g = rnd(S, H * n, seed=2)
    want = torch.einsum("shk,hjk->shj", seen(x, where), seen(w, where))
    want = want.reshape(S, H * n)
    close(ops.head_linear(put(x, where), put(w, where)), want, where)
    buf = torch.zeros(S, H * n + 5, device=where[0], dtype=where[1])
    ops.head_linear(put(x, where), put(w, where), gate=put(g, where),
                    out=buf[:, :H * n])
    close(buf[:, :H * n], want * torch.sigmoid(seen(g, where)), where)
    assert buf[:, H * n:].abs().max() == 0
