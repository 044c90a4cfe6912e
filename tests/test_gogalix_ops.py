"""Gogalix's mechanisms one by one against the plain oracle: on the CPU the
reference path, on the GPU (marked) every HIP kernel in f32 and bf16, at sizes
that take the vector, the matrix-core and the any-size forms."""
import math

import pytest
import torch

import rbg_amd.ops as ops
from tests import gogalix_oracle as oracle
from tests.test_bitatar_ops import (BF16, F32, WHERE, close, i32, layout, put,
                                    rnd, seen)
from tests.test_notadra_ops import pages_of

# -- stream, gates ---------------------------------------------------------------


def branch(T, W, where, seed, bias, route=None):
    """A branch, and what it adds to the stream."""
    rows = rnd(T if route is None else route.rows.numel(), W, seed=seed)
    wide = rnd(T, W + 24, seed=seed + 1, scale=2.0)
    gb, ls, b = (rnd(W, seed=seed + i) for i in (2, 3, 4))
    y = seen(rows, where)
    if route is not None:
        y = (y[route.inv.cpu().long()].view(T, -1, W) *
             route.weights.double().cpu().unsqueeze(-1)).sum(1)
    z = seen(wide, where)[:, 8:8 + W]           # a slice of a projection
    if bias:
        y = y + b.float().double()
    add = y * ls.float().double() * torch.sigmoid(z + gb.float().double())
    return ops.Branch(put(rows, where), put(wide, where)[:, 8:8 + W],
                      put(gb, where, F32), put(ls, where, F32),
                      put(b, where, F32) if bias else None, route), add


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W", [48, 256, 2056, 5120, 37, 1030])
def test_gate_norm(where, W):
    T, eps = 5, 3e-2                    # an eps that shows
    x = rnd(T, W, seed=1, scale=0.3)
    one, each = torch.tensor([1.7]), 1 + 0.3 * rnd(W, seed=3).float()
    xs, want = put(x, where, F32), x.float().double()
    h = ops.gate_norm(xs, [], put(one, where, F32), eps, where[1])
    assert h.dtype == where[1]
    close(h, oracle.norm(want, one.double(), eps), where)
    b1, add1 = branch(T, W, where, 10, False)
    b2, add2 = branch(T, W, where, 20, True)
    h = ops.gate_norm(xs, [b1, b2], put(each, where, F32), eps, where[1])
    want = want + add1 + add2
    close(xs, want, where, 2e-6)        # the stream is f32 in every mode
    close(h, oracle.norm(want, each.double(), eps), where)
    assert ops.gate_norm(xs, [b2], None, eps, where[1]) is None
    close(xs, want + add2, where, 2e-6)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W,top", [(64, 3), (35, 1), (2048, 8)])
def test_weighed_experts_in_the_norm(where, W, top):
    T, E = 6, 12
    route = ops.moe_route(put(rnd(T, E, seed=5), where, F32),
                          put(rnd(E, seed=6), where, F32), 1, 1, top, 16,
                          softmax=True)
    b1, add1 = branch(T, W, where, 10, True)
    b2, add2 = branch(T, W, where, 20, False, route)
    x = rnd(T, W, seed=1)
    xs, one = put(x, where, F32), torch.tensor([0.6])
    h = ops.gate_norm(xs, [b1, b2], put(one, where, F32), 1e-5, where[1])
    want = x.float().double() + add1 + add2
    close(xs, want, where, 2e-6)
    close(h, oracle.norm(want, one.double(), 1e-5), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("F", [40, 33])
@pytest.mark.parametrize("bias", [True, False])
def test_silu_glu(where, F, bias):
    seg = F + -F % 8
    y = rnd(6, 2 * seg + 8, scale=2.0)
    bg, bu = rnd(F, seed=1), rnd(F, seed=2)
    yd, ys = put(y, where), seen(y, where)
    out = torch.zeros(6, F, device=where[0], dtype=where[1])
    ops.silu_glu(yd[:, 8:8 + F], yd[:, 8 + seg:8 + seg + F],
                 *([put(b, where, F32) for b in (bg, bu)] if bias
                   else [None, None]), out)
    g, u = ys[:, 8:8 + F], ys[:, 8 + seg:8 + seg + F]
    if bias:
        g, u = g + bg.float().double(), u + bu.float().double()
    close(out, oracle.silu(g) * u, where)


# -- short convolution -------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W,taps", [(64, 4), (50, 2), (32, 7), (16, 1),
                                    (40, 3), (24, 19)])
def test_short_conv_portions(where, W, taps):
    """Portions down to one token, shorter and longer than the past, of two
    sequences on dirty slots; the input is a slice of wider rows."""
    n = [61, 40]
    xs = [seen(rnd(t, W, seed=t), where) for t in n]
    w = rnd(W, taps, seed=9, scale=0.5)
    want = [oracle.short_conv(x, w.float().double()) for x in xs]
    ring = torch.full((4, taps, W), 7.0, device=where[0], dtype=where[1])
    slots, at = i32([3, 1], where), [0, 0]
    for portion in [(17, 2), (1, 1), (2, 3), (2, 2), (35, 30), (4, 2)]:
        ends = [a + p for a, p in zip(at, portion)]
        lay = layout(at, ends, where)
        rows = torch.cat([x[a:e] for x, a, e in zip(xs, at, ends)])
        wide = put(torch.nn.functional.pad(rows, (8, 16)), where)
        h = ops.short_conv(wide[:, 8:8 + W], put(w.T, where, F32), ring,
                           lay.prefill_tiles(max(ops.CONV_TILE, taps)),
                           i32([0, portion[0], sum(portion)], where),
                           i32(at, where), slots)
        close(h, torch.cat([y[a:e] for y, a, e in zip(want, at, ends)]), where)
        at = ends
    assert at == n and (ring[[0, 2]] == 7.0).all()


# -- gated delta rule --------------------------------------------------------------


def delta_case(where, H, G, D, E, taps, T, per_channel, seed=0, rate=-1.0,
               fixed=None):
    """Projections with gaps between their segments, and the oracle's rows.
    ``rate`` shifts the decays' logarithms: at 3 a state is gone in a token.
    ``fixed``: another case whose weights are taken."""
    def seg(n):
        return n + -n % 8
    offs = [0, seg(G * D), 2 * seg(G * D)]
    C = offs[2] + seg(H * E)
    qkv = rnd(T, C + 16, seed=seed)
    qkv[:, :C] *= 1.5
    beta, gate = rnd(T, H, seed=seed + 1, scale=2.0), rnd(T, H * E,
                                                          seed=seed + 2)
    z = rnd(T, H * D if per_channel else H, seed=seed + 3, scale=2.0)
    f = fixed or dict(
        conv=torch.cat([torch.nn.functional.pad(rnd(n, taps, seed=seed + 4 + i,
                                                    scale=0.6),
                                                (0, 0, 0, -n % 8))
                        for i, n in enumerate((G * D, G * D, H * E))]),
        a_log=rnd(H, seed=seed + 7) + rate,
        dt=rnd(z.shape[1], seed=seed + 8), norm=1 + 0.3 * rnd(E, seed=seed + 9))
    ys = seen(qkv, where)
    f32 = {k: t.float().double() for k, t in f.items()}

    def conv(at, n, size):
        cols = slice(at, at + n * size)
        return oracle.short_conv(ys[:, cols], f32["conv"][cols]).view(T, n,
                                                                      size)
    q = oracle.unit(conv(offs[0], G, D)) * D ** -0.5
    k, v = oracle.unit(conv(offs[1], G, D)), conv(offs[2], H, E)
    q, k = (t.repeat_interleave(H // G, dim=1) for t in (q, k))
    zs, dt = seen(z, where), f32["dt"]
    if per_channel:
        g = oracle.decay(zs.view(T, H, D), f32["a_log"].view(H, 1),
                         dt.view(H, D))
    else:
        g = oracle.decay(zs, f32["a_log"], dt).unsqueeze(-1).expand(T, H, D)
    o = oracle.recurrence(q, k, v, g, torch.sigmoid(seen(beta, where)))
    eps, zg = 1e-4, seen(gate, where)
    want = (oracle.rms(o, eps) * f32["norm"]).reshape(T, -1) * (
        torch.sigmoid(zg) if per_channel else oracle.silu(zg))
    params = ops.GatedDelta(
        put(f["a_log"], where, F32), put(f["dt"], where, F32),
        put(f["norm"], where, F32), G, not per_channel, D ** -0.5, 1e-6, eps)
    return dict(qkv=put(qkv, where), beta=put(beta, where), z=put(z, where),
                gate=put(gate, where), p=params, offs=offs, want=want, C=C,
                conv=put(f["conv"].T, where, F32), fixed=f)


def run_delta(c, lo, hi, at, cu, state, ring, slots, out, lay, chunk=True):
    """Rows [lo, hi) of a case: one row per sequence as a decode step, or
    portions."""
    rows = slice(lo, hi)
    args = (c["beta"][rows], c["z"][rows], c["gate"][rows], state, slots)
    if cu is None:
        ops.gated_delta(c["p"], c["qkv"][rows], c["offs"], *args, None, at,
                        out[rows], conv=(c["conv"], ring))
        return
    x = ops.short_conv(c["qkv"][rows][:, :c["C"]], c["conv"], ring,
                       lay.prefill_tiles(ops.CONV_TILE), cu, at, slots)
    ops.gated_delta(c["p"], x, c["offs"], *args, cu, at, out[rows],
                    chunks=(lay.prefill_tiles(ops.DELTA_CHUNK),
                            lay.prefill_tile_cu(ops.DELTA_CHUNK))
                    if chunk else None)


#               H  G  D    E    taps
DELTA_SIZES = [(4, 2, 64, 32, 4), (2, 2, 24, 40, 3), (3, 1, 128, 128, 2),
               (2, 1, 12, 7, 5), (1, 1, 33, 96, 4), (2, 1, 160, 24, 1),
               (1, 1, 96, 200, 4), (4, 4, 32, 64, 1)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,E,taps", DELTA_SIZES)
@pytest.mark.parametrize("per_channel", [True, False])
@pytest.mark.parametrize("rate", [-3.0, 0.0, 3.0])
def test_gated_delta_portions(where, H, G, D, E, taps, per_channel, rate):
    """Portions of 2..37 tokens, by chunks and (any head size) token by token,
    single tokens as decode steps, on a slot full of somebody else's state."""
    T = 65
    c = delta_case(where, H, G, D, E, taps, T, per_channel, seed=D, rate=rate)
    state = torch.full((3, H, D, E), 5.0, device=where[0])
    ring = torch.full((3, taps, c["C"]), 5.0, device=where[0], dtype=where[1])
    out = torch.zeros(T, H * E, device=where[0], dtype=where[1])
    at = 0
    for i, n in enumerate([37, 1, 2, 1, 1, 5, 15, 3]):
        lay = layout([at], [at + n], where)
        run_delta(c, at, at + n, i32([at], where),
                  i32([0, n], where) if n > 1 else None, state, ring,
                  i32([2], where), out, lay, chunk=i != 5)
        at += n
    assert at == T
    close(out, c["want"], where)
    assert (state[1] == 5.0).all() and (ring[1] == 5.0).all()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("per_channel", [True, False])
def test_gated_delta_batch(where, per_channel):
    """Unequal sequences in one launch, each on its own slot; then a decode
    step of all of them, whose heads share keys and their past."""
    H, G, D, E, taps = 4, 1, 40, 48, 4
    lens = [3, 17, 33, 2]
    cases = []
    for n in lens:
        cases.append(delta_case(where, H, G, D, E, taps, n + 1, per_channel,
                                seed=n, fixed=cases[0]["fixed"] if cases
                                else None))
    both = dict(cases[0])
    for name in ("qkv", "beta", "z", "gate"):
        both[name] = torch.cat([c[name][:-1] for c in cases] +
                               [c[name][-1:] for c in cases])
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    lay = layout([0] * 4, lens, where)
    T = cu[-1]
    out = torch.zeros(T + 4, H * E, device=where[0], dtype=where[1])
    state = torch.full((6, H, D, E), 3.0, device=where[0])
    ring = torch.full((6, taps, both["C"]), 3.0, device=where[0],
                      dtype=where[1])
    slots = i32([5, 2, 4, 1], where)
    run_delta(both, 0, T, i32([0] * 4, where), i32(cu, where), state, ring,
              slots, out, lay)
    run_delta(both, T, T + 4, i32(lens, where), None, state, ring, slots, out,
              None)
    for i, (c, a, b) in enumerate(zip(cases, cu, cu[1:])):
        close(torch.cat([out[a:b], out[T + i:T + i + 1]]), c["want"], where)


@pytest.mark.parametrize("where", WHERE)
def test_one_key_is_kept_and_written_over(where):
    """Without decay and with full steps a key returns the value written last,
    however long ago; the read-out sees the current token's write."""
    H, D, E, T = 1, 8, 8, 50
    key = torch.eye(D, dtype=torch.float64)
    qkv = torch.zeros(T, 24, dtype=torch.float64)
    vals = rnd(T, E, seed=3)
    for t in range(T):
        j = 0 if t in (0, 30, 49) else 1 + t % (D - 1)
        qkv[t, :8] = qkv[t, 8:16] = key[j] * 30     # silu(30) is 30
        qkv[t, 16:] = vals[t]
    qkv[40, :8] = key[0] * 30                       # reads what 30 wrote
    big = torch.full((T, 1), 40.0, dtype=torch.float64)
    p = ops.GatedDelta(*(put(t, where, F32) for t in (
        torch.tensor([-40.0]), torch.zeros(1), torch.ones(E))), 1, False, 1.0,
        1e-6, 1e-9)
    state = torch.zeros(2, 1, D, E, device=where[0])
    out = torch.zeros(T, E, device=where[0], dtype=where[1])
    lay = layout([0], [T], where)
    x = torch.cat([oracle.silu(qkv[:, :16]), qkv[:, 16:]], 1)
    ops.gated_delta(p, put(x, where), [0, 8, 16], put(big, where),
                    put(-big, where), put(big.expand(T, E), where), state,
                    i32([1], where), i32([0, T], where), i32([0], where), out,
                    chunks=(lay.prefill_tiles(ops.DELTA_CHUNK),
                            lay.prefill_tile_cu(ops.DELTA_CHUNK)))
    vs = oracle.rms(seen(vals, where), 1e-9)
    close(out[40], vs[30], where)
    close(out[49], vs[49], where)
    close(state[1, 0, 0], seen(vals, where)[49], where, 1e-5)


# -- differential attention --------------------------------------------------------

#            H   G   D    DV
DIFF_SIZES = [(4, 2, 32, 32), (3, 3, 8, 16), (8, 1, 64, 80), (2, 2, 128, 128),
              (10, 1, 40, 96), (2, 1, 16, 256), (20, 1, 16, 8), (2, 1, 10, 36),
              (2, 1, 136, 24), (2, 1, 128, 256)]


def diff_case(where, H, G, D, DV, n, scale, window, seed=0):
    """Every third query singles one key out with each map, just inside the
    window, just outside, or at a page's edge."""
    q, k, v = rnd(n, H, 2, D, seed=seed), rnd(n, G, 2, D, seed=seed + 1), \
        rnd(n, G, DV, seed=seed + 2)
    for i in range(0, n, 3):
        back = [window - 1, window, 0, i - i // 16 * 16, window // 2]
        for m in (0, 1):
            j = max(0, i - back[(i // 3 + 2 * m) % 5])
            for h in range(H):
                key = k[j, h // (H // G), m]
                q[i, h, m] = key * 14 / scale / (key * key).sum()
    return tuple(seen(t, where) for t in (q, k, v))


def diff_want(q, k, v, scale, window, lam, diff, eps):
    per = q.shape[1] // k.shape[1]
    k, v = (t.repeat_interleave(per, dim=1) for t in (k, v))
    a1, a2 = (oracle.window_attention(q[:, :, m], k[:, :, m], v, scale, window)
              for m in (0, 1))
    return oracle.difference(a1, a2, lam, diff, eps)


def difference(where, lam, diff, eps):
    return ops.Difference(put(torch.tensor([lam]), where, F32), 1 - diff, eps)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,DV", DIFF_SIZES)
@pytest.mark.parametrize("window", [1, 19, 64, 65, 500])
def test_difference_prefill_portions(where, H, G, D, DV, window):
    """Portions cut anywhere, over keys in shuffled pages, other rows of the
    pages poisoned."""
    n, scale, lam, diff, eps = 150, 0.7 / math.sqrt(D), 0.45, 0.3, 1e-3
    q, k, v = diff_case(where, H, G, D, DV, n, scale, window, D)
    want = diff_want(q, k, v, scale, window, lam, diff, eps).reshape(n, -1)
    kp, vp, tables = pages_of(k.flatten(2), v, where, [n])
    at = 0
    for m in [70, 2, 3, 75]:
        lay = layout([at], [at + m], where, tables=tables)
        buf = torch.zeros(m, H * DV + 8, device=where[0], dtype=where[1])
        # rows of q are a slice of something wider
        qd = put(torch.nn.functional.pad(q[at:at + m].reshape(m, -1), (0, 8)),
                 where)[:, :H * 2 * D].unflatten(1, (H, 2 * D))
        ops.paged_prefill(qd, kp, vp, lay.paged_view(), buf[:, :H * DV], scale,
                          0.0, False, window=window,
                          diff=difference(where, lam, diff, eps))
        close(buf[:, :H * DV], want[at:at + m], where)
        assert (buf[:, H * DV:] == 0).all()
        at += m


@pytest.mark.parametrize("where", WHERE)
def test_difference_prefill_batch_after_decode_rows(where):
    H, G, D, DV, scale, window = 4, 2, 32, 48, 0.2, 21
    starts, ends = [7, 0, 40, 15], [8, 130, 42, 64]
    parts = [diff_case(where, H, G, D, DV, e, scale, window, seed=e)
             for e in ends]
    kp, vp, tables = pages_of(torch.cat([p[1] for p in parts]).flatten(2),
                              torch.cat([p[2] for p in parts]), where, ends)
    lay = layout(starts, ends, where, num_decode=1, tables=tables)
    q = torch.cat([p[0][s:] for p, s in zip(parts[1:], starts[1:])]).flatten(2)
    out = torch.zeros(q.shape[0], H * DV, device=where[0], dtype=where[1])
    ops.paged_prefill(put(q, where), kp, vp, lay.paged_view(), out, scale, 0.0,
                      False, window=window,
                      diff=difference(where, 1.2, 0.7, 1e-4))
    at = 0
    for p, s in zip(parts[1:], starts[1:]):
        want = diff_want(*p, scale, window, 1.2, 0.7, 1e-4)[s:].flatten(1)
        close(out[at:at + len(want)], want, where)
        at += len(want)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,DV", DIFF_SIZES)
@pytest.mark.parametrize("window", [1, 16, 130, 1000])
def test_difference_decode(where, H, G, D, DV, window):
    """Contexts around page, step and window borders."""
    scale, lam, diff, eps = 0.7 / math.sqrt(D), -0.3, 0.5, 1e-3
    ctxs = [1, 15, 17, 32, 127, 129, 130, 131, 161, 290]
    parts, qs, wants = [], [], []
    for b, c in enumerate(ctxs):
        q, k, v = diff_case(where, H, G, D, DV, c, scale, window, seed=c)
        # the maps look at the two sides of the window's edge, and at itself
        for m in (0, 1):
            j = max(0, c - 1 - [window - 1, window, 0][(b + m) % 3])
            key = k[j, :, m].repeat_interleave(H // G, dim=0)
            q[c - 1, :, m] = key * 14 / scale / \
                (key * key).sum(-1, keepdim=True)
        q = seen(q, where)
        parts.append((k, v))
        qs.append(q[-1].flatten(1))
        lo = max(0, c - window)         # the last row alone
        per = H // G
        ks, vs = (t[lo:].repeat_interleave(per, dim=1) for t in (k, v))
        a = []
        for m in (0, 1):
            w = torch.softmax((ks[:, :, m] * q[-1, :, m]).sum(-1) * scale, 0)
            a.append((w.unsqueeze(-1) * vs).sum(0))
        wants.append(oracle.difference(a[0], a[1], lam, diff, eps).flatten())
    kp, vp, tables = pages_of(torch.cat([p[0] for p in parts]).flatten(2),
                              torch.cat([p[1] for p in parts]), where, ctxs)
    wide = max(len(t.pages) for t in tables)
    bt = i32([t.pages + [0] * (wide - len(t.pages)) for t in tables], where)
    for splits in (0, 1, 3):
        out = torch.zeros(len(ctxs), H * DV, device=where[0], dtype=where[1])
        ops.paged_decode(put(torch.stack(qs), where), kp, vp, bt,
                         i32(ctxs, where), out, scale, 0.0, False, splits,
                         window=window, diff=difference(where, lam, diff, eps))
        for b in range(len(ctxs)):
            close(out[b], wants[b], where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sink,cap", [(False, 0.0), (True, 30.0)])
@pytest.mark.parametrize("window", [1, 33, 64])
def test_window_of_ordinary_heads(where, sink, cap, window):
    """The window with the options that other designs use."""
    H, G, D, DV, n, scale = 4, 2, 32, 32, 170, 0.3
    q, k, v = diff_case(where, H, G, D, DV, n, scale, window)
    q, k = q[:, :, 0], k[:, :, 0]
    want = torch.zeros(n, H, DV, dtype=torch.float64)
    for i in range(n):
        lo = max(0, i - window + 1)
        for h in range(H):
            s = k[lo:i + 1, h // 2] @ q[i, h] * scale
            s = cap * torch.tanh(s / cap) if cap else s
            if sink:
                s = torch.cat([s, torch.zeros(1, dtype=s.dtype)])
            p = torch.softmax(s, 0)[:i + 1 - lo]
            want[i, h] = p @ v[lo:i + 1, h // 2]
    kp, vp, tables = pages_of(k, v, where, [n])
    lay = layout([0], [n], where, tables=tables)
    out = torch.zeros(n, H * DV, device=where[0], dtype=where[1])
    ops.paged_prefill(put(q, where), kp, vp, lay.paged_view(), out, scale, cap,
                      sink, window=window)
    close(out, want.flatten(1), where)
    for splits in (1, 2):
        one = torch.zeros(1, H * DV, device=where[0], dtype=where[1])
        ops.paged_decode(put(q[n - 1:], where), kp, vp,
                         i32([tables[0].pages], where), i32([n], where), one,
                         scale, cap, sink, splits, window=window)
        close(one, want[n - 1:].flatten(1), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("G,D,DV", [(2, 32, 16), (1, 10, 7)])
def test_plain_paged_store(where, G, D, DV):
    """Keys and values go to the pages as they are; the queries stay."""
    T, H = 5, 3
    sizes = [H * D, G * D, G * DV]
    offs, at = [], 0
    for n in sizes:
        offs.append(at)
        at += n + -n % 8
    y = put(rnd(T, at), where)
    before = y.clone()
    k = torch.full((4, G, 16, D), 9.0, device=where[0], dtype=where[1])
    v = torch.full((4, G, 16, DV), 9.0, device=where[0], dtype=where[1])
    slots = [17, 40, 16, 63, 31]
    ops.rope_store_paged(y, None, None, i32(range(T), where),
                         i32(slots, where), H, D, k, v, offs)
    assert torch.equal(y, before)
    for t, name, at in ((k, D, offs[1]), (v, DV, offs[2])):
        flat = t.permute(0, 2, 1, 3).reshape(64, -1)
        assert torch.equal(flat[slots], y[:, at:at + G * name])
        rest = [s for s in range(64) if s not in slots]
        assert (flat[rest] == 9.0).all()


# -- experts -----------------------------------------------------------------------


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("T,E,top", [(7, 16, 3), (1, 8, 2), (80, 8, 1),
                                     (5, 6, 6), (300, 128, 8), (40, 520, 3),
                                     (3, 1, 1)])
def test_softmax_route(where, T, E, top):
    logits = rnd(T, E, seed=E + T, scale=2.0).float()
    bias = rnd(E, seed=2).float()
    r = ops.moe_route(put(logits, where, F32), put(bias, where, F32), 1, 1,
                      top, 16, softmax=True)
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    owner = {}
    for e, at, m in r.tiles[:n].cpu().tolist():
        owner.update({i: e for i in range(at, at + m)})
    inv = r.inv.cpu().view(T, top).tolist()
    assert sorted(sum(inv, [])) == list(range(T * top))
    for t in range(T):
        want = oracle.route(logits[t].double() + bias.double(), top)
        got = {owner[i]: w for i, w in zip(inv[t], r.weights[t].tolist())}
        assert sorted(got) == sorted(e for e, _ in want)
        for e, w in want:
            assert got[e] == pytest.approx(w.item(), rel=1e-5)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("T,E,top,F,K", [
    (1, 16, 3, 24, 48), (3, 4, 2, 40, 136), (20, 8, 2, 96, 256),
    (150, 4, 2, 136, 72), (400, 4, 3, 264, 200), (5, 6, 2, 14, 21)])
@pytest.mark.parametrize("tile", [16, 32, 64, 128])
def test_gated_experts(where, T, E, top, F, K, tile):
    if tile > 16 and (where[1] == F32 or 2 * F % 8 or K % 8):
        pytest.skip("these sizes have one form")
    logits = rnd(T, E, seed=3, scale=3.0).float()
    logits[:, E - 1] -= 2.0             # unequal experts, perhaps an empty one
    r = ops.moe_route(put(logits, where, F32),
                      put(torch.zeros(E), where, F32), 1, 1, top, tile,
                      softmax=True)
    x = rnd(T, K)
    gate, up = (rnd(E, F, K, seed=s, scale=2 / math.sqrt(K)) for s in (1, 2))
    n = r.tiles.shape[0] if r.count is None else int(r.count)
    owner = torch.zeros(T * top, dtype=torch.long)
    for e, at, m in r.tiles[:n].tolist():
        owner[at:at + m] = e
    w = ops.interleave_glu(gate, up)
    h = ops.expert_linear(put(x, where), put(w, where), r, gather=True,
                          swiglu=True)
    assert h.shape == (T * top, F)
    xs = seen(x, where)[r.rows.cpu().long()]
    g, u = seen(gate, where), seen(up, where)
    want = torch.stack([oracle.silu(g[e] @ t) * (u[e] @ t)
                        for e, t in zip(owner, xs)])
    close(h, want, where)


@pytest.mark.gpu
def test_decode_softplus_of_tiny_and_large_logits():
    """The decay's logarithm keeps its relative precision where softplus is
    tiny, and does not overflow where it is large."""
    where = ("cuda", F32)
    z = torch.tensor([-60.0, -20.0, -9.0, -1.0, 0.0, 3.0, 30.0, 90.0])
    n = len(z)
    a_log = torch.tensor([16.0, 9.0, 5.0, 0.0, 0.0, -1.0, -4.0, -6.0])
    state = torch.ones(2, n, 8, 8, device="cuda")
    qkv = torch.zeros(1, 2 * n * 8 + n * 8, device="cuda")
    p = ops.GatedDelta(put(a_log, where), put(torch.zeros(n), where),
                       put(torch.ones(8), where), n, True, 1.0, 1e-6, 1e-6)
    out = torch.zeros(1, n * 8, device="cuda")
    ops.gated_delta(p, qkv, [0, n * 8, 2 * n * 8],
                    torch.zeros(1, n, device="cuda"), put(z.view(1, n), where),
                    torch.zeros(1, n * 8, device="cuda"), state,
                    i32([1], where), None, i32([4], where), out)
    want = -torch.exp(a_log.double()) * torch.log1p(torch.exp(z.double()))
    got = torch.log(state[1, :, 0, 0].double().cpu())
    assert torch.allclose(got, want, rtol=3e-5, atol=3e-7)
