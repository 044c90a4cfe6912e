"""Plain implementation of the Gogalix design, one function per mechanism.

Numerics oracle for tests/test_gogalix*.py: whole sequences, loops over tokens,
no cache, no batching, no kernels, and nothing imported from rbg_amd.  It
computes in the dtype of the weights it is given (the tests use float64).
"""
import torch

UNIT_EPS = 1e-6


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, gain, eps):
    """RMS norm whose weight is one number."""
    return rms(x, eps) * gain


def silu(z):
    return z * torch.sigmoid(z)


# -- delta rule ------------------------------------------------------------------


def short_conv(x, taps):
    """x [T, C]; taps [C, n], the last one is the current token's; then silu."""
    n = taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(n):
            if t - j >= 0:
                out[t] += taps[:, n - 1 - j] * x[t - j]
    return silu(out)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def decay(logits, a_log, dt_bias):
    """Factor per token on the state, in (0, 1)."""
    return torch.exp(-torch.exp(a_log) *
                     torch.nn.functional.softplus(logits + dt_bias,
                                                  threshold=40))


def recurrence(q, k, v, g, beta):
    """q, k [T, H, D], v [T, H, E], g [T, H, D], beta [T, H] -> o [T, H, E].
    The read-out sees the current token's write."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(T):
        S = S * g[t].unsqueeze(-1)
        seen = (S * k[t].unsqueeze(-1)).sum(1)
        u = beta[t].unsqueeze(-1) * (v[t] - seen)
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out.append((S * q[t].unsqueeze(-1)).sum(1))
    return torch.stack(out)


def delta(h, p, mixer, eps, per_channel):
    T, H, G = h.shape[0], mixer["heads"], mixer["kv_heads"]
    D, E = mixer["dim"], mixer["vdim"]
    q = unit(short_conv(h @ p["q"].T, p["q.conv"]).view(T, G, D)) * D ** -0.5
    k = unit(short_conv(h @ p["k"].T, p["k.conv"]).view(T, G, D))
    v = short_conv(h @ p["v"].T, p["v.conv"]).view(T, H, E)
    q, k = (t.repeat_interleave(H // G, dim=1) for t in (q, k))
    beta = torch.sigmoid(h @ p["b"].T)
    if per_channel:
        logits = ((h @ p["a1"].T) @ p["a2"].T).view(T, H, D)
        g = decay(logits, p["A_log"].view(H, 1), p["dt_bias"].view(H, D))
        gate = torch.sigmoid((h @ p["g1"].T) @ p["g2"].T)
    else:
        g = decay(h @ p["a"].T, p["A_log"], p["dt_bias"])
        g = g.unsqueeze(-1).expand(T, H, D)
        gate = silu(h @ p["g"].T)
    o = rms(recurrence(q, k, v, g, beta), eps) * p["norm"]
    return (o.reshape(T, H * E) * gate) @ p["o"].T


# -- differential attention ------------------------------------------------------


def window_attention(q, k, v, scale, window):
    """q [T, H, D], k [T, H, D], v [T, H, E]: position i sees the `window`
    positions up to itself."""
    out = []
    for i in range(q.shape[0]):
        lo = max(0, i - window + 1)
        s = (k[lo:i + 1] * q[i]).sum(-1) * scale        # [keys, H]
        w = torch.softmax(s, dim=0)
        out.append((w.unsqueeze(-1) * v[lo:i + 1]).sum(0))
    return torch.stack(out)


def difference(a1, a2, lam, diff, eps):
    return rms(a1 - lam * a2, eps) * (1 - diff)


def lam_of(p, diff):
    return (torch.exp((p["lq1"] * p["lk1"]).sum()) -
            torch.exp((p["lq2"] * p["lk2"]).sum()) + diff)


def keys_values(h, p, mixer):
    T, G = h.shape[0], mixer["kv_heads"]
    return ((h @ p["k"].T).view(T, G, 2, mixer["dim"]),
            (h @ p["v"].T).view(T, G, mixer["vdim"]))


def attention(h, p, mixer, kv, eps):
    T, H, G = h.shape[0], mixer["heads"], mixer["kv_heads"]
    q = (h @ p["q"].T).view(T, H, 2, mixer["dim"])
    k, v = (t.repeat_interleave(H // G, dim=1) for t in kv)
    a1, a2 = (window_attention(q[:, :, m], k[:, :, m], v, mixer["scale"],
                               mixer["mask"]["size"]) for m in (0, 1))
    o = difference(a1, a2, lam_of(p, mixer["diff"]), mixer["diff"], eps)
    return o.reshape(T, -1) @ p["o"].T


# -- feed-forwards ---------------------------------------------------------------


def dense(h, p):
    act = silu(h @ p["gate"].T + p["gate.b"]) * (h @ p["up"].T + p["up.b"])
    return act @ p["down"].T + p["down.b"]


def route(logits, top):
    """[(expert, weight)] of one token: softmax over the chosen alone."""
    order = sorted(range(len(logits)), key=lambda e: -logits[e].item())[:top]
    w = torch.softmax(logits[order], dim=0)
    return list(zip(order, w))


def experts(h, p, top):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(p["router"] @ h[t] + p["router.b"], top):
            act = silu(p[f"e{e}.gate"] @ h[t]) * (p[f"e{e}.up"] @ h[t])
            out[t] += w * (p[f"e{e}.down"] @ act)
    return out


# -- model -----------------------------------------------------------------------


def sub(weights, prefix):
    return {n[len(prefix):]: t for n, t in weights.items()
            if n.startswith(prefix)}


def gated(y, h, w, which):
    """A branch's result under its layer scale and its input's gate."""
    gate = torch.sigmoid(h @ w["rg" + which].T + w[f"rg{which}.b"])
    return y * w["ls" + which] * gate


def forward(tokens, config, weights):
    """Logits [T, vocab] of one sequence, and the residual stream after
    every layer [layers, T, width]."""
    eps = config["norm"]["eps"]
    x = weights["embed"][torch.tensor(tokens)] * config["embedding"]["scale"]
    streams, kv = [], {}
    for i, layer in enumerate(config["layers"]):
        w, mixer = sub(weights, f"l{i}."), layer["mixer"]
        h, p = norm(x, w["norm1"], eps), sub(w, "mix.")
        if layer["type"] == "attention":
            src = mixer.get("kv_from")
            if src is None:
                src = i
                kv[i] = keys_values(h, p, mixer)
            y = attention(h, p, mixer, kv[src], eps)
        else:
            y = delta(h, p, mixer, eps, layer["type"] == "channel_delta")
        y = gated(y, h, w, "1")
        if layer["mlp"] is not None:
            p = sub(w, "mlp.")
            f = dense(h, p) if layer["mlp"]["kind"] == "dense" else \
                experts(h, p, layer["mlp"]["router"]["top"])
            y = y + gated(f, h, w, "2")
        x = x + y
        streams.append(x)
    x = norm(x, weights["final.norm"], eps)
    return x @ weights["head"].T, torch.stack(streams)
