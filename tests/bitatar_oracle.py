"""Plain implementation of the Bitatar design, one function per mechanism.

Numerics oracle for tests/test_bitatar*.py: whole sequences, loops over time,
no cache, no batching, no kernels, and nothing imported from rbg_amd.  It
computes in the dtype of the weights it is given (the tests use float64).
"""
import math

import torch


def group_norm(x, w, groups, eps):
    """x [T, width]: each of `groups` equal parts divided by its own RMS."""
    T, width = x.shape
    parts = x.reshape(T, groups, width // groups)
    rms = torch.sqrt((parts * parts).mean(-1, keepdim=True) + eps)
    return (parts / rms).reshape(T, width) * w


def rms_norm(x, w, eps):
    return group_norm(x, w, 1, eps)


def conv_residual(h, w):
    """h + causal depthwise convolution of h; w [width, taps]."""
    T, width = h.shape
    taps = w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            src = t - taps + 1 + j
            if src >= 0:
                out[t] += w[:, j] * h[src]
    return out


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(
        math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def dense_ff(x, p):
    return (gelu_tanh(x @ p["gate"].T) * (x @ p["up"].T)) @ p["down"].T


def delta_inputs(h, p, heads, dim):
    """Per-token vectors of the recurrence, each [T, heads, dim]."""
    T = h.shape[0]
    r = (h @ p["r"].T).view(T, heads, dim)
    k = (h @ p["k"].T).view(T, heads, dim)
    v = (h @ p["v"].T).view(T, heads, dim)
    z = torch.tanh(h @ p["w1"].T) @ p["w2"].T + p["w0"]
    w = torch.exp(-math.exp(-0.5) * torch.sigmoid(z)).view(T, heads, dim)
    a = torch.sigmoid(h @ p["a"].T + p["a.b"]).view(T, heads, dim)
    return r, w, k, v, a


def delta_recurrence(r, w, k, v, a, state=None):
    """S <- diag(w) S - (a*u)(u^T S) + k v^T (old S on the right), o = S^T r.
    Inputs [T, heads, dim]; returns (o, final S [heads, dim, dim])."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=r.dtype) if state is None \
        else state.clone()
    u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    o = torch.zeros(T, H, v.shape[-1], dtype=r.dtype)
    for t in range(T):
        for h in range(H):
            old = S[h]
            new = w[t, h][:, None] * old
            new = new - torch.outer(a[t, h] * u[t, h], u[t, h] @ old)
            new = new + torch.outer(k[t, h], v[t, h])
            S[h] = new
            o[t, h] = new.T @ r[t, h]
    return o, S


def delta_output(o, h, p, eps):
    T, H, D = o.shape
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    o = o.reshape(T, H * D) * p["norm"] * torch.sigmoid(h @ p["g"].T)
    return o @ p["o"].T


def general_delta(h, p, mixer, eps):
    r, w, k, v, a = delta_inputs(h, p, mixer["heads"], mixer["dim"])
    o, _ = delta_recurrence(r, w, k, v, a)
    return delta_output(o, h, p, eps)


def window_attention(q, k, v, scale, window):
    """q,k [T, H, D], v [T, H, Dv]; i sees j with 0 <= i-j < window."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(H):
            s = (k[lo:i + 1, h] @ q[i, h]) * scale
            s = torch.exp(s - s.max())
            out[i, h] = (s / s.sum()) @ v[lo:i + 1, h]
    return out


def latent_attention(h, p, mixer, eps):
    T = h.shape[0]
    H, D, Dv = mixer["heads"], mixer["dim"], mixer["vdim"]
    q = (h @ p["q"].T).view(T, H, D)
    c = rms_norm(h @ p["dkv"].T, p["dkv.norm"], eps)
    k = (c @ p["uk"].T).view(T, H, D)
    v = (c @ p["uv"].T).view(T, H, Dv)
    o = window_attention(q, k, v, mixer["scale"], mixer["mask"]["size"])
    o = o.reshape(T, H * Dv) * torch.sigmoid(h @ p["g"].T)
    return o @ p["o"].T


MIXERS = {"general_delta": general_delta, "latent_attention": latent_attention}


def sub(weights, prefix):
    return {n[len(prefix):]: t for n, t in weights.items()
            if n.startswith(prefix)}


def forward(tokens, config, weights):
    """Logits [T, vocab] of one sequence, and the residual stream after
    every layer [layers, T, width]."""
    eps, groups = config["norm"]["eps"], config["norm"]["groups"]
    x = weights["embed"][torch.tensor(tokens)] * config["embedding"]["scale"]
    streams = []
    for i, layer in enumerate(config["layers"]):
        w = sub(weights, f"l{i}.")
        h = conv_residual(group_norm(x, w["norm1"], groups, eps), w["canon1"])
        add = MIXERS[layer["type"]](h, sub(w, "mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            add = add + dense_ff(group_norm(x, w["norm2"], groups, eps),
                                 sub(w, "mlp."))
        x = x + add
        streams.append(x)
    x = group_norm(x, weights["final.norm"], groups, eps)
    return x @ weights["head"].T, torch.stack(streams)
