"""Plain implementation of the Notadra design, one function per mechanism.

Numerics oracle for tests/test_notadra*.py: whole sequences, loops over tokens,
no cache, no batching, no kernels, and nothing imported from rbg_amd.  It
computes in the dtype of the weights it is given (the tests use float64).
"""
import math

import torch


def norm(x, w, eps):
    """RMS norm; the weight is stored as its distance from one."""
    rms = torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return x / rms * (1 + w)


def embedding(tokens, embed, bigram, cfg):
    """Token rows plus a hashed row for (previous token, token)."""
    out = []
    for t, tok in enumerate(tokens):
        if t == 0:
            row = cfg["buckets"]
        else:
            row = (tokens[t - 1] * cfg["mul_prev"] +
                   tok * cfg["mul_cur"]) % cfg["buckets"]
        out.append(embed[tok] + bigram[row])
    return torch.stack(out)


def frequencies(rot):
    """Angle per position of every rotated pair, and the factor on cos/sin."""
    n, base = rot["dims"], rot["base"]
    plain = [base ** (-2 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if sc is None:
        return plain, 1.0

    def dim_of(turns):
        return n * math.log(sc["original"] / (turns * 2 * math.pi)) / \
            (2 * math.log(base))
    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), n - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0), 1)
        out.append(f / sc["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot, first=0):
    """x [T, heads, dim]: rows at positions first, first + 1, ..."""
    freqs, mult = frequencies(rot)
    half = rot["dims"] // 2
    out = x.clone()
    for t in range(x.shape[0]):
        a = torch.tensor([(first + t) * f for f in freqs], dtype=x.dtype)
        c, s = torch.cos(a) * mult, torch.sin(a) * mult
        u, v = x[t, :, :half], x[t, :, half:2 * half]
        out[t, :, :half] = u * c - v * s
        out[t, :, half:2 * half] = v * c + u * s
    return out


def sink_attention(q, k, v, scale, softcap):
    """Causal; q [T, H, D], k [T, G, D], v [T, G, Dv]; scores are squashed
    into (-softcap, softcap), and the softmax has a silent key of score 0."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    k = k.repeat_interleave(per, dim=1)         # head h reads key head h // per
    v = v.repeat_interleave(per, dim=1)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        s = (k[:i + 1] * q[i]).sum(-1) * scale  # [keys, heads]
        s = softcap * torch.tanh(s / softcap)
        m = s.max(0).values.clamp(min=0)
        e = torch.exp(s - m)
        p = e / (torch.exp(-m) + e.sum(0))
        out[i] = (p.unsqueeze(-1) * v[:i + 1]).sum(0)
    return out


def keys_values(h, p, mixer):
    T, G = h.shape[0], mixer["kv_heads"]
    k = (h @ p["k"].T + p["k.b"]).view(T, G, mixer["dim"])
    v = (h @ p["v"].T + p["v.b"]).view(T, G, mixer["vdim"])
    return rotate(k, mixer["rot"]), v


def attention(h, p, mixer, kv):
    T, H = h.shape[0], mixer["heads"]
    q = (h @ p["q"].T + p["q.b"]).view(T, H, mixer["dim"])
    o = sink_attention(rotate(q, mixer["rot"]), *kv, mixer["scale"],
                       mixer["softcap"])
    return o.reshape(T, -1) @ p["o"].T


def route(logits, correction, router):
    """[(expert, weight)] of one token, from its router logits."""
    s = torch.sigmoid(logits)
    choice = (s + correction).tolist()
    n = len(choice)
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = n // groups["count"]
    totals = []
    for g in range(groups["count"]):
        best = sorted(choice[g * size:(g + 1) * size], reverse=True)[:2]
        totals.append((sum(best), g))
    kept = {g for _, g in sorted(totals, reverse=True)[:groups["keep"]]}
    order = sorted((e for e in range(n) if e // size in kept),
                   key=lambda e: choice[e], reverse=True)
    return [(e, s[e]) for e in order[:router["top"]]]


def expert(x, up, down):
    return torch.relu(x @ up.T) ** 2 @ down.T


def experts(h, p, mlp):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(p["router"] @ h[t], p["correction"], mlp["router"]):
            out[t] += w * expert(h[t], p[f"e{e}.up"], p[f"e{e}.down"])
    return out


def sub(weights, prefix):
    return {n[len(prefix):]: t for n, t in weights.items()
            if n.startswith(prefix)}


def forward(tokens, config, weights):
    """Logits [T, vocab] of one sequence, and the residual stream after
    every layer [layers, T, width]."""
    eps = config["norm"]["eps"]
    x = embedding(tokens, weights["embed"], weights["bigram"],
                  config["embedding"]["bigram"])
    streams, kv = [], {}
    for i, layer in enumerate(config["layers"]):
        w, mixer = sub(weights, f"l{i}."), layer["mixer"]
        h, p = norm(x, w["norm1"], eps), sub(w, "mix.")
        src = mixer.get("kv_from")
        if src is None:
            src = i
            kv[i] = keys_values(h, p, mixer)
        x = x + norm(attention(h, p, mixer, kv[src]), w["norm1b"], eps)
        if layer["mlp"] is not None:
            y = experts(norm(x, w["norm2"], eps), sub(w, "mlp."),
                        layer["mlp"])
            x = x + norm(y, w["norm2b"], eps)
        streams.append(x)
    x = norm(x, weights["final.norm"], eps)
    return x @ weights["head"].T * config["logit_scale"], torch.stack(streams)
