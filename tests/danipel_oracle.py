"""Plain implementation of the Danipel design, one function per mechanism.

Numerics oracle for tests/test_danipel*.py: whole sequences, loops over tokens,
no cache, no batching, no kernels, and nothing imported from rbg_amd.  It
computes in the dtype of the weights it is given (the tests use float64).
"""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def tanh_norm(x, alpha, w, b):
    """Dynamic tanh: no statistics of the row."""
    return torch.tanh(alpha * x) * w + b


def gelu_tanh(z):
    inner = math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)
    return 0.5 * z * (1 + torch.tanh(inner))


# -- hyper-connections -----------------------------------------------------------


def gather(streams, weights):
    """What a sublayer reads: a weighed sum of the streams [S, T, W]."""
    u = torch.zeros_like(streams[0])
    for s in range(streams.shape[0]):
        u = u + weights[s] * streams[s]
    return u


def scatter(streams, mix, out, y, mult):
    """New streams from the old ones, mix[from, to], and a sublayer's y."""
    new = []
    for to in range(streams.shape[0]):
        x = mult * out[to] * y
        for frm in range(streams.shape[0]):
            x = x + mix[frm, to] * streams[frm]
        new.append(x)
    return torch.stack(new)


# -- rotary positions ------------------------------------------------------------


def frequencies(rot):
    """Angle per position of every pair, and the factor on cosine and sine."""
    dims, base, s = rot["dims"], rot["base"], rot.get("scaling")
    freqs = [base ** (-2 * i / dims) for i in range(dims // 2)]
    if not s:
        return freqs, 1.0

    def dim(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / \
            (2 * math.log(base))
    lo = max(math.floor(dim(s["fast"])), 0)
    hi = min(math.ceil(dim(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1


def rotate(x, rot, interleaved, first=0):
    """x [T, .., dims], row t at position first + t."""
    freqs, mult = frequencies(rot)
    half = rot["dims"] // 2
    out = torch.empty_like(x)
    for t in range(x.shape[0]):
        for i, f in enumerate(freqs):
            a = (first + t) * f
            c, s = math.cos(a) * mult, math.sin(a) * mult
            i0, i1 = (2 * i, 2 * i + 1) if interleaved else (i, i + half)
            u, v = x[t, ..., i0], x[t, ..., i1]
            out[t, ..., i0] = u * c - v * s
            out[t, ..., i1] = v * c + u * s
    return out


# -- latent attention ------------------------------------------------------------


def causal_attention(q, k, v, scale, sink=None):
    """q, k [T, H, D], v [T, H, E]; sink [H]: a logit without key or value."""
    out = []
    for i in range(q.shape[0]):
        s = (k[:i + 1] * q[i]).sum(-1) * scale          # [keys, H]
        if sink is not None:
            s = torch.cat([s, sink.view(1, -1)])
        w = torch.softmax(s, dim=0)[:i + 1]
        out.append((w.unsqueeze(-1) * v[:i + 1]).sum(0))
    return torch.stack(out)


def latent_attention(h, p, m, eps, interleaved):
    """Sink and query latent as far as their tensors are there."""
    T, H, D, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    if "dq" in p:
        q = (rms(h @ p["dq"].T, eps) * p["dq.norm"]) @ p["uq"].T
    else:
        q = h @ p["q"].T
    q = q.view(T, H, D + R)
    low = h @ p["dkv"].T
    c = rms(low[:, :m["kv_rank"]], eps) * p["dkv.norm"]
    kr = rotate(low[:, m["kv_rank"]:], m["rot"], interleaved)
    qr = rotate(q[..., D:], m["rot"], interleaved)
    k = torch.cat([(c @ p["uk"].T).view(T, H, D),
                   kr.unsqueeze(1).expand(T, H, R)], dim=-1)
    v = (c @ p["uv"].T).view(T, H, m["vdim"])
    o = causal_attention(torch.cat([q[..., :D], qr], dim=-1), k, v,
                         m["scale"], p.get("sink"))
    return o.reshape(T, -1) @ p["o"].T


# -- feed-forwards ---------------------------------------------------------------


def dense(h, p):
    return (gelu_tanh(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def clamped_glu(gate, up, limit):
    g = gate.clamp(max=limit)
    u = up.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(h, p, name, limit):
    act = clamped_glu(h @ p[name + ".gate"].T, h @ p[name + ".up"].T, limit)
    return act @ p[name + ".down"].T


def route(logits, correction, top, scale):
    """[(expert, weight)] of one token: chosen by softmax score + correction,
    weighed by the chosen ones' shares of their scores."""
    s = torch.softmax(logits, dim=0)
    order = sorted(range(len(s)), key=lambda e: -(s + correction)[e].item())
    total = sum(s[e] for e in order[:top]) + 1e-20
    return [(e, s[e] / total * scale) for e in order[:top]]


def experts(h, p, mlp):
    r = mlp["router"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(p["router"] @ h[t], p["correction"], r["top"],
                          r["scale"]):
            y = h[t] if e >= r["experts"] else \
                expert(h[t], p, f"e{e}", mlp["expert"]["limit"])
            out[t] += w * y
    if mlp.get("shared"):
        out = out + expert(h, p, "shared", mlp["shared"]["limit"])
    return out


# -- model -----------------------------------------------------------------------


def sub(weights, prefix):
    return {n[len(prefix):]: t for n, t in weights.items()
            if n.startswith(prefix)}


def sublayer(xs, w, which, mult, f):
    n = "norm" + which
    hc = sub(w, f"hc{which}.")
    h = tanh_norm(gather(xs, hc["in"]), w[n + ".alpha"], w[n], w[n + ".b"])
    return scatter(xs, hc["mix"], hc["out"], f(h), mult)


def forward(tokens, config, weights):
    """Logits [T, vocab] of one sequence, and the sum of its streams after
    every layer [layers, T, width]."""
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x = weights["embed"][torch.tensor(tokens)] * config["embedding"]["scale"]
    xs = torch.stack([x] * config["streams"])
    sums = []
    for i, layer in enumerate(config["layers"]):
        w, mlp = sub(weights, f"l{i}."), layer["mlp"]
        xs = sublayer(xs, w, "1", mult, lambda h: latent_attention(
            h, sub(w, "mix."), layer["mixer"], eps,
            layer["type"] == "latent_attention"))
        if mlp is not None:
            p = sub(w, "mlp.")
            xs = sublayer(xs, w, "2", mult, lambda h: dense(h, p)
                          if mlp["kind"] == "dense" else experts(h, p, mlp))
        sums.append(xs.sum(0))
    n = "final.norm"
    h = tanh_norm(xs.sum(0), weights[n + ".alpha"], weights[n],
                  weights[n + ".b"])
    return h @ weights["head"].T, torch.stack(sums)
