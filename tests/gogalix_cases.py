"""Small Gogalix models for the tests: configuration, weights, and the oracle's
answers (float64, tests/gogalix_oracle.py)."""
import math

import torch

from tests import gogalix_oracle as oracle
from tests.bitatar_cases import prompt, rel_err, row_errs, save  # noqa: F401

VOCAB = 101


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(ff=24, n=6, top=2):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": n, "top": top}}


def delta(heads=4, kv_heads=2, dim=16, vdim=24, taps=3, mlp=dense(),
          kind="delta"):
    return {"type": kind, "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": taps}}


def channel(**kw):
    return delta(kind="channel_delta", **kw)


def attention(heads=4, kv_heads=2, dim=8, vdim=24, window=13, scale=0.4,
              diff=0.35, kv_from=None, mlp=dense()):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "mask": {"size": window}, "scale": scale, "diff": diff}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mlp": mlp, "mixer": m}


def config(layers, width=48, vocab=VOCAB, eps=1e-4, scale=1.5):
    return {"architecture": "Gogalix", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": scale}}


def shapes(cfg, ranks=(5, 12)):
    """ranks: of the low-rank maps to decays and to gates."""
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": ()}
    for i, spec in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", spec["mixer"], spec["mlp"]
        out[p + "norm1"] = ()
        H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        if spec["type"] == "attention":
            mix = {"q": (H * 2 * D, w)}
            if m.get("kv_from") is None:
                mix.update(k=(G * 2 * D, w), v=(G * E, w))
            mix.update({n: (D,) for n in ("lq1", "lk1", "lq2", "lk2")})
        else:
            mix = {"q": (G * D, w), "k": (G * D, w), "v": (H * E, w)}
            mix.update({n + ".conv": (s[0], m["conv"])
                        for n, s in list(mix.items())})
            mix.update(b=(H, w), A_log=(H,), norm=(E,))
            if spec["type"] == "delta":
                mix.update(a=(H, w), dt_bias=(H,), g=(H * E, w))
            else:
                mix.update(a1=(ranks[0], w), a2=(H * D, ranks[0]),
                           dt_bias=(H * D,), g1=(ranks[1], w),
                           g2=(H * E, ranks[1]))
        mix["o"] = (w, H * E)
        out.update({p + "mix." + n: s for n, s in mix.items()})
        for b in ("1", "2")[:1 if mlp is None else 2]:
            out[p + "ls" + b] = (w,)
            out[p + "rg" + b] = (w, w)
            out[p + f"rg{b}.b"] = (w,)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            for n, s in (("gate", (ff, w)), ("up", (ff, w)),
                         ("down", (w, ff))):
                out[p + "mlp." + n] = s
                out[p + f"mlp.{n}.b"] = s[:1]
            continue
        n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        for e in range(n):
            out[f"{p}mlp.e{e}.gate"] = out[f"{p}mlp.e{e}.up"] = (ff, w)
            out[f"{p}mlp.e{e}.down"] = (w, ff)
        out[p + "mlp.router"] = (n, w)
        out[p + "mlp.router.b"] = (n,)
    return out


def weights(cfg, seed=0, sharpen=3.0, ranks=(5, 12)):
    """bf16 values.  Queries of attention are sharpened so that single keys
    stand out.  Tokens are of two kinds, far apart along one direction that the
    routers look at, and router biases are spread: rounding does not change
    which experts are chosen.  Decays range from almost none to fast."""
    gen = torch.Generator().manual_seed(seed)
    kind = torch.randn(cfg["width"], generator=gen).sign()
    out = {}
    for name, shape in shapes(cfg, ranks).items():
        t = torch.randn(shape, generator=gen)
        layer = cfg["layers"][int(name[1:].split(".")[0])] \
            if name.startswith("l") else None
        if "norm" in name.split(".")[-1]:
            t = 1 + 0.2 * t
        elif name == "embed":
            t += 2.0 * kind * (torch.arange(shape[0]) % 2 * 2 - 1).view(-1, 1)
        elif name.endswith("router"):
            side = (torch.arange(shape[0]) % 2 * 2 - 1).view(-1, 1)
            t = (0.1 * t + 4.0 * side * kind / math.sqrt(shape[1])) / \
                math.sqrt(shape[1])
        elif name.endswith("router.b"):
            t = 0.7 * torch.randperm(shape[0], generator=gen) - 1
        elif name.endswith("A_log"):
            t = 1.5 * t - 1
        elif name.endswith("dt_bias"):
            t = t - 2
        elif name.endswith(".conv"):
            t = 0.5 * t
        elif name[-3:] in ("ls1", "ls2"):
            t = 0.8 + 0.3 * t
        elif name[-3:] in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.3 * t
        elif name.endswith(".b"):
            t = 0.3 * t
        elif len(shape) == 2:
            t = t / math.sqrt(shape[1])
            if name.endswith("mix.q") and layer["type"] == "attention":
                t = t * sharpen
        out[name] = t.bfloat16()
    return out


def answers(tokens, cfg, w):
    return oracle.forward(tokens, cfg, {n: t.double() for n, t in w.items()})[0]
