"""Small Notadra models for the tests: configuration, weights, and the oracle's
answers (float64, tests/notadra_oracle.py)."""
import math

import torch

from tests import notadra_oracle as oracle
from tests.bitatar_cases import prompt, rel_err, row_errs, save  # noqa: F401

VOCAB = 101


def rot(dims=8, base=1000.0, factor=4.0, original=64, fast=8.0, slow=1.0):
    return {"dims": dims, "base": base,
            "scaling": {"factor": factor, "original": original, "fast": fast,
                        "slow": slow}}


def attention(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.3, softcap=20.0,
              kv_from=None, **kw):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale, "softcap": softcap, "rot": rot(**kw)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def experts(ff=24, n=8, top=2, count=4, keep=2):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": n, "top": top,
                       "groups": {"count": count, "keep": keep}}}


def layer(mixer=None, mlp=None, **kw):
    return {"type": "attention", "mixer": mixer or attention(**kw),
            "mlp": experts() if mlp is None else mlp or None}


def config(layers, width=48, vocab=VOCAB, eps=1e-4, logit_scale=0.7,
           buckets=37, mul_prev=13, mul_cur=5):
    return {"architecture": "Notadra", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps},
            "logit_scale": logit_scale,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev,
                                     "mul_cur": mul_cur}}}


def shapes(cfg):
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": (w,),
           "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, w)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        out[p + "norm1"] = out[p + "norm1b"] = (w,)
        sizes = {"q": m["heads"] * m["dim"]}
        if m.get("kv_from") is None:
            sizes.update(k=m["kv_heads"] * m["dim"],
                         v=m["kv_heads"] * m["vdim"])
        for name, n in sizes.items():
            out[p + "mix." + name] = (n, w)
            out[p + "mix." + name + ".b"] = (n,)
        out[p + "mix.o"] = (w, m["heads"] * m["vdim"])
        if spec["mlp"] is None:
            continue
        out[p + "norm2"] = out[p + "norm2b"] = (w,)
        n, ff = spec["mlp"]["router"]["experts"], spec["mlp"]["expert"]["ff"]
        for e in range(n):
            out[f"{p}mlp.e{e}.up"] = (ff, w)
            out[f"{p}mlp.e{e}.down"] = (w, ff)
        out[p + "mlp.router"] = (n, w)
        out[p + "mlp.correction"] = (n,)
    return out


def weights(cfg, seed=0, sharpen=2.5):
    """bf16 values.  Queries are sharpened so that single keys stand out.
    Tokens are of two kinds, far apart along one direction that the routers
    look at: each kind has its experts, and rounding does not change who is
    chosen."""
    gen = torch.Generator().manual_seed(seed)
    kind = torch.randn(cfg["width"], generator=gen).sign()
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=gen)
        if "norm" in name.split(".")[-1]:
            t = 0.3 * t
        elif name == "embed":
            t += 3.0 * kind * (torch.arange(shape[0]) % 2 * 2 - 1).view(-1, 1)
        elif name.endswith("correction"):
            t = 0.2 * t - 0.7               # choice scores of both signs
        elif name.endswith(".b"):
            t = 0.3 * t
        elif name.endswith("router"):
            side = (torch.arange(shape[0]) // 2 % 2 * 2 - 1).view(-1, 1)
            t = (0.1 * t + 4.0 * side * kind / math.sqrt(shape[1])) / \
                math.sqrt(shape[1])
        elif len(shape) == 2 and name != "bigram":
            t = t / math.sqrt(shape[1])
            if name.endswith("mix.q"):
                t = t * sharpen
        out[name] = t.bfloat16()
    return out


def answers(tokens, cfg, w):
    return oracle.forward(tokens, cfg, {n: t.double() for n, t in w.items()})[0]
