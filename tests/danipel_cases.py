"""Small Danipel models for the tests: configuration, weights, and the oracle's
answers (float64, tests/danipel_oracle.py)."""
import math

import torch

from tests import danipel_oracle as oracle
from tests.bitatar_cases import prompt, rel_err, row_errs, save  # noqa: F401

VOCAB = 101
YARN = {"factor": 6.0, "original": 40, "fast": 4.0, "slow": 0.5}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(ff=24, n=5, identity=3, top=2, scale=1.8, limit=0.9, shared=(32, 0.6)):
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
           "router": {"experts": n, "identity": identity, "top": top,
                      "scale": scale}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def direct(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, scale=0.3,
           base=300.0, scaling=YARN, mlp=dense(), kind="latent_attention"):
    rot = {"dims": rot_dim, "base": base}
    if scaling:
        rot["scaling"] = scaling
    return {"type": kind, "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim,
                      "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": rot}}


def indirect(q_rank=32, scaling=None, **kw):
    out = direct(kind="latent_attention_2", scaling=scaling, **kw)
    out["mixer"]["q_rank"] = q_rank
    return out


def config(layers, width=48, vocab=VOCAB, eps=3e-2, scale=1.4, streams=2,
           mult=0.6):
    return {"architecture": "Danipel", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "streams": streams,
            "residual_mult": mult}


def norm_shapes(name, w):
    return {name: (w,), name + ".b": (w,), name + ".alpha": ()}


def shapes(cfg):
    w, v, n = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {"embed": (v, w), "head": (v, w), **norm_shapes("final.norm", w)}
    for i, spec in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", spec["mixer"], spec["mlp"]
        for b in ("1", "2")[:1 if mlp is None else 2]:
            out.update(norm_shapes(p + "norm" + b, w))
            out.update({p + f"hc{b}.in": (n,), p + f"hc{b}.out": (n,),
                        p + f"hc{b}.mix": (n, n)})
        H, R = m["heads"], m["kv_rank"]
        qk = H * (m["dim"] + m["rot_dim"])
        if spec["type"] == "latent_attention":
            mix = {"q": (qk, w), "sink": (H,)}
        else:
            mix = {"dq": (m["q_rank"], w), "dq.norm": (m["q_rank"],),
                   "uq": (qk, m["q_rank"])}
        mix.update({"dkv": (R + m["rot_dim"], w), "dkv.norm": (R,),
                    "uk": (H * m["dim"], R), "uv": (H * m["vdim"], R),
                    "o": (w, H * m["vdim"])})
        out.update({p + "mix." + name: s for name, s in mix.items()})
        if mlp is None:
            continue
        parts = {"": mlp.get("ff")}
        if mlp["kind"] == "moe":
            r = mlp["router"]
            parts = {f"e{e}.": mlp["expert"]["ff"]
                     for e in range(r["experts"])}
            every = r["experts"] + r["identity"]
            out[p + "mlp.router"] = (every, w)
            out[p + "mlp.correction"] = (every,)
            if mlp.get("shared"):
                parts["shared."] = mlp["shared"]["ff"]
        for part, ff in parts.items():
            out[p + f"mlp.{part}gate"] = out[p + f"mlp.{part}up"] = (ff, w)
            out[p + f"mlp.{part}down"] = (w, ff)
    return out


def weights(cfg, seed=0, sharpen=3.0):
    """bf16 values.  Queries are sharpened so that single keys stand out, and
    sinks matter.  Tokens are of two kinds, far apart along one direction that
    the routers look at, and corrections are spread: rounding does not change
    which experts are chosen."""
    gen = torch.Generator().manual_seed(seed)
    kind = torch.randn(cfg["width"], generator=gen).sign()
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=gen)
        last = name.split(".")[-1]
        if last == "alpha":
            t = 0.6 + 0.2 * torch.rand(shape, generator=gen)
        elif last.startswith("norm"):
            t = 1 + 0.2 * t
        elif last == "b":
            t = 0.3 * t
        elif last == "in":
            t = 1 / cfg["streams"] + 0.3 * t
        elif last == "out":
            t = 0.8 + 0.4 * t
        elif last == "mix":
            t = torch.eye(shape[0]) + 0.25 * t
        elif last == "sink":
            t = 1.5 + t
        elif name == "embed":
            t += 2.0 * kind * (torch.arange(shape[0]) % 2 * 2 - 1).view(-1, 1)
        elif last == "router":
            side = (torch.arange(shape[0]) % 2 * 2 - 1).view(-1, 1)
            t = (0.1 * t + 6.0 * side * kind / math.sqrt(shape[1])) / \
                math.sqrt(shape[1])
        elif last == "correction":
            t = 0.04 * torch.randperm(shape[0], generator=gen) - 0.1
        elif len(shape) == 2:
            t = t / math.sqrt(shape[1])
            if last in ("q", "uq"):
                t = t * sharpen
        out[name] = t.bfloat16()
    return out


def answers(tokens, cfg, w):
    return oracle.forward(tokens, cfg, {n: t.double() for n, t in w.items()})[0]
