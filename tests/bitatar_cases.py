"""Small Bitatar models for the tests: configuration, weights, model folder,
and the oracle's answers (float64, tests/bitatar_oracle.py)."""
import json
import math
import os

import torch

from tests import bitatar_oracle as oracle


def config(layers, width=48, vocab=101, groups=3, taps=3, eps=1e-5,
           scale=3.5):
    return {"architecture": "Bitatar", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps, "groups": groups},
            "embedding": {"scale": scale}, "canon": {"taps": taps}}


def delta(heads=2, dim=12, ff=40):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def latent(heads=3, dim=8, vdim=16, rank=24, window=21, scale=0.6, ff=40):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "kv_rank": rank, "mask": {"size": window},
                      "scale": scale},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def shapes(cfg, decay_rank=10):
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (w,)
        out[p + "canon1"] = (w, cfg["canon"]["taps"])
        if layer["type"] == "general_delta":
            n = m["heads"] * m["dim"]
            for name in ("r", "k", "v", "a", "g"):
                out[p + "mix." + name] = (n, w)
            for name in ("a.b", "w0", "norm"):
                out[p + "mix." + name] = (n,)
            out[p + "mix.w1"] = (decay_rank, w)
            out[p + "mix.w2"] = (n, decay_rank)
            out[p + "mix.o"] = (w, n)
        else:
            qk, vo, r = (m["heads"] * m["dim"], m["heads"] * m["vdim"],
                         m["kv_rank"])
            out.update({p + "mix.q": (qk, w), p + "mix.dkv": (r, w),
                        p + "mix.dkv.norm": (r,), p + "mix.uk": (qk, r),
                        p + "mix.uv": (vo, r), p + "mix.g": (vo, w),
                        p + "mix.o": (w, vo)})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (w,), p + "mlp.gate": (ff, w),
                        p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return out


def weights(cfg, seed=0, decay_rank=10, sharpen=2.0):
    """bf16 values.  Queries are sharpened so that single keys stand out: a
    key too many or too few at a window's edge changes the logits."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg, decay_rank).items():
        t = torch.randn(shape, generator=gen)
        if name.endswith("norm") or name[-5:] in ("norm1", "norm2"):
            t = 1 + 0.2 * t
        elif name.endswith("canon1"):
            t = 0.4 * t
        elif len(shape) == 2:
            t = t / math.sqrt(shape[1])
            if name.endswith("mix.q"):
                t = t * sharpen
        out[name] = t.bfloat16()
    return out


_TAGS = {torch.bfloat16: "BF16", torch.float32: "F32"}


def save(folder, cfg, w):
    """config.json + model.safetensors, written by hand."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    meta, blobs, at = {}, [], 0
    for name, t in w.items():
        raw = t.contiguous().view(-1).view(torch.uint8).numpy().tobytes()
        meta[name] = {"dtype": _TAGS[t.dtype], "shape": list(t.shape),
                      "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(meta).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(len(head).to_bytes(8, "little") + head + b"".join(blobs))
    return str(folder)


def answers(tokens, cfg, w):
    return oracle.forward(tokens, cfg, {n: t.double() for n, t in w.items()})[0]


def prompt(n, vocab=101, seed=0):
    gen = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, vocab, (n,), generator=gen).tolist()


def row_errs(got, want):
    """Per row: RMS of the difference over the RMS of all answers."""
    d = (got.double().cpu() - want).pow(2).mean(-1).sqrt()
    return d / want.pow(2).mean().sqrt()


def rel_err(got, want):
    return row_errs(got, want).max().item()
