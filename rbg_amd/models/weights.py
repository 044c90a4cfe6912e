"""Where a model's tensors come from: a safetensors file or a seed.

The file format is an 8-byte little-endian header length, that many bytes of
JSON (name -> dtype, shape, data_offsets relative to the header's end), and the
raw little-endian data.
"""
from __future__ import annotations

import json
import math
import mmap
import os
import zlib
from typing import Dict, Optional, Set, Tuple

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32,
           "F64": torch.float64, "I64": torch.int64, "I32": torch.int32,
           "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8,
           "BOOL": torch.bool}


class WeightSource:
    """take() one tensor by name, as stored (weights keep their dtype)."""

    def shape(self, name: str, default: Tuple[int, ...]) -> Tuple[int, ...]:
        raise NotImplementedError

    def take(self, name: str, shape: Tuple[int, ...], init: str = "linear"
             ) -> torch.Tensor:
        raise NotImplementedError

    def finish(self, optional: Set[str] = frozenset()) -> None:
        """Called when a model has everything it needs."""


class SafetensorsSource(WeightSource):
    def __init__(self, path: str, device: torch.device):
        if os.path.isdir(path):
            path = os.path.join(path, "model.safetensors")
        self.path, self.device = path, device
        with open(path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        n = int.from_bytes(self._map[:8], "little")
        if n > len(self._map) - 8:
            raise ValueError(f"{path}: header longer than the file")
        self._meta: Dict[str, dict] = json.loads(self._map[8:8 + n])
        self._meta.pop("__metadata__", None)
        self._base = 8 + n
        self._taken: Set[str] = set()

    def shape(self, name, default):
        return tuple(self._entry(name)["shape"])

    def _entry(self, name: str) -> dict:
        if name not in self._meta:
            raise KeyError(f"{self.path} has no tensor {name!r}")
        return self._meta[name]

    def take(self, name, shape, init="linear"):
        e = self._entry(name)
        if tuple(e["shape"]) != tuple(shape):
            raise ValueError(f"tensor {name!r} is {e['shape']}, the "
                             f"configuration needs {list(shape)}")
        lo, hi = e["data_offsets"]
        dtype = _DTYPES[e["dtype"]]
        if (hi - lo != math.prod(shape) * dtype.itemsize or lo < 0 or
                self._base + hi > len(self._map)):
            raise ValueError(f"tensor {name!r}: bad data_offsets")
        self._taken.add(name)
        raw = bytearray(self._map[self._base + lo:self._base + hi])
        t = torch.frombuffer(raw, dtype=dtype) if raw else \
            torch.empty(0, dtype=dtype)
        return t.view(tuple(shape)).to(self.device)

    def finish(self, optional=frozenset()):
        rest = set(self._meta) - self._taken - set(optional)
        if rest:
            raise ValueError(f"{self.path}: tensors that the model does not "
                             f"use: {sorted(rest)[:8]}")


class RandomSource(WeightSource):
    """Seeded weights; a tensor depends on (seed, name) only, so every
    parallel degree sees the same model."""

    def __init__(self, seed: int, device: torch.device,
                 dtype: torch.dtype = torch.bfloat16):
        self.seed, self.device, self.dtype = seed, device, dtype

    def shape(self, name, default):
        return tuple(default)

    def take(self, name, shape, init="linear"):
        gen = torch.Generator(device=self.device)
        gen.manual_seed(self.seed * 1000003 + zlib.crc32(name.encode()))
        t = torch.empty(shape, device=self.device, dtype=self.dtype)
        if init == "ones":
            return t.fill_(1.0)
        if init == "zeros":
            return t.zero_()
        if init == "eye":
            return t.copy_(torch.eye(*shape))
        scale = 1.0
        if init == "linear":
            scale = 1.0 / math.sqrt(shape[-1])
        elif init == "conv":
            scale = 0.5 / math.sqrt(shape[-1])
        elif init == "rate":        # of a decay, before its softplus
            return t.normal_(-3.0, 1.0, generator=gen)
        return t.normal_(0.0, scale, generator=gen)


def open_weights(path: str, seed: int, device: torch.device) -> WeightSource:
    if path:
        return SafetensorsSource(path, device)
    return RandomSource(seed, device)
