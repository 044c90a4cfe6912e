"""Rotary position tables, computed in float64 on the host.

``rot`` is a configuration's rotation: dims (rotated leading dimensions of a
head), base, and optionally a YaRN-style scaling (factor, original, fast, slow):
pairs that turn more than ``fast`` times over the original length keep their
frequency, those that turn less than ``slow`` times are slowed down by
``factor``, with a linear ramp over the pair index between.
"""
from __future__ import annotations

import json
import math
from typing import Any, Dict, Iterable, Tuple

import torch


def rotation(rot: Dict[str, Any]) -> Tuple[torch.Tensor, float]:
    """Angle per position of each pair (float64), and the factor that cosine
    and sine are multiplied by."""
    dims, base = int(rot["dims"]), float(rot["base"])
    if dims <= 0 or dims % 2:
        raise ValueError(f"rotated dimensions must be even, not {dims}")
    pair = torch.arange(dims // 2, dtype=torch.float64)
    freq = base ** (-2.0 * pair / dims)
    scaling = rot.get("scaling")
    if not scaling:
        return freq, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_turning(times: float) -> float:
        return dims * math.log(original / (2 * math.pi * times)) / \
            (2 * math.log(base))
    first = max(math.floor(pair_turning(float(scaling["fast"]))), 0)
    last = min(math.ceil(pair_turning(float(scaling["slow"]))), dims - 1)
    ramp = ((pair - first) / max(last - first, 0.001)).clamp(0, 1)
    return (freq / factor * ramp + freq * (1 - ramp),
            0.1 * math.log(factor) + 1.0)


def rotary_table(rot: Dict[str, Any], positions: int,
                 device: torch.device) -> torch.Tensor:
    """f32 [positions, dims] = [cosines | sines]."""
    freq, mult = rotation(rot)
    angle = torch.outer(torch.arange(positions, dtype=torch.float64), freq)
    return (torch.cat([angle.cos(), angle.sin()], dim=1) * mult).float().to(
        device)


def assign_tables(mixers: Iterable, positions: int,
                  device: torch.device) -> None:
    """Gives every mixer with a rotation (``rot``) its table (``cos_sin``); one
    per distinct rotation."""
    tables: Dict[str, torch.Tensor] = {}
    for mixer in mixers:
        if mixer.rot is None:
            continue
        key = json.dumps(mixer.rot, sort_keys=True)
        if key not in tables:
            tables[key] = rotary_table(mixer.rot, positions, device)
        mixer.cos_sin = tables[key]
