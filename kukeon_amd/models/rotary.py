"""Rotary angle tables.

`angle_table` covers plain rotary frequencies and two rescalings of them,
told apart by the keys of `scaling`:

* `fast` / `slow` (YaRN): frequencies whose wavelength exceeds the original
  context are divided by `factor`, short wavelengths are kept, and a linear
  ramp over the pair index blends the two; cos and sin are then scaled by
  0.1 ln(factor) + 1.
* `low` / `high` (the bands of Llama 3.1): a frequency that turns more than
  `high` times over the original context is kept, one that turns less than
  `low` times is divided by `factor`, and those between are blended linearly
  in the number of turns; cos and sin are not scaled.

Angles are formed in float64 and the table is stored in fp32, one row per
position: [cos_0 .. cos_(n-1) | sin_0 .. sin_(n-1)] with n = dims / 2.
"""
from __future__ import annotations

import math
from typing import Optional

import torch


def pair_frequencies(dims: int, base: float,
                     scaling: Optional[dict] = None):
    """-> (freq [dims/2] float64, amplitude) for pair i = dims 2i, 2i+1."""
    n = dims // 2
    i = torch.arange(n, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64),
                  -2.0 * i / dims)
    amp = 1.0
    if scaling and "low" in scaling:
        factor = float(scaling["factor"])
        low, high = float(scaling["low"]), float(scaling["high"])
        turns = float(scaling["original"]) * f / (2.0 * math.pi)
        s = (turns - low) / (high - low) if high != low else turns * 0.0
        f = torch.where(turns > high, f, torch.where(
            turns < low, f / factor, (1.0 - s) * f / factor + s * f))
    elif scaling:
        factor = float(scaling["factor"])
        orig = float(scaling["original"])

        def pair_of(turns: float) -> float:
            # pair index whose wavelength makes `turns` rotations over
            # the original context
            return dims * math.log(orig / (2.0 * math.pi * turns)) / \
                (2.0 * math.log(base))

        lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
        hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        f = f / factor * ramp + f * (1.0 - ramp)
        amp = 0.1 * math.log(factor) + 1.0
    return f, amp


def angle_table(positions: int, dims: int, base: float,
                scaling: Optional[dict] = None) -> torch.Tensor:
    f, amp = pair_frequencies(dims, base, scaling)
    ang = torch.arange(positions, dtype=torch.float64)[:, None] * f[None, :]
    return torch.cat([ang.cos() * amp, ang.sin() * amp], dim=1).float()


def scaling_key(scaling: Optional[dict]) -> tuple:
    """A frequency rescaling as a value to keep in a frozen configuration."""
    return tuple(sorted((k, float(v)) for k, v in (scaling or {}).items()))


def attach_tables(mixers, positions: int, device) -> None:
    """Give every mixer that rotates (its configuration has `rot_dims`) its
    angle table `cs` for positions 0 .. positions-1; equal ones are shared."""
    tables = {}
    for mx in mixers:
        if not hasattr(mx.m, "rot_dims"):
            continue
        scaling = getattr(mx.m, "rot_scaling", ())
        key = (mx.m.rot_dims, mx.m.rot_base, scaling)
        if key not in tables:
            tables[key] = angle_table(positions, mx.m.rot_dims,
                                      mx.m.rot_base, dict(scaling)).to(device)
        mx.cs = tables[key]


def pairs_from_half(dims: int, n: int) -> torch.Tensor:
    """Row order that turns the half layout of a part of n entries, of which
    the first `dims` rotate (entry i with i + dims/2), into the pair layout:
    new[2i] = old[i], new[2i+1] = old[i + dims/2]."""
    half = dims // 2
    order = []
    for i in range(half):
        order += [i, i + half]
    return torch.tensor(order + list(range(dims, n)), dtype=torch.long)
