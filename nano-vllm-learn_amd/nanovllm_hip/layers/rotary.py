"""Rotation tables: fp32 [max_position, dims] = cos | sin of position * frequency, one copy per device shared by all layers.
Angles are reduced in double precision, so a table entry is the correctly rounded one at any position."""
import math

import torch

_TABLES = {}


def frequencies(dims, base, scaling=None):
    """base^(-2i/dims) per pair.  scaling = dict(factor, low, high, original), as in Llama 3.1: a pair that turns fewer than `low` times over `original`
    positions is slowed down by `factor`, one that turns more than `high` times is kept, between the two the share of the kept frequency grows
    linearly with the number of turns."""
    freq = float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    if scaling is None:
        return freq
    turns = float(scaling["original"]) * freq / (2.0 * math.pi)
    low, high = float(scaling["low"]), float(scaling["high"])
    kept = ((turns - low) / (high - low)).clamp(0.0, 1.0) if high > low else (turns > low).double()
    return (1.0 - kept) * freq / float(scaling["factor"]) + kept * freq


def rotation_table(dims, base, max_position, device, scaling=None):
    key = (dims, float(base), max_position, str(device), None if scaling is None else tuple(sorted((k, float(v)) for k, v in scaling.items())))
    if key not in _TABLES:
        angle = torch.arange(max_position, dtype=torch.float64)[:, None] * frequencies(dims, base, scaling)[None, :]
        _TABLES[key] = torch.cat((angle.cos(), angle.sin()), dim=1).float().contiguous().to(device)
    return _TABLES[key]


def halves_to_pairs(width, dims):
    """Index that brings the pairs (i, i + dims / 2) of the first `dims` of `width` dimensions next to each other, as the kernels turn them."""
    half = torch.arange(dims // 2)
    return torch.cat((torch.stack((half, half + dims // 2), dim=1).reshape(-1), torch.arange(dims, width)))
