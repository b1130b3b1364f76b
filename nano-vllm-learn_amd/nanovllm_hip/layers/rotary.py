"""Rotation tables: fp32 [max_position, dims] = cos | sin of position * base^(-2i/dims), one copy per device shared by all layers.
Angles are reduced in double precision, so a table entry is the correctly rounded one at any position."""
import torch

_TABLES = {}


def rotation_table(dims, base, max_position, device):
    key = (dims, float(base), max_position, str(device))
    if key not in _TABLES:
        freq = float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
        angle = torch.arange(max_position, dtype=torch.float64)[:, None] * freq[None, :]
        _TABLES[key] = torch.cat((angle.cos(), angle.sin()), dim=1).float().contiguous().to(device)
    return _TABLES[key]
