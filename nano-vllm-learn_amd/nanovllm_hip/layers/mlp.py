"""Dense feed-forwards.
ClampedGLU: down(g sigmoid(alpha g) (u + 1)), g = min(gate, limit), u = clamp(up, -limit, limit).  GeluGLU: down(gelu(gate) up), the tanh form.
PolyNormMLP: down(a N(z) + b N(z^2) + c N(z^3) + e), z = up(x), powers by element, N(v) = v / sqrt(mean(v^2) + eps) over a token's values."""
import torch
import torch.nn.functional as F
from torch import nn

from .. import ops
from .linear import linear, padded, round_up


class GatedMLP(nn.Module):
    """down(unit(gate, up)); `unit`: the fused projection's `glu`, `rows_unit`: the same over rows."""

    def __init__(self, in_width, in_cols, ff, dtype, unit, rows_unit):
        super().__init__()
        self.in_width, self.in_cols, self.ff, self.dtype, self.unit, self.rows_unit = in_width, in_cols, ff, dtype, unit, rows_unit
        self.cols = round_up(ff, 64)

    def load(self, get):
        assert get("gate").shape == (self.ff, self.in_width)
        self.register_buffer("w_gate_up", torch.cat([padded(get(n), self.cols, self.in_cols) for n in ("gate", "up")]).to(self.dtype).contiguous())
        self.register_buffer("w_down", padded(get("down"), self.in_cols, self.cols).to(self.dtype).contiguous())

    def forward(self, x):
        if x.dtype == torch.bfloat16 and x.shape[0] <= ops.LINEAR_SMALL_M_MAX:
            act = ops.fused_linear(x, self.w_gate_up, epilogue="silu_mul", glu=self.unit)
        else:
            act = self.rows_unit(F.linear(x, self.w_gate_up))
        return linear(act, self.w_down)

    def decode(self, xp, rows, bufs):
        mid = bufs.packed(self.cols)
        ops.fused_linear(xp, self.w_gate_up, x_packed_rows=rows, epilogue="silu_mul", glu=self.unit, out_packed=mid, want_out=False,
                         workspace=bufs.workspace)
        return ops.fused_linear(mid, self.w_down, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_gate_up, "silu_mul"), (self.w_down, "none")]


class ClampedGLU(GatedMLP):
    def __init__(self, in_width, in_cols, ff, limit, dtype, alpha=1.702):
        super().__init__(in_width, in_cols, ff, dtype, (float(limit), alpha), lambda rows: ops.clamped_glu(rows, float(limit), alpha))
        self.limit, self.alpha = float(limit), alpha


class GeluGLU(GatedMLP):
    def __init__(self, in_width, in_cols, ff, dtype):
        super().__init__(in_width, in_cols, ff, dtype, "gelu", ops.gelu_glu)


class PolyNormMLP(nn.Module):
    def __init__(self, in_width, in_cols, ff, eps, dtype):
        super().__init__()
        self.in_width, self.in_cols, self.ff, self.eps, self.dtype = in_width, in_cols, ff, eps, dtype
        self.cols = round_up(ff, 64)

    def load(self, get):
        assert get("up").shape == (self.ff, self.in_width) and get("act").numel() == 4
        self.register_buffer("w_up", padded(get("up"), self.cols, self.in_cols).to(self.dtype).contiguous())
        self.register_buffer("w_down", padded(get("down"), self.in_cols, self.cols).to(self.dtype).contiguous())
        self.register_buffer("coef", get("act").float().contiguous())

    def forward(self, x):
        return linear(ops.poly_norm(linear(x, self.w_up), self.coef, self.eps, self.ff), self.w_down)

    def decode(self, xp, rows, bufs):
        z = ops.fused_linear(xp, self.w_up, x_packed_rows=rows, workspace=bufs.workspace)
        mid = bufs.packed(self.cols)
        ops.poly_norm(z, self.coef, self.eps, self.ff, packed=mid)
        return ops.fused_linear(mid, self.w_down, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_up, "none"), (self.w_down, "none")]
