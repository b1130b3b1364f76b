"""Dense feed-forward with a clamped gated unit: down(g sigmoid(alpha g) (u + 1)), g = min(gate, limit), u = clamp(up, -limit, limit)."""
import torch
import torch.nn.functional as F
from torch import nn

from .. import ops
from .linear import linear, padded, round_up


class ClampedGLU(nn.Module):
    def __init__(self, in_width, in_cols, ff, limit, dtype, alpha=1.702):
        super().__init__()
        self.in_width, self.in_cols, self.ff, self.limit, self.alpha, self.dtype = in_width, in_cols, ff, float(limit), alpha, dtype
        self.cols = round_up(ff, 64)

    def load(self, get):
        assert get("gate").shape == (self.ff, self.in_width)
        self.register_buffer("w_gate_up", torch.cat([padded(get(n), self.cols, self.in_cols) for n in ("gate", "up")]).to(self.dtype).contiguous())
        self.register_buffer("w_down", padded(get("down"), self.in_cols, self.cols).to(self.dtype).contiguous())

    def forward(self, x):
        if x.dtype == torch.bfloat16 and x.shape[0] <= ops.LINEAR_SMALL_M_MAX:
            act = ops.fused_linear(x, self.w_gate_up, epilogue="silu_mul", glu=(self.limit, self.alpha))
        else:
            act = ops.clamped_glu(F.linear(x, self.w_gate_up), self.limit, self.alpha)
        return linear(act, self.w_down)

    def decode(self, xp, rows, bufs):
        mid = bufs.packed(self.cols)
        ops.fused_linear(xp, self.w_gate_up, x_packed_rows=rows, epilogue="silu_mul", glu=(self.limit, self.alpha), out_packed=mid, want_out=False,
                         workspace=bufs.workspace)
        return ops.fused_linear(mid, self.w_down, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_gate_up, "silu_mul"), (self.w_down, "none")]
