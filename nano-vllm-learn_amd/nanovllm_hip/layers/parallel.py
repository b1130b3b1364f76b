"""Two mixers side by side on the same rows: softmax attention over pages and a selective scan, one projection in front of both.  Their outputs are returned as they
are, with the weights of their norms: half the sum of the normed ones is taken where the residual streams are updated (ops.stream_mix)."""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded


class ParallelMixer(nn.Module):
    mixes = ()

    def __init__(self, in_width, in_cols, left, right):
        super().__init__()
        self.in_width, self.in_cols, self.left, self.right = in_width, in_cols, left, right
        self.step_ok = left.step_ok and right.step_ok
        self.segment_units = right.segment_units

    def load(self, get):
        for name in ("left", "right"):
            getattr(self, name).load(lambda n: get(f"{name}.{n}"))
            self.register_buffer(f"{name}_out", padded(get(f"{name}.out").float(), self.in_cols))
        self.register_buffer("w_in", torch.cat([self.left.w_qkv, self.right.w_in]).contiguous())
        self.left.w_qkv = self.right.w_in = None             # (one projection for both)

    def _result(self, left, right):
        return dict(y=left, post=(right, self.left_out, self.right_out, 0.5))

    def forward(self, x, positions, step):
        a, cut = linear(x, self.w_in), self.left.proj_cols
        return self._result(linear(self.left.attend(a[:, :cut], positions, step), self.left.w_o), linear(self.right.scan(a[:, cut:], positions, step), self.right.w_o))

    def decode(self, xp, rows, positions, step, bufs):
        """Fused decode: fragment-packed rows in, output rows out (eight launches)."""
        a, cut = ops.fused_linear(xp, self.w_in, x_packed_rows=rows, workspace=bufs.workspace), self.left.proj_cols
        left = ops.fused_linear(self.left.decode_attend(a[:, :cut], positions, step, bufs), self.left.w_o, x_packed_rows=rows, workspace=bufs.workspace)
        right = ops.fused_linear(self.right.decode_scan(a[:, cut:], rows, positions, step, bufs), self.right.w_o, x_packed_rows=rows, workspace=bufs.workspace)
        return self._result(left, right)

    def linears(self):
        return [(w, "none") for w in (self.w_in, self.left.w_o, self.right.w_x, self.right.w_o)]
