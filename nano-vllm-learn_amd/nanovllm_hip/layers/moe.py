"""Mixture of experts: a sigmoid router with choice corrections over groups of neighbouring experts, or a softmax over the chosen logits, and small gated
feed-forwards without biases (SiLU, or the clamped unit).
The module returns the chosen experts' outputs and weights; ops.residual_norm adds their weighted sum to the stream."""
import torch
from torch import nn

from .. import ops
from .linear import padded, round_up


class MixtureOfExperts(nn.Module):
    def __init__(self, in_width, in_cols, ff, experts, top, dtype, groups=1, keep=1, scale=1.0, softmax=False, unit=None):
        """softmax: the router is a linear layer with a bias ("router.b"), the weights are the softmax over the chosen logits.  unit: (limit, alpha) of the
        clamped gated unit."""
        super().__init__()
        assert not softmax or groups == 1
        self.softmax, self.unit = softmax, unit
        assert experts % groups == 0 and 0 < keep <= groups and 0 < top <= keep * (experts // groups), f"{experts} experts, {groups} groups, {keep} kept, top {top}"
        self.in_width, self.in_cols, self.ff, self.cols, self.dtype = in_width, in_cols, ff, round_up(ff, 64), dtype
        self.experts, self.top, self.groups, self.keep, self.scale = experts, top, groups, keep, float(scale)

    def load(self, get):
        """get(name) -> tensor of the checkpoint (names below the feed-forward's prefix)."""
        e, f, c, d = self.experts, self.cols, self.in_cols, self.dtype
        device = get("router").device
        gate_up, down = torch.zeros(e, 2 * f, c, dtype=d, device=device), torch.zeros(e, c, f, dtype=d, device=device)
        assert get("router").shape == (e, self.in_width) and get("e0.gate").shape == (self.ff, self.in_width)
        for i in range(e):
            gate_up[i, :self.ff, :self.in_width], gate_up[i, f:f + self.ff, :self.in_width] = get(f"e{i}.gate"), get(f"e{i}.up")
            down[i, :self.in_width, :self.ff] = get(f"e{i}.down")
        self.register_buffer("w_gate_up", gate_up)
        self.register_buffer("w_down", down)
        self.register_buffer("router", padded(get("router"), e, c).to(d).contiguous())
        self.register_buffer("correction", get("router.b" if self.softmax else "correction").float().contiguous())

    def forward(self, x):
        """x [rows, in_cols] -> (expert outputs [rows * top, in_cols], weights fp32 [rows, top])."""
        ids, weights = ops.moe_route(x, self.router, self.correction, self.top, self.groups, self.keep, self.scale, self.softmax)
        small = x.dtype == torch.bfloat16 and x.shape[0] <= ops.LINEAR_SMALL_M_MAX
        dispatch = None if small else ops.moe_dispatch(ids, self.experts, x.dtype)
        act = ops.moe_gemm(x, self.w_gate_up, ids, True, dispatch, self.unit)
        return ops.moe_gemm(act, self.w_down, ids, False, dispatch), weights
