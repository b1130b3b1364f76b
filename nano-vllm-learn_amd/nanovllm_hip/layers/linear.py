"""The linear layer every model uses: weight-streaming HIP kernel for decode-sized batches, vendor GEMM otherwise."""
import torch
import torch.nn.functional as F


def linear(x, weight, bias=None):
    """F.linear; decode-sized batches on the GPU take the weight-streaming HIP kernel (ops.linear_small_m), anything
    else (prefill, fp32 models, CPU tests) goes to the vendor GEMM."""
    if x.is_cuda and x.dtype == torch.bfloat16 and x.numel() // x.shape[-1] <= 64 and x.shape[-1] % 64 == 0 and weight.shape[0] % 16 == 0:
        from .. import ops
        return ops.linear_small_m(x, weight, bias)
    return F.linear(x, weight, bias)


def round_up(n, m):
    return (n + m - 1) // m * m


def padded(t, *shape):
    """`t` in the leading corner of a zero tensor of `shape`."""
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


class DecodeBuffers:
    """Scratch of a fused decode path for one number of 16-row tiles: fragment-order activations by width and the split-K workspace (zero-filled once)."""

    def __init__(self, rows, device, linears, stream_cols):
        from .. import ops
        self.rows16, self.device, self._packed = round_up(rows, 16), device, {}
        need = max([16] + [ops.linear_workspace_bytes(rows, w.shape[0], w.shape[1], epi) for w, epi in linears])
        self.workspace = torch.zeros(need, dtype=torch.uint8, device=device)
        self.stream = torch.zeros(self.rows16 * stream_cols, dtype=torch.bfloat16, device=device)       # what a layer's projections read, in fragment order
        for w, _ in linears:
            self.packed(w.shape[1])

    def packed(self, cols):
        """One buffer per width, never the stream's: what one launch writes the next launch on the stream consumes, so equal widths can share."""
        if cols not in self._packed:
            self._packed[cols] = torch.zeros(self.rows16 * cols, dtype=torch.bfloat16, device=self.device)
        return self._packed[cols]
