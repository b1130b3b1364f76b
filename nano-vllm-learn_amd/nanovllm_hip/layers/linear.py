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
