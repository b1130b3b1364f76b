"""Tensor-level wrappers over the C ABI (include/nvh_attn.h).

Same function names and argument meaning as the helpers the reference's attention modules call
(store_kvcache: nanovllm/layers/attention.py:44-55; flash_attn_with_kvcache / flash_attn_varlen_func:
call sites attention.py:93-101, oracle bodies nanovllm/layers/attention_sdpa.py:65-182), so parity
tests read like the reference.  Everything runs on torch's CURRENT stream and is graph-capture safe:
no host synchronisation, no host reads of device data.  There is no fallback: tensors must live on
a GPU and the HIP library must load.
"""
from __future__ import annotations

import ctypes

import torch

from . import _lib
from ._lib import NVH_BF16, NVH_F32

_workspaces: dict[tuple, torch.Tensor] = {}
_retired_workspaces: list[torch.Tensor] = []


def _stream():
    return torch.cuda.current_stream().cuda_stream


def _out_code(dtype):
    if dtype == torch.bfloat16:
        return NVH_BF16
    if dtype == torch.float32:
        return NVH_F32
    raise TypeError(f"output dtype {dtype} unsupported (bfloat16 or float32)")


def _require_gpu_bf16(**tensors):
    for name, t in tensors.items():
        if not t.is_cuda:
            raise RuntimeError(f"{name} must be a GPU tensor: the hip attention backend has no CPU path")
        if t.dtype != torch.bfloat16:
            raise TypeError(f"{name} must be bfloat16 (the reference's runtime dtype), got {t.dtype}")


def _require_i32(**tensors):
    for name, t in tensors.items():
        if not t.is_cuda or t.dtype != torch.int32:
            raise TypeError(f"{name} must be an int32 GPU tensor, got {t.dtype} on {t.device}")


# --------------------------------------------------------------------------------------- store
def store_kvcache(key: torch.Tensor, value: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                  slot_mapping: torch.Tensor) -> None:
    """cache.view(-1, KVH*D)[slot_mapping[i]] = key[i] / value[i]; rows with slot < 0 are skipped.

    key/value [N, KVH, D] with contiguous inner dims and any row stride (attention.py:49-55)."""
    n, kvh, hd = key.shape
    d = kvh * hd
    _require_gpu_bf16(key=key, value=value, k_cache=k_cache, v_cache=v_cache)
    _require_i32(slot_mapping=slot_mapping)
    assert value.shape == key.shape
    assert key.stride(-1) == 1 and value.stride(-1) == 1                 # attention.py:51
    assert key.stride(1) == hd and value.stride(1) == hd                 # attention.py:52
    assert k_cache.stride(1) == d and v_cache.stride(1) == d             # attention.py:53
    assert k_cache.is_contiguous() and v_cache.is_contiguous()
    assert slot_mapping.numel() == n and slot_mapping.is_contiguous()    # attention.py:54
    rc = _lib.load().nvh_store_kvcache(key.data_ptr(), value.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                                       slot_mapping.data_ptr(), n, kvh, hd, key.stride(0), value.stride(0),
                                       NVH_BF16, _stream())
    _lib.check(rc, "nvh_store_kvcache")


# --------------------------------------------------------------------------------------- decode
def decode_workspace_bytes(batch, num_heads, head_dim, max_blocks, block_size) -> int:
    return int(_lib.load().nvh_paged_decode_workspace(batch, num_heads, head_dim, max_blocks, block_size))


def reserve_workspace(device, nbytes: int, kind: str = "chunked") -> torch.Tensor:
    """Grow (never shrink) the per-device decode scratch.  Call before graph capture with the largest shape; all layers
    share it (they run back to back on ONE stream — the reference runs one process per GPU and one stream per process;
    callers that launch decode attention on several streams concurrently must pass their own `workspace=` per stream).
    ZERO-FILLED once (the contract of nvh_attn.h): the buffer starts with a fixed header of arrival tickets (one uint32 per
    (sequence, kv head) pair, each on a 128-byte line of its own) and the counters of the fused qkv + attention launch; the chunk
    records behind it are plain fp32 rows published with write-through stores and need no initial value.  Every launch returns the
    tickets and counters it used to zero, so one buffer serves all layers, shapes and graph replays; ONE launch at a time per
    workspace; after a launch that was aborted mid-flight (a device fault, a killed process) zero-fill it again.  The split +
    combine variants (tests, A/B) keep their partials in a buffer of their own (`kind`)."""
    idx = torch.device(device).index
    idx = torch.cuda.current_device() if idx is None else idx
    idx = (idx, kind)
    ws = _workspaces.get(idx)
    if ws is None or ws.numel() < nbytes:
        if ws is not None and torch.cuda.is_current_stream_capturing():
            return torch.zeros(nbytes, dtype=torch.uint8, device=device)   # graph-pool memory, not cached
        if ws is not None:
            _retired_workspaces.append(ws)                 # a captured graph may still point at it: never freed
        ws = torch.zeros(max(nbytes, 1 << 20), dtype=torch.uint8, device=device)
        if not torch.cuda.is_current_stream_capturing():
            _workspaces[idx] = ws
    return ws


def _decode_common(q, k_cache, v_cache, cache_seqlens, block_table, softmax_scale, out, out_dtype, workspace=None, kind="chunked"):
    squeeze = q.dim() == 4
    if squeeze:
        assert q.shape[1] == 1, "Decode stage should have seq_len=1"      # attention_sdpa.py:133
        q3 = q[:, 0]
    else:
        q3 = q
    b, h, hd = q3.shape
    nb, bs, kvh, hd2 = k_cache.shape
    assert hd2 == hd and v_cache.shape == k_cache.shape
    _require_gpu_bf16(q=q, k_cache=k_cache, v_cache=v_cache)
    _require_i32(cache_seqlens=cache_seqlens, block_table=block_table)
    assert q3.stride(-1) == 1 and q3.stride(1) == hd
    assert k_cache.is_contiguous() and v_cache.is_contiguous()
    assert block_table.dim() == 2 and block_table.shape[0] == b and block_table.stride(1) == 1
    assert cache_seqlens.numel() == b and cache_seqlens.is_contiguous()
    if softmax_scale is None:
        softmax_scale = hd ** -0.5
    out_dtype = out_dtype or torch.bfloat16
    if out is None:
        out = torch.empty((b, h, hd), dtype=out_dtype, device=q.device)
    else:
        assert out.shape == (b, h, hd) and out.is_contiguous() and out.dtype == out_dtype
    max_blocks = block_table.shape[1]
    need = decode_workspace_bytes(b, h, hd, max_blocks, bs)
    if workspace is not None:
        assert workspace.is_cuda and workspace.dtype == torch.uint8 and workspace.is_contiguous() and workspace.numel() >= need
        ws = workspace
    else:
        ws = reserve_workspace(q.device, need, kind)
    return squeeze, q3, b, h, hd, kvh, bs, max_blocks, float(softmax_scale), out, ws


def flash_attn_with_kvcache(q, k_cache, v_cache, cache_seqlens, block_table, softmax_scale=None, causal=True,
                            out=None, out_dtype=None, out_packed=None, variant=None, waves=0, chunks=0, workspace=None):
    """Decode attention, drop-in for the call at attention.py:99-101.

    q [B, 1, H, D] (or [B, H, D]); caches [NB, bs, KVH, D]; cache_seqlens int32 [B] (0 -> zero row);
    block_table int32 [B, max_blocks].  `causal` is accepted for signature parity; with one query per
    sequence it has no effect.  Returns [B, 1, H, D] (or [B, H, D]).  out_packed: optional flat bf16 buffer of
    ceil(B/16)*16*H*D elements that also receives the result in MFMA-fragment order (pack_rows layout) for fused_linear.
    variant ("chunked" | "split_mfma" | "split_valu"), waves, chunks: tests / A-B only (nvh_paged_decode_variant); the module
    path never passes them.  workspace: a caller-owned ZERO-FILLED uint8 buffer of decode_workspace_bytes() (one per stream
    that may run decode attention concurrently); default: the per-device buffer of reserve_workspace()."""
    squeeze, q3, b, h, hd, kvh, bs, max_blocks, scale, out, ws = _decode_common(
        q, k_cache, v_cache, cache_seqlens, block_table, softmax_scale, out, out_dtype, workspace,
        "split" if variant in ("split_mfma", "split_valu") else "chunked")
    tail = (q3.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), block_table.data_ptr(), cache_seqlens.data_ptr(), b, h, kvh, hd, bs,
            max_blocks, q3.stride(0), block_table.stride(0), scale, NVH_BF16, _out_code(out.dtype), ws.data_ptr(), ws.numel(), _stream())
    if variant is not None or waves or chunks:
        assert out_packed is None
        rc = _lib.load().nvh_paged_decode_variant(_lib.DECODE_VARIANTS[variant or "chunked"], int(waves), int(chunks), out.data_ptr(), *tail)
    elif out_packed is not None:
        _require_gpu_bf16(out_packed=out_packed)
        assert out_packed.is_contiguous() and out_packed.numel() >= ((b + 15) // 16) * 16 * h * hd
        rc = _lib.load().nvh_paged_decode_packed(out.data_ptr(), out_packed.data_ptr(), *tail)
    else:
        rc = _lib.load().nvh_paged_decode(out.data_ptr(), *tail)
    _lib.check(rc, "nvh_paged_decode")
    return out.unsqueeze(1) if squeeze else out


def decode_step(q, k_new, v_new, k_cache, v_cache, slot_mapping, cache_seqlens, block_table, softmax_scale=None,
                out=None, out_dtype=None):
    """store_kvcache(k_new, v_new, ...) followed by flash_attn_with_kvcache(q, ...) as one C-ABI call
    (the two calls at attention.py:84-86 and :99-101)."""
    squeeze, q3, b, h, hd, kvh, bs, max_blocks, scale, out, ws = _decode_common(
        q, k_cache, v_cache, cache_seqlens, block_table, softmax_scale, out, out_dtype)
    _require_gpu_bf16(k_new=k_new, v_new=v_new)
    _require_i32(slot_mapping=slot_mapping)
    assert k_new.shape == (b, kvh, hd) and v_new.shape == (b, kvh, hd)
    assert k_new.stride(-1) == 1 and v_new.stride(-1) == 1 and k_new.stride(1) == hd and v_new.stride(1) == hd
    assert slot_mapping.numel() == b and slot_mapping.is_contiguous()
    rc = _lib.load().nvh_decode_step(out.data_ptr(), q3.data_ptr(), k_new.data_ptr(), v_new.data_ptr(),
                                     k_cache.data_ptr(), v_cache.data_ptr(), slot_mapping.data_ptr(),
                                     block_table.data_ptr(), cache_seqlens.data_ptr(), b, h, kvh, hd, bs, max_blocks,
                                     q3.stride(0), k_new.stride(0), v_new.stride(0), block_table.stride(0), scale,
                                     NVH_BF16, _out_code(out.dtype), ws.data_ptr(), ws.numel(), _stream())
    _lib.check(rc, "nvh_decode_step")
    return out.unsqueeze(1) if squeeze else out


# --------------------------------------------------------------------------------------- prefill
PV16_MIN_KEYS = 512       # fp16 P V (nvh_prefill_varlen_pv16) by default from this many keys per sequence on (40.5 vs 42.0 us at 32 x 512; below, the conversion launch costs what it saves)


def flash_attn_varlen_func(q, k, v, max_seqlen_q, cu_seqlens_q, max_seqlen_k, cu_seqlens_k, softmax_scale=None,
                           causal=True, block_table=None, out_dtype=None, kernel=None, short_waves=0, pv_fp16=None):
    """Packed varlen causal attention, drop-in for the call at attention.py:93-96.

    q [Tq, H, D]; without block_table k/v are [Tk, KVH, D] (any row stride); with block_table they are
    the paged caches [NB, bs, KVH, D] and sequence i reads its keys through block_table[i].
    kernel ("auto" | "tiled" | "short" | "tiled_f16v"), short_waves: tests / A-B only (nvh_prefill_varlen_variant).
    pv_fp16: P V on the fp16 matrix pipe (nvh_prefill_varlen_pv16: V converted to fp16 rows in a scratch buffer with a range guard, P rounded to
    11 bits; a V value that does not fit fp16 makes the kernel itself fall back to the exact form, no host read).  None (default) = where it pays and
    is invisible: bf16 output (whose own rounding, 2^-9 |o|, is 8x coarser than P's), no block_table, max_seqlen_k >= PV16_MIN_KEYS or a batch the
    short-sequence kernel takes (head_dim 64, <= 128 keys, >= 128 (sequence, kv head) pairs: it converts V inside the kernel); True = always
    (no block_table); False = never (P as bf16 hi + lo, 6e-6).  Error of the fp16 form <= 2^-12 * max|v|: 4.5e-4 on the reference goldens (the
    reference's flash backend rounds P to a single bf16, 8 bits).  DESIGN.md section 12.2."""
    if kernel is not None or short_waves or block_table is not None:
        assert not pv_fp16 or kernel == "tiled_f16v", "pv_fp16 goes with the default kernel choice and packed k / v rows"
        pv_fp16 = False
    elif pv_fp16 is None:
        # ... or on the short-sequence kernel's shapes (it converts its resident V images itself: no extra launch; the library's rule, prefill_mfma.hip launch_short)
        short = (q.shape[2] == 64 and 64 < int(max_seqlen_k) <= 128 and int(max_seqlen_q) <= int(max_seqlen_k)
                 and (cu_seqlens_q.numel() - 1) * k.shape[1] >= 128)
        pv_fp16 = (out_dtype in (None, torch.bfloat16)) and (int(max_seqlen_k) >= PV16_MIN_KEYS or short)
    if not causal:
        raise NotImplementedError("the reference only ever calls this with causal=True (attention.py:96)")
    tq, h, hd = q.shape
    if kernel == "tiled_f16v":                                  # measurement variant: v already converted to fp16 by the caller
        assert v.dtype == torch.float16 and v.is_cuda and block_table is None
        _require_gpu_bf16(q=q, k=k)
    else:
        _require_gpu_bf16(q=q, k=k, v=v)
    _require_i32(cu_seqlens_q=cu_seqlens_q, cu_seqlens_k=cu_seqlens_k)
    assert q.stride(-1) == 1 and q.stride(1) == hd
    batch = cu_seqlens_q.numel() - 1
    assert cu_seqlens_k.numel() == batch + 1
    if softmax_scale is None:
        softmax_scale = hd ** -0.5
    out = torch.empty((tq, h, hd), dtype=out_dtype or torch.bfloat16, device=q.device)
    if block_table is not None:
        _require_i32(block_table=block_table)
        nb, bs, kvh, hd2 = k.shape
        assert hd2 == hd and v.shape == k.shape and k.is_contiguous() and v.is_contiguous()
        assert block_table.shape[0] == batch and block_table.stride(1) == 1
        max_blocks, bt_stride, bt_ptr = block_table.shape[1], block_table.stride(0), block_table.data_ptr()
        k_stride = v_stride = kvh * hd
    else:
        tk, kvh, hd2 = k.shape
        assert hd2 == hd and v.shape == k.shape
        assert k.stride(-1) == 1 and v.stride(-1) == 1 and k.stride(1) == hd and v.stride(1) == hd
        bs, max_blocks, bt_stride, bt_ptr = 0, 0, 0, None
        k_stride, v_stride = k.stride(0), v.stride(0)
    tail = (out.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr(), cu_seqlens_q.data_ptr(), cu_seqlens_k.data_ptr(), bt_ptr, batch,
            int(max_seqlen_q), int(max_seqlen_k), h, kvh, hd, bs, max_blocks, q.stride(0), k_stride, v_stride, bt_stride,
            float(softmax_scale), NVH_BF16, _out_code(out.dtype), _stream())
    if pv_fp16:
        lib = _lib.load()
        if int(max_seqlen_k) <= 128 and not lib.nvh_prefill_pv16_uses_scratch(batch, int(max_seqlen_q), int(max_seqlen_k), kvh, hd):
            sc_ptr, sc_bytes = None, 0                           # the short-sequence kernel converts V in LDS: one launch, no scratch
        else:
            scratch = torch.empty(lib.nvh_prefill_pv16_scratch_bytes(tk, kvh, hd), dtype=torch.uint8, device=q.device)
            sc_ptr, sc_bytes = scratch.data_ptr(), scratch.numel()
        rc = lib.nvh_prefill_varlen_pv16(out.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr(), cu_seqlens_q.data_ptr(), cu_seqlens_k.data_ptr(), batch,
                                         int(max_seqlen_q), int(max_seqlen_k), tk, h, kvh, hd, q.stride(0), k_stride, v_stride, float(softmax_scale),
                                         NVH_BF16, _out_code(out.dtype), sc_ptr, sc_bytes, _stream())
        _lib.check(rc, "nvh_prefill_varlen_pv16")
        return out
    if kernel is not None or short_waves:
        rc = _lib.load().nvh_prefill_varlen_variant(_lib.PREFILL_KERNELS[kernel or "auto"], int(short_waves), *tail)
    else:
        rc = _lib.load().nvh_prefill_varlen(*tail)
    _lib.check(rc, "nvh_prefill_varlen")
    return out


# --------------------------------------------------------------------------------------- rope + store (next row f2)
def rope_store(qkv, positions, cos_sin, num_heads, num_kv_heads, head_dim, k_cache=None, v_cache=None, slot_mapping=None,
               q_norm_weight=None, k_norm_weight=None, eps=1e-6):
    """In-place (optional per-head RMSNorm ->) neox RoPE on the q and k parts of the fused projection output
    `qkv` [N, (H+2KVH)*D], then k/v rows -> paged cache at slot_mapping (skipped when no cache is bound or slot < 0).
    Equivalent to q_norm/k_norm + rotary_emb + store_kvcache of the reference (qwen3.py:108-116, attention.py:84-86)."""
    _require_gpu_bf16(qkv=qkv)
    n = qkv.shape[0]
    assert qkv.dim() == 2 and qkv.stride(1) == 1 and qkv.shape[1] == (num_heads + 2 * num_kv_heads) * head_dim
    assert positions.dtype == torch.int64 and positions.is_cuda and positions.numel() == n and positions.is_contiguous()
    assert cos_sin.dtype == torch.float32 and cos_sin.is_cuda and cos_sin.is_contiguous() and cos_sin.shape[1] == head_dim
    have_cache = k_cache is not None and k_cache.numel() > 0 and slot_mapping is not None
    if have_cache:
        _require_gpu_bf16(k_cache=k_cache, v_cache=v_cache)
        _require_i32(slot_mapping=slot_mapping)
        assert k_cache.is_contiguous() and v_cache.is_contiguous() and k_cache.stride(1) == num_kv_heads * head_dim
        assert slot_mapping.numel() == n and slot_mapping.is_contiguous()
    if q_norm_weight is not None:
        _require_gpu_bf16(q_norm_weight=q_norm_weight, k_norm_weight=k_norm_weight)
    rc = _lib.load().nvh_rope_store(qkv.data_ptr(), positions.data_ptr(), cos_sin.data_ptr(),
                                    q_norm_weight.data_ptr() if q_norm_weight is not None else None,
                                    k_norm_weight.data_ptr() if k_norm_weight is not None else None, float(eps),
                                    k_cache.data_ptr() if have_cache else None, v_cache.data_ptr() if have_cache else None,
                                    slot_mapping.data_ptr() if have_cache else None,
                                    n, num_heads, num_kv_heads, head_dim, qkv.stride(0), NVH_BF16, _stream())
    _lib.check(rc, "nvh_rope_store")


# --------------------------------------------------------------------------------------- row-wise ops around the attention block
def add_rmsnorm(x, weight, eps, residual=None):
    """RMSNorm.forward(x[, residual]) of the reference (layernorm.py:43-50) in one launch.  `residual`, when given, is
    updated IN PLACE to x + residual (bf16) and the norm is taken of the fp32 sum.  Returns the normalised tensor."""
    _require_gpu_bf16(x=x, weight=weight)
    hidden = x.shape[-1]
    x2 = x.view(-1, hidden)
    assert x2.stride(1) == 1 and weight.numel() == hidden and weight.is_contiguous()
    out = torch.empty((x2.shape[0], hidden), dtype=torch.bfloat16, device=x.device)
    r2 = None
    if residual is not None:
        _require_gpu_bf16(residual=residual)
        r2 = residual.view(-1, hidden)
        assert r2.shape == x2.shape and r2.stride(1) == 1
    rc = _lib.load().nvh_add_rmsnorm(out.data_ptr(), x2.data_ptr(), r2.data_ptr() if r2 is not None else None, weight.data_ptr(), float(eps),
                                     x2.shape[0], hidden, x2.stride(0), out.stride(0), r2.stride(0) if r2 is not None else 0, NVH_BF16, _stream())
    _lib.check(rc, "nvh_add_rmsnorm")
    return out.view(x.shape)


def residual_add_pack(residual, y, packed=None):
    """residual += y in place (bf16, one rounding) and, optionally, the updated rows in fragment order into `packed`
    (nvh_residual_add_pack): the step after a tensor-parallel all-reduce in the fused decode layer."""
    _require_gpu_bf16(residual=residual, y=y)
    assert residual.dim() == 2 and residual.shape == y.shape and residual.stride(1) == 1 and y.stride(1) == 1
    m, hidden = residual.shape
    if packed is not None:
        _require_gpu_bf16(packed=packed)
        assert packed.is_contiguous() and packed.numel() >= ((m + 15) // 16) * 16 * hidden
    rc = _lib.load().nvh_residual_add_pack(residual.data_ptr(), y.data_ptr(), packed.data_ptr() if packed is not None else None, m, hidden,
                                           residual.stride(0), y.stride(0), NVH_BF16, _stream())
    _lib.check(rc, "nvh_residual_add_pack")
    return residual


def silu_mul(gate_up):
    """SiluAndMul.forward (activation.py:11-14): silu(gate_up[..., :I]) * gate_up[..., I:]."""
    _require_gpu_bf16(gate_up=gate_up)
    inter = gate_up.shape[-1] // 2
    g2 = gate_up.view(-1, 2 * inter)
    assert g2.stride(1) == 1
    out = torch.empty((g2.shape[0], inter), dtype=torch.bfloat16, device=gate_up.device)
    rc = _lib.load().nvh_silu_mul(out.data_ptr(), g2.data_ptr(), g2.shape[0], inter, g2.stride(0), out.stride(0), NVH_BF16, _stream())
    _lib.check(rc, "nvh_silu_mul")
    return out.view(*gate_up.shape[:-1], inter)


LINEAR_SMALL_M_MAX = 64


def linear_small_m(x, weight, bias=None, silu_mul=False):
    """F.linear(x, weight, bias) for at most 64 rows, streaming `weight` [N, K] once; with silu_mul=True `weight` is the
    merged gate_up projection and the result is SiLU(x gate^T) * (x up^T) (projection + activation.py:11-14 in one launch)."""
    _require_gpu_bf16(x=x, weight=weight)
    k = x.shape[-1]
    x2 = x.view(-1, k)
    n = weight.shape[0]
    assert x2.shape[0] <= LINEAR_SMALL_M_MAX and x2.stride(1) == 1 and weight.is_contiguous() and weight.shape[1] == k
    inter = n // 2 if silu_mul else 0
    out = torch.empty((x2.shape[0], inter if silu_mul else n), dtype=torch.bfloat16, device=x.device)
    if bias is not None:
        _require_gpu_bf16(bias=bias)
        assert bias.numel() == n and bias.is_contiguous()
    rc = _lib.load().nvh_linear_small_m(out.data_ptr(), x2.data_ptr(), weight.data_ptr(), bias.data_ptr() if bias is not None else None,
                                        x2.shape[0], n, k, inter, x2.stride(0), out.stride(0), NVH_BF16, _stream())
    _lib.check(rc, "nvh_linear_small_m")
    return out.view(*x.shape[:-1], out.shape[1])


def pack_rows(x, rows=None):
    """[M, C] bf16 -> the MFMA-fragment order the streaming GEMM reads at full address rate (nvh_pack_index):
    [ceil(M/16)][C/32][lane = 16 * (col/8 % 4) + row % 16][8], rows padded with zeros.  Torch-side helper (tests, first layer)."""
    m, c = x.shape
    assert c % 32 == 0
    mt = (max(m, rows or m) + 15) // 16
    xp = torch.zeros((mt * 16, c), dtype=x.dtype, device=x.device)
    xp[:m] = x
    return xp.view(mt, 16, c // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous().view(-1)


def unpack_rows(xp, m, c):
    """Inverse of pack_rows: flat fragment-order buffer -> [m, c]."""
    mt = xp.numel() // (16 * c)
    return xp.view(mt, c // 32, 4, 16, 8).permute(0, 3, 1, 2, 4).reshape(mt * 16, c)[:m]


def linear_workspace_bytes(m, n, k, epilogue="none") -> int:
    return int(_lib.load().nvh_linear_small_m_workspace(m, n, k, _EPI_CODES[epilogue]))


_EPI_CODES = {"none": _lib.EPI_NONE, "silu_mul": _lib.EPI_SILU_MUL, "residual_add": _lib.EPI_RESIDUAL_ADD, "rope_store": _lib.EPI_ROPE_STORE}


def fused_linear(x, weight, *, bias=None, norm_weight=None, norm_eps=1e-6, norm_folded=False, epilogue="none", out=None, rope=None,
                 x_packed_rows=None, out_packed=None, workspace=None, want_out=True, candidates=None, prefetch=None, glu=None, x_groups=None):
    """nvh_linear_small_m_ex: x [M<=64, K] . weight[N, K]^T with an optional RMSNorm prologue and one of the epilogues
    "none" (+bias) | "silu_mul" | "residual_add" (out = the residual stream, updated in place) | "rope_store"
    (rope = dict(positions, cos_sin, k_cache, v_cache, slot_mapping, num_heads, num_kv_heads, head_dim); returns q [M, H*D]).
    Streaming form: x_packed_rows = M when `x` is a flat fragment-order buffer (pack_rows); out_packed = a flat bf16 buffer
    that receives the result in fragment order as well; workspace = a ZERO-FILLED uint8 buffer of linear_workspace_bytes()
    (needed for K > 1024); want_out=False skips the row-major output when out_packed is given ("none" / "silu_mul");
    candidates = (val float32 [groups, stride], idx int32 [groups, stride]) with groups = linear_candidate_groups(n, k):
    per workgroup and row the best bf16 output and its column ("none" only) — with want_out=False the outputs themselves are
    never written (LM head + greedy arg-max in one pass; finish with greedy_advance_candidates).
    prefetch = a contiguous CUDA tensor the NEXT launch will stream (the following projection's weights): the CUs this launch
    leaves idle read it into the caches first (a hint; results do not depend on it).
    glu = (limit, alpha): "silu_mul" applies the clamped gated unit of clamped_glu() instead of SiLU(g) * u; "gelu": gelu_tanh(g) * u.
    x_groups = (count, weight rows): `x` holds `count` packed buffers of equal size, each group of weight rows is applied to its own ("none" only)."""
    d, out = _linear_desc(x, weight, bias=bias, norm_weight=norm_weight, norm_eps=norm_eps, norm_folded=norm_folded, epilogue=epilogue, out=out,
                          rope=rope, x_packed_rows=x_packed_rows, out_packed=out_packed, workspace=workspace, want_out=want_out,
                          candidates=candidates, prefetch=prefetch)
    if glu == "gelu":
        d.glu_gelu = 1
    elif glu is not None:
        d.glu_limit, d.glu_alpha = float(glu[0]), float(glu[1])
    if x_groups is not None:
        d.x_groups, d.x_group_rows = int(x_groups[0]), int(x_groups[1])
        d.x_group_stride = x.numel() // d.x_groups
        assert x_packed_rows is not None and x.numel() % d.x_groups == 0
    rc = _lib.load().nvh_linear_small_m_ex(ctypes.byref(d), NVH_BF16, _stream())
    _lib.check(rc, "nvh_linear_small_m_ex")
    return out


def _linear_desc(x, weight, *, bias=None, norm_weight=None, norm_eps=1e-6, norm_folded=False, epilogue="none", out=None, rope=None,
                 x_packed_rows=None, out_packed=None, workspace=None, want_out=True, candidates=None, prefetch=None):
    """Build the nvh_linear_desc of fused_linear's arguments; returns (descriptor, out)."""
    _require_gpu_bf16(x=x, weight=weight)
    n, k = weight.shape
    if x_packed_rows is not None:
        m = int(x_packed_rows)
        assert x.dim() == 1 and x.numel() >= ((m + 15) // 16) * 16 * k and x.is_contiguous()
    else:
        m = x.shape[0]
        assert x.shape[1] == k and x.stride(1) == 1
    assert weight.is_contiguous() and m <= LINEAR_SMALL_M_MAX
    d = _lib.LinearDesc()
    d.x, d.w, d.m, d.n, d.k = x.data_ptr(), weight.data_ptr(), m, n, k
    d.x_row_stride = k if x_packed_rows is not None else x.stride(0)
    d.x_packed = 1 if x_packed_rows is not None else 0
    d.bias = bias.data_ptr() if bias is not None else None
    if norm_folded:                                   # `weight` already carries the norm weight: w * diag(g)
        assert norm_weight is None
        d.norm_folded, d.norm_eps = 1, float(norm_eps)
    if norm_weight is not None:
        _require_gpu_bf16(norm_weight=norm_weight)
        assert norm_weight.numel() == k
        d.norm_weight, d.norm_eps = norm_weight.data_ptr(), float(norm_eps)
    if epilogue == "none":
        d.epilogue, cols = _lib.EPI_NONE, n
    elif epilogue == "silu_mul":
        d.epilogue, d.silu_inter, cols = _lib.EPI_SILU_MUL, n // 2, n // 2
    elif epilogue == "residual_add":
        assert out is not None and out.shape == (m, n) and out.dtype == torch.bfloat16 and out.stride(1) == 1
        d.epilogue, cols = _lib.EPI_RESIDUAL_ADD, n
    elif epilogue == "rope_store":
        h, kvh, hd = rope["num_heads"], rope["num_kv_heads"], rope["head_dim"]
        _require_i32(slot_mapping=rope["slot_mapping"])
        assert rope["positions"].dtype == torch.int64 and rope["cos_sin"].dtype == torch.float32 and rope["cos_sin"].is_contiguous()
        assert rope["k_cache"].is_contiguous() and rope["v_cache"].is_contiguous()
        d.epilogue, cols = _lib.EPI_ROPE_STORE, h * hd
        d.positions, d.cos_sin = rope["positions"].data_ptr(), rope["cos_sin"].data_ptr()
        d.k_cache, d.v_cache, d.slot_mapping = rope["k_cache"].data_ptr(), rope["v_cache"].data_ptr(), rope["slot_mapping"].data_ptr()
        d.h, d.kvh, d.hd = h, kvh, hd
    else:
        raise ValueError(epilogue)
    if out_packed is not None:
        _require_gpu_bf16(out_packed=out_packed)
        assert out_packed.is_contiguous() and out_packed.numel() >= ((m + 15) // 16) * 16 * cols
        d.out_packed = out_packed.data_ptr()
    if workspace is not None:
        assert workspace.is_cuda and workspace.dtype == torch.uint8 and workspace.is_contiguous()
        d.workspace, d.workspace_bytes = workspace.data_ptr(), workspace.numel()
    if candidates is not None:
        cv, ci = candidates
        assert epilogue == "none" and cv.dtype == torch.float32 and ci.dtype == torch.int32 and cv.is_cuda and ci.is_cuda
        assert cv.shape == ci.shape and cv.dim() == 2 and cv.is_contiguous() and ci.is_contiguous()
        assert cv.shape[0] >= linear_candidate_groups(n, k) > 0 and cv.shape[1] >= m
        d.candidate_val, d.candidate_idx, d.candidate_stride = cv.data_ptr(), ci.data_ptr(), cv.stride(0)
    if prefetch is not None:
        assert prefetch.is_cuda and prefetch.is_contiguous()
        d.prefetch, d.prefetch_bytes = prefetch.data_ptr(), prefetch.numel() * prefetch.element_size()
    if out is None and (want_out or (out_packed is None and candidates is None)):
        out = torch.empty((m, cols), dtype=torch.bfloat16, device=x.device)
    if out is not None:
        d.out, d.out_row_stride = out.data_ptr(), out.stride(0)
    return d, out


QKV_ATTEND_MODES = {"auto": 0, "two_launches": 1, "one_launch": 2, "two_launches_kv_prefetch": 3}


def qkv_rope_attend(x, weight, *, rope, context_lens, block_tables, bias=None, norm_eps=1e-6, norm_folded=True, x_packed_rows=None,
                    q_out=None, attn_out=None, attn_out_packed=None, softmax_scale=None, workspace=None, linear_workspace=None, prefetch=None,
                    mode="auto", spin_limit=0, missing_producers=0):
    """nvh_qkv_rope_attend: the front of a decode layer in ONE launch — fused_linear(..., epilogue="rope_store") followed by
    flash_attn_with_kvcache on its q rows and the caches it has just extended (models/qwen3.py:104-117 with
    layers/attention.py:84-86 and :99-101 inside).  Shapes the one-launch kernel does not serve (head_dim 128, k > 1024,
    row-major x, ...) run as the two launches with the same results.  Returns (q [M, H*D], attn_out [M, H, D], one_launch: bool).
    workspace = the decode workspace (default: the per-device one); linear_workspace = fused_linear's (split-K, k > 1024 only).
    mode / spin_limit / missing_producers: tests and A/B only (nvh_qkv_rope_attend_variant)."""
    d, q = _linear_desc(x, weight, bias=bias, norm_eps=norm_eps, norm_folded=norm_folded, epilogue="rope_store", out=q_out, rope=rope,
                        x_packed_rows=x_packed_rows, workspace=linear_workspace, prefetch=prefetch)
    h, kvh, hd = rope["num_heads"], rope["num_kv_heads"], rope["head_dim"]
    m = d.m
    k_cache = rope["k_cache"]
    bs = k_cache.shape[1]
    _require_i32(context_lens=context_lens, block_tables=block_tables)
    assert block_tables.dim() == 2 and block_tables.shape[0] == m and block_tables.stride(1) == 1
    assert context_lens.numel() == m and context_lens.is_contiguous()
    if attn_out is None:
        attn_out = torch.empty((m, h, hd), dtype=torch.bfloat16, device=q.device)
    else:
        assert attn_out.shape == (m, h, hd) and attn_out.is_contiguous() and attn_out.dtype == torch.bfloat16
    if attn_out_packed is not None:
        _require_gpu_bf16(attn_out_packed=attn_out_packed)
        assert attn_out_packed.is_contiguous() and attn_out_packed.numel() >= ((m + 15) // 16) * 16 * h * hd
    max_blocks = block_tables.shape[1]
    need = decode_workspace_bytes(m, h, hd, max_blocks, bs)
    if workspace is not None:
        assert workspace.is_cuda and workspace.dtype == torch.uint8 and workspace.is_contiguous() and workspace.numel() >= need
        ws = workspace
    else:
        ws = reserve_workspace(q.device, need)
    scale = float(hd ** -0.5 if softmax_scale is None else softmax_scale)
    fused = ctypes.c_int(0)
    rc = _lib.load().nvh_qkv_rope_attend_variant(
        QKV_ATTEND_MODES[mode], int(spin_limit), int(missing_producers), ctypes.byref(fused), ctypes.byref(d), attn_out.data_ptr(),
        attn_out_packed.data_ptr() if attn_out_packed is not None else None, block_tables.data_ptr(), context_lens.data_ptr(), bs, max_blocks,
        block_tables.stride(0), scale, NVH_BF16, ws.data_ptr(), ws.numel(), _stream())
    _lib.check(rc, "nvh_qkv_rope_attend")
    return q, attn_out, bool(fused.value)


def qkv_rope_attend_status(workspace=None, device=None) -> int:
    """Host-synchronous: non-zero after a one-launch call whose consumers gave up waiting for a producer (its rows are NaN)."""
    ws = workspace if workspace is not None else reserve_workspace(device if device is not None else torch.device("cuda", torch.cuda.current_device()), 1)
    v = ctypes.c_uint32(0)
    _lib.check(_lib.load().nvh_qkv_rope_attend_status(ws.data_ptr(), ctypes.byref(v)), "nvh_qkv_rope_attend_status")
    return int(v.value)


def linear_candidate_groups(n, k) -> int:
    return int(_lib.load().nvh_linear_small_m_candidate_groups(n, k))


def greedy_advance_candidates(cand_val, cand_idx, groups, n_rows, input_ids, positions, context_lens, slot_mapping, block_tables, block_size,
                              tokens_log, row_steps, embed=None):
    """greedy_advance on the candidate records of fused_linear(candidates=...) instead of logits.
    embed = (weight [vocab, hidden], hidden_out [n_rows, hidden], hidden_packed or None): the same launch also looks up the
    chosen tokens' embedding rows for the next step (row-major and, optionally, in fragment order)."""
    _require_i32(context_lens=context_lens, slot_mapping=slot_mapping, block_tables=block_tables)
    for t in (input_ids, positions, tokens_log, row_steps):
        assert t.dtype == torch.int64 and t.is_cuda
    if embed is not None:
        w, hid, packed = embed
        _require_gpu_bf16(embed_weight=w, hidden_out=hid)
        assert w.is_contiguous() and hid.shape == (n_rows, w.shape[1]) and hid.stride(1) == 1
        assert packed is None or (packed.dtype == torch.bfloat16 and packed.is_cuda and packed.numel() >= ((n_rows + 15) // 16) * 16 * w.shape[1])
        rc = _lib.load().nvh_greedy_advance_candidates_embed(
            cand_val.data_ptr(), cand_idx.data_ptr(), groups, cand_val.stride(0), n_rows, input_ids.data_ptr(), positions.data_ptr(),
            context_lens.data_ptr(), slot_mapping.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), block_size,
            tokens_log.data_ptr(), tokens_log.stride(0), row_steps.data_ptr(), w.data_ptr(), w.shape[0], w.shape[1], hid.data_ptr(), hid.stride(0),
            None if packed is None else packed.data_ptr(), NVH_BF16, _stream())
        _lib.check(rc, "nvh_greedy_advance_candidates_embed")
        return
    rc = _lib.load().nvh_greedy_advance_candidates(cand_val.data_ptr(), cand_idx.data_ptr(), groups, cand_val.stride(0), n_rows,
                                                   input_ids.data_ptr(), positions.data_ptr(), context_lens.data_ptr(), slot_mapping.data_ptr(),
                                                   block_tables.data_ptr(), block_tables.stride(0), block_size, tokens_log.data_ptr(),
                                                   tokens_log.stride(0), row_steps.data_ptr(), _stream())
    _lib.check(rc, "nvh_greedy_advance_candidates")


def argmax_rows(logits):
    """Greedy token per row: argmax over the last dim of bf16 logits [M, N] (ties -> lowest index), int64."""
    _require_gpu_bf16(logits=logits)
    assert logits.dim() == 2 and logits.stride(1) == 1
    out = torch.empty(logits.shape[0], dtype=torch.int64, device=logits.device)
    rc = _lib.load().nvh_argmax_rows(out.data_ptr(), logits.data_ptr(), logits.shape[0], logits.shape[1], logits.stride(0), NVH_BF16, _stream())
    _lib.check(rc, "nvh_argmax_rows")
    return out


def greedy_advance(logits, input_ids, positions, context_lens, slot_mapping, block_tables, block_size, tokens_log, row_steps):
    """argmax_rows fused with the between-steps bookkeeping of a greedy decode session (nvh_greedy_advance): appends the
    token to `tokens_log[row_steps[r], r]` and rewrites next step's input_ids / positions / context_lens / slot_mapping in place."""
    _require_gpu_bf16(logits=logits)
    _require_i32(context_lens=context_lens, slot_mapping=slot_mapping, block_tables=block_tables)
    m = logits.shape[0]
    assert logits.dim() == 2 and logits.stride(1) == 1 and block_tables.stride(1) == 1
    for t in (input_ids, positions, tokens_log, row_steps):
        assert t.dtype == torch.int64 and t.is_cuda
    assert tokens_log.dim() == 2 and tokens_log.shape[1] >= m and tokens_log.stride(1) == 1
    rc = _lib.load().nvh_greedy_advance(logits.data_ptr(), m, logits.shape[1], logits.stride(0), input_ids.data_ptr(), positions.data_ptr(),
                                        context_lens.data_ptr(), slot_mapping.data_ptr(), block_tables.data_ptr(), block_tables.stride(0),
                                        block_size, tokens_log.data_ptr(), tokens_log.stride(0), row_steps.data_ptr(), NVH_BF16, _stream())
    _lib.check(rc, "nvh_greedy_advance")


# --------------------------------------------------------------------------------------- fp32-residual row ops, recurrence, latent attention
def _act_code(*tensors):
    """Activation type of a call: every tensor bf16, or every tensor fp32."""
    dtype = tensors[0].dtype
    for t in tensors:
        if not t.is_cuda:
            raise RuntimeError("the hip layers have no CPU path: GPU tensors only")
        if t.dtype != dtype:
            raise TypeError(f"activations and weights of one call share a type, got {dtype} and {t.dtype}")
    return _out_code(dtype)


def _ptr(t):
    return t.data_ptr() if t is not None else None


def _require_f32(**tensors):
    for name, t in tensors.items():
        if not t.is_cuda or t.dtype != torch.float32 or not t.is_contiguous():
            raise TypeError(f"{name} must be a contiguous fp32 GPU tensor, got {t.dtype} on {t.device}")


def embed_rows(tokens, embed, scale, packed=None, positions=None, table=None, copy=None, want_rows=True):
    """(fp32 stream [rows, cols], the same in the activation type — the stream itself for fp32) = embed[tokens] * scale (+ table[positions], fp32).
    packed (bf16): the second form in fragment order into this buffer instead; want_rows=False: no second form.  copy (fp32): the stream a second time."""
    code = _act_code(embed)
    assert tokens.dtype == torch.int64 and tokens.is_cuda and tokens.is_contiguous() and embed.is_contiguous()
    rows, cols = tokens.numel(), embed.shape[1]
    x = torch.empty((rows, cols), dtype=torch.float32, device=embed.device)
    xb = torch.empty((rows, cols), dtype=embed.dtype, device=embed.device) if embed.dtype != torch.float32 and packed is None and want_rows else None
    if table is not None:
        _require_f32(table=table)
        assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows and table.shape[1] == cols
    if copy is not None:
        _require_f32(copy=copy)
        assert copy.shape == x.shape
    if packed is not None:
        _require_gpu_bf16(embed=embed, packed=packed)
        assert packed.is_contiguous() and packed.numel() >= ((rows + 15) // 16) * 16 * cols
    rc = _lib.load().nvh_embed_rows(x.data_ptr(), _ptr(xb), _ptr(packed), tokens.data_ptr(), embed.data_ptr(), float(scale), rows, cols, embed.shape[0], _ptr(copy),
                                    _ptr(positions) if table is not None else None, _ptr(table), table.shape[0] if table is not None else 0, code, _stream())
    _lib.check(rc, "nvh_embed_rows")
    return x, xb if xb is not None else x


def norm_residual(x, weight, eps, n, dtype, y=None, packed=None, want_rows=True):
    """y given: x (fp32 stream, in place) += rmsnorm(y) * weight; returns the new stream in `dtype` (x itself for fp32).  y None: returns
    rmsnorm(x) * weight in `dtype`, x unchanged.  The mean runs over the first n columns; packed (bf16): the rows also in fragment order."""
    _require_f32(x=x, weight=weight)
    rows, cols = x.shape
    assert weight.numel() == cols
    xb = None
    if want_rows and (dtype != torch.float32 or y is None):
        xb = torch.empty((rows, cols), dtype=dtype, device=x.device)
    d = _lib.NormResidualDesc()
    d.x, d.w, d.eps, d.rows, d.cols, d.n = x.data_ptr(), weight.data_ptr(), float(eps), rows, cols, int(n)
    d.xb = xb.data_ptr() if xb is not None else None
    if packed is not None:
        _require_gpu_bf16(packed=packed)
        assert packed.is_contiguous() and packed.numel() >= ((rows + 15) // 16) * 16 * cols
        d.packed = packed.data_ptr()
    if y is not None:
        assert y.shape == x.shape and y.stride(1) == 1 and y.dtype == dtype and y.is_cuda
        d.y, d.y_stride = y.data_ptr(), y.stride(0)
    _lib.check(_lib.load().nvh_norm_residual(ctypes.byref(d), _out_code(dtype), _stream()), "nvh_norm_residual")
    return xb if xb is not None else x


def clamped_glu(gate_up, limit, alpha):
    """g sigmoid(alpha g) (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit); rows hold gate | up."""
    code = _act_code(gate_up)
    inter = gate_up.shape[1] // 2
    assert gate_up.dim() == 2 and gate_up.stride(1) == 1
    out = torch.empty((gate_up.shape[0], inter), dtype=gate_up.dtype, device=gate_up.device)
    rc = _lib.load().nvh_clamped_glu(out.data_ptr(), gate_up.data_ptr(), gate_up.shape[0], inter, gate_up.stride(0), out.stride(0), float(limit), float(alpha),
                                     code, _stream())
    _lib.check(rc, "nvh_clamped_glu")
    return out


def gelu_glu(gate_up):
    """gelu(gate) * up with the tanh form of gelu; rows hold gate | up."""
    code = _act_code(gate_up)
    inter = gate_up.shape[1] // 2
    assert gate_up.dim() == 2 and gate_up.stride(1) == 1
    out = torch.empty((gate_up.shape[0], inter), dtype=gate_up.dtype, device=gate_up.device)
    rc = _lib.load().nvh_gelu_glu(out.data_ptr(), gate_up.data_ptr(), gate_up.shape[0], inter, gate_up.stride(0), out.stride(0), code, _stream())
    _lib.check(rc, "nvh_gelu_glu")
    return out


def rglru_chunk_tokens() -> int:
    return int(_lib.load().nvh_rglru_chunk_tokens())


def rglru_step_supported(block) -> bool:
    return bool(_lib.load().nvh_rglru_step_supported(int(block)))


def _rglru_desc(yx, p, positions, state_slots, state, conv_state):
    code = _act_code(yx, p["ra"], p["ri"], conv_state)
    blocks, block, _ = p["ra"].shape
    width = blocks * block
    taps = p["conv_w"].shape[0]
    _require_f32(conv_w=p["conv_w"], conv_b=p["conv_b"], ra_b=p["ra_b"], ri_b=p["ri_b"], rate=p["rate"], state=state)
    _require_i32(state_slots=state_slots)
    assert yx.stride(1) == 1 and yx.shape[1] == 2 * width and p["ra"].is_contiguous() and p["ri"].is_contiguous() and p["ri"].shape == p["ra"].shape
    assert p["conv_w"].shape == (taps, width) and all(p[n].numel() == width for n in ("conv_b", "ra_b", "ri_b", "rate"))
    assert state.shape[1] == width and conv_state.shape == (state.shape[0], taps, width) and conv_state.is_contiguous()
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == yx.shape[0]
    d = _lib.RglruDesc()
    d.yx, d.yx_stride, d.width, d.block, d.blocks, d.taps = yx.data_ptr(), yx.stride(0), width, block, blocks, taps
    d.conv_w, d.conv_b, d.ra, d.ri = p["conv_w"].data_ptr(), p["conv_b"].data_ptr(), p["ra"].data_ptr(), p["ri"].data_ptr()
    d.ra_b, d.ri_b, d.rate = p["ra_b"].data_ptr(), p["ri_b"].data_ptr(), p["rate"].data_ptr()
    d.positions, d.state_slots, d.state, d.conv_state = positions.data_ptr(), state_slots.data_ptr(), state.data_ptr(), conv_state.data_ptr()
    return d, width, code


def rglru_chunks(yx, params, positions, state_slots, chunks, segment, summaries, state, conv_state, out=None, generic=False):
    """Gated linear recurrence over portions of sequences.  yx [rows, 2 * width] = gate branch | recurrent branch; params = dict(conv_w [taps, width],
    conv_b, ra / ri [blocks, block, block], ra_b, ri_b, rate); chunks int32 [n, 4] = (first row, rows, sequence, index in its portion), portions cut every
    `segment` tokens (a multiple of rglru_chunk_tokens()); summaries: some portion has more than one segment.  state [slots, width] fp32 and conv_state
    [slots, taps, width] are updated.  Rows no segment covers are left alone in `out` (they belong to another launch)."""
    d, width, code = _rglru_desc(yx, params, positions, state_slots, state, conv_state)
    _require_i32(chunks=chunks)
    assert chunks.dim() == 2 and chunks.shape[1] == 4 and chunks.is_contiguous()
    rows = yx.shape[0]
    if out is None:
        out = torch.empty((rows, width), dtype=yx.dtype, device=yx.device)
    assert out.shape == (rows, width) and out.stride(1) == 1 and out.dtype == yx.dtype
    scratch = torch.empty((2, chunks.shape[0], width), dtype=torch.float32, device=yx.device)
    d.chunks, d.n_chunks, d.s_loc, d.a_cum = chunks.data_ptr(), chunks.shape[0], scratch[0].data_ptr(), scratch[1].data_ptr()
    d.segment, d.summaries = int(segment), int(summaries)
    d.out, d.out_stride = out.data_ptr(), out.stride(0)
    _lib.check(_lib.load().nvh_rglru_chunks(ctypes.byref(d), int(generic), code, _stream()), "nvh_rglru_chunks")
    return out


def rglru_step(yx, params, positions, state_slots, state, conv_state, out=None, out_packed=None, want_out=True):
    """One new token per sequence (row i = sequence i), the whole recurrence in one launch (bf16).  out_packed: also in fragment order."""
    d, width, code = _rglru_desc(yx, params, positions, state_slots, state, conv_state)
    rows = yx.shape[0]
    assert state_slots.numel() >= rows
    if out is None and want_out:
        out = torch.empty((rows, width), dtype=yx.dtype, device=yx.device)
    if out is not None:
        assert out.shape == (rows, width) and out.stride(1) == 1 and out.dtype == yx.dtype
        d.out, d.out_stride = out.data_ptr(), out.stride(0)
    if out_packed is not None:
        _require_gpu_bf16(out_packed=out_packed)
        assert out_packed.is_contiguous() and out_packed.numel() >= ((rows + 15) // 16) * 16 * width
        d.out_packed = out_packed.data_ptr()
    _lib.check(_lib.load().nvh_rglru_step(ctypes.byref(d), rows, code, _stream()), "nvh_rglru_step")
    return out


def latent_prep(a, q_rank, q_weight, eps, positions, cos_sin, kv_rank=0, kv_weight=None, cache=None, slots=None, cq_packed=None):
    """Row ops behind the down-projections: returns the normed query latent [rows, q_cols]; with `cache` given also norms the key latent, rotates the
    shared key part and stores the row.  `a` rows: query latent (q_cols) | key latent (kv_cols) | shared key part (rot_cols)."""
    code = _act_code(a)
    rows, q_cols = a.shape[0], q_weight.numel()
    _require_f32(q_weight=q_weight, cos_sin=cos_sin)
    assert a.stride(1) == 1 and positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    d = _lib.LatentPrepDesc()
    d.a, d.a_stride, d.rows, d.q_rank, d.q_cols, d.q_w, d.eps = a.data_ptr(), a.stride(0), rows, q_rank, q_cols, q_weight.data_ptr(), float(eps)
    cq = None
    if cq_packed is None:
        cq = torch.empty((rows, q_cols), dtype=a.dtype, device=a.device)
        d.cq = cq.data_ptr()
    else:
        _require_gpu_bf16(cq_packed=cq_packed)
        assert cq_packed.is_contiguous() and cq_packed.numel() >= ((rows + 15) // 16) * 16 * q_cols
        d.cq_packed = cq_packed.data_ptr()
    if cache is not None:
        _require_f32(kv_weight=kv_weight)
        _require_i32(slots=slots)
        _act_code(a, cache)
        kv_cols = kv_weight.numel()
        assert cache.is_contiguous() and slots.numel() == rows and slots.is_contiguous() and a.shape[1] >= q_cols + cache.shape[-1]
        d.kv_rank, d.kv_cols, d.kv_w, d.rot, d.rot_cols = kv_rank, kv_cols, kv_weight.data_ptr(), cos_sin.shape[1], cache.shape[-1] - kv_cols
        d.cache, d.slots, d.positions, d.cos_sin, d.max_position = cache.data_ptr(), slots.data_ptr(), positions.data_ptr(), cos_sin.data_ptr(), cos_sin.shape[0]
    _lib.check(_lib.load().nvh_latent_prep(ctypes.byref(d), code, _stream()), "nvh_latent_prep")
    return cq


def latent_attend_mfma(kv_cols, rot_cols, block_size) -> bool:
    return bool(_lib.load().nvh_latent_attend_mfma(kv_cols, rot_cols, block_size))


def latent_splits(rows, heads, max_context, mfma, cache_cols=576) -> int:
    """Context splits of one latent-attention launch.  MFMA form: as many workgroups as the 256 CUs hold at once (two LDS images of 64 cache rows
    each), every split the same number of 64-key tiles."""
    tiles = (max_context + 63) // 64
    if not mfma:
        return max(1, min(512 // max(1, rows * heads), tiles, 64))
    resident = 256 * (2 if 4 * 64 * cache_cols * 2 + 16384 <= 163840 else 1)
    groups = 1 if heads <= 16 else (heads + 31) // 32
    splits = max(1, min(resident // (rows * groups), tiles, 64))
    per = -(-tiles // splits)
    return -(-tiles // per)


def latent_attention(q, cache, block_tables, positions, cos_sin, w_uk, w_uv, scale, rot, max_context, row_seq=None, out=None, out_packed=None, want_out=True,
                     splits=None, generic=False):
    """Causal latent attention of single rows (row i attends positions 0 .. positions[i] of sequence row_seq[i], or i): q [rows, heads, dim_cols +
    qrot_cols] unrotated | rotated part (turned here); cache pages [blocks, block_size, kv_cols + rot_cols]; w_uk [heads, kv_cols, dim_cols],
    w_uv [heads, v_cols, kv_cols].  Returns [rows, heads * v_cols].  generic=True forces the plain kernel (tests)."""
    code = _act_code(q, cache, w_uk, w_uv)
    rows = q.shape[0]
    heads, kv_cols, dim_cols = w_uk.shape
    v_cols, cols, block_size = w_uv.shape[1], cache.shape[2], cache.shape[1]
    _require_f32(cos_sin=cos_sin)
    _require_i32(block_tables=block_tables)
    assert q.dim() == 2 and q.stride(1) == 1 and q.shape[1] % heads == 0 and w_uk.is_contiguous() and w_uv.is_contiguous() and cache.is_contiguous()
    assert w_uv.shape == (heads, v_cols, kv_cols) and block_tables.dim() == 2 and block_tables.stride(1) == 1
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    mfma = code == NVH_BF16 and row_seq is None and not generic and latent_attend_mfma(kv_cols, cols - kv_cols, block_size)
    splits = splits or latent_splits(rows, heads, max_context, mfma, cols)
    qa = torch.empty((rows, heads, cols), dtype=q.dtype, device=q.device)
    part_o = torch.empty((rows, splits, heads, kv_cols), dtype=torch.float32, device=q.device)
    part_ml = torch.empty((rows, splits, heads, 2), dtype=torch.float32, device=q.device)
    if out is None and want_out:
        out = torch.empty((rows, heads * v_cols), dtype=q.dtype, device=q.device)
    d = _lib.LatentAttnDesc()
    d.q, d.q_stride, d.rows, d.heads, d.dim_cols, d.qrot_cols = q.data_ptr(), q.stride(0), rows, heads, dim_cols, q.shape[1] // heads - dim_cols
    d.cache, d.kv_cols, d.rot, d.rot_cols, d.block_size = cache.data_ptr(), kv_cols, int(rot), cols - kv_cols, block_size
    d.block_tables, d.bt_stride, d.max_blocks = block_tables.data_ptr(), block_tables.stride(0), block_tables.shape[1]
    if row_seq is not None:
        _require_i32(row_seq=row_seq)
        assert row_seq.numel() == rows and row_seq.is_contiguous()
        d.row_seq = row_seq.data_ptr()
    else:
        assert block_tables.shape[0] >= rows
    d.positions, d.cos_sin, d.max_position = positions.data_ptr(), cos_sin.data_ptr(), cos_sin.shape[0]
    d.w_uk, d.w_uv, d.v_cols, d.scale = w_uk.data_ptr(), w_uv.data_ptr(), v_cols, float(scale)
    d.qa, d.part_o, d.part_ml, d.splits = qa.data_ptr(), part_o.data_ptr(), part_ml.data_ptr(), splits
    if out is not None:
        assert out.shape == (rows, heads * v_cols) and out.stride(1) == 1 and out.dtype == q.dtype
        d.out, d.out_stride = out.data_ptr(), out.stride(0)
    if out_packed is not None:
        _require_gpu_bf16(out_packed=out_packed)
        assert out_packed.is_contiguous() and out_packed.numel() >= ((rows + 15) // 16) * 16 * heads * v_cols
        d.out_packed = out_packed.data_ptr()
    _lib.check(_lib.load().nvh_latent_attention(ctypes.byref(d), int(generic), code, _stream()), "nvh_latent_attention")
    return out


def latent_gather(cache, cu_k, total, block_tables):
    """The cache rows of every key of the sequences, packed [total, cols]."""
    code = _act_code(cache)
    _require_i32(cu_k=cu_k, block_tables=block_tables)
    batch = cu_k.numel() - 1
    assert cache.is_contiguous() and cu_k.is_contiguous() and block_tables.shape[0] >= batch and block_tables.stride(1) == 1
    out = torch.empty((total, cache.shape[2]), dtype=cache.dtype, device=cache.device)
    rc = _lib.load().nvh_latent_gather(out.data_ptr(), cache.data_ptr(), cu_k.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), batch, total,
                                       cache.shape[2], cache.shape[1], code, _stream())
    _lib.check(rc, "nvh_latent_gather")
    return out


def latent_prefill_supported(dk, dv) -> bool:
    return bool(_lib.load().nvh_latent_prefill_supported(dk, dv))


def latent_prefill(q, k, k_rot, v, cu_q, cu_k, max_q, positions, cos_sin, scale, out=None):
    """Causal attention of prompt portions in expanded form: q [rows, heads, dk] (rotated part not turned yet), k [keys, heads, dim_cols], k_rot
    [keys, >= dk - dim_cols] shared by the heads, v [keys, heads, dv] (all with any row stride).  Returns [rows, heads * dv] (bf16)."""
    _require_gpu_bf16(q=q, k=k, k_rot=k_rot, v=v)
    _require_i32(cu_q=cu_q, cu_k=cu_k)
    _require_f32(cos_sin=cos_sin)
    rows, heads, dk = q.shape
    dim_cols, dv = k.shape[2], v.shape[2]
    assert k.shape[1] == heads and v.shape[1] == heads and q.stride(1) == dk and k.stride(1) == dim_cols and v.stride(1) == dv
    assert q.stride(2) == 1 and k.stride(2) == 1 and v.stride(2) == 1 and k_rot.stride(1) == 1 and k_rot.shape[1] >= dk - dim_cols
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows and cu_q.numel() == cu_k.numel()
    if out is None:
        out = torch.empty((rows, heads * dv), dtype=torch.bfloat16, device=q.device)
    assert out.shape == (rows, heads * dv) and out.stride(1) == 1
    d = _lib.LatentPrefillDesc()
    d.q, d.k, d.k_rot, d.v, d.out = q.data_ptr(), k.data_ptr(), k_rot.data_ptr(), v.data_ptr(), out.data_ptr()
    d.q_stride, d.k_stride, d.kr_stride, d.v_stride, d.out_stride = q.stride(0), k.stride(0), k_rot.stride(0), v.stride(0), out.stride(0)
    d.cu_q, d.cu_k, d.positions, d.cos_sin, d.max_position, d.rot = (cu_q.data_ptr(), cu_k.data_ptr(), positions.data_ptr(), cos_sin.data_ptr(),
                                                                     cos_sin.shape[0], cos_sin.shape[1])
    d.batch, d.heads, d.dim_cols, d.dk, d.dv, d.max_q, d.scale_log2 = cu_q.numel() - 1, heads, dim_cols, dk, dv, int(max_q), float(scale) * 1.4426950408889634
    _lib.check(_lib.load().nvh_latent_prefill(ctypes.byref(d), NVH_BF16, _stream()), "nvh_latent_prefill")
    return out


# --------------------------------------------------------------------------------------- paged sink/window attention
def _packed_ok(packed, rows, cols):
    _require_gpu_bf16(packed=packed)
    assert packed.is_contiguous() and packed.numel() >= ((rows + 15) // 16) * 16 * cols


def attn_prep(qkv, heads, kv_heads, dk, dv, positions, cos_sin, cache, slots, q_weight=None, k_weight=None, q_n=0, k_n=0, eps=0.0, head_norm=False, v_cos_sin=None):
    """Row ops behind a q | k | v projection: optional RMS norm over all query and all key columns (means over q_n / k_n of them; head_norm: over every head
    by itself, weights [dk] shared by the heads), rotation of interleaved pairs of the first cos_sin.shape[1] dimensions of every head (None: no rotation), of
    values by v_cos_sin, keys and values into the cache [pages, block_size, kv_heads * (dk + dv)] (inside a page: [kv head][keys | values]).  The queries are rewritten in place."""
    code = _act_code(qkv, cache)
    rows = qkv.shape[0]
    _require_i32(slots=slots)
    assert qkv.dim() == 2 and qkv.stride(1) == 1 and qkv.shape[1] >= heads * dk + kv_heads * (dk + dv)
    assert cache.dim() == 3 and cache.is_contiguous() and cache.shape[2] == kv_heads * (dk + dv)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows and slots.numel() == rows and slots.is_contiguous()
    d = _lib.AttnPrepDesc()
    d.qkv, d.qkv_stride, d.rows, d.heads, d.kv_heads, d.dk, d.dv = qkv.data_ptr(), qkv.stride(0), rows, heads, kv_heads, dk, dv
    if q_weight is not None:
        _require_f32(q_weight=q_weight, k_weight=k_weight)
        assert (q_weight.numel(), k_weight.numel()) == ((dk, dk) if head_norm else (heads * dk, kv_heads * dk))
        d.head_norm = int(head_norm)
        d.q_w, d.k_w, d.q_n, d.k_n, d.eps = q_weight.data_ptr(), k_weight.data_ptr(), int(q_n), int(k_n), float(eps)
    d.positions = positions.data_ptr()
    if cos_sin is not None:
        _require_f32(cos_sin=cos_sin)
        d.cos_sin, d.max_position, d.rot = cos_sin.data_ptr(), cos_sin.shape[0], cos_sin.shape[1]
    if v_cos_sin is not None:
        _require_f32(v_cos_sin=v_cos_sin)
        assert cos_sin is None or cos_sin.shape[0] == v_cos_sin.shape[0]
        d.v_cos_sin, d.max_position, d.v_rot = v_cos_sin.data_ptr(), v_cos_sin.shape[0], v_cos_sin.shape[1]
    d.cache, d.slots, d.block_size = cache.data_ptr(), slots.data_ptr(), cache.shape[1]
    _lib.check(_lib.load().nvh_attn_prep(ctypes.byref(d), code, _stream()), "nvh_attn_prep")


def paged_attend_supported(dk, dv, block_size) -> bool:
    return bool(_lib.load().nvh_paged_attend_supported(int(dk), int(dv), int(block_size)))


def paged_attend_splits(rows, kv_heads, heads, max_context, window=0, keep_first=0, chunk=0) -> int:
    """Context splits of one launch over single rows: about two workgroups per CU, none with fewer than two 64-key tiles."""
    window = window or chunk
    seen = min(max_context, window + keep_first + 126) if window else max_context
    tiles = (seen + 63) // 64
    groups = rows * kv_heads * ((heads // kv_heads + 7) // 8)
    splits = max(1, min(512 // max(1, groups), (tiles + 1) // 2, 64))
    per = -(-tiles // splits)
    return -(-tiles // per)


def _paged_desc(q, cache, block_tables, heads, kv_heads, dk, dv, scale, window, keep_first, sink, out, chunk=0, turn=None):
    code = _act_code(q, cache)
    rows = q.shape[0]
    _require_i32(block_tables=block_tables)
    assert q.dim() == 2 and q.stride(1) == 1 and q.shape[1] >= heads * dk and cache.dim() == 3 and cache.is_contiguous() and cache.shape[2] == kv_heads * (dk + dv)
    assert block_tables.dim() == 2 and block_tables.stride(1) == 1
    d = _lib.PagedAttendDesc()
    d.q, d.q_stride, d.rows, d.heads, d.kv_heads, d.dk, d.dv = q.data_ptr(), q.stride(0), rows, heads, kv_heads, dk, dv
    d.cache, d.block_size, d.block_tables, d.bt_stride = cache.data_ptr(), cache.shape[1], block_tables.data_ptr(), block_tables.stride(0)
    d.scale, d.window, d.keep_first, d.splits, d.chunk = float(scale), int(window), int(keep_first), 1, int(chunk)
    if turn is not None:
        _require_f32(turn=turn)
        d.o_cos_sin, d.max_position, d.o_rot = turn.data_ptr(), turn.shape[0], turn.shape[1]
    if sink is not None:
        _require_f32(sink=sink)
        assert sink.numel() == heads
        d.sink = sink.data_ptr()
    if out is not None:
        assert out.shape == (rows, heads * dv) and out.stride(1) == 1 and out.dtype == q.dtype
        d.out, d.out_stride = out.data_ptr(), out.stride(0)
    return d, code


SCORE_BYTES = 256 << 20        # scores talk_rows keeps in memory at a time: more rows run in several launches


def talk_rows_supported(heads, dk, dv, block_size) -> bool:
    return bool(_lib.load().nvh_talk_rows_supported(int(heads), int(dk), int(dv), int(block_size)))


TALK_PROMPT_MAX = 2000.0       # largest entry of a mixing matrix talk_prompt takes


def talk_prompt_supported(heads, kv_heads, dk, dv, block_size, softcap) -> bool:
    return bool(_lib.load().nvh_talk_prompt_supported(int(heads), int(kv_heads), int(dk), int(dv), int(block_size), float(softcap)))


def _set_talk(d, talk, softcap, heads):
    _require_f32(talk=talk)
    assert talk.shape == (heads, heads)
    d.talk, d.softcap = talk.data_ptr(), float(softcap)


def talk_rows(q, cache, block_tables, positions, heads, kv_heads, dk, dv, scale, max_context, talk, softcap=0.0, window=0, keep_first=0, sink=None, row_seq=None, out=None,
              out_packed=None, want_out=True, splits=None, generic=False):
    """paged_attend_rows with scores capped (softcap tanh(scale q . k / softcap); 0: not) and mixed across the heads by talk [heads, heads] before the softmax."""
    rows = q.shape[0]
    if out is None and want_out:
        out = torch.empty((rows, heads * dv), dtype=q.dtype, device=q.device)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    if row_seq is not None:
        _require_i32(row_seq=row_seq)
        assert row_seq.numel() == rows and row_seq.is_contiguous()
    else:
        assert block_tables.shape[0] >= rows
    lib = _lib.load()
    # 64-key tiles a row sees at most: all of its context, or those a window and the kept first tokens touch
    tiles = (max_context + 63) // 64
    if window:
        tiles = min(tiles, (window + 126) // 64 + (keep_first + 63) // 64)
    cols = int(lib.nvh_talk_score_cols(heads))
    step = max(1, SCORE_BYTES // (tiles * 64 * cols * 4))
    fast = q.dtype == torch.bfloat16 and row_seq is None and not generic and talk_rows_supported(heads, dk, dv, cache.shape[1])
    assert out_packed is None or step >= rows, "packed rows are few"
    for r in range(0, rows, step):
        n = min(step, rows - r)
        d, code = _paged_desc(q[r:r + n], cache, block_tables if row_seq is not None else block_tables[r:], heads, kv_heads, dk, dv, scale, window, keep_first, sink,
                              out[r:r + n] if out is not None else None)
        _set_talk(d, talk, softcap, heads)
        d.positions = positions[r:].data_ptr()
        d.row_seq = row_seq[r:].data_ptr() if row_seq is not None else None
        scores = torch.empty((n, tiles * 64, cols), dtype=torch.float32, device=q.device)
        d.scores, d.span = scores.data_ptr(), tiles * 64
        if fast:
            d.splits = splits or paged_attend_splits(n, kv_heads, heads, max_context, window, keep_first)
        if d.splits > 1:
            part = torch.empty((n, heads, d.splits, dv + 4), dtype=torch.float32, device=q.device)
            tickets = reserve_workspace(q.device, int(lib.nvh_talk_ticket_bytes(n, kv_heads, heads)), "paged_attend")
            d.part, d.tickets = part.data_ptr(), tickets.data_ptr()
        if out_packed is not None:
            _packed_ok(out_packed, rows, heads * dv)
            d.out_packed = out_packed.data_ptr()
        _lib.check(lib.nvh_talk_rows(ctypes.byref(d), int(generic), code, _stream()), "nvh_talk_rows")
    return out


def talk_prompt(q, cache, block_tables, cu_q, cu_k, max_q, heads, kv_heads, dk, dv, scale, talk, softcap=0.0, window=0, keep_first=0, sink=None, out=None):
    """paged_attend_prompt with capped scores mixed across the heads (see talk_rows)."""
    _require_gpu_bf16(q=q)
    _require_i32(cu_q=cu_q, cu_k=cu_k)
    if out is None:
        out = torch.empty((q.shape[0], heads * dv), dtype=q.dtype, device=q.device)
    d, code = _paged_desc(q, cache, block_tables, heads, kv_heads, dk, dv, scale, window, keep_first, sink, out)
    assert cu_q.numel() == cu_k.numel() and cu_q.is_contiguous() and cu_k.is_contiguous() and block_tables.shape[0] >= cu_q.numel() - 1
    d.cu_q, d.cu_k, d.batch, d.max_q = cu_q.data_ptr(), cu_k.data_ptr(), cu_q.numel() - 1, int(max_q)
    _set_talk(d, talk, softcap, heads)
    _lib.check(_lib.load().nvh_talk_prompt(ctypes.byref(d), code, _stream()), "nvh_talk_prompt")
    return out


def paged_attend_rows(q, cache, block_tables, positions, heads, kv_heads, dk, dv, scale, max_context, window=0, keep_first=0, sink=None, row_seq=None, out=None,
                      out_packed=None, want_out=True, splits=None, generic=False, chunk=0, turn=None):
    """Attention of single query rows over the pages (row i: sequence row_seq[i], or i; sees its own position and before, with window > 0 only what is
    nearer than `window` or among the first keep_first tokens, with chunk > 0 only what lies in its own chunk of that many positions, or among those; sink
    [heads] joins the softmax; turn [positions, dims]: the output is turned back by the angles of its position).  Returns [rows, heads * dv].
    generic=True forces the plain kernel (tests)."""
    rows = q.shape[0]
    if out is None and want_out:
        out = torch.empty((rows, heads * dv), dtype=q.dtype, device=q.device)
    d, code = _paged_desc(q, cache, block_tables, heads, kv_heads, dk, dv, scale, window, keep_first, sink, out, chunk, turn)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    d.positions = positions.data_ptr()
    if row_seq is not None:
        _require_i32(row_seq=row_seq)
        assert row_seq.numel() == rows and row_seq.is_contiguous()
        d.row_seq = row_seq.data_ptr()
    else:
        assert block_tables.shape[0] >= rows
    if code == NVH_BF16 and row_seq is None and not generic and paged_attend_supported(dk, dv, cache.shape[1]):
        d.splits = splits or paged_attend_splits(rows, kv_heads, heads, max_context, window, keep_first, chunk)
    if d.splits > 1:
        part = torch.empty((rows, heads, d.splits, dv + 4), dtype=torch.float32, device=q.device)
        tickets = reserve_workspace(q.device, paged_attend_ticket_bytes(rows, kv_heads, heads), "paged_attend")
        d.part, d.tickets = part.data_ptr(), tickets.data_ptr()
    if out_packed is not None:
        _packed_ok(out_packed, rows, heads * dv)
        d.out_packed = out_packed.data_ptr()
    _lib.check(_lib.load().nvh_paged_attend_rows(ctypes.byref(d), int(generic), code, _stream()), "nvh_paged_attend_rows")
    return out


def paged_attend_ticket_bytes(rows, kv_heads, heads) -> int:
    return int(_lib.load().nvh_paged_attend_ticket_bytes(rows, kv_heads, heads))


def paged_attend_prompt(q, cache, block_tables, cu_q, cu_k, max_q, heads, kv_heads, dk, dv, scale, window=0, keep_first=0, sink=None, out=None, chunk=0, turn=None):
    """Attention of prompt portions over the pages (bf16): rows cu_q[b] .. of q are the last ones of sequence b, which has cu_k[b + 1] - cu_k[b] keys;
    visibility, sink and turn as in paged_attend_rows.  Returns [rows, heads * dv]."""
    _require_gpu_bf16(q=q)
    _require_i32(cu_q=cu_q, cu_k=cu_k)
    if out is None:
        out = torch.empty((q.shape[0], heads * dv), dtype=q.dtype, device=q.device)
    d, code = _paged_desc(q, cache, block_tables, heads, kv_heads, dk, dv, scale, window, keep_first, sink, out, chunk, turn)
    assert cu_q.numel() == cu_k.numel() and cu_q.is_contiguous() and cu_k.is_contiguous() and block_tables.shape[0] >= cu_q.numel() - 1
    d.cu_q, d.cu_k, d.batch, d.max_q = cu_q.data_ptr(), cu_k.data_ptr(), cu_q.numel() - 1, int(max_q)
    _lib.check(_lib.load().nvh_paged_attend_prompt(ctypes.byref(d), code, _stream()), "nvh_paged_attend_prompt")
    return out


# --------------------------------------------------------------------------------------- lightning attention
def lightning_supported(dk, dv) -> bool:
    return bool(_lib.load().nvh_lightning_supported(int(dk), int(dv)))


def _lightning_desc(qkv, decay, positions, state_slots, state, out):
    code = _act_code(qkv)
    slots, heads, dk, dv = state.shape
    rows = qkv.shape[0]
    _require_f32(decay=decay, state=state)
    _require_i32(state_slots=state_slots)
    assert qkv.dim() == 2 and qkv.stride(1) == 1 and qkv.shape[1] >= heads * (2 * dk + dv) and decay.numel() == heads
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    if out is None:
        out = torch.empty((rows, heads * dv), dtype=qkv.dtype, device=qkv.device)
    assert out.shape == (rows, heads * dv) and out.stride(1) == 1 and out.dtype == qkv.dtype
    d = _lib.LightningDesc()
    d.qkv, d.qkv_stride, d.rows, d.heads, d.dk, d.dv = qkv.data_ptr(), qkv.stride(0), rows, heads, dk, dv
    d.decay, d.positions, d.state_slots, d.state = decay.data_ptr(), positions.data_ptr(), state_slots.data_ptr(), state.data_ptr()
    d.out, d.out_stride = out.data_ptr(), out.stride(0)
    return d, out, code


def lightning_chunks(qkv, decay, positions, state_slots, chunks, summaries, state, out=None, generic=False):
    """Lightning attention over portions of sequences.  qkv rows: q (heads * dk) | k (heads * dk) | v (heads * dv), SiLU not applied yet; chunks int32 [n, 4] =
    (first row, rows, sequence, index in its portion); summaries: some portion has more than one segment; state [slots, heads, dk, dv] fp32 is
    updated.  Rows no segment covers are left alone in `out`."""
    d, out, code = _lightning_desc(qkv, decay, positions, state_slots, state, out)
    _require_i32(chunks=chunks)
    assert chunks.dim() == 2 and chunks.shape[1] == 4 and chunks.is_contiguous()
    d.chunks, d.n_chunks, d.summaries = chunks.data_ptr(), chunks.shape[0], int(summaries)
    if summaries:
        seg = torch.empty((chunks.shape[0], *state.shape[1:]), dtype=torch.float32, device=qkv.device)
        d.seg_state = seg.data_ptr()
    _lib.check(_lib.load().nvh_lightning_chunks(ctypes.byref(d), int(generic), code, _stream()), "nvh_lightning_chunks")
    return out


def lightning_step(qkv, decay, positions, state_slots, state, out=None):
    """One new token per sequence (row i = sequence i), bf16."""
    d, out, code = _lightning_desc(qkv, decay, positions, state_slots, state, out)
    assert state_slots.numel() >= qkv.shape[0]
    _lib.check(_lib.load().nvh_lightning_step(ctypes.byref(d), code, _stream()), "nvh_lightning_step")
    return out


def norm_gate(x, gate, weight, eps, n, packed=None):
    """rmsnorm(x over n columns) * weight * sigmoid(gate); packed (bf16): in fragment order into this buffer, returns None."""
    code = _act_code(x, gate)
    _require_f32(weight=weight)
    rows, cols = x.shape
    assert gate.shape == x.shape and x.stride(1) == 1 and gate.stride(1) == 1 and weight.numel() == cols
    out = None
    if packed is None:
        out = torch.empty((rows, cols), dtype=x.dtype, device=x.device)
    else:
        _packed_ok(packed, rows, cols)
    rc = _lib.load().nvh_norm_gate(out.data_ptr() if out is not None else None, packed.data_ptr() if packed is not None else None, x.data_ptr(), gate.data_ptr(),
                                   weight.data_ptr(), float(eps), rows, cols, int(n), x.stride(0), gate.stride(0), cols, code, _stream())
    _lib.check(rc, "nvh_norm_gate")
    return out


# --------------------------------------------------------------------------------------- several residual streams, the token before
def _rows_desc(d, positions, rows, step):
    """Where rows stand in their sequences (utils/step.py StepMeta)."""
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    _require_i32(state_slots=step.state_slots)
    d.positions, d.state_slots = positions.data_ptr(), step.state_slots.data_ptr()
    if step.cu_rows is not None:
        _require_i32(row_seq=step.row_seq, cu_rows=step.cu_rows)
        assert step.row_seq.numel() == rows and step.state_slots.numel() >= step.cu_rows.numel() - 1
        d.row_seq, d.cu_rows = step.row_seq.data_ptr(), step.cu_rows.data_ptr()
        if hasattr(d, "sequences"):
            d.sequences = step.cu_rows.numel() - 1
    else:
        assert step.num_decode == rows and step.state_slots.numel() >= rows


def bigram_embed(tokens, positions, step, embed, bigram, mul_prev, mul_cur, last_token):
    """embed[token] + bigram[(previous token * mul_prev + token * mul_cur) mod buckets] (the last of the buckets + 1 rows for a sequence's first token) as fp32
    rows; last_token int64 [slots] carries the previous token from step to step."""
    code, rows, cols = _act_code(embed, bigram), tokens.numel(), embed.shape[1]
    assert tokens.dtype == torch.int64 and tokens.is_cuda and tokens.is_contiguous() and embed.is_contiguous() and bigram.is_contiguous() and bigram.shape[1] == cols
    assert last_token.dtype == torch.int64 and last_token.is_cuda and last_token.is_contiguous()
    x = torch.empty((rows, cols), dtype=torch.float32, device=embed.device)
    d = _lib.BigramEmbedDesc()
    _rows_desc(d, positions, rows, step)
    d.x, d.tokens, d.last_token, d.embed, d.bigram = x.data_ptr(), tokens.data_ptr(), last_token.data_ptr(), embed.data_ptr(), bigram.data_ptr()
    d.buckets, d.mul_prev, d.mul_cur, d.rows, d.cols, d.vocab = bigram.shape[0] - 1, int(mul_prev), int(mul_cur), rows, cols, embed.shape[0]
    _lib.check(_lib.load().nvh_bigram_embed(ctypes.byref(d), code, _stream()), "nvh_bigram_embed")
    return x


def stream_mix(x, streams, dtype, n, update=None, read=None, norm=None, packed=None, want_rows=True, out=None, shift=None):
    """Hyper-connections between two sublayers.  x: [rows, streams, cols] (fp32), or [rows, cols] where all streams are alike.
    update = dict(y, mix [from, to], out [to]): x_t <- sum_s mix[s, t] x_s + out[t] y (into `out`, or in place); with post = (y2, w, w2, scale) y is
    scale (rms(y) w + rms(y2) w2) first, eps of the norm, as norm = (.., eps) or update["eps"].  Of the new streams u = sum_s read[s] x_s (None: plain sum);
    norm = (weight, groups, eps): returns its RMS norm in `groups` equal parts of the n columns (in `dtype`; packed: in fragment order too); norm None: returns u (fp32).
    shift = dict(positions, step, shift, ring, mu, packed), single tokens: token_shift of the normed rows with these arguments in the same launch."""
    alike = x.dim() == 2
    rows, cols = x.shape[0], x.shape[-1]
    _require_f32(x=x)
    assert alike or x.shape[1] == streams
    d = _lib.StreamMixDesc()
    d.xin, d.xin_row, d.xin_stream = x.data_ptr(), cols if alike else streams * cols, 0 if alike else cols
    d.rows, d.cols, d.n, d.streams, d.groups = rows, cols, int(n), int(streams), 1
    if update is not None:
        y = update["y"]
        _require_f32(mix=update["mix"], out=update["out"])
        assert y.shape == (rows, cols) and y.stride(1) == 1 and y.dtype == dtype and y.is_cuda and update["mix"].shape == (streams, streams) and update["out"].numel() == streams
        d.y, d.y_stride, d.mix, d.out = y.data_ptr(), y.stride(0), update["mix"].data_ptr(), update["out"].data_ptr()
        if update.get("post") is not None:
            y2, w, w2, scale = update["post"]
            _require_f32(w=w, w2=w2)
            assert y2.shape == (rows, cols) and y2.stride(1) == 1 and y2.dtype == dtype and y2.is_cuda and w.numel() == w2.numel() == cols
            d.y2, d.y2_stride, d.y_w, d.y2_w, d.y_scale, d.eps = y2.data_ptr(), y2.stride(0), w.data_ptr(), w2.data_ptr(), float(scale), float(update["eps"])
        if out is None:
            assert not alike, "streams that are all alike need somewhere to go"
            out = x
        _require_f32(out=out)
        assert out.shape == (rows, streams, cols)
        d.xout = out.data_ptr()
    if read is not None:
        _require_f32(read=read)
        assert read.numel() == streams
        setattr(d, "in", read.data_ptr())
    if norm is None:
        res = torch.empty((rows, cols), dtype=torch.float32, device=x.device)
        d.sum = res.data_ptr()
    else:
        weight, d.groups, eps = norm
        _require_f32(weight=weight)
        assert weight.numel() == cols and (update is None or update.get("post") is None or update["eps"] == eps)
        d.w, d.eps, res = weight.data_ptr(), float(eps), None
        if want_rows:
            res = torch.empty((rows, cols), dtype=dtype, device=x.device)
            d.h = res.data_ptr()
        if packed is not None:
            _packed_ok(packed, rows, cols)
            d.packed = packed.data_ptr()
        if shift is not None:
            ring, mu, dst, step, positions = (shift[k] for k in ("ring", "mu", "packed", "step", "positions"))
            d.mixes, d.shifted_mix = 0 if mu is None else mu.shape[0], (rows + 15) // 16 * 16 * cols
            _require_f32(shift=shift["shift"])
            _require_gpu_bf16(ring=ring, packed=dst)
            _require_i32(state_slots=step.state_slots)
            assert shift["shift"].numel() == cols and ring.is_contiguous() and ring.shape[1:] == (3 if d.mixes else 2, cols)
            assert dst.is_contiguous() and dst.numel() >= max(d.mixes, 1) * d.shifted_mix
            assert step.num_decode == rows and step.state_slots.numel() >= rows and positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
            if mu is not None:
                _require_f32(mu=mu)
                assert mu.shape[1] == cols
                d.mu = mu.data_ptr()
            d.shift, d.ring, d.depth, d.shifted = shift["shift"].data_ptr(), ring.data_ptr(), ring.shape[1], dst.data_ptr()
            d.positions, d.state_slots = positions.data_ptr(), step.state_slots.data_ptr()
    _lib.check(_lib.load().nvh_stream_mix(ctypes.byref(d), _out_code(dtype), _stream()), "nvh_stream_mix")
    return res


def token_shift(h, positions, step, shift, ring, mu=None, packed=None):
    """s = h + (h' - h) shift with h' the previous token's h; without mu returns s [1, rows, cols], with mu [mixes, cols] s + (s' - s) mu[k] for every k
    [mixes, rows, cols]; packed (bf16): in fragment order into this buffer (one after the other), returns None.  ring [slots, 2 or 3 with mu, cols] carries h."""
    code = _act_code(h, ring)
    _require_f32(shift=shift)
    rows, cols = h.shape
    mixes = 0 if mu is None else mu.shape[0]
    assert h.stride(1) == 1 and shift.numel() == cols and ring.is_contiguous() and ring.shape[1:] == (3 if mixes else 2, cols)
    d = _lib.TokenShiftDesc()
    _rows_desc(d, positions, rows, step)
    d.h, d.h_stride, d.rows, d.cols, d.shift, d.mixes, d.ring, d.depth = h.data_ptr(), h.stride(0), rows, cols, shift.data_ptr(), mixes, ring.data_ptr(), ring.shape[1]
    if mixes:
        _require_f32(mu=mu)
        assert mu.shape == (mixes, cols)
        d.mu = mu.data_ptr()
    out, count = None, max(mixes, 1)
    if packed is None:
        out = torch.empty((count, rows, cols), dtype=h.dtype, device=h.device)
        d.out, d.out_mix = out.data_ptr(), rows * cols
    else:
        d.packed, d.out, d.out_mix = 1, packed.data_ptr(), (rows + 15) // 16 * 16 * cols
        _require_gpu_bf16(packed=packed)
        assert packed.is_contiguous() and packed.numel() >= count * d.out_mix
    _lib.check(_lib.load().nvh_token_shift(ctypes.byref(d), code, _stream()), "nvh_token_shift")
    return out


def causal_conv(x, positions, step, weight, bias, ring, packed=None, want_rows=True):
    """silu(bias + sum over taps of weight[tap] x), weight [taps, cols] with the last tap on the current token; ring [slots, taps, cols] carries x."""
    code = _act_code(x, ring)
    _require_f32(weight=weight, bias=bias)
    rows, cols = x.shape
    taps = weight.shape[0]
    assert x.stride(1) == 1 and weight.shape[1] == cols and bias.numel() == cols and ring.is_contiguous() and ring.shape[1:] == (taps, cols)
    d = _lib.CausalConvDesc()
    _rows_desc(d, positions, rows, step)
    d.x, d.x_stride, d.rows, d.cols, d.taps, d.w, d.b, d.ring = x.data_ptr(), x.stride(0), rows, cols, taps, weight.data_ptr(), bias.data_ptr(), ring.data_ptr()
    out = None
    if want_rows:
        out = torch.empty((rows, cols), dtype=x.dtype, device=x.device)
        d.out = out.data_ptr()
    if packed is not None:
        _packed_ok(packed, rows, cols)
        d.packed = packed.data_ptr()
    _lib.check(_lib.load().nvh_causal_conv(ctypes.byref(d), code, _stream()), "nvh_causal_conv")
    return out


# --------------------------------------------------------------------------------------- selective scan
def scan_states(n) -> int:
    """States the kernels keep for n of them (a power of two; 0: too many)."""
    return int(_lib.load().nvh_scan_states(int(n)))


def _scan_desc(x, dt, bc, z, p, positions, state_slots, state, out):
    code = _act_code(x, dt, bc, z)
    rows, (inner, n) = x.shape[0], p["a_log2"].shape
    _require_f32(a_log2=p["a_log2"], d=p["d"], dt_bias=p["dt_bias"], state=state)
    _require_i32(state_slots=state_slots)
    assert x.shape[1] == z.shape[1] == p["d"].numel() == p["dt_bias"].numel() == inner and z.shape[0] == dt.shape[0] == bc.shape[0] == rows and bc.shape[1] >= 2 * n
    assert x.stride(1) == z.stride(1) == dt.stride(1) == bc.stride(1) == 1 and state.shape[1:] == (inner, n)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    d = _lib.ScanDesc()
    d.x, d.x_stride, d.dt, d.dt_stride, d.bc, d.bc_stride, d.z, d.z_stride = x.data_ptr(), x.stride(0), dt.data_ptr(), dt.stride(0), bc.data_ptr(), bc.stride(0), z.data_ptr(), z.stride(0)
    d.dt_bias, d.a_log2, d.d, d.rows, d.inner, d.n = p["dt_bias"].data_ptr(), p["a_log2"].data_ptr(), p["d"].data_ptr(), rows, inner, n
    d.positions, d.state_slots, d.state = positions.data_ptr(), state_slots.data_ptr(), state.data_ptr()
    if out is not None:
        assert out.shape == (rows, inner) and out.stride(1) == 1 and out.dtype == x.dtype
        d.out, d.out_stride = out.data_ptr(), out.stride(0)
    return d, code


def scan_chunks(x, dt, bc, z, params, positions, state_slots, chunks, summaries, state, out=None):
    """Selective scan over portions of sequences: x, dt (in front of bias and softplus), z [rows, inner]; bc rows B (n) | C (n); params = dict(a_log2 [inner, n], d,
    dt_bias); chunks int32 [n, 4] = (first row, rows, sequence, index in its portion); summaries: some portion has more than one segment; state [slots, inner, n]
    fp32 is updated.  Returns (scan + d x) silu(z); rows no segment covers are left alone in `out`."""
    if out is None:
        out = torch.empty((x.shape[0], x.shape[1]), dtype=x.dtype, device=x.device)
    d, code = _scan_desc(x, dt, bc, z, params, positions, state_slots, state, out)
    _require_i32(chunks=chunks)
    assert dt.shape[1] == x.shape[1] and chunks.dim() == 2 and chunks.shape[1] == 4 and chunks.is_contiguous()
    d.chunks, d.n_chunks, d.summaries = chunks.data_ptr(), chunks.shape[0], int(summaries)
    if summaries:
        seg, seg_dt = (torch.empty((chunks.shape[0], *s), dtype=torch.float32, device=x.device) for s in (state.shape[1:], state.shape[1:2]))
        d.seg_state, d.seg_dt = seg.data_ptr(), seg_dt.data_ptr()
    _lib.check(_lib.load().nvh_scan_chunks(ctypes.byref(d), code, _stream()), "nvh_scan_chunks")
    return out


def scan_step(x, dt, bc, z, params, positions, state_slots, state, out=None, out_packed=None, want_out=True):
    """One new token per sequence (row i = sequence i), bf16; dt [rows, rank] is multiplied by params["w_dt"] [inner, rank] first."""
    rows, w = x.shape[0], params["w_dt"]
    if out is None and want_out:
        out = torch.empty((rows, x.shape[1]), dtype=x.dtype, device=x.device)
    d, code = _scan_desc(x, dt, bc, z, params, positions, state_slots, state, out)
    _act_code(x, w)
    assert w.is_contiguous() and w.shape[0] == x.shape[1] and dt.shape[1] >= w.shape[1] and state_slots.numel() >= rows
    d.w_dt, d.rank = w.data_ptr(), w.shape[1]
    if out_packed is not None:
        _packed_ok(out_packed, rows, x.shape[1])
        d.out_packed = out_packed.data_ptr()
    _lib.check(_lib.load().nvh_scan_step(ctypes.byref(d), code, _stream()), "nvh_scan_step")
    return out


# --------------------------------------------------------------------------------------- time mixing with a decaying matrix state
def wkv_supported(dim) -> bool:
    return bool(_lib.load().nvh_wkv_supported(int(dim)))


def _wkv_desc(r, k, v, g, z, p, eps, n, positions, state_slots, state, out):
    code = _act_code(r, k, v, g, z)
    slots, heads, dim, dv = state.shape
    rows, cols = r.shape[0], heads * dim
    _require_f32(w0=p["w0"], u=p["u"], norm=p["norm"], state=state)
    _require_i32(state_slots=state_slots)
    assert dv == dim and all(t.shape[0] == rows and t.shape[1] >= cols and t.stride(1) == 1 and t.stride(0) == r.stride(0) for t in (r, k, v, g))
    assert z.shape[0] == rows and z.stride(1) == 1 and all(p[t].numel() == cols for t in ("w0", "u", "norm"))
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == rows
    d = _lib.WkvDesc()
    d.r, d.k, d.v, d.g, d.stride, d.z, d.z_stride = r.data_ptr(), k.data_ptr(), v.data_ptr(), g.data_ptr(), r.stride(0), z.data_ptr(), z.stride(0)
    d.w0, d.u, d.norm, d.eps, d.n, d.rows, d.heads, d.dim = p["w0"].data_ptr(), p["u"].data_ptr(), p["norm"].data_ptr(), float(eps), int(n), rows, heads, dim
    d.positions, d.state_slots, d.state = positions.data_ptr(), state_slots.data_ptr(), state.data_ptr()
    if out is not None:
        assert out.shape == (rows, cols) and out.stride(1) == 1 and out.dtype == r.dtype
        d.out, d.out_stride = out.data_ptr(), out.stride(0)
    return d, code


def wkv_chunks(r, k, v, g, z, params, eps, n, positions, state_slots, chunks, summaries, state, out=None, generic=False):
    """Time mixing over portions of sequences: r, k, v, g, z [rows, heads * dim]; params = dict(w0, u, norm [heads * dim]); decays exp(-exp(z + w0)); n: columns of a
    head the norm counts; chunks int32 [n, 4] = (first row, rows, sequence, index in its portion); summaries: some portion has more than one segment; state
    [slots, heads, dim, dim] fp32 is updated.  Rows no segment covers are left alone in `out`.  generic=True forces the plain kernel (tests)."""
    if out is None:
        out = torch.empty((r.shape[0], state.shape[1] * state.shape[2]), dtype=r.dtype, device=r.device)
    d, code = _wkv_desc(r, k, v, g, z, params, eps, n, positions, state_slots, state, out)
    _require_i32(chunks=chunks)
    assert z.shape[1] >= state.shape[1] * state.shape[2] and chunks.dim() == 2 and chunks.shape[1] == 4 and chunks.is_contiguous()
    d.chunks, d.n_chunks, d.summaries = chunks.data_ptr(), chunks.shape[0], int(summaries)
    if summaries:
        seg, dec = (torch.empty((chunks.shape[0], *s), dtype=torch.float32, device=r.device) for s in (state.shape[1:], state.shape[1:3]))
        d.seg_state, d.seg_decay = seg.data_ptr(), dec.data_ptr()
    _lib.check(_lib.load().nvh_wkv_chunks(ctypes.byref(d), int(generic), code, _stream()), "nvh_wkv_chunks")
    return out


def wkv_step(r, k, v, g, z, params, eps, n, positions, state_slots, state, out=None, out_packed=None, want_out=True):
    """One new token per sequence (row i = sequence i), bf16; z [rows, rank]: decays of params["w2"] tanh(z) with w2 [heads * dim, rank]."""
    rows, w2, cols = r.shape[0], params["w2"], state.shape[1] * state.shape[2]
    if out is None and want_out:
        out = torch.empty((rows, cols), dtype=r.dtype, device=r.device)
    d, code = _wkv_desc(r, k, v, g, z, params, eps, n, positions, state_slots, state, out)
    _act_code(r, w2)
    assert w2.is_contiguous() and w2.shape[0] >= cols and z.shape[1] >= w2.shape[1] and state_slots.numel() >= rows
    d.w2, d.rank = w2.data_ptr(), w2.shape[1]
    if out_packed is not None:
        _packed_ok(out_packed, rows, cols)
        d.out_packed = out_packed.data_ptr()
    _lib.check(_lib.load().nvh_wkv_step(ctypes.byref(d), code, _stream()), "nvh_wkv_step")
    return out


# --------------------------------------------------------------------------------------- mixture of experts
def moe_route(x, router, correction, top, groups=1, keep=1, scale=1.0, softmax=False):
    """(chosen experts int32 [rows, top], weights fp32 [rows, top]) of rows x against router [experts, cols].  softmax: the choice goes by the logits with
    `correction` as their bias, the weights are the softmax over the chosen ones; otherwise sigmoid scores, corrections for the choice only, groups."""
    code = _act_code(x, router)
    _require_f32(correction=correction)
    rows, cols = x.shape
    experts = router.shape[0]
    assert router.is_contiguous() and router.shape[1] == cols and x.stride(1) == 1 and correction.numel() == experts
    ids = torch.empty((rows, top), dtype=torch.int32, device=x.device)
    weights = torch.empty((rows, top), dtype=torch.float32, device=x.device)
    d = _lib.MoeRouteDesc()
    d.x, d.x_stride, d.router, d.correction = x.data_ptr(), x.stride(0), router.data_ptr(), correction.data_ptr()
    d.rows, d.cols, d.experts, d.top, d.groups, d.keep, d.scale = rows, cols, experts, int(top), int(groups), int(keep), float(scale)
    d.ids, d.weights, d.softmax = ids.data_ptr(), weights.data_ptr(), int(softmax)
    _lib.check(_lib.load().nvh_moe_route(ctypes.byref(d), code, _stream()), "nvh_moe_route")
    return ids, weights


def moe_dispatch(ids, experts, dtype, tile_rows=None):
    """(slot_pair, tiles, rows per tile): the pairs row * top + k sorted by expert, cut into tiles of one expert each; nothing comes back to the host."""
    _require_i32(ids=ids)
    assert ids.is_contiguous()
    lib, pairs = _lib.load(), ids.numel()
    tile_rows = tile_rows or int(lib.nvh_moe_tile_rows(pairs, experts, _out_code(dtype)))
    max_tiles = pairs // tile_rows + min(experts, pairs)
    slots = torch.empty(pairs, dtype=torch.int32, device=ids.device)
    tiles = torch.empty((pairs // tile_rows + experts, 4), dtype=torch.int32, device=ids.device)
    counts = torch.empty((lib.nvh_moe_dispatch_blocks(pairs), experts), dtype=torch.int32, device=ids.device)
    _lib.check(lib.nvh_moe_dispatch(slots.data_ptr(), tiles.data_ptr(), counts.data_ptr(), ids.data_ptr(), pairs, experts, tile_rows, tiles.shape[0], _stream()),
               "nvh_moe_dispatch")
    return slots, tiles[:max_tiles], tile_rows


def moe_gemm(x, weight, ids, glu, dispatch=None, unit=None):
    """Expert products per pair p = row * top + k: glu: silu(x[row] . gate_e) * (x[row] . up_e) with weight [experts, 2 * n, k], or with unit = (limit, alpha)
    the clamped unit g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit); otherwise x[p] . w_e with
    weight [experts, n, k].  dispatch: what moe_dispatch returned; None: the form for at most 64 rows (bf16)."""
    code = _act_code(x, weight)
    experts, n, k = weight.shape
    n = n // 2 if glu else n
    pairs, top = ids.numel(), ids.shape[1]
    assert weight.is_contiguous() and x.dim() == 2 and x.stride(1) == 1 and x.shape == (ids.shape[0] if glu else pairs, k) and (glu or x.is_contiguous())
    out = torch.empty((pairs, n), dtype=x.dtype, device=x.device)
    d = _lib.MoeGemmDesc()
    d.out, d.x, d.x_stride, d.w = out.data_ptr(), x.data_ptr(), x.stride(0), weight.data_ptr()
    d.pairs, d.top, d.experts, d.n, d.k, d.glu = pairs, top, experts, n, k, int(glu)
    if unit is not None:
        assert glu and unit[1] != 0.0
        d.limit, d.alpha = float(unit[0]), float(unit[1])
    if dispatch is None:
        _require_i32(ids=ids)
        assert ids.is_contiguous()
        d.ids = ids.data_ptr()
    else:
        slots, tiles, d.tile_rows = dispatch
        assert slots.numel() == pairs and tiles.is_contiguous()
        d.slot_pair, d.tiles, d.max_tiles = slots.data_ptr(), tiles.data_ptr(), tiles.shape[0]
    _lib.check(_lib.load().nvh_moe_gemm(ctypes.byref(d), code, _stream()), "nvh_moe_gemm")
    return out


# --------------------------------------------------------------------------------------- residual and output of models with one norm per layer
def residual_norm(x, dtype, y=None, experts=None, weight=None, bias=None, eps=0.0, n=0, packed=None, want_rows=True, post=None, mult=1.0, base=None, shift=None):
    """x (fp32 stream, in place) += y + the weighted sum of experts = (outputs [rows * top, cols], weights [rows, top]), or mult times the layer norm of that sum
    with post = (weight, bias); += base [rows, cols], += shift [cols] (fp32) where given; with weight given returns the layer norm
    of the new rows (mean and variance over n columns) in `dtype`, and in fragment order into `packed` (bf16)."""
    _require_f32(x=x)
    rows, cols = x.shape
    code = _out_code(dtype)
    d = _lib.ResidualNormDesc()
    d.x, d.rows, d.cols, d.n, d.eps = x.data_ptr(), rows, cols, int(n) or cols, float(eps)
    if y is not None:
        assert y.shape == x.shape and y.stride(1) == 1 and y.dtype == dtype and y.is_cuda
        d.y, d.y_stride = y.data_ptr(), y.stride(0)
    if experts is not None:
        e, ew = experts
        _require_f32(ew=ew)
        assert ew.shape[0] == rows and e.shape == (ew.numel(), cols) and e.is_contiguous() and e.dtype == dtype and e.is_cuda
        d.e, d.ew, d.top = e.data_ptr(), ew.data_ptr(), ew.shape[1]
    d.mult = float(mult)
    if post is not None:
        _require_f32(post_weight=post[0], post_bias=post[1])
        assert post[0].numel() == cols and post[1].numel() == cols
        d.post_w, d.post_b = post[0].data_ptr(), post[1].data_ptr()
    if base is not None:
        _require_f32(base=base)
        assert base.shape == x.shape
        d.base = base.data_ptr()
    if shift is not None:
        _require_f32(shift=shift)
        assert shift.numel() == cols
        d.shift = shift.data_ptr()
    out = None
    if weight is not None:
        _require_f32(weight=weight, bias=bias)
        assert weight.numel() == cols and bias.numel() == cols
        d.w, d.b = weight.data_ptr(), bias.data_ptr()
        if want_rows:
            out = torch.empty((rows, cols), dtype=dtype, device=x.device)
            d.xb = out.data_ptr()
        if packed is not None:
            _packed_ok(packed, rows, cols)
            d.packed = packed.data_ptr()
    _lib.check(_lib.load().nvh_residual_norm(ctypes.byref(d), code, _stream()), "nvh_residual_norm")
    return out


def poly_norm(z, coef, eps, n, packed=None):
    """coef[0] N(z) + coef[1] N(z^2) + coef[2] N(z^3) + coef[3] with N(v) = v / sqrt(mean over n columns of v^2 + eps), zero past n; packed (bf16): in fragment
    order into this buffer, returns None."""
    code = _act_code(z)
    _require_f32(coef=coef)
    rows, cols = z.shape
    assert z.stride(1) == 1 and coef.numel() == 4
    out = None
    if packed is None:
        out = torch.empty((rows, cols), dtype=z.dtype, device=z.device)
    else:
        _packed_ok(packed, rows, cols)
    _lib.check(_lib.load().nvh_poly_norm(_ptr(out), _ptr(packed), z.data_ptr(), coef.data_ptr(), float(eps), rows, cols, int(n), z.stride(0), cols, code, _stream()), "nvh_poly_norm")
    return out


def softcap_(x, cap):
    """cap * tanh(x / cap) in place (rows with any stride)."""
    code = _act_code(x)
    assert x.dim() == 2 and x.stride(1) == 1
    for rows in x.split(65535):
        _lib.check(_lib.load().nvh_softcap(rows.data_ptr(), float(cap), rows.shape[0], rows.shape[1], rows.stride(0), code, _stream()), "nvh_softcap")
    return x
