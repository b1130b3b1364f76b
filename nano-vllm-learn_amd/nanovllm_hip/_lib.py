"""ctypes binding of libnvh_attn.so (C ABI: include/nvh_attn.h).

The library is the product; there is no CPU or PyTorch fallback.  If it is missing or fails to
load, every op raises — loudly — instead of computing something else.
"""
import ctypes
import os

import torch  # noqa: F401  (imported first on purpose: libnvh_attn.so binds to the HIP runtime torch loaded)

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.environ.get("NVH_LIB_PATH") or os.path.join(_HERE, "lib", "libnvh_attn.so")   # override: A/B of two builds
_subset = None                                                                             # architecture whose kernels alone may be built (build.py --model)

NVH_BF16 = 0
NVH_F32 = 1
IPC_HANDLE_BYTES = 64                                                         # NVH_COMM_IPC_HANDLE_BYTES
AR_EPI_NONE, AR_EPI_RESIDUAL_ADD = 0, 1

class LinearDesc(ctypes.Structure):
    """nvh_linear_desc (include/nvh_attn.h)."""
    _fields_ = [("out", ctypes.c_void_p), ("x", ctypes.c_void_p), ("w", ctypes.c_void_p), ("bias", ctypes.c_void_p),
                ("m", ctypes.c_int32), ("n", ctypes.c_int32), ("k", ctypes.c_int32), ("silu_inter", ctypes.c_int32),
                ("x_row_stride", ctypes.c_int64), ("out_row_stride", ctypes.c_int64),
                ("norm_weight", ctypes.c_void_p), ("norm_eps", ctypes.c_float), ("epilogue", ctypes.c_int32),
                ("positions", ctypes.c_void_p), ("cos_sin", ctypes.c_void_p), ("k_cache", ctypes.c_void_p), ("v_cache", ctypes.c_void_p),
                ("slot_mapping", ctypes.c_void_p), ("h", ctypes.c_int32), ("kvh", ctypes.c_int32), ("hd", ctypes.c_int32),
                ("norm_folded", ctypes.c_int32), ("x_packed", ctypes.c_int32), ("out_packed", ctypes.c_void_p),
                ("workspace", ctypes.c_void_p), ("workspace_bytes", ctypes.c_size_t),
                ("candidate_val", ctypes.c_void_p), ("candidate_idx", ctypes.c_void_p), ("candidate_stride", ctypes.c_int64),
                ("prefetch", ctypes.c_void_p), ("prefetch_bytes", ctypes.c_size_t),
                ("glu_limit", ctypes.c_float), ("glu_alpha", ctypes.c_float), ("glu_gelu", ctypes.c_int32),
                ("x_groups", ctypes.c_int32), ("x_group_rows", ctypes.c_int32), ("x_group_stride", ctypes.c_int32)]


class NormResidualDesc(ctypes.Structure):
    """nvh_norm_residual_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("xb", ctypes.c_void_p), ("packed", ctypes.c_void_p), ("y", ctypes.c_void_p),
                ("w", ctypes.c_void_p), ("eps", ctypes.c_float), ("rows", ctypes.c_int32), ("cols", ctypes.c_int32), ("n", ctypes.c_int32),
                ("y_stride", ctypes.c_int64)]


class RglruDesc(ctypes.Structure):
    """nvh_rglru_desc (include/nvh_attn.h)."""
    _fields_ = [("yx", ctypes.c_void_p), ("yx_stride", ctypes.c_int64), ("width", ctypes.c_int32), ("block", ctypes.c_int32),
                ("blocks", ctypes.c_int32), ("taps", ctypes.c_int32), ("conv_w", ctypes.c_void_p), ("conv_b", ctypes.c_void_p),
                ("ra", ctypes.c_void_p), ("ri", ctypes.c_void_p), ("ra_b", ctypes.c_void_p), ("ri_b", ctypes.c_void_p),
                ("rate", ctypes.c_void_p), ("chunks", ctypes.c_void_p), ("n_chunks", ctypes.c_int32), ("segment", ctypes.c_int32), ("summaries", ctypes.c_int32), ("positions", ctypes.c_void_p),
                ("state_slots", ctypes.c_void_p), ("state", ctypes.c_void_p), ("conv_state", ctypes.c_void_p), ("s_loc", ctypes.c_void_p),
                ("a_cum", ctypes.c_void_p), ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64), ("out_packed", ctypes.c_void_p)]


class LatentPrepDesc(ctypes.Structure):
    """nvh_latent_prep_desc (include/nvh_attn.h)."""
    _fields_ = [("a", ctypes.c_void_p), ("a_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("q_rank", ctypes.c_int32),
                ("q_cols", ctypes.c_int32), ("kv_rank", ctypes.c_int32), ("kv_cols", ctypes.c_int32), ("rot", ctypes.c_int32),
                ("rot_cols", ctypes.c_int32), ("q_w", ctypes.c_void_p), ("kv_w", ctypes.c_void_p), ("eps", ctypes.c_float),
                ("cq", ctypes.c_void_p), ("cq_packed", ctypes.c_void_p), ("cache", ctypes.c_void_p), ("slots", ctypes.c_void_p),
                ("positions", ctypes.c_void_p), ("cos_sin", ctypes.c_void_p), ("max_position", ctypes.c_int32)]


class LatentAttnDesc(ctypes.Structure):
    """nvh_latent_attn_desc (include/nvh_attn.h)."""
    _fields_ = [("q", ctypes.c_void_p), ("q_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("heads", ctypes.c_int32),
                ("dim_cols", ctypes.c_int32), ("qrot_cols", ctypes.c_int32), ("cache", ctypes.c_void_p), ("kv_cols", ctypes.c_int32),
                ("rot", ctypes.c_int32), ("rot_cols", ctypes.c_int32), ("block_size", ctypes.c_int32), ("block_tables", ctypes.c_void_p),
                ("bt_stride", ctypes.c_int64), ("max_blocks", ctypes.c_int32), ("row_seq", ctypes.c_void_p), ("positions", ctypes.c_void_p),
                ("cos_sin", ctypes.c_void_p), ("max_position", ctypes.c_int32), ("w_uk", ctypes.c_void_p), ("w_uv", ctypes.c_void_p),
                ("v_cols", ctypes.c_int32), ("scale", ctypes.c_float), ("qa", ctypes.c_void_p), ("part_o", ctypes.c_void_p),
                ("part_ml", ctypes.c_void_p), ("splits", ctypes.c_int32), ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64),
                ("out_packed", ctypes.c_void_p)]


class LatentPrefillDesc(ctypes.Structure):
    """nvh_latent_prefill_desc (include/nvh_attn.h)."""
    _fields_ = [("q", ctypes.c_void_p), ("k", ctypes.c_void_p), ("k_rot", ctypes.c_void_p), ("v", ctypes.c_void_p),
                ("out", ctypes.c_void_p), ("q_stride", ctypes.c_int64), ("k_stride", ctypes.c_int64), ("kr_stride", ctypes.c_int64),
                ("v_stride", ctypes.c_int64), ("out_stride", ctypes.c_int64), ("cu_q", ctypes.c_void_p), ("cu_k", ctypes.c_void_p),
                ("positions", ctypes.c_void_p), ("cos_sin", ctypes.c_void_p), ("max_position", ctypes.c_int32), ("rot", ctypes.c_int32),
                ("batch", ctypes.c_int32), ("heads", ctypes.c_int32), ("dim_cols", ctypes.c_int32), ("dk", ctypes.c_int32),
                ("dv", ctypes.c_int32), ("max_q", ctypes.c_int32), ("scale_log2", ctypes.c_float)]


class AttnPrepDesc(ctypes.Structure):
    """nvh_attn_prep_desc (include/nvh_attn.h)."""
    _fields_ = [("qkv", ctypes.c_void_p), ("qkv_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("heads", ctypes.c_int32),
                ("kv_heads", ctypes.c_int32), ("dk", ctypes.c_int32), ("dv", ctypes.c_int32), ("q_w", ctypes.c_void_p),
                ("k_w", ctypes.c_void_p), ("q_n", ctypes.c_int32), ("k_n", ctypes.c_int32), ("eps", ctypes.c_float),
                ("positions", ctypes.c_void_p), ("cos_sin", ctypes.c_void_p), ("max_position", ctypes.c_int32), ("rot", ctypes.c_int32),
                ("cache", ctypes.c_void_p), ("slots", ctypes.c_void_p), ("block_size", ctypes.c_int32), ("head_norm", ctypes.c_int32),
                ("v_cos_sin", ctypes.c_void_p), ("v_rot", ctypes.c_int32)]


class PagedAttendDesc(ctypes.Structure):
    """nvh_paged_attend_desc (include/nvh_attn.h)."""
    _fields_ = [("q", ctypes.c_void_p), ("q_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("heads", ctypes.c_int32),
                ("kv_heads", ctypes.c_int32), ("dk", ctypes.c_int32), ("dv", ctypes.c_int32), ("cache", ctypes.c_void_p),
                ("block_size", ctypes.c_int32), ("block_tables", ctypes.c_void_p), ("bt_stride", ctypes.c_int64),
                ("row_seq", ctypes.c_void_p), ("positions", ctypes.c_void_p), ("cu_q", ctypes.c_void_p), ("cu_k", ctypes.c_void_p),
                ("batch", ctypes.c_int32), ("max_q", ctypes.c_int32), ("scale", ctypes.c_float), ("window", ctypes.c_int32),
                ("keep_first", ctypes.c_int32), ("sink", ctypes.c_void_p), ("splits", ctypes.c_int32), ("part", ctypes.c_void_p),
                ("tickets", ctypes.c_void_p), ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64),
                ("out_packed", ctypes.c_void_p), ("talk", ctypes.c_void_p), ("softcap", ctypes.c_float), ("scores", ctypes.c_void_p),
                ("span", ctypes.c_int32), ("chunk", ctypes.c_int32), ("o_cos_sin", ctypes.c_void_p), ("max_position", ctypes.c_int32), ("o_rot", ctypes.c_int32)]


class LightningDesc(ctypes.Structure):
    """nvh_lightning_desc (include/nvh_attn.h)."""
    _fields_ = [("qkv", ctypes.c_void_p), ("qkv_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("heads", ctypes.c_int32),
                ("dk", ctypes.c_int32), ("dv", ctypes.c_int32), ("decay", ctypes.c_void_p), ("positions", ctypes.c_void_p),
                ("state_slots", ctypes.c_void_p), ("state", ctypes.c_void_p), ("chunks", ctypes.c_void_p), ("n_chunks", ctypes.c_int32),
                ("summaries", ctypes.c_int32), ("seg_state", ctypes.c_void_p), ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64)]


class MoeRouteDesc(ctypes.Structure):
    """nvh_moe_route_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("x_stride", ctypes.c_int64), ("router", ctypes.c_void_p), ("correction", ctypes.c_void_p),
                ("rows", ctypes.c_int32), ("cols", ctypes.c_int32), ("experts", ctypes.c_int32), ("top", ctypes.c_int32),
                ("groups", ctypes.c_int32), ("keep", ctypes.c_int32), ("scale", ctypes.c_float), ("ids", ctypes.c_void_p),
                ("weights", ctypes.c_void_p), ("softmax", ctypes.c_int32)]


class MoeGemmDesc(ctypes.Structure):
    """nvh_moe_gemm_desc (include/nvh_attn.h)."""
    _fields_ = [("out", ctypes.c_void_p), ("x", ctypes.c_void_p), ("x_stride", ctypes.c_int64), ("w", ctypes.c_void_p),
                ("pairs", ctypes.c_int32), ("top", ctypes.c_int32), ("experts", ctypes.c_int32), ("n", ctypes.c_int32),
                ("k", ctypes.c_int32), ("glu", ctypes.c_int32), ("ids", ctypes.c_void_p), ("slot_pair", ctypes.c_void_p),
                ("tiles", ctypes.c_void_p), ("max_tiles", ctypes.c_int32), ("tile_rows", ctypes.c_int32),
                ("limit", ctypes.c_float), ("alpha", ctypes.c_float)]


class ResidualNormDesc(ctypes.Structure):
    """nvh_residual_norm_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("y", ctypes.c_void_p), ("y_stride", ctypes.c_int64), ("e", ctypes.c_void_p),
                ("ew", ctypes.c_void_p), ("top", ctypes.c_int32), ("w", ctypes.c_void_p), ("b", ctypes.c_void_p), ("eps", ctypes.c_float),
                ("rows", ctypes.c_int32), ("cols", ctypes.c_int32), ("n", ctypes.c_int32), ("xb", ctypes.c_void_p),
                ("packed", ctypes.c_void_p), ("post_w", ctypes.c_void_p), ("post_b", ctypes.c_void_p), ("mult", ctypes.c_float),
                ("base", ctypes.c_void_p), ("shift", ctypes.c_void_p)]


class BigramEmbedDesc(ctypes.Structure):
    """nvh_bigram_embed_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("tokens", ctypes.c_void_p), ("positions", ctypes.c_void_p), ("row_seq", ctypes.c_void_p),
                ("cu_rows", ctypes.c_void_p), ("state_slots", ctypes.c_void_p), ("last_token", ctypes.c_void_p),
                ("embed", ctypes.c_void_p), ("bigram", ctypes.c_void_p), ("buckets", ctypes.c_int64), ("mul_prev", ctypes.c_int64),
                ("mul_cur", ctypes.c_int64), ("rows", ctypes.c_int32), ("cols", ctypes.c_int32), ("vocab", ctypes.c_int32)]


class StreamMixDesc(ctypes.Structure):
    """nvh_stream_mix_desc (include/nvh_attn.h)."""
    _fields_ = [("xin", ctypes.c_void_p), ("xin_row", ctypes.c_int64), ("xin_stream", ctypes.c_int64), ("xout", ctypes.c_void_p),
                ("rows", ctypes.c_int32), ("cols", ctypes.c_int32), ("n", ctypes.c_int32), ("streams", ctypes.c_int32),
                ("y", ctypes.c_void_p), ("y_stride", ctypes.c_int64), ("y2", ctypes.c_void_p), ("y2_stride", ctypes.c_int64),
                ("y_w", ctypes.c_void_p), ("y2_w", ctypes.c_void_p), ("y_scale", ctypes.c_float), ("mix", ctypes.c_void_p),
                ("out", ctypes.c_void_p), ("in", ctypes.c_void_p), ("sum", ctypes.c_void_p), ("w", ctypes.c_void_p),
                ("groups", ctypes.c_int32), ("eps", ctypes.c_float), ("h", ctypes.c_void_p), ("packed", ctypes.c_void_p), ("shift", ctypes.c_void_p),
                ("mu", ctypes.c_void_p), ("mixes", ctypes.c_int32), ("depth", ctypes.c_int32), ("ring", ctypes.c_void_p),
                ("shifted", ctypes.c_void_p), ("shifted_mix", ctypes.c_int64), ("positions", ctypes.c_void_p), ("state_slots", ctypes.c_void_p)]


class TokenShiftDesc(ctypes.Structure):
    """nvh_token_shift_desc (include/nvh_attn.h)."""
    _fields_ = [("h", ctypes.c_void_p), ("h_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("cols", ctypes.c_int32),
                ("shift", ctypes.c_void_p), ("mu", ctypes.c_void_p), ("mixes", ctypes.c_int32), ("out", ctypes.c_void_p),
                ("out_mix", ctypes.c_int64), ("packed", ctypes.c_int32), ("ring", ctypes.c_void_p), ("depth", ctypes.c_int32),
                ("positions", ctypes.c_void_p), ("row_seq", ctypes.c_void_p), ("cu_rows", ctypes.c_void_p),
                ("state_slots", ctypes.c_void_p), ("sequences", ctypes.c_int32)]


class CausalConvDesc(ctypes.Structure):
    """nvh_causal_conv_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("x_stride", ctypes.c_int64), ("rows", ctypes.c_int32), ("cols", ctypes.c_int32),
                ("taps", ctypes.c_int32), ("w", ctypes.c_void_p), ("b", ctypes.c_void_p), ("out", ctypes.c_void_p),
                ("packed", ctypes.c_void_p), ("ring", ctypes.c_void_p), ("positions", ctypes.c_void_p), ("row_seq", ctypes.c_void_p),
                ("cu_rows", ctypes.c_void_p), ("state_slots", ctypes.c_void_p), ("sequences", ctypes.c_int32)]


class ScanDesc(ctypes.Structure):
    """nvh_scan_desc (include/nvh_attn.h)."""
    _fields_ = [("x", ctypes.c_void_p), ("x_stride", ctypes.c_int64), ("dt", ctypes.c_void_p), ("dt_stride", ctypes.c_int64),
                ("dt_bias", ctypes.c_void_p), ("bc", ctypes.c_void_p), ("bc_stride", ctypes.c_int64), ("z", ctypes.c_void_p),
                ("z_stride", ctypes.c_int64), ("a_log2", ctypes.c_void_p), ("d", ctypes.c_void_p), ("rows", ctypes.c_int32),
                ("inner", ctypes.c_int32), ("n", ctypes.c_int32), ("positions", ctypes.c_void_p), ("state_slots", ctypes.c_void_p),
                ("state", ctypes.c_void_p), ("chunks", ctypes.c_void_p), ("n_chunks", ctypes.c_int32), ("summaries", ctypes.c_int32),
                ("seg_state", ctypes.c_void_p), ("seg_dt", ctypes.c_void_p), ("w_dt", ctypes.c_void_p), ("rank", ctypes.c_int32),
                ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64), ("out_packed", ctypes.c_void_p)]


class WkvDesc(ctypes.Structure):
    """nvh_wkv_desc (include/nvh_attn.h)."""
    _fields_ = [("r", ctypes.c_void_p), ("k", ctypes.c_void_p), ("v", ctypes.c_void_p), ("g", ctypes.c_void_p), ("stride", ctypes.c_int64),
                ("z", ctypes.c_void_p), ("z_stride", ctypes.c_int64), ("w0", ctypes.c_void_p), ("u", ctypes.c_void_p),
                ("norm", ctypes.c_void_p), ("eps", ctypes.c_float), ("n", ctypes.c_int32), ("rows", ctypes.c_int32),
                ("heads", ctypes.c_int32), ("dim", ctypes.c_int32), ("w2", ctypes.c_void_p), ("rank", ctypes.c_int32),
                ("positions", ctypes.c_void_p), ("state_slots", ctypes.c_void_p), ("state", ctypes.c_void_p), ("chunks", ctypes.c_void_p),
                ("n_chunks", ctypes.c_int32), ("summaries", ctypes.c_int32), ("seg_state", ctypes.c_void_p),
                ("seg_decay", ctypes.c_void_p), ("out", ctypes.c_void_p), ("out_stride", ctypes.c_int64), ("out_packed", ctypes.c_void_p)]


EPI_NONE, EPI_SILU_MUL, EPI_RESIDUAL_ADD, EPI_ROPE_STORE = 0, 1, 2, 3
PREFILL_KERNELS = {"auto": 0, "tiled": 1, "short": 2, "tiled_f16v": 3}                         # NVH_PREFILL_* (nvh_prefill_varlen_variant)
DECODE_VARIANTS = {"chunked": 0, "split_mfma": 1, "split_valu": 2, "chunked_p128": 3, "chunked_p256": 4, "chunked_p64": 5}      # NVH_DECODE_* (nvh_paged_decode_variant)

_c_i32p = ctypes.c_void_p
_SIGS = {
    "nvh_version": (ctypes.c_int, []),
    "nvh_last_error": (ctypes.c_char_p, []),
    "nvh_store_kvcache": (ctypes.c_int, [ctypes.c_void_p] * 4 + [_c_i32p, ctypes.c_int, ctypes.c_int, ctypes.c_int,
                                          ctypes.c_int64, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_paged_decode_workspace": (ctypes.c_size_t, [ctypes.c_int] * 5),
    "nvh_paged_decode": (ctypes.c_int, [ctypes.c_void_p] * 4 + [_c_i32p, _c_i32p] + [ctypes.c_int] * 6 +
                         [ctypes.c_int64, ctypes.c_int64, ctypes.c_float, ctypes.c_int, ctypes.c_int,
                          ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_paged_decode_variant": (ctypes.c_int, [ctypes.c_int] * 3 + [ctypes.c_void_p] * 4 + [_c_i32p, _c_i32p] + [ctypes.c_int] * 6 +
                                 [ctypes.c_int64, ctypes.c_int64, ctypes.c_float, ctypes.c_int, ctypes.c_int,
                                  ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_paged_decode_packed": (ctypes.c_int, [ctypes.c_void_p] * 5 + [_c_i32p, _c_i32p] + [ctypes.c_int] * 6 +
                                [ctypes.c_int64, ctypes.c_int64, ctypes.c_float, ctypes.c_int, ctypes.c_int,
                                 ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_decode_step": (ctypes.c_int, [ctypes.c_void_p] * 6 + [_c_i32p] * 3 + [ctypes.c_int] * 6 +
                        [ctypes.c_int64] * 4 + [ctypes.c_float, ctypes.c_int, ctypes.c_int,
                                                ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_prefill_varlen": (ctypes.c_int, [ctypes.c_void_p] * 4 + [_c_i32p] * 3 + [ctypes.c_int] * 8 +
                           [ctypes.c_int64] * 4 + [ctypes.c_float, ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_prefill_varlen_variant": (ctypes.c_int, [ctypes.c_int] * 2 + [ctypes.c_void_p] * 4 + [_c_i32p] * 3 + [ctypes.c_int] * 8 +
                                   [ctypes.c_int64] * 4 + [ctypes.c_float, ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_prefill_pv16_scratch_bytes": (ctypes.c_size_t, [ctypes.c_int] * 3),
    "nvh_prefill_pv16_uses_scratch": (ctypes.c_int, [ctypes.c_int] * 5),
    "nvh_prefill_varlen_pv16": (ctypes.c_int, [ctypes.c_void_p] * 4 + [_c_i32p] * 2 + [ctypes.c_int] * 7 + [ctypes.c_int64] * 3 +
                                [ctypes.c_float, ctypes.c_int, ctypes.c_int, ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_bf16_rows_to_f16": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_int64, ctypes.c_int64, ctypes.c_void_p]),
    "nvh_rope_store": (ctypes.c_int, [ctypes.c_void_p] * 5 + [ctypes.c_float] + [ctypes.c_void_p] * 3 + [ctypes.c_int] * 4 +
                       [ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_add_rmsnorm": (ctypes.c_int, [ctypes.c_void_p] * 4 + [ctypes.c_float, ctypes.c_int, ctypes.c_int] + [ctypes.c_int64] * 3 +
                        [ctypes.c_int, ctypes.c_void_p]),
    "nvh_residual_add_pack": (ctypes.c_int, [ctypes.c_void_p] * 3 + [ctypes.c_int, ctypes.c_int, ctypes.c_int64, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_silu_mul": (ctypes.c_int, [ctypes.c_void_p] * 2 + [ctypes.c_int, ctypes.c_int, ctypes.c_int64, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_linear_small_m": (ctypes.c_int, [ctypes.c_void_p] * 4 + [ctypes.c_int] * 4 + [ctypes.c_int64, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_argmax_rows": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_greedy_advance": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_int64] + [ctypes.c_void_p] * 5 +
                           [ctypes.c_int64, ctypes.c_int, ctypes.c_void_p, ctypes.c_int64, ctypes.c_void_p, ctypes.c_int, ctypes.c_void_p]),
    "nvh_linear_small_m_ex": (ctypes.c_int, [ctypes.POINTER(LinearDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_linear_small_m_workspace": (ctypes.c_size_t, [ctypes.c_int] * 4),
    "nvh_qkv_rope_attend": (ctypes.c_int, [ctypes.POINTER(LinearDesc), ctypes.c_void_p, ctypes.c_void_p, _c_i32p, _c_i32p, ctypes.c_int, ctypes.c_int,
                                           ctypes.c_int64, ctypes.c_float, ctypes.c_int, ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_qkv_rope_attend_variant": (ctypes.c_int, [ctypes.c_int, ctypes.c_uint32, ctypes.c_int, ctypes.POINTER(ctypes.c_int), ctypes.POINTER(LinearDesc),
                                                   ctypes.c_void_p, ctypes.c_void_p, _c_i32p, _c_i32p, ctypes.c_int, ctypes.c_int, ctypes.c_int64,
                                                   ctypes.c_float, ctypes.c_int, ctypes.c_void_p, ctypes.c_size_t, ctypes.c_void_p]),
    "nvh_qkv_rope_attend_status": (ctypes.c_int, [ctypes.c_void_p, ctypes.POINTER(ctypes.c_uint32)]),
    "nvh_pack_index": (ctypes.c_int64, [ctypes.c_int] * 3),
    "nvh_linear_small_m_candidate_groups": (ctypes.c_int, [ctypes.c_int] * 2),
    "nvh_comm_alloc": (ctypes.c_int, [ctypes.POINTER(ctypes.c_void_p), ctypes.c_size_t]),
    "nvh_comm_free": (ctypes.c_int, [ctypes.c_void_p]),
    "nvh_comm_ipc_export": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_void_p]),
    "nvh_comm_ipc_open": (ctypes.c_int, [ctypes.c_void_p, ctypes.POINTER(ctypes.c_void_p)]),
    "nvh_comm_ipc_close": (ctypes.c_int, [ctypes.c_void_p]),
    "nvh_allreduce_stage_bytes": (ctypes.c_size_t, [ctypes.c_int, ctypes.c_int]),
    "nvh_allreduce_flag_bytes": (ctypes.c_size_t, [ctypes.c_int]),
    "nvh_allreduce_status": (ctypes.c_int, [ctypes.c_void_p, ctypes.POINTER(ctypes.c_uint32), ctypes.POINTER(ctypes.c_uint32)]),
    "nvh_allreduce_oneshot": (ctypes.c_int, [ctypes.c_void_p] * 6 + [ctypes.c_int] * 4 + [ctypes.c_int64, ctypes.c_int64, ctypes.c_size_t,
                                                                        ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_greedy_advance_candidates": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_int] +
                                      [ctypes.c_void_p] * 5 + [ctypes.c_int64, ctypes.c_int, ctypes.c_void_p, ctypes.c_int64,
                                                                ctypes.c_void_p, ctypes.c_void_p]),
    "nvh_greedy_advance_candidates_embed": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_int] +
                                            [ctypes.c_void_p] * 5 + [ctypes.c_int64, ctypes.c_int, ctypes.c_void_p, ctypes.c_int64,
                                                                      ctypes.c_void_p] +
                                            [ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_void_p, ctypes.c_int64, ctypes.c_void_p, ctypes.c_int,
                                             ctypes.c_void_p]),
    "nvh_embed_rows": (ctypes.c_int, [ctypes.c_void_p] * 5 + [ctypes.c_float] + [ctypes.c_int] * 3 + [ctypes.c_void_p] * 3 + [ctypes.c_int] * 2 + [ctypes.c_void_p]),
    "nvh_norm_residual": (ctypes.c_int, [ctypes.POINTER(NormResidualDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_clamped_glu": (ctypes.c_int, [ctypes.c_void_p] * 2 + [ctypes.c_int] * 2 + [ctypes.c_int64] * 2 + [ctypes.c_float] * 2 + [ctypes.c_int, ctypes.c_void_p]),
    "nvh_gelu_glu": (ctypes.c_int, [ctypes.c_void_p] * 2 + [ctypes.c_int] * 2 + [ctypes.c_int64] * 2 + [ctypes.c_int, ctypes.c_void_p]),
    "nvh_rglru_chunk_tokens": (ctypes.c_int, []),
    "nvh_rglru_step_supported": (ctypes.c_int, [ctypes.c_int]),
    "nvh_rglru_chunks": (ctypes.c_int, [ctypes.POINTER(RglruDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_rglru_step": (ctypes.c_int, [ctypes.POINTER(RglruDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_latent_prep": (ctypes.c_int, [ctypes.POINTER(LatentPrepDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_latent_attend_mfma": (ctypes.c_int, [ctypes.c_int] * 3),
    "nvh_latent_attention": (ctypes.c_int, [ctypes.POINTER(LatentAttnDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_latent_gather": (ctypes.c_int, [ctypes.c_void_p] * 4 + [ctypes.c_int64] + [ctypes.c_int] * 5 + [ctypes.c_void_p]),
    "nvh_latent_prefill_supported": (ctypes.c_int, [ctypes.c_int] * 2),
    "nvh_latent_prefill": (ctypes.c_int, [ctypes.POINTER(LatentPrefillDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_attn_prep": (ctypes.c_int, [ctypes.POINTER(AttnPrepDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_paged_attend_supported": (ctypes.c_int, [ctypes.c_int] * 3),
    "nvh_paged_attend_ticket_bytes": (ctypes.c_size_t, [ctypes.c_int] * 3),
    "nvh_paged_attend_rows": (ctypes.c_int, [ctypes.POINTER(PagedAttendDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_paged_attend_prompt": (ctypes.c_int, [ctypes.POINTER(PagedAttendDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_talk_rows_supported": (ctypes.c_int, [ctypes.c_int] * 4),
    "nvh_talk_score_cols": (ctypes.c_int, [ctypes.c_int]),
    "nvh_talk_ticket_bytes": (ctypes.c_size_t, [ctypes.c_int] * 3),
    "nvh_talk_rows": (ctypes.c_int, [ctypes.POINTER(PagedAttendDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_talk_prompt_supported": (ctypes.c_int, [ctypes.c_int] * 5 + [ctypes.c_float]),
    "nvh_talk_prompt": (ctypes.c_int, [ctypes.POINTER(PagedAttendDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_lightning_supported": (ctypes.c_int, [ctypes.c_int] * 2),
    "nvh_lightning_chunks": (ctypes.c_int, [ctypes.POINTER(LightningDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_lightning_step": (ctypes.c_int, [ctypes.POINTER(LightningDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_norm_gate": (ctypes.c_int, [ctypes.c_void_p] * 5 + [ctypes.c_float] + [ctypes.c_int] * 3 + [ctypes.c_int64] * 3 + [ctypes.c_int, ctypes.c_void_p]),
    "nvh_moe_route": (ctypes.c_int, [ctypes.POINTER(MoeRouteDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_moe_dispatch_blocks": (ctypes.c_int, [ctypes.c_int]),
    "nvh_moe_dispatch": (ctypes.c_int, [ctypes.c_void_p] * 4 + [ctypes.c_int] * 4 + [ctypes.c_void_p]),
    "nvh_moe_tile_rows": (ctypes.c_int, [ctypes.c_int] * 3),
    "nvh_moe_gemm": (ctypes.c_int, [ctypes.POINTER(MoeGemmDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_residual_norm": (ctypes.c_int, [ctypes.POINTER(ResidualNormDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_poly_norm": (ctypes.c_int, [ctypes.c_void_p] * 4 + [ctypes.c_float] + [ctypes.c_int] * 3 + [ctypes.c_int64] * 2 + [ctypes.c_int, ctypes.c_void_p]),
    "nvh_softcap": (ctypes.c_int, [ctypes.c_void_p, ctypes.c_float, ctypes.c_int, ctypes.c_int, ctypes.c_int64, ctypes.c_int, ctypes.c_void_p]),
    "nvh_bigram_embed": (ctypes.c_int, [ctypes.POINTER(BigramEmbedDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_stream_mix": (ctypes.c_int, [ctypes.POINTER(StreamMixDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_token_shift": (ctypes.c_int, [ctypes.POINTER(TokenShiftDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_causal_conv": (ctypes.c_int, [ctypes.POINTER(CausalConvDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_scan_states": (ctypes.c_int, [ctypes.c_int]),
    "nvh_scan_chunks": (ctypes.c_int, [ctypes.POINTER(ScanDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_scan_step": (ctypes.c_int, [ctypes.POINTER(ScanDesc), ctypes.c_int, ctypes.c_void_p]),
    "nvh_wkv_supported": (ctypes.c_int, [ctypes.c_int]),
    "nvh_wkv_chunks": (ctypes.c_int, [ctypes.POINTER(WkvDesc), ctypes.c_int, ctypes.c_int, ctypes.c_void_p]),
    "nvh_wkv_step": (ctypes.c_int, [ctypes.POINTER(WkvDesc), ctypes.c_int, ctypes.c_void_p]),
}
EXPORTS = tuple(_SIGS)

_lib = None


class NvhLibraryError(RuntimeError):
    pass


class _Subset:
    """A library with the kernels of one model: entry points it does not hold raise when they are asked for."""

    def __init__(self, lib, path):
        self._lib, self._path = lib, path

    def __getattr__(self, name):
        try:
            return getattr(self._lib, name)
        except AttributeError as e:
            raise NvhLibraryError(f"{self._path} does not hold {name}: build the whole library with `python nano-vllm-learn_amd/build.py`") from e


def subset_path(architecture):
    return os.path.join(_HERE, "lib", f"libnvh_{architecture.lower()}.so")


def use_subset(architecture):
    """Where the whole library is not built, load the one with this architecture's kernels (before anything is loaded)."""
    global _subset
    _subset = architecture


def load():
    """Load (once) and return the library: libnvh_attn.so, or the subset chosen by use_subset() where only that is built.  Raises
    NvhLibraryError if neither is there."""
    global _lib
    if _lib is not None:
        return _lib
    whole = os.path.exists(LIB_PATH) or "NVH_LIB_PATH" in os.environ or _subset is None
    path = LIB_PATH if whole else subset_path(_subset)
    if not os.path.exists(path):
        raise NvhLibraryError(
            f"{LIB_PATH} not found: build it with `python nano-vllm-learn_amd/build.py` "
            "(the hip attention backend has no fallback path)")
    try:
        lib = ctypes.CDLL(path)
    except OSError as e:
        raise NvhLibraryError(f"cannot load {path}: {e}") from e
    subset = not whole
    for name, (res, args) in _SIGS.items():
        try:
            fn = getattr(lib, name)
        except AttributeError as e:
            if subset:
                continue
            raise NvhLibraryError(f"{path} does not export {name}") from e
        fn.restype = res
        fn.argtypes = args
    _lib = _Subset(lib, path) if subset else lib
    return _lib


def check(rc, what):
    """Turn a non-zero return code into the exception the reference's callers expect."""
    if rc == 0:
        return
    msg = load().nvh_last_error().decode(errors="replace")
    text = f"{what} failed (code {rc}): {msg}"
    if "out of memory" in msg.lower():
        raise torch.cuda.OutOfMemoryError(text)        # bench_my.py:13-17 maps this to "OOM"
    raise RuntimeError(text)
