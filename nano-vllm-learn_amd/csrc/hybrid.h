// Shared pieces of the gated-linear-recurrence / latent-attention kernels: activation-type helpers (bf16 or true fp32 rows) and the
// launcher interface between api_hybrid.hip and the kernel files.
#pragma once
#include "../../include/nvh_attn.h"
#include "common.h"
#include "kernels.h"

namespace nvh {

// an activation is either bf16 (stored as uint16_t) or float
__device__ __forceinline__ float act_ld(const uint16_t* p) { return __uint_as_float((uint32_t)*p << 16); }
__device__ __forceinline__ float act_ld(const float* p) { return *p; }
__device__ __forceinline__ void act_st(uint16_t* p, float v) { *p = (uint16_t)pack_bf16x2(v, 0.f); }
__device__ __forceinline__ void act_st(float* p, float v) { *p = v; }
__device__ __forceinline__ f32x4 act_ld4(const uint16_t* p) {
    const u32x2 r = *reinterpret_cast<const u32x2*>(p);
    return f32x4{bf16_lo(r[0]), bf16_hi(r[0]), bf16_lo(r[1]), bf16_hi(r[1])};
}
__device__ __forceinline__ f32x4 act_ld4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ void act_st4(uint16_t* p, f32x4 v) { *reinterpret_cast<u32x2*>(p) = u32x2{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])}; }
__device__ __forceinline__ void act_st4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
// the value an activation has after it was stored once
__device__ __forceinline__ float act_round(float v, const uint16_t*) { return (float)(__bf16)v; }
__device__ __forceinline__ float act_round(float v, const float*) { return v; }

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + __expf(-x)); }

// sum over a 256-thread workgroup; `lds` holds at least 4 floats and is free again after the next barrier
__device__ __forceinline__ float block_sum256(float v, float* lds) {
    v = group_sum<16>(v);
    v = sum_xor16(v);
    v = sum_xor32(v);
    if ((threadIdx.x & 63) == 0) lds[threadIdx.x >> 6] = v;
    __syncthreads();
    return lds[0] + lds[1] + lds[2] + lds[3];
}

// ---- row-wise ops (hybrid_ops.hip)
int launch_embed_rows(float* x, void* xb, void* packed, const int64_t* tokens, const void* embed, float scale, int rows, int cols, int vocab, float* copy,
                      const int64_t* positions, const float* table, int max_position, int f32, hipStream_t stream);
using NormResidualArgs = nvh_norm_residual_desc;
int launch_norm_residual(const NormResidualArgs& a, int f32, hipStream_t stream);
int launch_clamped_glu(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, float limit, float alpha, int f32, hipStream_t stream);
int launch_gelu_glu(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, int f32, hipStream_t stream);

// ---- gated linear recurrence (rglru.hip)
constexpr int kRglruChunk = 64;  // tokens a workgroup scans at a time
using RglruArgs = nvh_rglru_desc;
int launch_rglru_chunks(const RglruArgs& a, int f32, int generic, hipStream_t stream);
int launch_rglru_step(const RglruArgs& a, int rows, hipStream_t stream);
bool rglru_step_supported(int block);

// ---- latent attention (latent_attention.hip, latent_prefill.hip)
using LatentPrepArgs = nvh_latent_prep_desc;
int launch_latent_prep(const LatentPrepArgs& a, int f32, hipStream_t stream);

using LatentAttnArgs = nvh_latent_attn_desc;
int launch_latent_absorb(const LatentAttnArgs& a, int f32, hipStream_t stream);
int launch_latent_attend(const LatentAttnArgs& a, int f32, int generic, hipStream_t stream);
int launch_latent_value(const LatentAttnArgs& a, int f32, hipStream_t stream);
bool latent_mfma_supported(int kv_cols, int rot_cols, int block_size);

int launch_latent_gather(void* out, const void* cache, const int32_t* cu_k, const int32_t* block_tables, int64_t bt_stride, int batch, int total, int cols,
                         int block_size, int f32, hipStream_t stream);
using LatentPrefillArgs = nvh_latent_prefill_desc;
int launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t stream);
bool latent_prefill_supported(int dk, int dv);

}  // namespace nvh
