// Launcher interface of the paged sink/window attention, lightning attention and mixture-of-experts kernels (the api_*.hip files validate), and the pieces
// their kernels share.
#pragma once
#include "hybrid.h"

namespace nvh {

using AttnPrepArgs = nvh_attn_prep_desc;
using PagedAttendArgs = nvh_paged_attend_desc;
using LightningArgs = nvh_lightning_desc;
using MoeRouteArgs = nvh_moe_route_desc;
using MoeGemmArgs = nvh_moe_gemm_desc;
using ResidualNormArgs = nvh_residual_norm_desc;

constexpr int kRowPieces = 16;                       // 8-element pieces a thread of a row kernel holds at most: rows of up to 256 * 16 * 8 elements
constexpr int kMaxRowCols = 256 * kRowPieces * 8;
constexpr int kAttendTicketWords = 32;               // one arrival ticket per 128-byte line
constexpr int kRowsHeads = 8;                        // query heads of one key/value head a pass over single rows holds at most
constexpr int kLightningChunk = 64;                  // tokens a workgroup takes at a time
constexpr int kMoeMaxExperts = 1024;

int launch_attn_prep(const AttnPrepArgs& a, int f32, hipStream_t stream);
bool paged_attend_supported(int dk, int dv, int block_size);
inline int paged_attend_groups(int heads, int kv_heads) { return (heads / kv_heads + kRowsHeads - 1) / kRowsHeads; }      // passes per key/value head
int launch_paged_attend_rows(const PagedAttendArgs& a, int f32, int generic, hipStream_t stream);
int launch_paged_attend_prompt(const PagedAttendArgs& a, hipStream_t stream);

__host__ __device__ constexpr int score_cols(int heads) { return (heads + 3) / 4 * 4; }          // row length of PagedAttendArgs::scores
bool talk_rows_supported(int heads, int dk, int dv, int block_size);
int launch_talk_rows(const PagedAttendArgs& a, int f32, int generic, hipStream_t stream);
bool talk_prompt_supported(int heads, int kv_heads, int dk, int dv, int block_size);
constexpr float kTalkPromptCap = 1e4f;               // it takes capped scores only
int launch_talk_prompt(const PagedAttendArgs& a, hipStream_t stream);

bool lightning_supported(int dk, int dv);
int launch_lightning_chunks(const LightningArgs& a, int f32, int generic, hipStream_t stream);
int launch_lightning_step(const LightningArgs& a, hipStream_t stream);
int launch_norm_gate(void* out, void* packed, const void* x, const void* gate, const float* w, float eps, int rows, int cols, int n, int64_t x_stride,
                     int64_t gate_stride, int64_t out_stride, int f32, hipStream_t stream);

int launch_moe_route(const MoeRouteArgs& a, int f32, hipStream_t stream);
int moe_dispatch_blocks(int pairs);
int launch_moe_dispatch(int32_t* slot_pair, int32_t* tiles, int32_t* counts, const int32_t* ids, int pairs, int experts, int tile_rows, int max_tiles,
                        hipStream_t stream);
int moe_tile_rows(int pairs, int experts, int f32);
int launch_moe_gemm(const MoeGemmArgs& a, int f32, hipStream_t stream);

int launch_residual_norm(const ResidualNormArgs& a, int f32, hipStream_t stream);
int launch_poly_norm(void* out, void* packed, const void* z, const float* coef, float eps, int rows, int cols, int n, int64_t z_stride, int64_t out_stride, int f32,
                     hipStream_t stream);
int launch_softcap(void* x, float cap, int rows, int cols, int64_t stride, int f32, hipStream_t stream);

// ---- 8 elements of an activation row
struct f32x8 {
    f32x4 a, b;
};
__device__ __forceinline__ f32x8 unpack8(u32x4 r) {
    return {f32x4{bf16_lo(r[0]), bf16_hi(r[0]), bf16_lo(r[1]), bf16_hi(r[1])}, f32x4{bf16_lo(r[2]), bf16_hi(r[2]), bf16_lo(r[3]), bf16_hi(r[3])}};
}
__device__ __forceinline__ f32x8 act_ld8(const uint16_t* p) { return unpack8(*reinterpret_cast<const u32x4*>(p)); }
__device__ __forceinline__ f32x8 act_ld8(const float* p) { return {*reinterpret_cast<const f32x4*>(p), *reinterpret_cast<const f32x4*>(p + 4)}; }
__device__ __forceinline__ void act_st8(uint16_t* p, const f32x8& v) {
    *reinterpret_cast<u32x4*>(p) = u32x4{pack_bf16x2(v.a[0], v.a[1]), pack_bf16x2(v.a[2], v.a[3]), pack_bf16x2(v.b[0], v.b[1]), pack_bf16x2(v.b[2], v.b[3])};
}
__device__ __forceinline__ void act_st8(float* p, const f32x8& v) {
    *reinterpret_cast<f32x4*>(p) = v.a;
    *reinterpret_cast<f32x4*>(p + 4) = v.b;
}
__device__ __forceinline__ float sum4(f32x4 v) { return (v[0] + v[1]) + (v[2] + v[3]); }

__device__ __forceinline__ float wave_sum64(float v) {
    v = group_sum<16>(v);
    v = sum_xor16(v);
    return sum_xor32(v);
}
// sums of two values over a 256-thread workgroup; `lds` holds 8 floats and is free again after the next barrier
__device__ __forceinline__ void block_sum256x2(float& u, float& v, float* lds) {
    u = wave_sum64(u);
    v = wave_sum64(v);
    if ((threadIdx.x & 63) == 0) {
        lds[threadIdx.x >> 6] = u;
        lds[4 + (threadIdx.x >> 6)] = v;
    }
    __syncthreads();
    u = lds[0] + lds[1] + lds[2] + lds[3];
    v = lds[4] + lds[5] + lds[6] + lds[7];
}

// sums of N values over a 256-thread workgroup; `lds` holds 4 * N floats and is free again after the next barrier
template <int N>
__device__ __forceinline__ void block_sums256(float (&v)[N], float* lds) {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = wave_sum64(v[i]);
    if ((threadIdx.x & 63) == 0) {
#pragma unroll
        for (int i = 0; i < N; ++i) lds[4 * i + (threadIdx.x >> 6)] = v[i];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = lds[4 * i] + lds[4 * i + 1] + lds[4 * i + 2] + lds[4 * i + 3];
}

__device__ __forceinline__ void wave_lds_sync() {    // LDS written by other lanes of this wave is visible behind it
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
}

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + __expf(-z)); }

// ---- keys a query at position `pos` sees, as 64-key tiles: the tiles of the kept first tokens, then those of the window
struct VisibleTiles {
    int kept, first, count;                          // tiles [0, kept), then [first, first + count - kept)
    __device__ __forceinline__ int tile(int i) const { return i < kept ? i : first + i - kept; }
};
// the first key, kept ones aside, that a query at `pos` sees through a window (the last `window` tokens; 0: all) or in its chunk (chunk > 0)
__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
    if (chunk > 0) return pos - pos % chunk;
    return window > 0 && pos >= window ? pos - window + 1 : 0;
}
// lo: first_seen of the first query that walks along, last_pos: position of the last one
__device__ __forceinline__ VisibleTiles visible_from(int lo, int last_pos, int keep_first) {
    VisibleTiles v;
    v.first = lo >> 6;
    const int k = (keep_first + 63) >> 6;
    v.kept = k < v.first ? k : v.first;
    v.count = v.kept + ((last_pos + 64) >> 6) - v.first;
    return v;
}
// first_pos .. last_pos: positions of the queries that walk together
__device__ __forceinline__ VisibleTiles visible_tiles(int first_pos, int last_pos, int window, int keep_first) {
    return visible_from(first_seen(first_pos, window, 0), last_pos, keep_first);
}

// 4 columns of a head's output at `pos`, from dimension d on (a multiple of 4), turned back: interleaved pairs of the first `rot` dimensions, table rows cos | sin
__device__ __forceinline__ f32x4 turn_back(f32x4 v, const float* table, int64_t pos, int max_position, int rot, int d) {
    if (d >= rot) return v;
    const float* cs = table + (pos < max_position ? pos : max_position - 1) * rot;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
        if (d + 2 * p >= rot) continue;
        const float c = cs[d / 2 + p], s = cs[rot / 2 + d / 2 + p], x = v[2 * p], y = v[2 * p + 1];
        v[2 * p] = x * c + y * s;
        v[2 * p + 1] = y * c - x * s;
    }
    return v;
}

}  // namespace nvh
