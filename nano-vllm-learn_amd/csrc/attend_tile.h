// The MFMA tile of the prompt-attention kernels that read keys and values from LDS images of 64 rows (unequal widths DK, DV):
// 4 waves x QT x 16 query rows, S^T = K Q^T and O^T = V^T P^T with the weights as bf16 hi + lo halves, online softmax in the log2 domain.
// A kernel stages the images (16-byte pieces swizzled by swz_k / swz_v), fills the query fragments and says which keys a query sees.
#pragma once
#include <type_traits>

#include "hybrid.h"

namespace nvh {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

template <int OFF>
__device__ __forceinline__ u32x2 ds_read_tr16(uint32_t lds_addr) {
    static_assert(OFF >= 0 && OFF < 65536, "ds offset field is 16 bits");
    u32x2 r;
    asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(r) : "v"(lds_addr), "n"(OFF) : "memory");
    return r;
}
__device__ __forceinline__ uint32_t lds_addr_of(const void* p) { return (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)p; }
__device__ __forceinline__ float max3f(float x, float y, float z) {
    float r;
    asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(x), "v"(y), "v"(z));
    return r;
}
// workgroup barrier behind this wave's LDS traffic only (a __syncthreads() would drain the loads in flight)
__device__ __forceinline__ void lds_only_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
// 16 bytes per lane from global memory to 1024 consecutive LDS bytes
__device__ __forceinline__ void dma16(const void* src, unsigned char* lds_wave_base) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src, (__attribute__((address_space(3))) void*)lds_wave_base, 16, 0, 0);
}
// 16-byte pieces of a row are xor-ed inside groups of 8 (rows of an odd number of 128-byte lines) or 16 (even)
template <int W>
__device__ __forceinline__ int swz_k(int row) { return (W / 64) & 1 ? ((row >> 1) & 7) : (row & 15); }
template <int W>
__device__ __forceinline__ int swz_v(int row) { return W == 64 ? (row & 6) : ((2 * row) & 14); }

// LDS of a tile walk: V images of both buffers, then their K images (V offsets fit a DS immediate)
template <int DK, int DV>
struct TileImages {
    static constexpr int BN = 64, KROW = DK * 2, VROW = DV * 2, KIMG = BN * KROW, VIMG = BN * VROW;
    static constexpr int KP = DK / 8, VP = DV / 8;   // 16-byte pieces per row == DMA instructions per image
    static constexpr int NK = KP / 4, NV = VP / 4;   // ... per wave
    static constexpr size_t BYTES = (size_t)2 * (KIMG + VIMG);
    static __device__ __forceinline__ unsigned char* k(unsigned char* lds, int buf) { return lds + 2 * VIMG + buf * KIMG; }
    static __device__ __forceinline__ unsigned char* v(unsigned char* lds, int buf) { return lds + buf * VIMG; }
};

// One workgroup's attention over n_tiles tiles of 64 keys; wave w holds query rows 16 QT w .. of the workgroup's 64 QT.  The kernel says
//   stage(it, buf)       starts the NK + NV DMA instructions per wave that fill buffer `buf` with tile `it`
//   query(qs, st)        query fragment: row lq of sub-tile qs, columns 32 st + 8 lg .. (B operand of S^T)
//   first_key(it)        key of the tile's first row; covers(kv0): this wave sees something of that tile; masked(kv0): but not all of it:
//   sees(kv0, qs, off)   key kv0 + 4 lg + off counts for the lane's query of sub-tile qs
//   row(qs)              where the lane's query of sub-tile qs goes, or null; last(qs, d, v): what becomes of its 4 output columns from d on
// start: score (log2 domain) of a softmax entry without key and value, -inf for none.
// (The sums, the fragments and the tile loop live in ONE function: split up, the same code takes 32 registers more.)
template <int DK, int DV, int QT, typename Stage, typename Query, typename FirstKey, typename Covers, typename Masked, typename Sees, typename Row, typename Last>
__device__ __forceinline__ void attend_walk(unsigned char* lds, int n_tiles, float scale_log2, float start, int lane, Stage stage, Query query, FirstKey first_key, Covers covers,
                                            Masked need_mask, Sees sees, Row row, Last last) {
    using Images = TileImages<DK, DV>;
    constexpr int BN = Images::BN, KROW = Images::KROW, VROW = Images::VROW, KIMG = Images::KIMG, VIMG = Images::VIMG, NK = Images::NK, NV = Images::NV;
    constexpr int STEPS = DK / 32, DT = DV / 16, NT = BN / 16;
    const int lq = lane & 15, lg = lane >> 4;
    f32x4 o[QT][DT];
    float m[QT], l[QT];                              // running maximum (log2 domain) and this lane's share of the sum
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        m[qs] = start;
        l[qs] = start > -INFINITY && lg == 0 ? 1.f : 0.f;
#pragma unroll
        for (int t = 0; t < DT; ++t) o[qs][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    stage(0, 0);
    bf16x8 qf[QT][STEPS];
#pragma unroll
    for (int qs = 0; qs < QT; ++qs)
#pragma unroll
        for (int st = 0; st < STEPS; ++st) qf[qs][st] = query(qs, st);
    uint32_t vaddr[DT];
    {
        const int R0 = 4 * lg + (lq >> 2), p = lq & 3, swz = swz_v<DV>(R0);    // rows R0, R0 + 16, R0 + 32 share a swizzle
#pragma unroll
        for (int t = 0; t < DT; ++t) vaddr[t] = lds_addr_of(lds + R0 * VROW + (p & 1) * 8 + (((2 * t + (p >> 1)) ^ swz) * 16));
    }
    auto tile_body = [&](auto bufc, const int it) {
        constexpr int buf = decltype(bufc)::value;
        if (it + 1 < n_tiles) {
            stage(it + 1, buf ^ 1);
            asm volatile("s_waitcnt vmcnt(%0)" ::"n"(NK + NV) : "memory");     // tile `it` has landed, tile it + 1 is in flight
        } else {
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        }
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        const unsigned char* kimg = lds + 2 * VIMG + buf * KIMG;
        const int kv0 = first_key(it);
        if (covers(kv0)) {
            f32x4 sT[QT][NT];
#pragma unroll
            for (int tt = 0; tt < NT; ++tt) {
#pragma unroll
                for (int qs = 0; qs < QT; ++qs) sT[qs][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
                const int R = 16 * tt + lq;
#pragma unroll
                for (int st = 0; st < STEPS; ++st) {
                    const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kimg + R * KROW + (((4 * st + lg) ^ swz_k<DK>(R)) * 16));
#pragma unroll
                    for (int qs = 0; qs < QT; ++qs) sT[qs][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qs][st], sT[qs][tt], 0, 0, 0);
                }
            }
            // the max chain reads the accumulators through inline asm: one statement that takes all of them carries the MFMA wait states
            if constexpr (QT == 1) asm volatile("s_nop 7" : "+v"(sT[0][0]), "+v"(sT[0][1]), "+v"(sT[0][2]), "+v"(sT[0][3]));
            else asm volatile("s_nop 7" : "+v"(sT[0][0]), "+v"(sT[0][1]), "+v"(sT[0][2]), "+v"(sT[0][3]), "+v"(sT[1][0]), "+v"(sT[1][1]), "+v"(sT[1][2]), "+v"(sT[1][3]));
            const bool masked = need_mask(kv0);
#pragma unroll
            for (int qs = 0; qs < QT; ++qs) {
                if (masked) {
#pragma unroll
                    for (int tt = 0; tt < NT; ++tt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) sT[qs][tt][r] = sees(kv0, qs, 16 * tt + r) ? sT[qs][tt][r] : -INFINITY;
                }
                float mx = max3f(sT[qs][0][0], sT[qs][0][1], sT[qs][0][2]);
                mx = max3f(mx, sT[qs][0][3], sT[qs][1][0]);
                mx = max3f(mx, sT[qs][1][1], sT[qs][1][2]);
                mx = max3f(mx, sT[qs][1][3], sT[qs][2][0]);
                mx = max3f(mx, sT[qs][2][1], sT[qs][2][2]);
                mx = max3f(mx, sT[qs][2][3], sT[qs][3][0]);
                mx = max3f(mx, sT[qs][3][1], sT[qs][3][2]);
                mx = max2(mx, sT[qs][3][3]);
                mx = max_xor16(mx);
                mx = max_xor32(mx);
                mx *= scale_log2;                                                  // (the host admits positive scales only)
                const float m_new = max2(m[qs], mx);
                const float m_use = m_new == -INFINITY ? 0.f : m_new;
                float psum = 0.f;
#pragma unroll
                for (int tt = 0; tt < NT; ++tt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const float e = fast_exp2(sT[qs][tt][r] * scale_log2 - m_use);
                        sT[qs][tt][r] = e;
                        psum += e;
                    }
                if (__builtin_amdgcn_ballot_w64(m_new != m[qs]) != 0) {
                    const float alpha = fast_exp2(m[qs] - m_use);
                    l[qs] *= alpha;
#pragma unroll
                    for (int t = 0; t < DT; ++t) o[qs][t] *= alpha;
                }
                l[qs] += psum;
                m[qs] = m_new;
            }
#pragma unroll
            for (int hh = 0; hh < BN / 32; ++hh) {
                bf16x8 p_hi[QT], p_lo[QT];
#pragma unroll
                for (int qs = 0; qs < QT; ++qs) {
                    u32x4 hraw, lraw;
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const float p0 = sT[qs][2 * hh + (j >> 1)][2 * (j & 1)], p1 = sT[qs][2 * hh + (j >> 1)][2 * (j & 1) + 1];
                        hraw[j] = pack_bf16x2(p0, p1);
                        lraw[j] = pack_bf16x2(p0 - bf16_lo(hraw[j]), p1 - bf16_hi(hraw[j]));
                    }
                    p_hi[qs] = *reinterpret_cast<const bf16x8*>(&hraw);
                    p_lo[qs] = *reinterpret_cast<const bf16x8*>(&lraw);
                }
                u32x2 vlo[DT], vhi[DT];
                if (hh == 0) {
#pragma unroll
                    for (int t = 0; t < DT; ++t) {
                        vlo[t] = ds_read_tr16<buf * VIMG>(vaddr[t]);
                        vhi[t] = ds_read_tr16<buf * VIMG + 16 * VROW>(vaddr[t]);
                    }
                } else {
#pragma unroll
                    for (int t = 0; t < DT; ++t) {
                        vlo[t] = ds_read_tr16<buf * VIMG + 32 * VROW>(vaddr[t]);
                        vhi[t] = ds_read_tr16<buf * VIMG + 48 * VROW>(vaddr[t]);
                    }
                }
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                __builtin_amdgcn_sched_barrier(0);
                bf16x8 vf[DT];
#pragma unroll
                for (int t = 0; t < DT; ++t) {
                    const u32x4 raw = {vlo[t][0], vlo[t][1], vhi[t][0], vhi[t][1]};
                    vf[t] = *reinterpret_cast<const bf16x8*>(&raw);
                }
#pragma unroll
                for (int t = 0; t < DT; ++t)
#pragma unroll
                    for (int qs = 0; qs < QT; ++qs) o[qs][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[t], p_hi[qs], o[qs][t], 0, 0, 0);
#pragma unroll
                for (int t = 0; t < DT; ++t)
#pragma unroll
                    for (int qs = 0; qs < QT; ++qs) o[qs][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[t], p_lo[qs], o[qs][t], 0, 0, 0);
            }
        }
        lds_only_barrier();                                                    // everyone's reads of this buffer are done
    };
    for (int it = 0; it < n_tiles; it += 2) {
        tile_body(std::integral_constant<int, 0>{}, it);
        if (it + 1 < n_tiles) tile_body(std::integral_constant<int, 1>{}, it + 1);
    }
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        float sum = sum_xor16(l[qs]);
        sum = sum_xor32(sum);
        uint16_t* out = row(qs);
        if (!out) continue;
        const float inv = sum > 0.f ? 1.f / sum : 0.f;
#pragma unroll
        for (int t = 0; t < DT; ++t) act_st4(out + 16 * t + 4 * lg, last(qs, 16 * t + 4 * lg, o[qs][t] * inv));
    }
}

// (sequence, head, query tile) of this workgroup: the query tiles of one (sequence, head) share one XCD's L2, heaviest tiles first (workgroups are
// dealt round-robin over the 8 XCDs).  Grid: heads x sequences x query tiles.
__device__ __forceinline__ void attend_unit(int heads, int& qt, int& head, int& b) {
    qt = gridDim.z - 1 - blockIdx.z;
    head = blockIdx.x;
    b = blockIdx.y;
    const int units = (int)(gridDim.x * gridDim.y);
    if ((units & 7) == 0) {
        const int lin = (int)blockIdx.x + (int)gridDim.x * ((int)blockIdx.y + (int)gridDim.y * (int)blockIdx.z);
        const int idx = lin >> 3, per = units >> 3, u = (lin & 7) + 8 * (idx % per);
        b = u / heads;
        head = u - b * heads;
        qt = (int)gridDim.z - 1 - idx / per;
    }
}

}  // namespace nvh
