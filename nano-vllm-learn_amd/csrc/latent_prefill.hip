// Causal attention of prompt portions in expanded latent form (gfx950 MFMA): the keys and values of every visible token have been expanded from the
// cached latents by two projections; a head's key is [its own unrotated part | the rotated part all heads share], key width DK != value width DV.
// Same tile scheme as prefill_mfma.hip (4 waves x QT x 16 query rows, 64-key tiles double-buffered through LDS by LDS-DMA, S^T = K Q^T and
// O^T = V^T P^T with the weights as bf16 hi + lo halves, online softmax in the log2 domain); what differs:
//   * a key row in LDS is gathered from two sources: each 16-byte piece comes from the expanded rows or from the shared rotated rows
//   * the query's rotated part is turned in registers while the fragments are loaded, so no launch of its own rotates queries
//   * unequal widths: DK in {64, 128, 192, 256}, DV in {64, 128}
// Algorithmic flops per launch: sum over sequences of 2 (DK + DV) heads (causal pairs).
#include <type_traits>

#include "hybrid.h"

namespace nvh {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
constexpr int BN = 64;

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
// 16-byte pieces of a row are xor-ed inside groups of 8 (rows of an odd number of 128-byte lines) or 16 (even)
template <int W>
__device__ __forceinline__ int swz_k(int row) { return (W / 64) & 1 ? ((row >> 1) & 7) : (row & 15); }
template <int W>
__device__ __forceinline__ int swz_v(int row) { return W == 64 ? (row & 6) : ((2 * row) & 14); }

template <int DK, int DV, int QT>
__global__ __launch_bounds__(256) void latent_prefill_kernel(const LatentPrefillArgs a) {
    constexpr int BM = 64 * QT, WR = 16 * QT;
    constexpr int KROW = DK * 2, VROW = DV * 2, KIMG = BN * KROW, VIMG = BN * VROW;
    constexpr int KP = DK / 8, VP = DV / 8;          // 16-byte pieces per row == DMA instructions per image
    constexpr int NK = KP / 4, NV = VP / 4;          // ... per wave
    constexpr int STEPS = DK / 32, DT = DV / 16, NT = BN / 16;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];        // V images of both buffers, then their K images (V offsets fit a DS immediate)
    int qt = gridDim.z - 1 - blockIdx.z, head = blockIdx.x, b = blockIdx.y;
    {
        // the q-tiles of one (sequence, head) share one XCD's L2, heaviest tiles first (workgroups are dealt round-robin over the 8 XCDs)
        const int units = (int)(gridDim.x * gridDim.y);
        if ((units & 7) == 0) {
            const int lin = (int)blockIdx.x + (int)gridDim.x * ((int)blockIdx.y + (int)gridDim.y * (int)blockIdx.z);
            const int idx = lin >> 3, per = units >> 3, u = (lin & 7) + 8 * (idx % per);
            b = u / a.heads;
            head = u - b * a.heads;
            qt = (int)gridDim.z - 1 - idx / per;
        }
    }
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, k_beg = a.cu_k[b], sk = a.cu_k[b + 1] - k_beg;
    const int q0 = qt * BM;
    if (q0 >= sq || sk <= 0) return;
    const int shift = sk - sq;                       // query r sees keys <= r + shift
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;

    f32x4 o[QT][DT];
    float m_run[QT], l_run[QT];
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        m_run[qs] = -INFINITY;
        l_run[qs] = 0.f;
#pragma unroll
        for (int t = 0; t < DT; ++t) o[qs][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    int kv_end = q0 + BM + shift;
    if (kv_end > sk) kv_end = sk;
    const int n_tiles = (kv_end + BN - 1) / BN;
    const int wave_first_key = q0 + wave * WR + shift, wave_last_key = wave_first_key + WR - 1;

    // ---- staging: this lane's piece of each DMA instruction: LDS row, source pointer of the sequence's first key, row stride
    const uint16_t *kp[NK], *vp_[NV];
    int64_t ks[NK];
    int kr[NK], vr_[NV];
#pragma unroll
    for (int j = 0; j < NK; ++j) {
        const int s = (wave * NK + j) * 64 + lane, R = s / KP, piece = (s - R * KP) ^ swz_k<DK>(R);
        const bool own = piece * 8 < a.dim_cols;
        kr[j] = R;
        ks[j] = own ? a.k_stride : a.kr_stride;
        kp[j] = own ? a.k + (int64_t)k_beg * a.k_stride + head * a.dim_cols + piece * 8 : a.k_rot + (int64_t)k_beg * a.kr_stride + (piece * 8 - a.dim_cols);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int s = (wave * NV + j) * 64 + lane, R = s / VP, piece = (s - R * VP) ^ swz_v<DV>(R);
        vr_[j] = R;
        vp_[j] = a.v + (int64_t)k_beg * a.v_stride + head * DV + piece * 8;
    }
    auto stage = [&](int tile, int buf) {
        unsigned char* kimg = lds + 2 * VIMG + buf * KIMG;
        unsigned char* vimg = lds + buf * VIMG;
        const int kv0 = tile * BN;
#pragma unroll
        for (int j = 0; j < NK; ++j) {
            const int row = kv0 + kr[j] < sk ? kv0 + kr[j] : sk - 1;           // rows past the end repeat the last key: masked
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(kp[j] + row * ks[j]),
                                             (__attribute__((address_space(3))) void*)(kimg + (wave * NK + j) * 1024), 16, 0, 0);
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int row = kv0 + vr_[j] < sk ? kv0 + vr_[j] : sk - 1;
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(vp_[j] + row * a.v_stride),
                                             (__attribute__((address_space(3))) void*)(vimg + (wave * NV + j) * 1024), 16, 0, 0);
        }
    };
    stage(0, 0);

    // ---- query fragments (B operand of S^T), the rotated part turned here
    int my_q[QT];
    bool q_ok[QT];
    bf16x8 qf[QT][STEPS];
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        my_q[qs] = q0 + wave * WR + 16 * qs + lq;
        q_ok[qs] = my_q[qs] < sq;
        const int64_t qrow = q_beg + (q_ok[qs] ? my_q[qs] : sq - 1);
        const uint16_t* qp = a.q + qrow * a.q_stride + (int64_t)head * DK + lg * 8;
        int64_t pos = a.positions[qrow];
        if (pos >= a.max_position) pos = a.max_position - 1;
        const float* cs = a.cos_sin + pos * a.rot;
#pragma unroll
        for (int st = 0; st < STEPS; ++st) {
            u32x4 raw = *reinterpret_cast<const u32x4*>(qp + st * 32);
            const int i0 = (32 * st + 8 * lg - a.dim_cols) / 2;               // first pair of this piece (dim_cols is a multiple of 32)
            if (32 * st >= a.dim_cols) {
#pragma unroll
                for (int k = 0; k < 4; ++k)
                    if (i0 + k < a.rot / 2) {
                        const float u = bf16_lo(raw[k]), v = bf16_hi(raw[k]), co = cs[i0 + k], si = cs[a.rot / 2 + i0 + k];
                        raw[k] = pack_bf16x2(u * co - v * si, v * co + u * si);
                    }
            }
            qf[qs][st] = *reinterpret_cast<const bf16x8*>(&raw);
        }
    }
    uint32_t vaddr[DT];
    {
        const int R0 = 4 * lg + (lq >> 2), p = lq & 3, swz = swz_v<DV>(R0);   // rows R0, R0 + 16, R0 + 32 share a swizzle
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
        const int kv0 = it * BN;
        if (kv0 <= wave_last_key) {
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
            const bool need_mask = kv0 + BN - 1 > wave_first_key || kv0 + BN > sk;
#pragma unroll
            for (int qs = 0; qs < QT; ++qs) {
                if (need_mask) {
                    const int q_pos = my_q[qs] + shift;
                    const int limit = (q_pos < sk - 1 ? q_pos : sk - 1) - kv0 - 4 * lg;
#pragma unroll
                    for (int tt = 0; tt < NT; ++tt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) sT[qs][tt][r] = (16 * tt + r <= limit) ? sT[qs][tt][r] : -INFINITY;
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
                mx *= a.scale_log2;                                            // the host admits positive scales only
                const float m_new = max2(m_run[qs], mx);
                const float m_use = m_new == -INFINITY ? 0.f : m_new;
                float psum = 0.f;
#pragma unroll
                for (int tt = 0; tt < NT; ++tt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const float e = fast_exp2(sT[qs][tt][r] * a.scale_log2 - m_use);
                        sT[qs][tt][r] = e;
                        psum += e;
                    }
                if (__builtin_amdgcn_ballot_w64(m_new != m_run[qs]) != 0) {
                    const float alpha = fast_exp2(m_run[qs] - m_use);
                    l_run[qs] *= alpha;
#pragma unroll
                    for (int t = 0; t < DT; ++t) o[qs][t] *= alpha;
                }
                l_run[qs] += psum;
                m_run[qs] = m_new;
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
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();                                          // everyone's reads of this buffer are done
        asm volatile("" ::: "memory");
    };
    for (int it = 0; it < n_tiles; it += 2) {
        tile_body(std::integral_constant<int, 0>{}, it);
        if (it + 1 < n_tiles) tile_body(std::integral_constant<int, 1>{}, it + 1);
    }
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        float l = sum_xor16(l_run[qs]);
        l = sum_xor32(l);
        if (!q_ok[qs]) continue;
        const float inv = l > 0.f ? 1.f / l : 0.f;
        uint16_t* orow = a.out + (int64_t)(q_beg + my_q[qs]) * a.out_stride + head * DV;
#pragma unroll
        for (int t = 0; t < DT; ++t) act_st4(orow + 16 * t + 4 * lg, o[qs][t] * inv);
    }
}

template <int DK, int DV, int QT>
int launch_one(const LatentPrefillArgs& a, hipStream_t stream) {
    constexpr size_t lds = (size_t)2 * BN * (DK + DV) * 2;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(latent_prefill_kernel<DK, DV, QT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    latent_prefill_kernel<DK, DV, QT><<<dim3(a.heads, a.batch, (a.max_q + 64 * QT - 1) / (64 * QT)), 256, lds, stream>>>(a);
    return check_launch("latent_prefill");
}
template <int DK, int DV>
int launch_dims(const LatentPrefillArgs& a, hipStream_t stream) {
    return a.max_q > 256 ? launch_one<DK, DV, 2>(a, stream) : launch_one<DK, DV, 1>(a, stream);
}

}  // namespace

bool latent_prefill_supported(int dk, int dv) { return (dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128); }

int launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t stream) {
    if (a.batch == 0 || a.max_q <= 0) return 0;
    switch (a.dk * 1000 + a.dv) {
        case 64064: return launch_dims<64, 64>(a, stream);
        case 64128: return launch_dims<64, 128>(a, stream);
        case 128064: return launch_dims<128, 64>(a, stream);
        case 128128: return launch_dims<128, 128>(a, stream);
        case 192064: return launch_dims<192, 64>(a, stream);
        case 192128: return launch_dims<192, 128>(a, stream);
        case 256064: return launch_dims<256, 64>(a, stream);
        case 256128: return launch_dims<256, 128>(a, stream);
        default: set_error("latent_prefill: key width %d / value width %d", a.dk, a.dv); return -2;
    }
}

}  // namespace nvh
