// Lightning attention: per head a matrix state with a constant decay d,   S = d S + k v^T,   o = S^T q,   q, k, v = silu of the projection's columns.
//
// Prompt portions (launch_lightning_chunks): a workgroup owns one (segment, head, 64 value columns) and takes 64 tokens at a time,
//   o_i = d^(i+1) S^T q_i + sum_{j <= i} d^(i-j) (q_i . k_j) v_j          S <- d^n S + sum_j d^(n-1-j) k_j v_j^T
// on MFMA tiles.  The state stays in fp32 accumulators, laid out so that they are the left operand of S^T q without a shuffle; everything decays touch
// (weights, state, decayed values) enters the MFMA as bf16 hi + lo halves.  q, k and v go through registers on their way to LDS (silu, one rounding),
// the next step's rows are fetched while this one computes.
// A portion of several segments: a SUMMARY walk leaves every segment's own contribution, a small launch turns those into states at segment starts, and
// the second walk begins there.  State pools are read by the launch in front and written by the last segment: no workgroup sees a half-updated one.
// Decoding (launch_lightning_step): one workgroup per (sequence, head, value slice) streams the state once: read, decay, add, multiply, write.
// A sequence's first token (position 0) takes the state as zero instead of reading it: slots need no clearing when reused.
#include "attend_tile.h"
#include "mixers.h"

namespace nvh {

namespace {

constexpr int C = kLightningChunk, VS = 64;          // tokens per step, value columns per workgroup
constexpr int PLD = C + 8;                           // row of the weights in LDS

__device__ __forceinline__ void split_hi_lo(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
    u32x4 h, l;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        h[j] = pack_bf16x2(v[2 * j], v[2 * j + 1]);
        l[j] = pack_bf16x2(v[2 * j] - bf16_lo(h[j]), v[2 * j + 1] - bf16_hi(h[j]));
    }
    hi = *reinterpret_cast<const bf16x8*>(&h);
    lo = *reinterpret_cast<const bf16x8*>(&l);
}

__device__ __forceinline__ u32x4 silu8(u32x4 r) {
#pragma unroll
    for (int k = 0; k < 4; ++k) r[k] = pack_bf16x2(silu_f(bf16_lo(r[k])), silu_f(bf16_hi(r[k])));
    return r;
}

template <int DK, bool SUMMARY>
__global__ __launch_bounds__(256) void lightning_walk_kernel(const LightningArgs a) {
    constexpr int KP = DK / 8, KROW = DK * 2, NQ = C * KP / 256, NV = C * (VS / 8) / 256, DT = DK / 16;
    constexpr bool kOdd = ((KROW / 128) & 1) != 0, kAhead = DK <= 128;         // (wider: no registers to fetch a step ahead)
    constexpr int TB = DT < 8 ? DT : 8;              // key tiles read at a time
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    unsigned char* kimg = smem;                                                // [C][DK] keys
    unsigned char* vimg = kimg + C * KROW;                                     // [C][VS] values
    unsigned char* qimg = vimg + C * VS * 2;                                   // [C][DK] queries
    uint16_t* p_lds = reinterpret_cast<uint16_t*>(qimg + C * KROW);            // [hi | lo][C][PLD] weights
    __shared__ float pw[C + 1];                                                // decay^0 .. decay^C
    auto swz = [](int r) { return kOdd ? ((r >> 1) & 7) : (r & 7); };
    auto swzv = [](int r) { return (r >> 1) & 7; };
    const int32_t* ch = a.chunks + 4 * blockIdx.x;
    const int row0 = ch[0], n_rows = ch[1], seq = ch[2];
    const int head = blockIdx.y, v0 = blockIdx.z * VS;
    const bool last = blockIdx.x + 1 == (unsigned)a.n_chunks || a.chunks[4 * (blockIdx.x + 1) + 3] == 0;
    if (SUMMARY && last) return;                     // (nothing follows it)
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const int64_t slot = a.state_slots[seq];
    const int64_t head_state = (int64_t)a.dk * a.dv;
    if (tid <= C) pw[tid] = powf(a.decay[head], (float)tid);

    // state: value column v0 + 16 wave + lq, key rows 16 t + 4 lg + r
    f32x4 S[DT];
#pragma unroll
    for (int t = 0; t < DT; ++t) S[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int sv = v0 + 16 * wave + lq;
    if constexpr (!SUMMARY) {
        const float* src = nullptr;
        if (a.summaries) src = a.seg_state + ((int64_t)blockIdx.x * a.heads + head) * head_state;
        else if (slot >= 0 && a.positions[row0] > 0) src = a.state + (slot * a.heads + head) * head_state;
        if (src) {
#pragma unroll
            for (int t = 0; t < DT; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) S[t][r] = src[(int64_t)(16 * t + 4 * lg + r) * a.dv + sv];
        }
    }
    const uint16_t* qkv = reinterpret_cast<const uint16_t*>(a.qkv);
    const int64_t k_off = (int64_t)a.heads * a.dk + head * DK, v_off = 2 * (int64_t)a.heads * a.dk + (int64_t)head * a.dv + v0, q_off = (int64_t)head * DK;
    u32x4 qr[NQ], kr[NQ], vr[NV];
    const u32x4 zero = {0u, 0u, 0u, 0u};
    auto fetch = [&](int t0) {                       // rows t0 .. of the segment; rows past its end are zero
#pragma unroll
        for (int j = 0; j < NQ; ++j) {
            const int e = j * 256 + tid, r = e / KP, c = (e - r * KP) * 8;
            const bool ok = t0 + r < n_rows;
            const uint16_t* p = qkv + (int64_t)(row0 + (ok ? t0 + r : 0)) * a.qkv_stride + c;
            kr[j] = ok ? *reinterpret_cast<const u32x4*>(p + k_off) : zero;
            if constexpr (!SUMMARY) qr[j] = ok ? *reinterpret_cast<const u32x4*>(p + q_off) : zero;
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int e = j * 256 + tid, r = e >> 3, c = (e & 7) * 8;
            const bool ok = t0 + r < n_rows;
            vr[j] = ok ? *reinterpret_cast<const u32x4*>(qkv + (int64_t)(row0 + t0 + r) * a.qkv_stride + v_off + c) : zero;
        }
    };
    if constexpr (kAhead) fetch(0);
    for (int t0 = 0; t0 < n_rows; t0 += C) {
        const int n = n_rows - t0 < C ? n_rows - t0 : C;
        if constexpr (!kAhead) fetch(t0);
        // (silu(0) = 0: rows past the end stay zero)
#pragma unroll
        for (int j = 0; j < NQ; ++j) {
            const int e = j * 256 + tid, r = e / KP, pc = e - r * KP;
            *reinterpret_cast<u32x4*>(kimg + r * KROW + (pc ^ swz(r)) * 16) = silu8(kr[j]);
            if constexpr (!SUMMARY) *reinterpret_cast<u32x4*>(qimg + r * KROW + (pc ^ swz(r)) * 16) = silu8(qr[j]);
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int e = j * 256 + tid, r = e >> 3, pc = e & 7;
            *reinterpret_cast<u32x4*>(vimg + r * VS * 2 + (pc ^ swzv(r)) * 16) = silu8(vr[j]);
        }
        if constexpr (kAhead) {
            if (t0 + C < n_rows) fetch(t0 + C);
        }
        lds_only_barrier();
        const int tr = 4 * lg + (lq >> 2), tp = lq & 3;                        // transposed reads: row and column quarter this lane addresses
        f32x4 o[4];                                  // o^T: value 16 wave + 4 lg + r, token 16 it + lq
        if constexpr (!SUMMARY) {
            // weights of this wave's 16 queries: D[key 16 jt + 4 lg + r][query 16 wave + lq]
            f32x4 s[4];
#pragma unroll
            for (int jt = 0; jt < 4; ++jt) s[jt] = f32x4{0.f, 0.f, 0.f, 0.f};
            const int Rq = 16 * wave + lq;
#pragma unroll
            for (int st = 0; st < DK / 32; ++st) {
                const bf16x8 qf = *reinterpret_cast<const bf16x8*>(qimg + Rq * KROW + ((4 * st + lg) ^ swz(Rq)) * 16);
#pragma unroll
                for (int jt = 0; jt < 4; ++jt) {
                    if (jt > wave) continue;         // keys behind every query of this wave
                    const int Rk = 16 * jt + lq;
                    const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kimg + Rk * KROW + ((4 * st + lg) ^ swz(Rk)) * 16);
                    s[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, s[jt], 0, 0, 0);
                }
            }
#pragma unroll
            for (int jt = 0; jt < 4; ++jt) {
                float p[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int back = Rq - (16 * jt + 4 * lg + r);
                    p[r] = back >= 0 ? s[jt][r] * pw[back >= 0 ? back : 0] : 0.f;
                }
                const u32x2 hi = {pack_bf16x2(p[0], p[1]), pack_bf16x2(p[2], p[3])};
                const u32x2 lo = {pack_bf16x2(p[0] - bf16_lo(hi[0]), p[1] - bf16_hi(hi[0])), pack_bf16x2(p[2] - bf16_lo(hi[1]), p[3] - bf16_hi(hi[1]))};
                const int at = Rq * PLD + 32 * (jt >> 1) + 8 * lg + 4 * (jt & 1);
                *reinterpret_cast<u32x2*>(p_lds + at) = hi;
                *reinterpret_cast<u32x2*>(p_lds + C * PLD + at) = lo;
            }
            // what the state gives: slots of a 32-wide step are key rows 16 (2 st) + 4 lg + 0..3 and 16 (2 st + 1) + 4 lg + 0..3
#pragma unroll
            for (int it = 0; it < 4; ++it) o[it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int st = 0; st < DK / 32; ++st) {
                const float v[8] = {S[2 * st][0], S[2 * st][1], S[2 * st][2], S[2 * st][3], S[2 * st + 1][0], S[2 * st + 1][1], S[2 * st + 1][2], S[2 * st + 1][3]};
                bf16x8 hi, lo;
                split_hi_lo(v, hi, lo);
#pragma unroll
                for (int it = 0; it < 4; ++it) {
                    const int R = 16 * it + lq;
                    const unsigned char* qrow = qimg + R * KROW + (lg & 1) * 8;
                    const u32x2 qa = *reinterpret_cast<const u32x2*>(qrow + ((4 * st + (lg >> 1)) ^ swz(R)) * 16);
                    const u32x2 qb = *reinterpret_cast<const u32x2*>(qrow + ((4 * st + 2 + (lg >> 1)) ^ swz(R)) * 16);
                    const u32x4 raw = {qa[0], qa[1], qb[0], qb[1]};
                    const bf16x8 qf = *reinterpret_cast<const bf16x8*>(&raw);
                    o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, qf, o[it], 0, 0, 0);
                    o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, qf, o[it], 0, 0, 0);
                }
            }
#pragma unroll
            for (int it = 0; it < 4; ++it) o[it] *= pw[16 * it + lq + 1];
            lds_only_barrier();                      // all weights are in LDS
        }
        // value fragments: lane = column 16 wave + lq, slots = keys 32 hh + 4 lg + 0..3 and the same + 16
        u32x2 vlo[2], vhi[2];
#pragma unroll
        for (int hh = 0; hh < 2; ++hh) {
            const int ra = 32 * hh + tr, rb = ra + 16, pc = 2 * wave + (tp >> 1);
            vlo[hh] = ds_read_tr16<0>(lds_addr_of(vimg + ra * VS * 2 + (pc ^ swzv(ra)) * 16 + (tp & 1) * 8));
            vhi[hh] = ds_read_tr16<0>(lds_addr_of(vimg + rb * VS * 2 + (pc ^ swzv(rb)) * 16 + (tp & 1) * 8));
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_sched_barrier(0);
        bf16x8 vf[2];
#pragma unroll
        for (int hh = 0; hh < 2; ++hh) {
            const u32x4 raw = {vlo[hh][0], vlo[hh][1], vhi[hh][0], vhi[hh][1]};
            vf[hh] = *reinterpret_cast<const bf16x8*>(&raw);
        }
        if constexpr (!SUMMARY) {
#pragma unroll
            for (int it = 0; it < 4; ++it)
#pragma unroll
                for (int hh = 0; hh < 2; ++hh) {
                    if (32 * hh > 16 * it + 15) continue;
                    const uint16_t* pr = p_lds + (16 * it + lq) * PLD + 32 * hh + 8 * lg;
                    o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[hh], *reinterpret_cast<const bf16x8*>(pr), o[it], 0, 0, 0);
                    o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[hh], *reinterpret_cast<const bf16x8*>(pr + C * PLD), o[it], 0, 0, 0);
                }
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                const int t = t0 + 16 * it + lq;
                if (t < n_rows) act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(row0 + t) * a.out_stride + (int64_t)head * a.dv + v0 + 16 * wave + 4 * lg, o[it]);
            }
        }
        // ---- the state behind these tokens
#pragma unroll
        for (int t = 0; t < DT; ++t) S[t] *= pw[n];
#pragma unroll
        for (int hh = 0; hh < 2; ++hh) {
            const u32x4 raw = *reinterpret_cast<const u32x4*>(&vf[hh]);
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int key = 32 * hh + (j < 4 ? 0 : 16) + 4 * lg + (j & 3);
                v[j] = (j & 1 ? bf16_hi(raw[j >> 1]) : bf16_lo(raw[j >> 1])) * pw[key < n ? n - 1 - key : 0];
            }
            bf16x8 hi, lo;
            split_hi_lo(v, hi, lo);
            const int ra = 32 * hh + tr, rb = ra + 16;
#pragma unroll
            for (int tb = 0; tb < DT; tb += TB) {
                u32x2 klo[TB], khi[TB];
#pragma unroll
                for (int t = 0; t < TB; ++t) {
                    const int pc = 2 * (tb + t) + (tp >> 1);
                    klo[t] = ds_read_tr16<0>(lds_addr_of(kimg + ra * KROW + (pc ^ swz(ra)) * 16 + (tp & 1) * 8));
                    khi[t] = ds_read_tr16<0>(lds_addr_of(kimg + rb * KROW + (pc ^ swz(rb)) * 16 + (tp & 1) * 8));
                }
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int t = 0; t < TB; ++t) {
                    const u32x4 kraw = {klo[t][0], klo[t][1], khi[t][0], khi[t][1]};
                    const bf16x8 kf = *reinterpret_cast<const bf16x8*>(&kraw);
                    S[tb + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, hi, S[tb + t], 0, 0, 0);
                    S[tb + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, lo, S[tb + t], 0, 0, 0);
                }
            }
        }
        lds_only_barrier();                          // everyone is done with the images
    }
    float* dst = nullptr;
    if constexpr (SUMMARY) dst = a.seg_state + ((int64_t)blockIdx.x * a.heads + head) * head_state;
    else if (last && slot >= 0) dst = a.state + (slot * a.heads + head) * head_state;
    if (dst) {
#pragma unroll
        for (int t = 0; t < DT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[(int64_t)(16 * t + 4 * lg + r) * a.dv + sv] = S[t][r];
    }
}

// contributions of the segments -> states at their starts, in place; one thread per state element, walking the segments of every portion
__global__ __launch_bounds__(256) void lightning_starts_kernel(const LightningArgs a) {
    const int64_t head_state = (int64_t)a.dk * a.dv, per = a.heads * head_state, e = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int first = blockIdx.y;                    // only a portion's first segment starts a walk
    if (e >= per || a.chunks[4 * first + 3] != 0) return;
    const float d = a.decay[e / head_state];
    const int64_t slot = a.state_slots[a.chunks[4 * first + 2]];
    float cur = slot >= 0 && a.positions[a.chunks[4 * first]] > 0 ? a.state[slot * per + e] : 0.f;
    for (int c = first; c < a.n_chunks && (c == first || a.chunks[4 * c + 3] != 0); ++c) {
        const bool more = c + 1 < a.n_chunks && a.chunks[4 * (c + 1) + 3] != 0;        // (the last segment left no contribution)
        const float own = more ? a.seg_state[c * per + e] : 0.f;
        a.seg_state[c * per + e] = cur;
        cur = powf(d, (float)a.chunks[4 * c + 1]) * cur + own;
    }
}

// ------------------------------------------------------------------------------------------------ token by token, any type and size
// one workgroup per (portion, head, 32 value columns); the state slice in LDS, 8 groups of key rows x 32 columns
template <typename T>
__global__ __launch_bounds__(256) void lightning_generic_kernel(const LightningArgs a) {
    extern __shared__ float lds_f[];                 // [dk][32] state, [2][dk] k and q, [8][32] sums
    float *S = lds_f, *kq = S + a.dk * 32, *red = kq + 2 * a.dk;
    const int first = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, c = tid & 31, rg = tid >> 5, col = blockIdx.z * 32 + c;
    if (a.chunks[4 * first + 3] != 0) return;        // a portion is walked whole from its first segment
    const int row0 = a.chunks[4 * first];
    int n_rows = a.chunks[4 * first + 1];
    for (int k = first + 1; k < a.n_chunks && a.chunks[4 * k + 3] != 0; ++k) n_rows += a.chunks[4 * k + 1];
    const int64_t slot = a.state_slots[a.chunks[4 * first + 2]], head_state = (int64_t)a.dk * a.dv;
    const bool ok = col < a.dv;
    float* pool = slot >= 0 ? a.state + (slot * a.heads + head) * head_state : nullptr;
    const bool carry = pool && a.positions[row0] > 0;
    for (int r = rg; r < a.dk; r += 8) S[r * 32 + c] = carry && ok ? pool[(int64_t)r * a.dv + col] : 0.f;
    const float d = a.decay[head];
    for (int t = 0; t < n_rows; ++t) {
        const T* x = reinterpret_cast<const T*>(a.qkv) + (int64_t)(row0 + t) * a.qkv_stride;
        for (int i = tid; i < a.dk; i += 256) {
            const float k = act_ld(x + (int64_t)a.heads * a.dk + head * a.dk + i), q = act_ld(x + head * a.dk + i);
            kq[i] = act_round(silu_f(k), (const T*)nullptr);
            kq[a.dk + i] = act_round(silu_f(q), (const T*)nullptr);
        }
        const float v = ok ? act_round(silu_f(act_ld(x + 2 * (int64_t)a.heads * a.dk + (int64_t)head * a.dv + col)), (const T*)nullptr) : 0.f;
        __syncthreads();
        float acc = 0.f;
        for (int r = rg; r < a.dk; r += 8) {
            const float s = d * S[r * 32 + c] + kq[r] * v;
            S[r * 32 + c] = s;
            acc += s * kq[a.dk + r];
        }
        red[rg * 32 + c] = acc;
        __syncthreads();
        if (rg == 0 && ok) {
            float s = 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k) s += red[k * 32 + c];
            act_st(reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t) * a.out_stride + (int64_t)head * a.dv + col, s);
        }
    }
    if (pool && ok)
        for (int r = rg; r < a.dk; r += 8) pool[(int64_t)r * a.dv + col] = S[r * 32 + c];
}

// ------------------------------------------------------------------------------------------------ one token per sequence (bf16)
// grid (heads, rows, dv / VC): VC / 4 lanes hold a state row's slice, 1024 / VC rows at a time
template <int VC>
__global__ __launch_bounds__(256) void lightning_step_kernel(const LightningArgs a) {
    constexpr int LN = VC / 4, RG = 256 / LN, UN = 8;
    extern __shared__ float lds_s[];                 // [2][dk] k and q, then [RG][VC] sums
    float *kq = lds_s, *red = lds_s + 2 * a.dk;
    const int head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, c = (tid % LN) * 4, rg = tid / LN, col = blockIdx.z * VC + c;
    const int64_t slot = a.state_slots[row], head_state = (int64_t)a.dk * a.dv;
    const bool carry = slot >= 0 && a.positions[row] > 0;
    float* pool = a.state + ((slot >= 0 ? slot : 0) * a.heads + head) * head_state + col;
    const uint16_t* x = reinterpret_cast<const uint16_t*>(a.qkv) + (int64_t)row * a.qkv_stride;
    f32x4 s[UN];
#pragma unroll
    for (int u = 0; u < UN; ++u) {                   // asked for before anything is computed
        const int r = rg + u * RG;
        s[u] = carry && r < a.dk ? *reinterpret_cast<const f32x4*>(pool + (int64_t)r * a.dv) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int i = tid; i < a.dk; i += 256) {
        kq[i] = act_round(silu_f(act_ld(x + (int64_t)a.heads * a.dk + head * a.dk + i)), (const uint16_t*)nullptr);
        kq[a.dk + i] = act_round(silu_f(act_ld(x + head * a.dk + i)), (const uint16_t*)nullptr);
    }
    f32x4 v = act_ld4(x + 2 * (int64_t)a.heads * a.dk + (int64_t)head * a.dv + col);
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = act_round(silu_f(v[k]), (const uint16_t*)nullptr);
    const float d = a.decay[head];
    __syncthreads();
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int r0 = 0; r0 < a.dk; r0 += UN * RG) {
        if (r0) {
#pragma unroll
            for (int u = 0; u < UN; ++u) {
                const int r = r0 + rg + u * RG;
                s[u] = carry && r < a.dk ? *reinterpret_cast<const f32x4*>(pool + (int64_t)r * a.dv) : f32x4{0.f, 0.f, 0.f, 0.f};
            }
        }
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            const int r = r0 + rg + u * RG;
            if (r >= a.dk) continue;
            const f32x4 n = s[u] * d + v * kq[r];
            acc += n * kq[a.dk + r];
            if (slot >= 0) *reinterpret_cast<f32x4*>(pool + (int64_t)r * a.dv) = n;
        }
    }
    *reinterpret_cast<f32x4*>(red + rg * VC + c) = acc;
    __syncthreads();
    if (rg == 0) {
        f32x4 o = acc;
        for (int k = 1; k < RG; ++k) o += *reinterpret_cast<const f32x4*>(red + k * VC + c);
        act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)row * a.out_stride + (int64_t)head * a.dv + col, o);
    }
}

// ------------------------------------------------------------------------------------------------ norm and gate behind the heads
template <typename T, int CH>
__global__ __launch_bounds__(256) void norm_gate_kernel(T* __restrict__ out, uint16_t* __restrict__ packed, const T* __restrict__ x, const T* __restrict__ gate,
                                                        const float* __restrict__ w, float eps, int cols, int n, int64_t x_stride, int64_t gate_stride, int64_t out_stride) {
    __shared__ float lds[4];
    const int64_t row = blockIdx.x;
    f32x8 v[CH], gt[CH];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        v[i] = gt[i] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (c < cols) {
            v[i] = act_ld8(x + row * x_stride + c);
            gt[i] = act_ld8(gate + row * gate_stride + c);
        }
        ss += sum4(v[i].a * v[i].a) + sum4(v[i].b * v[i].b);
    }
    const float inv = 1.f / sqrtf(block_sum256(ss, lds) / n + eps);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= cols) continue;
        f32x8 r = v[i];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            r.a[k] *= inv * w[c + k] * sigmoid_f(gt[i].a[k]);
            r.b[k] *= inv * w[c + 4 + k] * sigmoid_f(gt[i].b[k]);
        }
        if (packed) act_st8(packed + pack_index((int)row, c, cols), r);
        else act_st8(out + row * out_stride + c, r);
    }
}

template <int DK>
int walk_dk(const LightningArgs& a, hipStream_t stream) {
    constexpr size_t sum_lds = (size_t)C * (DK + VS) * 2, lds = sum_lds + (size_t)C * DK * 2 + (size_t)2 * C * PLD * 2;
    if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(lightning_walk_kernel<DK, false>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    const dim3 grid(a.n_chunks, a.heads, a.dv / VS);
    if (a.summaries) {
        lightning_walk_kernel<DK, true><<<grid, 256, sum_lds, stream>>>(a);
        int rc = check_launch("lightning summary");
        if (rc) return rc;
        const int64_t per = (int64_t)a.heads * a.dk * a.dv;
        lightning_starts_kernel<<<dim3((unsigned)((per + 255) / 256), a.n_chunks), 256, 0, stream>>>(a);
        rc = check_launch("lightning starts");
        if (rc) return rc;
    }
    lightning_walk_kernel<DK, false><<<grid, 256, lds, stream>>>(a);
    return check_launch("lightning walk");
}

template <typename T>
void norm_gate_t(void* out, void* packed, const void* x, const void* gate, const float* w, float eps, int rows, int cols, int n, int64_t xs, int64_t gs, int64_t os,
                 hipStream_t stream) {
    const int ch = (cols + 2047) / 2048;
    auto go = [&](auto k) {
        norm_gate_kernel<T, decltype(k)::value><<<rows, 256, 0, stream>>>((T*)out, (uint16_t*)packed, (const T*)x, (const T*)gate, w, eps, cols, n, xs, gs, os);
    };
    if (ch <= 1) go(std::integral_constant<int, 1>{});
    else if (ch <= 2) go(std::integral_constant<int, 2>{});
    else if (ch <= 4) go(std::integral_constant<int, 4>{});
    else if (ch <= 8) go(std::integral_constant<int, 8>{});
    else go(std::integral_constant<int, kRowPieces>{});
}

}  // namespace

bool lightning_supported(int dk, int dv) { return (dk == 64 || dk == 128 || dk == 256) && dv > 0 && dv % 64 == 0; }

int launch_lightning_chunks(const LightningArgs& a, int f32, int generic, hipStream_t stream) {
    if (!f32 && !generic && lightning_supported(a.dk, a.dv)) {
        switch (a.dk) {
            case 64: return walk_dk<64>(a, stream);
            case 128: return walk_dk<128>(a, stream);
            default: return walk_dk<256>(a, stream);
        }
    }
    const size_t lds = ((size_t)a.dk * 34 + 256) * 4;
    const dim3 grid(a.n_chunks, a.heads, (a.dv + 31) / 32);
    const void* fn = f32 ? reinterpret_cast<const void*>(lightning_generic_kernel<float>) : reinterpret_cast<const void*>(lightning_generic_kernel<uint16_t>);
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (f32) lightning_generic_kernel<float><<<grid, 256, lds, stream>>>(a);
    else lightning_generic_kernel<uint16_t><<<grid, 256, lds, stream>>>(a);
    return check_launch("lightning generic");
}

int launch_lightning_step(const LightningArgs& a, hipStream_t stream) {
    const bool wide = (int64_t)a.rows * a.heads * (a.dv / 64) >= 512;
    const size_t lds = (size_t)2 * a.dk * 4 + 1024 * 4;
    if (wide) lightning_step_kernel<64><<<dim3(a.heads, a.rows, a.dv / 64), 256, lds, stream>>>(a);
    else lightning_step_kernel<32><<<dim3(a.heads, a.rows, a.dv / 32), 256, lds, stream>>>(a);
    return check_launch("lightning step");
}

int launch_norm_gate(void* out, void* packed, const void* x, const void* gate, const float* w, float eps, int rows, int cols, int n, int64_t x_stride,
                     int64_t gate_stride, int64_t out_stride, int f32, hipStream_t stream) {
    if (f32) norm_gate_t<float>(out, nullptr, x, gate, w, eps, rows, cols, n, x_stride, gate_stride, out_stride, stream);
    else norm_gate_t<uint16_t>(out, packed, x, gate, w, eps, rows, cols, n, x_stride, gate_stride, out_stride, stream);
    return check_launch("norm_gate");
}

}  // namespace nvh
