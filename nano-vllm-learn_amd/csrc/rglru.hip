// Real-gated linear recurrent unit with a causal depthwise convolution in front of it:
//   u = conv(x)           y-branch gate applied at the end
//   r = sigmoid(ra u), i = sigmoid(ri u)            block-diagonal maps (MFMA)
//   log a = -rate r ; S = a S + sqrt(1 - a^2) i u ; out = S gelu(y)
// The recurrence and everything that enters it besides u is fp32; u is rounded once to the activation type.
//
// Prompt portions (launch_rglru_chunks): the host cuts a portion into segments; a workgroup owns one (segment, diagonal block) and walks the segment 64
// tokens at a time with the state in registers: convolution into LDS, both gates on MFMA tiles, and the scan of the 64 tokens IN the accumulator
// layout (a lane holds 4 consecutive tokens of one channel, the 4 lane groups 16 consecutive ones: compose 4 in the lane, two shuffles across the
// groups, a carry over the 16-token tiles), then S gelu(y) back out through LDS.
// A portion of one segment (many sequences at once) is one such walk.  Otherwise a SUMMARY walk first leaves (product of decays, end value) of every
// segment but the last, and the second walk of a segment starts from the composition of the ones before it.
// State and convolution ring are read by the walks and written by a small launch behind them: no workgroup can see a half-updated one.
// Decode (launch_rglru_step): one workgroup per 16 channels and 32 sequences does all of it in one launch.  Convolution inputs live in a ring of
// `taps` entries (input of position p at entry p % taps): the entry a step writes is the one no workgroup of that step reads.
// A sequence's first token (position 0) takes state and earlier inputs as zero instead of reading them: slots need no clearing when reused.
// Bytes per (token, channel) of a walk: 2 (x) + 2 (y) + 2 (out); about 50 vector instructions, 8 of them transcendental: issue-bound.
#include "hybrid.h"

namespace nvh {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
constexpr int CH = kRglruChunk;
constexpr int kGroup = 256;                          // channels one walking workgroup owns at most (16 waves x 16)

__device__ __forceinline__ float fast_sqrt(float x) { return __builtin_amdgcn_sqrtf(x); }
__device__ __forceinline__ float fast_sigmoid(float x) { return fast_rcp(1.f + fast_exp2(-kLog2e * x)); }
__device__ __forceinline__ float fast_gelu(float z) {
    const float t = (2.f * kLog2e * 0.7978845608028654f) * (z + 0.044715f * z * z * z);
    return z - z * fast_rcp(1.f + fast_exp2(t));
}
// decay a = exp(-rate r) and input sqrt(1 - a^2) i u; 1 - a^2 by its series where it would cancel
__device__ __forceinline__ void decay_and_input(float rate, float r, float ig, float u, float& a, float& b) {
    const float x = rate * r, y = 2.f * x;
    a = fast_exp2(-kLog2e * x);
    const float series = y * (1.f - y * (1.f / 2) * (1.f - y * (1.f / 3) * (1.f - y * (1.f / 4))));
    b = fast_sqrt(y < 0.06f ? series : 1.f - a * a) * ig * u;
}

// convolution input of the token `t` rows after the portion's first row (negative: before it, from the ring; before position 0: zero)
template <typename T>
__device__ __forceinline__ const T* conv_input(const RglruArgs& a, int seq_row0, int t, int64_t pos0, int slot, int ch) {
    if (t >= 0) return reinterpret_cast<const T*>(a.yx) + (int64_t)(seq_row0 + t) * a.yx_stride + a.width + ch;
    const int64_t p = pos0 + t;
    if (p < 0 || slot < 0) return nullptr;
    return reinterpret_cast<const T*>(a.conv_state) + ((int64_t)slot * a.taps + (int)(p % a.taps)) * a.width + ch;
}

__device__ __forceinline__ void fma8(float (&acc)[8], const u32x4 v, const float* w) {
    const f32x4 w0 = *reinterpret_cast<const f32x4*>(w), w1 = *reinterpret_cast<const f32x4*>(w + 4);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        const float wa = k < 2 ? w0[2 * k] : w1[2 * k - 4], wb = k < 2 ? w0[2 * k + 1] : w1[2 * k - 3];
        acc[2 * k] += wa * bf16_lo(v[k]);
        acc[2 * k + 1] += wb * bf16_hi(v[k]);
    }
}
__device__ __forceinline__ u32x4 pack8(const float (&v)[8]) {
    return u32x4{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7])};
}

// 8 channels x CNT consecutive tokens of the convolution; row(t) -> pointer of token t's input (null: zero).  Every input row is unpacked once.
template <int TAPS, int CNT, typename Row>
__device__ __forceinline__ void conv_run(const RglruArgs& a, int ch, int taps_rt, float (&acc)[CNT][8], Row row) {
    const f32x4 b0 = *reinterpret_cast<const f32x4*>(a.conv_b + ch), b1 = *reinterpret_cast<const f32x4*>(a.conv_b + ch + 4);
#pragma unroll
    for (int i = 0; i < CNT; ++i)
#pragma unroll
        for (int k = 0; k < 8; ++k) acc[i][k] = k < 4 ? b0[k] : b1[k - 4];
    if constexpr (TAPS > 0) {
        f32x4 w[TAPS][2];
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
            for (int q = 0; q < 2; ++q) w[j][q] = *reinterpret_cast<const f32x4*>(a.conv_w + (int64_t)j * a.width + ch + 4 * q);
        u32x4 v[CNT + TAPS - 1];
#pragma unroll
        for (int s = 0; s < CNT + TAPS - 1; ++s) {
            const uint16_t* p = row(s - (TAPS - 1));
            v[s] = p ? *reinterpret_cast<const u32x4*>(p) : u32x4{0, 0, 0, 0};
        }
#pragma unroll
        for (int s = 0; s < CNT + TAPS - 1; ++s)
#pragma unroll
            for (int k = 0; k < 8; ++k) {
                const float x = k & 1 ? bf16_hi(v[s][k >> 1]) : bf16_lo(v[s][k >> 1]);
#pragma unroll
                for (int i = 0; i < CNT; ++i)
                    if (s - i >= 0 && s - i < TAPS) acc[i][k] += w[s - i][k >> 2][k & 3] * x;
            }
    } else {
        for (int j = 0; j < taps_rt; ++j)
#pragma unroll
            for (int i = 0; i < CNT; ++i) {
                const uint16_t* p = row(i + j - (taps_rt - 1));
                if (p) fma8(acc[i], *reinterpret_cast<const u32x4*>(p), a.conv_w + (int64_t)j * a.width + ch);
            }
    }
}

// what a segment starts from (segment table index `seg`, channel ch)
__device__ __forceinline__ float walk_start(const RglruArgs& a, bool summary, bool more, int seg, int kth, int slot, int64_t pos0, int ch) {
    float cs = 0.f;
    if (kth == 0) {
        if (!summary && more) return a.a_cum[(int64_t)seg * a.width + ch];     // left there by the summary walk: the state itself is being replaced
        if (pos0 > 0 && slot >= 0) cs = a.state[(int64_t)slot * a.width + ch];
    } else if (!summary) {
        const int64_t first = (int64_t)(seg - kth) * a.width + ch;
        cs = a.s_loc[first];
        for (int k = 1; k < kth; ++k) cs = a.a_cum[first + (int64_t)k * a.width] * cs + a.s_loc[first + (int64_t)k * a.width];
    }
    return cs;
}

// ------------------------------------------------------------------------------------------------ prompt portions, MFMA form (bf16)
// grid (segments, blocks x channel groups of at most 256); a wave owns 16 channels
template <bool SUMMARY>
__global__ __launch_bounds__(1024) void rglru_walk_kernel(const RglruArgs a) {
    extern __shared__ __attribute__((aligned(16))) uint16_t u_lds[];           // [CH][block + 8] u; behind it [CH][group + 8] y, then out
    const int groups = (a.block + kGroup - 1) / kGroup, seg = blockIdx.x, blk = blockIdx.y / groups, g0 = (blockIdx.y - blk * groups) * kGroup;
    const int row0 = a.chunks[seg * 4], n = a.chunks[seg * 4 + 1], seq = a.chunks[seg * 4 + 2], kth = a.chunks[seg * 4 + 3];
    const bool more = seg + 1 < a.n_chunks && a.chunks[seg * 4 + 6] == seq;    // another segment of this sequence follows
    if (SUMMARY && !more) return;
    const int off0 = kth * a.segment, seq_row0 = row0 - off0;
    const int slot = a.state_slots[seq];
    const int64_t pos0 = a.positions[seq_row0];
    const int gcols = a.block - g0 < kGroup ? a.block - g0 : kGroup;           // this workgroup's channels of the block: g0 ..
    const int ld = a.block + 8, oct = a.block / 8, yld = gcols + 8, goct = gcols / 8;
    uint16_t* y_lds = u_lds + CH * ld;
    const int tid = threadIdx.x, threads = blockDim.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const uint16_t* yx = reinterpret_cast<const uint16_t*>(a.yx);
    const uint16_t* ra = reinterpret_cast<const uint16_t*>(a.ra) + (int64_t)blk * a.block * a.block;
    const uint16_t* ri = reinterpret_cast<const uint16_t*>(a.ri) + (int64_t)blk * a.block * a.block;
    const bool mine = 16 * wave < gcols;             // (a narrower last group leaves waves to the row work only)
    const int cg = mine ? 16 * wave + lq : lq, cb = g0 + cg, ch = blk * a.block + cb;
    const float rb = a.ra_b[ch], ib = a.ri_b[ch], rate = a.rate[ch];
    float ca = 1.f, cs = walk_start(a, SUMMARY, more, seg, kth, slot, pos0, ch);
    if (SUMMARY && kth == 0 && mine && lg == 0) a.a_cum[(int64_t)seg * a.width + ch] = cs;
    const int pairs = CH / 2 * oct;
    for (int t0 = 0; t0 < n; t0 += CH) {
        const int cnt = n - t0 < CH ? n - t0 : CH;
        // ---- u into LDS, two tokens x 8 channels a time; y beside it
        const bool inside = off0 + t0 >= a.taps - 1;                           // no tap reaches in front of the portion
        for (int e = tid; e < pairs; e += threads) {
            const int tp = e / oct, o = e - tp * oct, t = 2 * tp, c8 = blk * a.block + o * 8;
            u32x4 r0 = {0, 0, 0, 0}, r1 = {0, 0, 0, 0};
            if (t < cnt) {
                float acc[2][8];
                const int at = off0 + t0 + t;
                const uint16_t* base = yx + (int64_t)(seq_row0 + at) * a.yx_stride + a.width + c8;
                const int last = t + 1 < cnt ? 1 : 0;                          // (an odd tail repeats its last row: not used)
                if (inside && a.taps == 4)
                    conv_run<4, 2>(a, c8, 4, acc, [&](int s) { return base + (int64_t)(s < last ? s : last) * a.yx_stride; });
                else
                    conv_run<0, 2>(a, c8, a.taps, acc, [&](int s) { return conv_input<uint16_t>(a, seq_row0, at + (s < last ? s : last), pos0, slot, c8); });
                r0 = pack8(acc[0]);
                if (last) r1 = pack8(acc[1]);
            }
            *reinterpret_cast<u32x4*>(u_lds + t * ld + o * 8) = r0;
            *reinterpret_cast<u32x4*>(u_lds + (t + 1) * ld + o * 8) = r1;
        }
        if (!SUMMARY)
            for (int e = tid; e < cnt * goct; e += threads) {
                const int t = e / goct, o = e - t * goct;
                *reinterpret_cast<u32x4*>(y_lds + t * yld + o * 8) =
                    *reinterpret_cast<const u32x4*>(yx + (int64_t)(row0 + t0 + t) * a.yx_stride + blk * a.block + g0 + o * 8);
            }
        __syncthreads();
        if (mine) {
            f32x4 gr[4], gi[4];
#pragma unroll
            for (int m = 0; m < 4; ++m) gr[m] = gi[m] = f32x4{0.f, 0.f, 0.f, 0.f};
            const uint16_t* wr = ra + (int64_t)cb * a.block + 8 * lg;
            const uint16_t* wi = ri + (int64_t)cb * a.block + 8 * lg;
            bf16x8 br = *reinterpret_cast<const bf16x8*>(wr), bi = *reinterpret_cast<const bf16x8*>(wi);
            for (int k = 0; k < a.block; k += 32) {
                const int kn = k + 32 < a.block ? k + 32 : k;                  // the next step's weights travel under this one's products
                const bf16x8 nr = *reinterpret_cast<const bf16x8*>(wr + kn), ni = *reinterpret_cast<const bf16x8*>(wi + kn);
#pragma unroll
                for (int m = 0; m < 4; ++m) {
                    const bf16x8 ua = *reinterpret_cast<const bf16x8*>(u_lds + (16 * m + lq) * ld + k + 8 * lg);
                    gr[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, br, gr[m], 0, 0, 0);
                    gi[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, bi, gi[m], 0, 0, 0);
                }
                br = nr;
                bi = ni;
            }
            // ---- decays, inputs and the scan: this lane holds tokens 16 m + 4 lg + i of one channel
#pragma unroll
            for (int m = 0; m < 4; ++m) {
                if (16 * m >= cnt) break;
                float av[4], sv[4];
                float pa = 1.f, ps = 0.f;                                      // inclusive composition over the lane's 4 tokens
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = 16 * m + 4 * lg + i;
                    float dec, inp;
                    decay_and_input(rate, fast_sigmoid(gr[m][i] + rb), fast_sigmoid(gi[m][i] + ib), act_ld(u_lds + t * ld + cb), dec, inp);
                    if (t >= cnt) dec = 1.f, inp = 0.f;
                    ps = dec * ps + inp;
                    pa *= dec;
                    av[i] = pa;
                    sv[i] = ps;
                }
                float ga = pa, gs = ps;                                        // inclusive over the lane groups so far
                {
                    const float oa = __shfl_up(ga, 16), os = __shfl_up(gs, 16);
                    if (lg >= 1) { gs = ga * os + gs; ga *= oa; }
                }
                {
                    const float oa = __shfl_up(ga, 32), os = __shfl_up(gs, 32);
                    if (lg >= 2) { gs = ga * os + gs; ga *= oa; }
                }
                if (!SUMMARY) {
                    float xa = __shfl_up(ga, 16), xs = __shfl_up(gs, 16);
                    if (lg == 0) { xa = 1.f; xs = 0.f; }
                    const float before = xa * cs + xs;                      // the state in front of this lane's first token
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        uint16_t* p = y_lds + (16 * m + 4 * lg + i) * yld + cg;
                        act_st(p, (av[i] * before + sv[i]) * fast_gelu(act_ld(p)));
                    }
                }
                const float ta = __shfl(ga, 48 + lq), ts = __shfl(gs, 48 + lq);    // the whole tile
                cs = ta * cs + ts;
                ca *= ta;
            }
        }
        __syncthreads();
        if (!SUMMARY)
            for (int e = tid; e < cnt * goct; e += threads) {
                const int t = e / goct, o = e - t * goct;
                *reinterpret_cast<u32x4*>(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(row0 + t0 + t) * a.out_stride + blk * a.block + g0 + o * 8) =
                    *reinterpret_cast<const u32x4*>(y_lds + t * yld + o * 8);
            }
        // (the next tokens' y goes where these rows were read from: same threads, same places)
    }
    if (mine && lg == 0 && (SUMMARY || !more)) {
        a.s_loc[(int64_t)seg * a.width + ch] = cs;
        if (SUMMARY && kth) a.a_cum[(int64_t)seg * a.width + ch] = ca;
    }
}

// ------------------------------------------------------------------------------------------------ prompt portions, blocks of up to 256 channels
// The same walk with everything in flight early: x of the next 64 tokens and y of these travel by LDS-DMA under this step's arithmetic, both gates' weights
// of a wave's channels stay in registers for the whole segment (8 waves, 16 or 32 channels each), and u and y come into the accumulator layout through an
// MFMA with a 0/1 selection matrix (exact) instead of single-element LDS reads.
constexpr int HALO = 8;                              // rows in front of a step's 64 in the x image: taps <= HALO + 1

__device__ __forceinline__ void lds_barrier() {      // (a __syncthreads() would drain the DMA in flight)
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}

template <int KS> constexpr size_t scan_x_bytes() { return (size_t)(CH + HALO) * KS * 64 + 1024; }     // (the last DMA instruction may run over)
template <int KS> constexpr size_t scan_lds_bytes(int taps) {
    return 2 * scan_x_bytes<KS>() + (size_t)CH * (KS * 32 + 8) * 2 + (size_t)CH * KS * 64 + (size_t)(taps + 1) * KS * 128;
}

template <int KS, bool SUMMARY>                      // block = 32 KS
__global__ __launch_bounds__(512) void rglru_scan_kernel(const RglruArgs a) {
    constexpr int BLOCK = 32 * KS, OCT = 4 * KS, TILES = 2 * KS, NTW = (TILES + 7) / 8, LD = BLOCK + 8;
    constexpr int SWZ = OCT % 8 == 0 ? 7 : 3;        // y image: piece p of row r sits at p ^ (r & SWZ)
    constexpr int XINS = ((CH + HALO) * OCT + 63) / 64, YINS = OCT;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    uint16_t* x_lds = reinterpret_cast<uint16_t*>(smem);                       // [2][HALO + CH][BLOCK]
    constexpr int XBUF = scan_x_bytes<KS>() / 2;
    uint16_t* u_lds = x_lds + 2 * XBUF;                                        // [CH][LD]
    uint16_t* y_lds = u_lds + CH * LD;                                         // [CH][BLOCK] swizzled; out after the scan
    float* w_lds = reinterpret_cast<float*>(y_lds + CH * BLOCK);               // [taps + 1][BLOCK]: taps, then the bias
    const int seg = blockIdx.x, blk = blockIdx.y, c0 = blk * BLOCK;
    const int row0 = a.chunks[seg * 4], n = a.chunks[seg * 4 + 1], seq = a.chunks[seg * 4 + 2], kth = a.chunks[seg * 4 + 3];
    const bool more = seg + 1 < a.n_chunks && a.chunks[seg * 4 + 6] == seq;
    if (SUMMARY && !more) return;
    const int off0 = kth * a.segment, seq_row0 = row0 - off0;
    const int slot = a.state_slots[seq];
    const int64_t pos0 = a.positions[seq_row0];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const uint16_t* yx = reinterpret_cast<const uint16_t*>(a.yx);
    const uint16_t* xcol = yx + a.width + c0;
    auto dma = [&](const uint16_t* src, void* dst) {
        __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src, (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
    };
    auto stage_x = [&](int t0, int buf) {            // rows t0 - HALO .. t0 + CH - 1 of the segment, clamped to the portion's rows that exist
        const int lo = -off0, hi = n - 1;
#pragma unroll
        for (int j = 0; j < (XINS + 7) / 8; ++j) {
            const int ins = wave + 8 * j;
            if (ins < XINS) {
                const int s = ins * 64 + lane;
                int t = t0 - HALO + s / OCT;
                t = t < lo ? lo : (t > hi ? hi : t);
                dma(xcol + (int64_t)(row0 + t) * a.yx_stride + (s % OCT) * 8, x_lds + buf * XBUF + ins * 512);
            }
        }
    };
    auto stage_y = [&](int t0) {
#pragma unroll
        for (int j = 0; j < (YINS + 7) / 8; ++j) {
            const int ins = wave + 8 * j;
            if (ins < YINS) {
                const int s = ins * 64 + lane, r = s / OCT, t = t0 + r < n ? t0 + r : n - 1;
                dma(yx + (int64_t)(row0 + t) * a.yx_stride + c0 + ((s % OCT) ^ (r & SWZ)) * 8, y_lds + ins * 512);
            }
        }
    };
    stage_x(0, 0);
    for (int e = tid; e < (a.taps + 1) * BLOCK; e += 512) w_lds[e] = e < a.taps * BLOCK ? a.conv_w[(int64_t)(e / BLOCK) * a.width + c0 + e % BLOCK] : a.conv_b[c0 + e % BLOCK];

    // ---- this wave's channels: 16-channel tiles wave, wave + 8
    bf16x8 wr[NTW][KS], wi[NTW][KS], sel;
    float ca[NTW], cs[NTW], rb[NTW], ib[NTW], rate[NTW];
    {
        u32x4 one;                                   // 1.0 where this lane's k-slot is its own channel (tiles wave and wave + 8: the same half of a k-step)
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int want = 16 * (wave & 1) + lq - 8 * lg - 2 * k;
            one[k] = want == 0 ? 0x3F80u : (want == 1 ? 0x3F800000u : 0u);
        }
        sel = __builtin_bit_cast(bf16x8, one);
    }
#pragma unroll
    for (int j = 0; j < NTW; ++j) {
        const int nt = wave + 8 * j < TILES ? wave + 8 * j : 0, cb = 16 * nt + lq, ch = c0 + cb;
        const uint16_t* pr = reinterpret_cast<const uint16_t*>(a.ra) + ((int64_t)c0 + cb) * BLOCK + 8 * lg;
        const uint16_t* pi = reinterpret_cast<const uint16_t*>(a.ri) + ((int64_t)c0 + cb) * BLOCK + 8 * lg;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            wr[j][k] = *reinterpret_cast<const bf16x8*>(pr + 32 * k);
            wi[j][k] = *reinterpret_cast<const bf16x8*>(pi + 32 * k);
        }
        rb[j] = -kLog2e * a.ra_b[ch], ib[j] = -kLog2e * a.ri_b[ch], rate[j] = a.rate[ch];
        ca[j] = 1.f;
        cs[j] = walk_start(a, SUMMARY, more, seg, kth, slot, pos0, ch);
        if (SUMMARY && kth == 0 && wave + 8 * j < TILES && lg == 0) a.a_cum[(int64_t)seg * a.width + ch] = cs[j];
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    lds_barrier();
    if (off0 == 0)                                   // inputs in front of the portion: from the ring, zero in front of the sequence
        for (int e = tid; e < (a.taps - 1) * OCT; e += 512) {
            const int back = e / OCT + 1, o = e % OCT;
            const uint16_t* p = conv_input<uint16_t>(a, seq_row0, -back, pos0, slot, c0 + o * 8);
            *reinterpret_cast<u32x4*>(x_lds + (HALO - back) * BLOCK + o * 8) = p ? *reinterpret_cast<const u32x4*>(p) : u32x4{0, 0, 0, 0};
        }

    for (int t0 = 0, buf = 0; t0 < n; t0 += CH, buf ^= 1) {
        const int cnt = n - t0 < CH ? n - t0 : CH;
        // x of this step was asked for a step ago; only that step's own stores were issued behind it (vector-memory operations complete in order)
        if (t0 > 0) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(SUMMARY ? 0 : KS / 2) : "memory");
        lds_barrier();                               // x is in LDS for everyone; the last step's reads of u and y are done
        if (!SUMMARY) stage_y(t0);
        if (t0 + CH < n) stage_x(t0 + CH, buf ^ 1);
        // ---- u, four tokens x 8 channels a time
        const uint16_t* xs = x_lds + buf * XBUF;
        for (int e = tid; e < CH / 4 * OCT; e += 512) {
            const int t = 4 * (e / OCT), o = e % OCT;
            const float* wp = w_lds + o * 8;
            float acc[4][8];
            {
                const f32x4 b0 = *reinterpret_cast<const f32x4*>(wp + a.taps * BLOCK), b1 = *reinterpret_cast<const f32x4*>(wp + a.taps * BLOCK + 4);
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int k = 0; k < 8; ++k) acc[i][k] = k < 4 ? b0[k] : b1[k - 4];
            }
            const uint16_t* xp = xs + (HALO + t - (a.taps - 1)) * BLOCK + o * 8;
            if (a.taps == 4) {
                u32x4 v[7];
#pragma unroll
                for (int j = 0; j < 7; ++j) v[j] = *reinterpret_cast<const u32x4*>(xp + j * BLOCK);
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int i = 0; i < 4; ++i) fma8(acc[i], v[i + j], wp + j * BLOCK);
            } else {
                for (int j = 0; j < a.taps; ++j)
#pragma unroll
                    for (int i = 0; i < 4; ++i) fma8(acc[i], *reinterpret_cast<const u32x4*>(xp + (i + j) * BLOCK), wp + j * BLOCK);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) *reinterpret_cast<u32x4*>(u_lds + (t + i) * LD + o * 8) = pack8(acc[i]);
        }
        lds_barrier();
#pragma unroll 1
        for (int tm = 0; tm < CH; tm += 16) {        // 16 tokens at a time
            if (tm > 0 && tm >= cnt) break;
            f32x4 gr[NTW], gi[NTW];
#pragma unroll
            for (int j = 0; j < NTW; ++j) gr[j] = gi[j] = f32x4{0.f, 0.f, 0.f, 0.f};
            const uint16_t* u_row = u_lds + (tm + lq) * LD + 8 * lg;
#pragma unroll
            for (int k = 0; k < KS; ++k) {
                const bf16x8 ua = *reinterpret_cast<const bf16x8*>(u_row + 32 * k);
#pragma unroll
                for (int j = 0; j < NTW; ++j) {
                    gr[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, wr[j][k], gr[j], 0, 0, 0);
                    gi[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, wi[j][k], gi[j], 0, 0, 0);
                }
            }
            if (!SUMMARY && tm == 0) {               // y of this step is in LDS; x of the next may still travel
                if (t0 + CH < n) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(XINS / 8) : "memory");
                else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
                lds_barrier();
            }
#pragma unroll
            for (int j = 0; j < NTW; ++j) {
                if (wave + 8 * j >= TILES) break;
                const int nt = wave + 8 * j, cb = 16 * nt + lq, r = tm + lq;
                const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
                const f32x4 uu = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(u_row + 32 * (nt >> 1)), sel, zero, 0, 0, 0);
                f32x4 yv = zero;
                if (!SUMMARY)
                    yv = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(y_lds + r * BLOCK + (((nt >> 1) * 4 + lg) ^ (r & SWZ)) * 8), sel, zero,
                                                                 0, 0, 0);
                float av[4], sv[4];
                float pa = 1.f, ps = 0.f;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float rg = fast_rcp(1.f + fast_exp2(gr[j][i] * -kLog2e + rb[j])), ig = fast_rcp(1.f + fast_exp2(gi[j][i] * -kLog2e + ib[j]));
                    float dec, inp;
                    decay_and_input(rate[j], rg, ig, uu[i], dec, inp);
                    if (tm + 4 * lg + i >= cnt) dec = 1.f, inp = 0.f;
                    ps = dec * ps + inp;
                    pa *= dec;
                    av[i] = pa;
                    sv[i] = ps;
                }
                // across the four lane groups (4 tokens each): e = the even group of the pair, then both pairs' totals to everyone
                const auto swap16 = [](float v) { return __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false); };
                const auto swap32 = [](float v) { return __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false); };
                const bool odd = lg & 1;
                const float ea = __uint_as_float(swap16(pa)[0]), es = __uint_as_float(swap16(ps)[0]);
                const float ia = odd ? pa * ea : pa, is = odd ? pa * es + ps : ps;                  // inclusive inside the pair
                const auto ha = swap32(__uint_as_float(swap16(ia)[1])), hs = swap32(__uint_as_float(swap16(is)[1]));
                const float la = __uint_as_float(ha[0]), ls = __uint_as_float(hs[0]), ua_ = __uint_as_float(ha[1]), us_ = __uint_as_float(hs[1]);
                if (!SUMMARY) {
                    float before = lg >= 2 ? la * cs[j] + ls : cs[j];
                    before = odd ? ea * before + es : before;                                       // the state in front of this lane's first token
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const int ro = tm + 4 * lg + i;
                        act_st(y_lds + ro * BLOCK + ((cb >> 3) ^ (ro & SWZ)) * 8 + (cb & 7), (av[i] * before + sv[i]) * fast_gelu(yv[i]));
                    }
                }
                cs[j] = ua_ * (la * cs[j] + ls) + us_;
                ca[j] *= la * ua_;
            }
        }
        if (!SUMMARY) {
            lds_barrier();
            for (int e = tid; e < cnt * OCT; e += 512) {
                const int r = e / OCT, p = e % OCT;
                *reinterpret_cast<u32x4*>(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(row0 + t0 + r) * a.out_stride + c0 + p * 8) =
                    *reinterpret_cast<const u32x4*>(y_lds + r * BLOCK + (p ^ (r & SWZ)) * 8);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < NTW; ++j) {
        const int nt = wave + 8 * j, ch = c0 + 16 * nt + lq;
        if (nt < TILES && lg == 0 && (SUMMARY || !more)) {
            a.s_loc[(int64_t)seg * a.width + ch] = cs[j];
            if (SUMMARY && kth) a.a_cum[(int64_t)seg * a.width + ch] = ca[j];
        }
    }
}

// ------------------------------------------------------------------------------------------------ prompt portions, any type and size
// one workgroup per (segment, 64 channels of a diagonal block): gates by plain dot products over LDS tiles, scan by one thread per channel
template <typename T, bool SUMMARY>
__global__ __launch_bounds__(256) void rglru_walk_generic_kernel(const RglruArgs a) {
    constexpr int KT = 32;
    __shared__ float u_t[CH][KT + 1];
    __shared__ float wr_t[64][KT + 1], wi_t[64][KT + 1];
    __shared__ float dec[CH][65], inp[CH][65];
    const int seg = blockIdx.x;
    const int tiles = (a.block + 63) / 64, blk = blockIdx.y / tiles, n0 = (blockIdx.y % tiles) * 64;
    const int row0 = a.chunks[seg * 4], n = a.chunks[seg * 4 + 1], seq = a.chunks[seg * 4 + 2], kth = a.chunks[seg * 4 + 3];
    const bool more = seg + 1 < a.n_chunks && a.chunks[seg * 4 + 6] == seq;
    if (SUMMARY && !more) return;
    const int off0 = kth * a.segment, seq_row0 = row0 - off0;
    const int slot = a.state_slots[seq];
    const int64_t pos0 = a.positions[seq_row0];
    const T* ra = reinterpret_cast<const T*>(a.ra) + (int64_t)blk * a.block * a.block;
    const T* ri = reinterpret_cast<const T*>(a.ri) + (int64_t)blk * a.block * a.block;
    const int tid = threadIdx.x, c = tid & 63, tq = tid >> 6;
    const int ch = blk * a.block + n0 + c;
    const bool live = n0 + c < a.block;
    auto conv_at = [&](int t, int cc) {              // t: tokens behind the segment's first
        float s = a.conv_b[cc];
        for (int j = 0; j < a.taps; ++j) {
            const T* p = conv_input<T>(a, seq_row0, off0 + t - (a.taps - 1) + j, pos0, slot, cc);
            if (p) s += a.conv_w[(int64_t)j * a.width + cc] * act_ld(p);
        }
        return act_round(s, (const T*)nullptr);
    };
    float ca = 1.f, cs = live ? walk_start(a, SUMMARY, more, seg, kth, slot, pos0, ch) : 0.f;
    if (SUMMARY && kth == 0 && live && tid < 64) a.a_cum[(int64_t)seg * a.width + ch] = cs;
    for (int t0 = 0; t0 < n; t0 += CH) {
        const int cnt = n - t0 < CH ? n - t0 : CH;
        float gr[16], gi[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) gr[i] = gi[i] = 0.f;
        for (int k0 = 0; k0 < a.block; k0 += KT) {
            for (int e = tid; e < CH * KT; e += 256) {
                const int t = e / KT, k = e % KT;
                u_t[t][k] = t < cnt ? conv_at(t0 + t, blk * a.block + k0 + k) : 0.f;
            }
            for (int e = tid; e < 64 * KT; e += 256) {
                const int o = e / KT, k = e % KT;
                const bool ok = n0 + o < a.block;
                wr_t[o][k] = ok ? act_ld(ra + (int64_t)(n0 + o) * a.block + k0 + k) : 0.f;
                wi_t[o][k] = ok ? act_ld(ri + (int64_t)(n0 + o) * a.block + k0 + k) : 0.f;
            }
            __syncthreads();
            for (int k = 0; k < KT; ++k) {
                const float wr = wr_t[c][k], wi = wi_t[c][k];
#pragma unroll
                for (int i = 0; i < 16; ++i) {
                    const float u = u_t[tq * 16 + i][k];
                    gr[i] += wr * u;
                    gi[i] += wi * u;
                }
            }
            __syncthreads();
        }
        if (live) {
            const float rb = a.ra_b[ch], ib = a.ri_b[ch], rate = a.rate[ch];
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int t = tq * 16 + i;
                if (t < cnt) {
                    // (accurate exponentials: this form also serves the true fp32 model)
                    const float r = 1.f / (1.f + expf(-(gr[i] + rb))), ig = 1.f / (1.f + expf(-(gi[i] + ib)));
                    const float log_a = -rate * r;
                    dec[t][c] = expf(log_a);
                    inp[t][c] = sqrtf(-expm1f(2.f * log_a)) * ig * conv_at(t0 + t, ch);
                }
            }
        }
        __syncthreads();
        if (tid < 64 && live)
            for (int t = 0; t < cnt; ++t) {
                cs = dec[t][c] * cs + inp[t][c];
                ca *= dec[t][c];
                inp[t][c] = cs;
            }
        __syncthreads();
        if (!SUMMARY && live)
            for (int t = tq; t < cnt; t += 4) {
                const float y = act_ld(reinterpret_cast<const T*>(a.yx) + (int64_t)(row0 + t0 + t) * a.yx_stride + ch);
                act_st(reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t0 + t) * a.out_stride + ch, inp[t][c] * gelu_tanh_f(y));
            }
        __syncthreads();
    }
    if (tid < 64 && live && (SUMMARY || !more)) {
        a.s_loc[(int64_t)seg * a.width + ch] = cs;
        if (SUMMARY && kth) a.a_cum[(int64_t)seg * a.width + ch] = ca;
    }
}

// behind the walks: every sequence's last segment hands its end value to the state and the portion's last inputs to the ring
template <typename T>
__global__ __launch_bounds__(256) void rglru_keep_kernel(const RglruArgs a) {
    const int seg = blockIdx.x, ch = (blockIdx.y * 256 + threadIdx.x) * 4;
    const int row0 = a.chunks[seg * 4], n = a.chunks[seg * 4 + 1], seq = a.chunks[seg * 4 + 2], kth = a.chunks[seg * 4 + 3];
    const int slot = a.state_slots[seq];
    if (ch >= a.width || slot < 0 || (seg + 1 < a.n_chunks && a.chunks[seg * 4 + 6] == seq)) return;
    *reinterpret_cast<f32x4*>(a.state + (int64_t)slot * a.width + ch) = *reinterpret_cast<const f32x4*>(a.s_loc + (int64_t)seg * a.width + ch);
    const int portion = kth * a.segment + n, keep = portion < a.taps ? portion : a.taps;
    for (int j = 0; j < keep; ++j) {
        const int row = row0 + n - 1 - j;
        act_st4(reinterpret_cast<T*>(a.conv_state) + ((int64_t)slot * a.taps + (int)(a.positions[row] % a.taps)) * a.width + ch,
                act_ld4(reinterpret_cast<const T*>(a.yx) + (int64_t)row * a.yx_stride + a.width + ch));
    }
}

// ------------------------------------------------------------------------------------------------ one token per sequence (bf16)
// grid (width / 16 channel tiles, 32-row tiles); the 4 waves split the contraction over the diagonal block and add up through LDS.
// Everything whose address needs no result of this launch (gate weights, states, y) is asked for before the convolution.
template <int KW>                                    // contraction steps of 32 per wave held in registers (0: a loop)
__global__ __launch_bounds__(256) void rglru_step_kernel(const RglruArgs a, const int rows) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int per = a.block / 16, blk = blockIdx.x / per, nt = blockIdx.x % per;
    const int r0 = blockIdx.y * 32, nr = rows - r0 < 32 ? rows - r0 : 32;
    const int ld = a.block + 8, oct = a.block / 8, ksteps = a.block / 32;
    uint16_t* u_lds = reinterpret_cast<uint16_t*>(smem);                        // [32][block + 8]
    f32x4* red = reinterpret_cast<f32x4*>(smem + 32 * ld * 2);                  // [wave][2 gates x 2 row tiles][64 lanes]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const uint16_t* yx = reinterpret_cast<const uint16_t*>(a.yx);
    const uint16_t* wr = reinterpret_cast<const uint16_t*>(a.ra) + ((int64_t)blk * a.block + 16 * nt + lq) * a.block + 8 * lg;
    const uint16_t* wi = reinterpret_cast<const uint16_t*>(a.ri) + ((int64_t)blk * a.block + 16 * nt + lq) * a.block + 8 * lg;
    bf16x8 br[KW > 0 ? KW : 1], bi[KW > 0 ? KW : 1];
#pragma unroll
    for (int k = 0; k < KW; ++k) {
        const int ks = wave + 4 * k < ksteps ? wave + 4 * k : 0;
        br[k] = *reinterpret_cast<const bf16x8*>(wr + 32 * ks);
        bi[k] = *reinterpret_cast<const bf16x8*>(wi + 32 * ks);
    }
    // this thread's two outputs: (row tile m, lane of the C layout, half of its 4 rows)
    const int m = tid >> 7, cl = (tid >> 1) & 63, half = tid & 1;
    const int cb = 16 * nt + (cl & 15), ch0 = blk * a.block + cb;
    int slot[2];
    int64_t pos[2];
    float old[2], yv[2];
    uint16_t xin[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int row = 16 * m + 4 * (cl >> 4) + 2 * half + i, rc = r0 + (row < nr ? row : 0);
        slot[i] = a.state_slots[rc];
        pos[i] = a.positions[rc];
        yv[i] = act_ld(yx + (int64_t)rc * a.yx_stride + ch0);
        xin[i] = yx[(int64_t)rc * a.yx_stride + a.width + ch0];
        old[i] = slot[i] >= 0 ? a.state[(int64_t)slot[i] * a.width + ch0] : 0.f;
        if (pos[i] <= 0) old[i] = 0.f;
    }
    const float rb = a.ra_b[ch0], ib = a.ri_b[ch0], rate = a.rate[ch0];
    for (int e = tid; e < 32 * oct; e += 256) {
        const int row = e / oct, o = e - row * oct;
        u32x4 packed = {0, 0, 0, 0};
        if (row < nr) {
            const int sl = a.state_slots[r0 + row], ch = blk * a.block + o * 8;
            const int64_t ps = a.positions[r0 + row];
            float acc[1][8];
            auto in = [&](int s) { return conv_input<uint16_t>(a, r0 + row, s, ps, sl, ch); };
            if (a.taps == 4) conv_run<4, 1>(a, ch, 4, acc, in);
            else conv_run<0, 1>(a, ch, a.taps, acc, in);
            packed = pack8(acc[0]);
        }
        *reinterpret_cast<u32x4*>(u_lds + row * ld + o * 8) = packed;
    }
    __syncthreads();
    f32x4 g[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) g[q] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto product = [&](int ks, const bf16x8 wr_k, const bf16x8 wi_k) {
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const bf16x8 ua = *reinterpret_cast<const bf16x8*>(u_lds + (16 * q + lq) * ld + 32 * ks + 8 * lg);
            g[q] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, wr_k, g[q], 0, 0, 0);
            g[2 + q] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, wi_k, g[2 + q], 0, 0, 0);
        }
    };
    if constexpr (KW > 0) {
#pragma unroll
        for (int k = 0; k < KW; ++k)
            if (wave + 4 * k < ksteps) product(wave + 4 * k, br[k], bi[k]);
    } else {
        for (int ks = wave; ks < ksteps; ks += 4) product(ks, *reinterpret_cast<const bf16x8*>(wr + 32 * ks), *reinterpret_cast<const bf16x8*>(wi + 32 * ks));
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) red[(wave * 4 + q) * 64 + lane] = g[q];
    __syncthreads();
    f32x4 sr = {0.f, 0.f, 0.f, 0.f}, si = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
        sr += red[(w * 4 + m) * 64 + cl];
        si += red[(w * 4 + 2 + m) * 64 + cl];
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int row = 16 * m + 4 * (cl >> 4) + 2 * half + i;
        if (row >= nr) continue;
        float dec, inp;
        decay_and_input(rate, fast_sigmoid((half ? sr[2 + i] : sr[i]) + rb), fast_sigmoid((half ? si[2 + i] : si[i]) + ib), act_ld(u_lds + row * ld + cb), dec, inp);
        const float s = dec * old[i] + inp;
        if (slot[i] >= 0) {
            a.state[(int64_t)slot[i] * a.width + ch0] = s;
            reinterpret_cast<uint16_t*>(a.conv_state)[((int64_t)slot[i] * a.taps + (int)(pos[i] % a.taps)) * a.width + ch0] = xin[i];
        }
        const float o = s * fast_gelu(yv[i]);
        if (a.out) act_st(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(r0 + row) * a.out_stride + ch0, o);
        if (a.out_packed) act_st(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(r0 + row, ch0, a.width), o);
    }
}

constexpr size_t kMaxLds = 160 * 1024;
size_t walk_lds(int block) { return (size_t)CH * ((block + 8) + ((block < kGroup ? block : kGroup) + 8)) * 2; }
size_t step_lds(int block) { return (size_t)32 * (block + 8) * 2 + 16 * 64 * sizeof(f32x4); }
template <bool SUMMARY, int KS>
bool scan_ks(const RglruArgs& a, hipStream_t stream) {
    const size_t lds = scan_lds_bytes<KS>(a.taps);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rglru_scan_kernel<KS, SUMMARY>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
    rglru_scan_kernel<KS, SUMMARY><<<dim3(a.n_chunks, a.blocks), 512, lds, stream>>>(a);
    return true;
}
template <bool SUMMARY>
bool scan(const RglruArgs& a, hipStream_t stream) {
    if (a.taps > HALO + 1 || scan_lds_bytes<8>(a.taps) > kMaxLds) return false;
    switch (a.block / 32) {
        case 1: return scan_ks<SUMMARY, 1>(a, stream);
        case 2: return scan_ks<SUMMARY, 2>(a, stream);
        case 3: return scan_ks<SUMMARY, 3>(a, stream);
        case 4: return scan_ks<SUMMARY, 4>(a, stream);
        case 5: return scan_ks<SUMMARY, 5>(a, stream);
        case 6: return scan_ks<SUMMARY, 6>(a, stream);
        case 7: return scan_ks<SUMMARY, 7>(a, stream);
        case 8: return scan_ks<SUMMARY, 8>(a, stream);
        default: return false;
    }
}

template <bool SUMMARY>
int walk(const RglruArgs& a, int f32, int generic, hipStream_t stream) {
    const size_t lds = walk_lds(a.block);
    if (f32 || generic == 1 || lds > kMaxLds) {
        const dim3 grid(a.n_chunks, a.blocks * ((a.block + 63) / 64));
        if (f32) rglru_walk_generic_kernel<float, SUMMARY><<<grid, 256, 0, stream>>>(a);
        else rglru_walk_generic_kernel<uint16_t, SUMMARY><<<grid, 256, 0, stream>>>(a);
    } else if (generic == 2 || !scan<SUMMARY>(a, stream)) {
        const int waves = a.block < kGroup ? a.block / 16 : kGroup / 16;
        if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rglru_walk_kernel<SUMMARY>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
        rglru_walk_kernel<SUMMARY><<<dim3(a.n_chunks, a.blocks * ((a.block + kGroup - 1) / kGroup)), waves * 64, lds, stream>>>(a);
    }
    return check_launch("rglru_walk");
}

template <int KW>
void step_kw(const RglruArgs& a, int rows, hipStream_t stream) {
    const size_t lds = step_lds(a.block);
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rglru_step_kernel<KW>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
    rglru_step_kernel<KW><<<dim3(a.blocks * (a.block / 16), (rows + 31) / 32), 256, lds, stream>>>(a, rows);
}

}  // namespace

bool rglru_step_supported(int block) { return step_lds(block) <= kMaxLds; }

int launch_rglru_chunks(const RglruArgs& a, int f32, int generic, hipStream_t stream) {
    if (a.n_chunks == 0) return 0;
    int rc = a.summaries ? walk<true>(a, f32, generic, stream) : 0;
    if (!rc) rc = walk<false>(a, f32, generic, stream);
    if (rc) return rc;
    const dim3 grid(a.n_chunks, (a.width / 4 + 255) / 256);
    if (f32) rglru_keep_kernel<float><<<grid, 256, 0, stream>>>(a);
    else rglru_keep_kernel<uint16_t><<<grid, 256, 0, stream>>>(a);
    return check_launch("rglru_keep");
}

int launch_rglru_step(const RglruArgs& a, int rows, hipStream_t stream) {
    if (a.block <= 128) step_kw<1>(a, rows, stream);
    else if (a.block <= 256) step_kw<2>(a, rows, stream);
    else if (a.block <= 512) step_kw<4>(a, rows, stream);
    else step_kw<0>(a, rows, stream);
    return check_launch("rglru_step");
}

}  // namespace nvh
