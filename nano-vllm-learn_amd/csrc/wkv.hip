// Time mixing with a matrix state per head whose rows decay by their own factor at every token:
//   o_t = (S + diag(u) k_t v_t^T)^T r_t          S <- diag(w_t) S + k_t v_t^T          w_t = exp(-exp(z_t + w0))
// and behind it, per head: o / rms(o) * norm * silu(gate).  State, decays and everything between z and the weights are fp32.
//
// Prompt portions (launch_wkv_chunks): a workgroup owns one (segment, head) and takes 64 tokens at a time.  With L the running sum of the log decays over the
// chunk and m its value behind the first 32 tokens,
//   r~_t = r_t e^(L_(t-1) - m)        k~_j = k_j e^(m - L_j)
//   o_t = (e^m S)^T r~_t + sum_{j < t} (r~_t . k~_j) v_j + (r_t . u k_t) v_t          S <- e^L S + e^(L - m) sum_j k~_j v_j^T
// on MFMA tiles: every product that counts has its true size, r~ and k~ enter as bf16 hi + lo halves, S and the weights too.  A chunk in which a channel decays by
// more than 2^100 within 32 tokens would leave the range and is walked token by token on the same registers (no result depends on which way was taken but by
// rounding).  The state stays in fp32 accumulators, laid out so that they are the left operand of S^T r without a shuffle.  Rows go straight to registers, a chunk
// ahead: a thread holds 2 channels of 8 tokens.
// A portion of several segments: a SUMMARY walk leaves every segment's own contribution and the sum of its log decays, a small launch turns those into states at
// segment starts, and the second walk begins there.
// Decoding (launch_wkv_step): one workgroup per (sequence, head) computes the decays from the low-rank row, streams the state once, norms and gates.
// A sequence's first token (position 0) takes the state as zero instead of reading it: slots need no clearing when reused.
#include "api_common.h"
#include "attend_tile.h"
#include "mixers.h"

namespace nvh {

namespace {

using WkvArgs = nvh_wkv_desc;
constexpr int C = 64;                                // tokens per chunk
constexpr int PLD = C + 8;                           // row of the weights in LDS
constexpr float kMaxDecay = 100.f;                   // log2 units a channel may decay in half a chunk on the MFMA way

__device__ __forceinline__ float log2_decay(float z) { return -kLog2e * __expf(z); }

__device__ __forceinline__ void split8(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
    u32x4 h, l;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        h[j] = pack_bf16x2(v[2 * j], v[2 * j + 1]);
        l[j] = pack_bf16x2(v[2 * j] - bf16_lo(h[j]), v[2 * j + 1] - bf16_hi(h[j]));
    }
    hi = *reinterpret_cast<const bf16x8*>(&h);
    lo = *reinterpret_cast<const bf16x8*>(&l);
}

template <int DIM>
struct WkvLds {
    static constexpr int WAVES = DIM / 16, ROW = DIM * 2, IMG = C * ROW;
    unsigned char r_hi[IMG], r_lo[IMG], k_hi[IMG], k_lo[IMG], v[IMG];          // (token by token: w as fp32 over r_hi and r_lo, k and r as they came over k_hi and k_lo)
    uint16_t p[2][C][PLD];                                                     // weights, hi | lo (token by token: outputs, [wave][16][16] fp32)
    float tot[8][DIM];                                                         // log decays by groups of 8 tokens
    float mid[DIM], full[DIM];
    float bonus[C];
    float red[WAVES][C];
};

// DIM / 16 waves; wave w holds value columns 16 w ..
template <int DIM, bool SUMMARY>
__global__ __launch_bounds__(DIM * 4) void wkv_walk_kernel(const WkvArgs a) {
    using Lds = WkvLds<DIM>;
    constexpr int ROW = DIM * 2, DT = DIM / 16, CP = DIM / 2, WAVES = Lds::WAVES;
    constexpr bool kOdd = ((ROW / 128) & 1) != 0;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    Lds& lds = *reinterpret_cast<Lds*>(smem);
    auto swz = [](int r) { return kOdd ? ((r >> 1) & 7) : (r & 7); };
    const int32_t* ch = a.chunks + 4 * blockIdx.x;
    const int row0 = ch[0], n_rows = ch[1], seq = ch[2];
    const int head = blockIdx.y;
    const bool last = blockIdx.x + 1 == (unsigned)a.n_chunks || a.chunks[4 * (blockIdx.x + 1) + 3] == 0;
    if (SUMMARY && last) return;                     // (nothing follows it)
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const int64_t slot = a.state_slots[seq];
    constexpr int64_t head_state = (int64_t)DIM * DIM;

    // state: value column 16 wave + lq, key rows 16 t + 4 lg + r
    f32x4 S[DT];
#pragma unroll
    for (int t = 0; t < DT; ++t) S[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int sv = 16 * wave + lq;
    if constexpr (!SUMMARY) {
        const float* src = nullptr;
        if (a.summaries) src = a.seg_state + ((int64_t)blockIdx.x * a.heads + head) * head_state;
        else if (slot >= 0 && a.positions[row0] > 0) src = a.state + (slot * a.heads + head) * head_state;
        if (src) {
#pragma unroll
            for (int t = 0; t < DT; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) S[t][r] = src[(16 * t + 4 * lg + r) * DIM + sv];
        }
    }
    // ---- this thread's rows of a chunk: channels 2 cp, 2 cp + 1 of tokens 8 tg ..; two 16-byte pieces of values; 4 gates of four tokens
    const int cp = tid % CP, tg = tid / CP;
    const int hc = head * DIM + 2 * cp;
    const float w0a = a.w0[hc], w0b = a.w0[hc + 1];
    float ua = 0.f, ub = 0.f;
    if constexpr (!SUMMARY) {
        ua = a.u[hc];
        ub = a.u[hc + 1];
    }
    uint32_t rr[8], kk[8], zz[8];
    u32x4 vv[2];
    u32x2 gg[4];
    auto fetch = [&](int t0) {                       // rows past the segment's end are zero (zz: not used)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int t = t0 + 8 * tg + i;
            const bool ok = t < n_rows;
            const int64_t row = row0 + (ok ? t : 0);
            kk[i] = ok ? *reinterpret_cast<const uint32_t*>(reinterpret_cast<const uint16_t*>(a.k) + row * a.stride + hc) : 0u;
            zz[i] = ok ? *reinterpret_cast<const uint32_t*>(reinterpret_cast<const uint16_t*>(a.z) + row * a.z_stride + hc) : 0u;
            if constexpr (!SUMMARY) rr[i] = ok ? *reinterpret_cast<const uint32_t*>(reinterpret_cast<const uint16_t*>(a.r) + row * a.stride + hc) : 0u;
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int e = j * DIM * 4 + tid, t = t0 + e / (DIM / 8), c = e % (DIM / 8) * 8;
            const bool ok = t < n_rows;
            vv[j] = ok ? *reinterpret_cast<const u32x4*>(reinterpret_cast<const uint16_t*>(a.v) + (int64_t)(row0 + t) * a.stride + head * DIM + c) : u32x4{0u, 0u, 0u, 0u};
        }
        if constexpr (!SUMMARY) {
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                const int t = t0 + 16 * it + lq;
                gg[it] = t < n_rows ? *reinterpret_cast<const u32x2*>(reinterpret_cast<const uint16_t*>(a.g) + (int64_t)(row0 + t) * a.stride + head * DIM + 16 * wave + 4 * lg)
                                    : u32x2{0u, 0u};
            }
        }
    };
    f32x4 nw = {0.f, 0.f, 0.f, 0.f};
    if constexpr (!SUMMARY) nw = *reinterpret_cast<const f32x4*>(a.norm + head * DIM + 16 * wave + 4 * lg);
    float dec_a = 0.f, dec_b = 0.f;
    fetch(0);
    for (int t0 = 0; t0 < n_rows; t0 += C) {
        const int n = n_rows - t0 < C ? n_rows - t0 : C;
        // ---- log decays of this thread's tokens, summed up
        float la[8], lb[8];                          // sums up to and with token i of the group
        {
            float sa = 0.f, sb = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const bool ok = 8 * tg + i < n;
                sa += ok ? log2_decay(bf16_lo(zz[i]) + w0a) : 0.f;
                sb += ok ? log2_decay(bf16_hi(zz[i]) + w0b) : 0.f;
                la[i] = sa;
                lb[i] = sb;
            }
            *reinterpret_cast<f32x2*>(&lds.tot[tg][2 * cp]) = f32x2{sa, sb};
        }
        lds_only_barrier();
        float oa = 0.f, ob = 0.f, ma = 0.f, mb = 0.f, fa = 0.f, fb = 0.f;
#pragma unroll
        for (int g = 0; g < 8; ++g) {
            const f32x2 s = *reinterpret_cast<const f32x2*>(&lds.tot[g][2 * cp]);
            oa += g < tg ? s[0] : 0.f;
            ob += g < tg ? s[1] : 0.f;
            if (g < 4) {
                ma += s[0];
                mb += s[1];
            }
            fa += s[0];
            fb += s[1];
        }
        dec_a += fa;
        dec_b += fb;
        // (every wave holds all channels: they agree)
        const bool strong = __builtin_amdgcn_ballot_w64(!(fminf(fminf(ma, fa - ma), fminf(mb, fb - mb)) >= -kMaxDecay)) != 0;
        const int pofs = (cp & 3) * 4;
        if (!strong) {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const int t = 8 * tg + i, at = t * ROW + (((cp >> 2) ^ swz(t)) * 16) + pofs;
                const float ia = oa + la[i], ib = ob + lb[i];
                const float ka = bf16_lo(kk[i]) * fast_exp2(ma - ia), kb = bf16_hi(kk[i]) * fast_exp2(mb - ib);
                const uint32_t kh = pack_bf16x2(ka, kb);
                *reinterpret_cast<uint32_t*>(lds.k_hi + at) = kh;
                *reinterpret_cast<uint32_t*>(lds.k_lo + at) = pack_bf16x2(ka - bf16_lo(kh), kb - bf16_hi(kh));
                if constexpr (!SUMMARY) {
                    const float ea = oa + (i ? la[i ? i - 1 : 0] : 0.f), eb = ob + (i ? lb[i ? i - 1 : 0] : 0.f);
                    const float ra = bf16_lo(rr[i]) * fast_exp2(ea - ma), rb = bf16_hi(rr[i]) * fast_exp2(eb - mb);
                    const uint32_t rh = pack_bf16x2(ra, rb);
                    *reinterpret_cast<uint32_t*>(lds.r_hi + at) = rh;
                    *reinterpret_cast<uint32_t*>(lds.r_lo + at) = pack_bf16x2(ra - bf16_lo(rh), rb - bf16_hi(rh));
                }
            }
        } else {
            float* w_f = reinterpret_cast<float*>(lds.r_hi);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const int t = 8 * tg + i;
                *reinterpret_cast<f32x2*>(w_f + t * DIM + 2 * cp) = f32x2{fast_exp2(log2_decay(bf16_lo(zz[i]) + w0a)), fast_exp2(log2_decay(bf16_hi(zz[i]) + w0b))};
                *reinterpret_cast<uint32_t*>(lds.k_hi + t * ROW + 4 * cp) = kk[i];
                if constexpr (!SUMMARY) *reinterpret_cast<uint32_t*>(lds.k_lo + t * ROW + 4 * cp) = rr[i];
            }
        }
        if constexpr (!SUMMARY) {                    // r . u k of the 8 tokens: over the lanes that hold a token's channels
            float d[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                d[i] = bf16_lo(rr[i]) * ua * bf16_lo(kk[i]) + bf16_hi(rr[i]) * ub * bf16_hi(kk[i]);
                d[i] = sum_xor16(group_sum<16>(d[i]));
                if constexpr (CP == 64) d[i] = sum_xor32(d[i]);
            }
            if (cp == 0) {
#pragma unroll
                for (int i = 0; i < 8; ++i) lds.bonus[8 * tg + i] = d[i];
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int e = j * DIM * 4 + tid, t = e / (DIM / 8), pc = e % (DIM / 8);
            *reinterpret_cast<u32x4*>(lds.v + t * ROW + (pc ^ swz(t)) * 16) = vv[j];
        }
        if (tg == 0) {
            *reinterpret_cast<f32x2*>(&lds.mid[2 * cp]) = f32x2{ma, mb};
            *reinterpret_cast<f32x2*>(&lds.full[2 * cp]) = f32x2{fa, fb};
        }
        u32x2 gate[4] = {gg[0], gg[1], gg[2], gg[3]};
        if (t0 + C < n_rows) fetch(t0 + C);
        lds_only_barrier();
        f32x4 o[4];                                  // o^T: value 16 wave + 4 lg + r, token 16 it + lq
        if (!strong) {
            const int tr = 4 * lg + (lq >> 2), tp = lq & 3;                    // transposed reads: row and column quarter this lane addresses
            if constexpr (!SUMMARY) {
                // weights: D[key 16 jt + 4 lg + r][query 16 qg + lq]; with 8 waves, two share a group of queries
                const int qg = wave & 3, Rq = 16 * qg + lq;
                f32x4 s[4];
#pragma unroll
                for (int jt = 0; jt < 4; ++jt) s[jt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int st = 0; st < DIM / 32; ++st) {
                    const int qat = Rq * ROW + ((4 * st + lg) ^ swz(Rq)) * 16;
                    const bf16x8 qh = *reinterpret_cast<const bf16x8*>(lds.r_hi + qat), ql = *reinterpret_cast<const bf16x8*>(lds.r_lo + qat);
#pragma unroll
                    for (int jt = 0; jt < 4; ++jt) {
                        if (jt > qg || (WAVES == 8 && (jt & 1) != wave >> 2)) continue;
                        const int Rk = 16 * jt + lq, kat = Rk * ROW + ((4 * st + lg) ^ swz(Rk)) * 16;
                        const bf16x8 kh = *reinterpret_cast<const bf16x8*>(lds.k_hi + kat), kl = *reinterpret_cast<const bf16x8*>(lds.k_lo + kat);
                        s[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, qh, s[jt], 0, 0, 0);
                        s[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, ql, s[jt], 0, 0, 0);
                        s[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, qh, s[jt], 0, 0, 0);
                    }
                }
                // products behind a branch: hipcc counts the wait states to their readers along one path into the join only
                asm volatile("s_nop 7" : "+v"(s[0]), "+v"(s[1]), "+v"(s[2]), "+v"(s[3]));
                const float bonus = lds.bonus[Rq];
#pragma unroll
                for (int jt = 0; jt < 4; ++jt) {
                    if (WAVES == 8 && (jt & 1) != wave >> 2) continue;
                    float p[4];
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const int back = Rq - (16 * jt + 4 * lg + r);
                        p[r] = back > 0 ? s[jt][r] : back == 0 ? bonus : 0.f;
                    }
                    const u32x2 hi = {pack_bf16x2(p[0], p[1]), pack_bf16x2(p[2], p[3])};
                    const u32x2 lo = {pack_bf16x2(p[0] - bf16_lo(hi[0]), p[1] - bf16_hi(hi[0])), pack_bf16x2(p[2] - bf16_lo(hi[1]), p[3] - bf16_hi(hi[1]))};
                    const int at = 32 * (jt >> 1) + 8 * lg + 4 * (jt & 1);
                    *reinterpret_cast<u32x2*>(&lds.p[0][Rq][at]) = hi;
                    *reinterpret_cast<u32x2*>(&lds.p[1][Rq][at]) = lo;
                }
                // what the state gives: slots of a 32-wide step are key rows 16 (2 st) + 4 lg + 0..3 and 16 (2 st + 1) + 4 lg + 0..3
#pragma unroll
                for (int it = 0; it < 4; ++it) o[it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int st = 0; st < DIM / 32; ++st) {
                    float sc[8];
#pragma unroll
                    for (int q = 0; q < 2; ++q) {
                        const f32x4 m4 = *reinterpret_cast<const f32x4*>(&lds.mid[16 * (2 * st + q) + 4 * lg]);
#pragma unroll
                        for (int r = 0; r < 4; ++r) sc[4 * q + r] = S[2 * st + q][r] * fast_exp2(m4[r]);
                    }
                    bf16x8 hi, lo;
                    split8(sc, hi, lo);
#pragma unroll
                    for (int it = 0; it < 4; ++it) {
                        const int R = 16 * it + lq, pa = ((4 * st + (lg >> 1)) ^ swz(R)) * 16 + (lg & 1) * 8, pb = ((4 * st + 2 + (lg >> 1)) ^ swz(R)) * 16 + (lg & 1) * 8;
                        const u32x2 ha = *reinterpret_cast<const u32x2*>(lds.r_hi + R * ROW + pa), hb = *reinterpret_cast<const u32x2*>(lds.r_hi + R * ROW + pb);
                        const u32x2 xa = *reinterpret_cast<const u32x2*>(lds.r_lo + R * ROW + pa), xb = *reinterpret_cast<const u32x2*>(lds.r_lo + R * ROW + pb);
                        const u32x4 hraw = {ha[0], ha[1], hb[0], hb[1]}, lraw = {xa[0], xa[1], xb[0], xb[1]};
                        const bf16x8 qh = *reinterpret_cast<const bf16x8*>(&hraw), ql = *reinterpret_cast<const bf16x8*>(&lraw);
                        o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, qh, o[it], 0, 0, 0);
                        o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, ql, o[it], 0, 0, 0);
                        o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, qh, o[it], 0, 0, 0);
                    }
                }
                lds_only_barrier();                  // all weights are in LDS
            }
            // value fragments: lane = column 16 wave + lq, slots = keys 32 hh + 4 lg + 0..3 and the same + 16
            u32x2 vlo[2], vhi[2];
#pragma unroll
            for (int hh = 0; hh < 2; ++hh) {
                const int ra = 32 * hh + tr, rb = ra + 16, pc = 2 * wave + (tp >> 1);
                vlo[hh] = ds_read_tr16<0>(lds_addr_of(lds.v + ra * ROW + (pc ^ swz(ra)) * 16 + (tp & 1) * 8));
                vhi[hh] = ds_read_tr16<0>(lds_addr_of(lds.v + rb * ROW + (pc ^ swz(rb)) * 16 + (tp & 1) * 8));
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
                        o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[hh], *reinterpret_cast<const bf16x8*>(&lds.p[0][16 * it + lq][32 * hh + 8 * lg]), o[it], 0, 0, 0);
                        o[it] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[hh], *reinterpret_cast<const bf16x8*>(&lds.p[1][16 * it + lq][32 * hh + 8 * lg]), o[it], 0, 0, 0);
                    }
            }
            // ---- the state behind these tokens, four key tiles at a time
#pragma unroll
            for (int tb = 0; tb < DT; tb += 4) {
                f32x4 M[4];
#pragma unroll
                for (int t = 0; t < 4; ++t) M[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int hh = 0; hh < 2; ++hh) {
                    const int ra = 32 * hh + tr, rb = ra + 16;
                    u32x2 ka[2][4], kb[2][4];
#pragma unroll
                    for (int t = 0; t < 4; ++t) {
                        const int pc = 2 * (tb + t) + (tp >> 1), pa = ra * ROW + (pc ^ swz(ra)) * 16 + (tp & 1) * 8, pb = rb * ROW + (pc ^ swz(rb)) * 16 + (tp & 1) * 8;
                        ka[0][t] = ds_read_tr16<0>(lds_addr_of(lds.k_hi + pa));
                        kb[0][t] = ds_read_tr16<0>(lds_addr_of(lds.k_hi + pb));
                        ka[1][t] = ds_read_tr16<0>(lds_addr_of(lds.k_lo + pa));
                        kb[1][t] = ds_read_tr16<0>(lds_addr_of(lds.k_lo + pb));
                    }
                    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                    for (int t = 0; t < 4; ++t)
#pragma unroll
                        for (int q = 0; q < 2; ++q) {
                            const u32x4 kraw = {ka[q][t][0], ka[q][t][1], kb[q][t][0], kb[q][t][1]};
                            M[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(&kraw), vf[hh], M[t], 0, 0, 0);
                        }
                }
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const f32x4 m4 = *reinterpret_cast<const f32x4*>(&lds.mid[16 * (tb + t) + 4 * lg]), f4 = *reinterpret_cast<const f32x4*>(&lds.full[16 * (tb + t) + 4 * lg]);
#pragma unroll
                    for (int r = 0; r < 4; ++r) S[tb + t][r] = fast_exp2(f4[r]) * S[tb + t][r] + fast_exp2(f4[r] - m4[r]) * M[t][r];
                }
            }
        } else {
            // ---- token by token; outputs of 16 tokens change lanes through a few LDS words of the wave
            const float* w_f = reinterpret_cast<const float*>(lds.r_hi);
            float* obuf = reinterpret_cast<float*>(lds.p) + wave * 256;
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                o[it] = f32x4{0.f, 0.f, 0.f, 0.f};
                for (int i = 0; i < 16 && 16 * it + i < n; ++i) {
                    const int t = 16 * it + i;
                    const float v = act_ld(reinterpret_cast<const uint16_t*>(lds.v + t * ROW + ((sv >> 3) ^ swz(t)) * 16) + (sv & 7));
                    float acc = 0.f;
#pragma unroll
                    for (int dt = 0; dt < DT; ++dt) {
                        const int key = 16 * dt + 4 * lg;
                        const f32x4 w4 = *reinterpret_cast<const f32x4*>(w_f + t * DIM + key), k4 = act_ld4(reinterpret_cast<const uint16_t*>(lds.k_hi + t * ROW) + key);
                        if constexpr (!SUMMARY) acc += sum4(act_ld4(reinterpret_cast<const uint16_t*>(lds.k_lo + t * ROW) + key) * S[dt]);
                        S[dt] = w4 * S[dt] + k4 * v;
                    }
                    if constexpr (!SUMMARY) {
                        acc = sum_xor16(acc);
                        acc = sum_xor32(acc) + lds.bonus[t] * v;
                        if (lg == 0) obuf[i * 16 + lq] = acc;
                    }
                }
                if constexpr (!SUMMARY) {
                    wave_lds_sync();
                    if (16 * it + lq < n) o[it] = *reinterpret_cast<const f32x4*>(obuf + lq * 16 + 4 * lg);
                    wave_lds_sync();
                }
            }
        }
        if constexpr (!SUMMARY) {
            // ---- norm over the head's columns, gate
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                float ss = sum4(o[it] * o[it]);
                ss = sum_xor16(ss);
                ss = sum_xor32(ss);
                if (lg == 0) lds.red[wave][16 * it + lq] = ss;
            }
            lds_only_barrier();
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                float ss = 0.f;
#pragma unroll
                for (int w = 0; w < WAVES; ++w) ss += lds.red[w][16 * it + lq];
                const float inv = 1.f / sqrtf(ss / a.n + a.eps);
                const int t = t0 + 16 * it + lq;
                const float g[4] = {bf16_lo(gate[it][0]), bf16_hi(gate[it][0]), bf16_lo(gate[it][1]), bf16_hi(gate[it][1])};
                f32x4 r;
#pragma unroll
                for (int k = 0; k < 4; ++k) r[k] = o[it][k] * inv * nw[k] * silu_f(g[k]);
                if (t < n_rows) act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(row0 + t) * a.out_stride + head * DIM + 16 * wave + 4 * lg, r);
            }
        }
    }
    float* dst = nullptr;
    if constexpr (SUMMARY) {
        dst = a.seg_state + ((int64_t)blockIdx.x * a.heads + head) * head_state;
        if (tg == 0) *reinterpret_cast<f32x2*>(a.seg_decay + (int64_t)blockIdx.x * a.heads * DIM + hc) = f32x2{dec_a, dec_b};
    } else if (last && slot >= 0) {
        dst = a.state + (slot * a.heads + head) * head_state;
    }
    if (dst) {
#pragma unroll
        for (int t = 0; t < DT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[(16 * t + 4 * lg + r) * DIM + sv] = S[t][r];
    }
}

// contributions of the segments -> states at their starts, in place; one thread per state element, walking the segments of every portion
__global__ __launch_bounds__(256) void wkv_starts_kernel(const WkvArgs a) {
    const int64_t per = (int64_t)a.heads * a.dim * a.dim, e = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int first = blockIdx.y;                    // only a portion's first segment starts a walk
    if (e >= per || a.chunks[4 * first + 3] != 0) return;
    const int64_t ch = e / a.dim, slot = a.state_slots[a.chunks[4 * first + 2]];
    float cur = slot >= 0 && a.positions[a.chunks[4 * first]] > 0 ? a.state[slot * per + e] : 0.f;
    for (int c = first; c < a.n_chunks && (c == first || a.chunks[4 * c + 3] != 0); ++c) {
        const bool more = c + 1 < a.n_chunks && a.chunks[4 * (c + 1) + 3] != 0;        // (the last segment left no contribution)
        const float own = more ? a.seg_state[c * per + e] : 0.f;
        a.seg_state[c * per + e] = cur;
        if (more) cur = fast_exp2(a.seg_decay[(int64_t)c * a.heads * a.dim + ch]) * cur + own;
    }
}

// ------------------------------------------------------------------------------------------------ token by token, any type and size
// one workgroup per (portion, head, 32 value columns); the state slice in LDS, 8 groups of key rows x 32 columns; norm and gate in a launch behind
template <typename T>
__global__ __launch_bounds__(256) void wkv_generic_kernel(const WkvArgs a) {
    extern __shared__ float lds_f[];                 // [dim][32] state, [4][dim] w, k, r, u, [8][32] sums
    float *S = lds_f, *wkr = S + a.dim * 32, *red = wkr + 4 * a.dim;
    const int first = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, c = tid & 31, rg = tid >> 5, col = blockIdx.z * 32 + c;
    if (a.chunks[4 * first + 3] != 0) return;        // a portion is walked whole from its first segment
    const int row0 = a.chunks[4 * first];
    int n_rows = a.chunks[4 * first + 1];
    for (int k = first + 1; k < a.n_chunks && a.chunks[4 * k + 3] != 0; ++k) n_rows += a.chunks[4 * k + 1];
    const int64_t slot = a.state_slots[a.chunks[4 * first + 2]], head_state = (int64_t)a.dim * a.dim;
    const bool ok = col < a.dim;
    float* pool = slot >= 0 ? a.state + (slot * a.heads + head) * head_state : nullptr;
    const bool carry = pool && a.positions[row0] > 0;
    for (int r = rg; r < a.dim; r += 8) S[r * 32 + c] = carry && ok ? pool[(int64_t)r * a.dim + col] : 0.f;
    for (int i = tid; i < a.dim; i += 256) wkr[3 * a.dim + i] = a.u[head * a.dim + i];
    for (int t = 0; t < n_rows; ++t) {
        const int64_t at = (int64_t)(row0 + t) * a.stride + head * a.dim;
        for (int i = tid; i < a.dim; i += 256) {
            const float z = act_ld(reinterpret_cast<const T*>(a.z) + (int64_t)(row0 + t) * a.z_stride + head * a.dim + i);
            wkr[i] = fast_exp2(log2_decay(z + a.w0[head * a.dim + i]));
            wkr[a.dim + i] = act_ld(reinterpret_cast<const T*>(a.k) + at + i);
            wkr[2 * a.dim + i] = act_ld(reinterpret_cast<const T*>(a.r) + at + i);
        }
        const float v = ok ? act_ld(reinterpret_cast<const T*>(a.v) + at + col) : 0.f;
        __syncthreads();
        float acc = 0.f;
        for (int r = rg; r < a.dim; r += 8) {
            const float s = S[r * 32 + c], kv = wkr[a.dim + r] * v;
            acc += (s + wkr[3 * a.dim + r] * kv) * wkr[2 * a.dim + r];
            S[r * 32 + c] = wkr[r] * s + kv;
        }
        red[rg * 32 + c] = acc;
        __syncthreads();
        if (rg == 0 && ok) {
            float s = 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k) s += red[k * 32 + c];
            act_st(reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t) * a.out_stride + head * a.dim + col, s);
        }
    }
    if (pool && ok)
        for (int r = rg; r < a.dim; r += 8) pool[(int64_t)r * a.dim + col] = S[r * 32 + c];
}

// one wave per (row of a portion, head), in place
template <typename T>
__global__ __launch_bounds__(256) void wkv_norm_gate_kernel(const WkvArgs a) {
    const int first = blockIdx.x, lane = threadIdx.x & 63, head = blockIdx.y;
    const int row0 = a.chunks[4 * first], n_rows = a.chunks[4 * first + 1];
    for (int t = blockIdx.z * 4 + (threadIdx.x >> 6); t < n_rows; t += gridDim.z * 4) {
        T* o = reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t) * a.out_stride + head * a.dim;
        const T* g = reinterpret_cast<const T*>(a.g) + (int64_t)(row0 + t) * a.stride + head * a.dim;
        float ss = 0.f;
        for (int c = lane; c < a.dim; c += 64) ss += act_ld(o + c) * act_ld(o + c);
        const float inv = 1.f / sqrtf(wave_sum64(ss) / a.n + a.eps);
        for (int c = lane; c < a.dim; c += 64) act_st(o + c, act_ld(o + c) * inv * a.norm[head * a.dim + c] * silu_f(act_ld(g + c)));
    }
}

// ------------------------------------------------------------------------------------------------ one token per sequence (bf16)
// grid (heads, rows); a thread holds 4 columns of DIM^2 / 1024 state rows; z: the low-rank row in front of its tanh
template <int DIM>
__global__ __launch_bounds__(256) void wkv_step_kernel(const WkvArgs a) {
    constexpr int LN = DIM / 4, RG = 256 / LN, NR = DIM / RG, TPC = 256 / DIM;
    extern __shared__ float low[];                   // [rank]
    __shared__ __attribute__((aligned(16))) float w_s[DIM], k_s[DIM], r_s[DIM], red[RG * DIM], part[4];
    const int head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, c = (tid % LN) * 4, rg = tid / LN;
    const int64_t slot = a.state_slots[row];
    const bool carry = slot >= 0 && a.positions[row] > 0;
    float* pool = a.state + ((slot >= 0 ? slot : 0) * a.heads + head) * (int64_t)(DIM * DIM) + c;
    f32x4 s[NR];
#pragma unroll
    for (int u = 0; u < NR; ++u)                     // asked for before anything is computed
        s[u] = carry ? *reinterpret_cast<const f32x4*>(pool + (rg + u * RG) * DIM) : f32x4{0.f, 0.f, 0.f, 0.f};
    const int64_t at = (int64_t)row * a.stride + head * DIM;
    const uint16_t* z = reinterpret_cast<const uint16_t*>(a.z) + (int64_t)row * a.z_stride;
    for (int i = tid; i < a.rank; i += 256) low[i] = tanhf(act_ld(z + i));
    const f32x4 v = act_ld4(reinterpret_cast<const uint16_t*>(a.v) + at + c);
    float bonus = 0.f;
    if (tid < DIM) {
        const float k = act_ld(reinterpret_cast<const uint16_t*>(a.k) + at + tid), r = act_ld(reinterpret_cast<const uint16_t*>(a.r) + at + tid);
        k_s[tid] = k;
        r_s[tid] = r;
        bonus = r * a.u[head * DIM + tid] * k;
    }
    bonus = wave_sum64(bonus);
    if ((tid & 63) == 0) part[tid >> 6] = bonus;
    __syncthreads();
    {
        const int chn = tid / TPC, sub = tid % TPC;  // TPC neighbouring lanes share a channel's row of the up-projection
        const uint16_t* w2 = reinterpret_cast<const uint16_t*>(a.w2) + (int64_t)(head * DIM + chn) * a.rank;
        float acc = 0.f;
        for (int p = sub * 8; p < a.rank; p += TPC * 8) {
            const f32x8 w = act_ld8(w2 + p);
            acc += sum4(w.a * *reinterpret_cast<const f32x4*>(low + p)) + sum4(w.b * *reinterpret_cast<const f32x4*>(low + p + 4));
        }
        if constexpr (TPC >= 2) acc += pair_in_row<1>(acc);
        if constexpr (TPC >= 4) acc += pair_in_row<2>(acc);
        if (sub == 0) w_s[chn] = fast_exp2(log2_decay(acc + a.w0[head * DIM + chn]));
    }
    bonus = part[0] + part[1] + part[2] + part[3];
    __syncthreads();
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < NR; ++u) {
        const int r = rg + u * RG;
        acc += s[u] * r_s[r];
        if (slot >= 0) *reinterpret_cast<f32x4*>(pool + r * DIM) = s[u] * w_s[r] + v * k_s[r];
    }
    if (rg == 0) acc += v * bonus;
    *reinterpret_cast<f32x4*>(red + rg * DIM + c) = acc;
    __syncthreads();
    float o = 0.f;
    if (tid < DIM) {
#pragma unroll
        for (int k = 0; k < RG; ++k) o += red[k * DIM + tid];
    }
    const float ss = wave_sum64(o * o);              // (threads past DIM hold zeros)
    if ((tid & 63) == 0) part[tid >> 6] = ss;
    __syncthreads();
    if (tid < DIM) {
        const float inv = 1.f / sqrtf((part[0] + part[1] + part[2] + part[3]) / a.n + a.eps);
        const float y = o * inv * a.norm[head * DIM + tid] * silu_f(act_ld(reinterpret_cast<const uint16_t*>(a.g) + at + tid));
        if (a.out) act_st(reinterpret_cast<uint16_t*>(a.out) + (int64_t)row * a.out_stride + head * DIM + tid, y);
        if (a.out_packed) act_st(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(row, head * DIM + tid, a.heads * DIM), y);
    }
}

template <int DIM>
int walk_dim(const WkvArgs& a, hipStream_t stream) {
    constexpr size_t lds = sizeof(WkvLds<DIM>);
    for (const void* fn : {reinterpret_cast<const void*>(wkv_walk_kernel<DIM, true>), reinterpret_cast<const void*>(wkv_walk_kernel<DIM, false>)})
        if (lds > 64 * 1024) (void)hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    const dim3 grid(a.n_chunks, a.heads);
    if (a.summaries) {
        wkv_walk_kernel<DIM, true><<<grid, DIM * 4, lds, stream>>>(a);
        int rc = check_launch("wkv summary");
        if (rc) return rc;
        const int64_t per = (int64_t)a.heads * DIM * DIM;
        wkv_starts_kernel<<<dim3((unsigned)((per + 255) / 256), a.n_chunks), 256, 0, stream>>>(a);
        rc = check_launch("wkv starts");
        if (rc) return rc;
    }
    wkv_walk_kernel<DIM, false><<<grid, DIM * 4, lds, stream>>>(a);
    return check_launch("wkv walk");
}

template <typename T>
int generic_t(const WkvArgs& a, hipStream_t stream) {
    const size_t lds = ((size_t)a.dim * 36 + 256) * 4;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(wkv_generic_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    wkv_generic_kernel<T><<<dim3(a.n_chunks, a.heads, (a.dim + 31) / 32), 256, lds, stream>>>(a);
    const int rc = check_launch("wkv generic");
    if (rc) return rc;
    wkv_norm_gate_kernel<T><<<dim3(a.n_chunks, a.heads, 16), 256, 0, stream>>>(a);
    return check_launch("wkv norm");
}

bool wkv_supported(int dim) { return dim == 64 || dim == 128; }

int check_wkv(const char* fn, const nvh_wkv_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->r && d->k && d->v && d->g && d->z && d->w0 && d->u && d->norm && d->positions && d->state_slots && d->state && (d->out || d->out_packed), NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->rows > 0 && d->heads > 0 && d->heads <= 65535 && d->dim > 0 && d->dim % 8 == 0 && d->dim <= 1024 && d->n > 0 && d->n <= d->dim, NVH_E_SHAPE, "%s: heads %d of %d (<= 1024)", fn,
            d->heads, d->dim);
    REQUIRE(d->stride % 8 == 0 && d->stride >= (int64_t)d->heads * d->dim && d->z_stride % 8 == 0 && (!d->out || (d->out_stride % 4 == 0 && d->out_stride >= (int64_t)d->heads * d->dim)),
            NVH_E_STRIDE, "%s: row strides", fn);
    REQUIRE(aligned16(d->r) && aligned16(d->k) && aligned16(d->v) && aligned16(d->g) && aligned16(d->z) && aligned16(d->w0) && aligned16(d->u) && aligned16(d->norm) && aligned16(d->state) &&
            aligned16(d->seg_state) && aligned16(d->seg_decay) && aligned16(d->out) && aligned16(d->out_packed), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

}  // namespace

}  // namespace nvh

using namespace nvh;

extern "C" {

int nvh_wkv_supported(int dim) { return wkv_supported(dim); }

int nvh_wkv_chunks(const nvh_wkv_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "wkv_chunks: null descriptor");
    if (d->n_chunks == 0) return 0;
    const int rc = check_wkv("wkv_chunks", d, dtype);
    if (rc) return rc;
    REQUIRE(d->chunks && d->n_chunks > 0 && d->n_chunks <= 65535 && d->out && d->z_stride >= (int64_t)d->heads * d->dim && (!d->summaries || (d->seg_state && d->seg_decay)), NVH_E_NULL,
            "wkv_chunks: %d segments or null pointer", d->n_chunks);
    if (dtype == NVH_F32) return generic_t<float>(*d, (hipStream_t)stream);
    if (generic || !wkv_supported(d->dim)) return generic_t<uint16_t>(*d, (hipStream_t)stream);
    return d->dim == 64 ? walk_dim<64>(*d, (hipStream_t)stream) : walk_dim<128>(*d, (hipStream_t)stream);
}

int nvh_wkv_step(const nvh_wkv_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "wkv_step: null descriptor");
    if (d->rows == 0) return 0;
    const int rc = check_wkv("wkv_step", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16 && wkv_supported(d->dim) && d->rows <= 65535 && d->w2 && aligned16(d->w2) && d->rank > 0 && d->rank % 8 == 0 && d->rank <= 8192 && d->z_stride >= d->rank &&
            (!d->out_packed || (d->heads * d->dim) % 32 == 0), NVH_E_SHAPE, "wkv_step: bf16, heads of %d, rank %d (%%8)", d->dim, d->rank);
    const dim3 grid(d->heads, d->rows);
    const size_t lds = (size_t)d->rank * 4;
    if (d->dim == 64) wkv_step_kernel<64><<<grid, 256, lds, (hipStream_t)stream>>>(*d);
    else wkv_step_kernel<128><<<grid, 256, lds, (hipStream_t)stream>>>(*d);
    return check_launch("wkv_step");
}

}  // extern "C"
