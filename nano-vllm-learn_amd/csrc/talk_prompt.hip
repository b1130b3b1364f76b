// Attention with mixed heads over prompt portions (gfx950 MFMA): scores are capped (tanh) and mixed across the heads before the softmax, so one workgroup holds all
// heads of 16 query rows and walks the visible keys 32 at a time:
//   1  S^T = K Q^T with the keys as fragments straight from the page, capped, to LDS: a wave takes its own heads, or the two heads of a pair of waves (they have the
//      same keys) over half of the keys.  cap tanh(t) = cap - 2 cap / (1 + exp(2 t)): the first term mixes to a constant per head, which a softmax does not see, so only
//      1 / (1 + exp(2 t)) is kept
//   2  the mixing matrix times these, 16 (query, key) pairs per product, in place: a wave takes whole pairs, all heads of them.  Both factors enter as the sum of two
//      fp16 numbers (22 bits; scaled by powers of two so that the second one is a normal number), the sums are fp32
//   3  every wave, for its own heads: online softmax (log2 domain: the matrix carries log2 e), O^T = V^T P^T with the weights as bf16 hi + lo
// Two barriers per 32 keys.  Values reach LDS by DMA, an image per key/value head that all waves read; with room for two images they are a step ahead.  The keys
// of the next step are on their way into registers meanwhile.  What no query of the tile sees is not read.  A sink starts the running maximum and sum.
// Algorithmic flops per launch: sum over sequences of (2 (DK + DV) + 2 heads) heads (visible pairs).
#include "attend_tile.h"
#include "talk.h"

namespace nvh {

namespace {

typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
typedef __fp16 f16x2 __attribute__((ext_vector_type(2)));

constexpr int kTile = 512;                           // scores of a head: 16 queries x 32 keys
constexpr float kMixGain = 16.f, kScoreGain = 4096.f;          // of the mixing matrix, of what step 1 keeps
constexpr size_t kLdsBytes = 160 * 1024;

// rows of scores in LDS (twice where a wave writes rows another one reads: PAIRS)
__host__ __device__ constexpr int rows_held(int heads, int hpw) { return hpw == 1 ? (heads + 3) / 4 * 4 : (heads + 15) / 16 * 16; }
// place of score i of head h: four groups of four heads read or written together lie in different banks
__device__ __forceinline__ int score_at(int h, int i) { return h * kTile + (i ^ (((h >> 2) & 3) * 16)); }

__device__ __forceinline__ uint32_t pack_f16(float x, float y) {
    const f16x2 v = __builtin_amdgcn_cvt_pkrtz(x, y);
    return __builtin_bit_cast(uint32_t, v);
}
__device__ __forceinline__ float f16_part(uint32_t v, int i) { return (float)__builtin_bit_cast(f16x2, v)[i]; }
// value tiles at two places, rows 0 .. 15 and (OFF bytes on) 16 .. 31 of each, transposed.  One statement with its wait: between a read and its wait the compiler
// might copy the register, and it would wait for the DMA in flight itself if it knew what is read
template <int OFF>
__device__ __forceinline__ void read_v2(bf16x8& v0, bf16x8& v1, uint32_t at0, uint32_t at1) {
    u32x2 a, b, c, d;
    asm volatile("ds_read_b64_tr_b16 %0, %4\n\tds_read_b64_tr_b16 %1, %4 offset:%6\n\tds_read_b64_tr_b16 %2, %5\n\tds_read_b64_tr_b16 %3, %5 offset:%6\n\ts_waitcnt lgkmcnt(0)"
                 : "=&v"(a), "=&v"(b), "=&v"(c), "=&v"(d) : "v"(at0), "v"(at1), "n"(OFF) : "memory");
    v0 = __builtin_bit_cast(bf16x8, u32x4{a[0], a[1], b[0], b[1]});
    v1 = __builtin_bit_cast(bf16x8, u32x4{c[0], c[1], d[0], d[1]});
}
// products that the vector pipe may read behind this: hipcc counts the wait states in between along one path into a join only
__device__ __forceinline__ void settle(f32x4& u, f32x4& v) { asm volatile("s_nop 7" : "+v"(u), "+v"(v)); }
// four numbers as their fp16 parts: hi of all four, then lo
__device__ __forceinline__ f16x8 split4(const float (&x)[4]) {
    u32x4 r;
    r[0] = pack_f16(x[0], x[1]);
    r[1] = pack_f16(x[2], x[3]);
    r[2] = pack_f16(fmaf(f16_part(r[0], 0), -1.f, x[0]), fmaf(f16_part(r[0], 1), -1.f, x[1]));                // (one mixed-precision instruction each)
    r[3] = pack_f16(fmaf(f16_part(r[1], 0), -1.f, x[2]), fmaf(f16_part(r[1], 1), -1.f, x[3]));
    return __builtin_bit_cast(f16x8, r);
}

// waves of HPW heads each; MT: tiles of 16 heads; PAIRS: step 1 in pairs of waves (HPW == 1, an even number of heads per key/value head).
// images: of a key/value head's values, 1 or 2; rate: 2 log2(e) scale / cap; unscale: what turns a mixed score as step 2 leaves it into the log2 domain; slack: 8 of
// that domain, as step 2 leaves it
template <int DK, int DV, int HPW, int MT, bool PAIRS>
__global__ __launch_bounds__(HPW == 1 ? 1024 : 512) void talk_prompt_kernel(const PagedAttendArgs a, const int q_tiles, const int images, const float rate,
                                                                                const float unscale, const float slack) {
    constexpr int STEPS = DK / 32, DT = DV / 16, KB = 32, VROW = DV * 2, VIMG = KB * VROW, VP = DV / 8, NV = VIMG / 1024;
    constexpr int SH = PAIRS ? 2 : HPW, HALVES = PAIRS ? 1 : 2;                // step 1: heads of a wave, halves of the keys
    constexpr int PB = HPW == 1 ? 1 : 2;                            // step 2: products at a time
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];        // [1 or 2][rows_held][kTile] scores, [images][kv heads] values, the mixing matrix
    int b, qt;
    {
        // one XCD takes a run of neighbouring query tiles, the longest walks first: what runs at once shares keys and values in its L2
        const int lin = blockIdx.x, total = gridDim.x, per = total >> 3, idx = total - 1 - (lin < per * 8 ? (lin & 7) * per + (lin >> 3) : lin);
        b = idx / q_tiles;
        qt = idx - b * q_tiles;
    }
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b], q0 = qt * 16;
    if (q0 >= sq || sk < sq) return;
    const int shift = sk - sq;                       // query row r has position r + shift
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), waves = blockDim.x >> 6, lq = lane & 15, lg = lane >> 4;
    const int heads = a.heads, ratio = heads / a.kv_heads, h0 = wave * HPW, s0 = PAIRS ? wave & ~1 : h0;
    const int rows = sq - q0 < 16 ? sq - q0 : 16, first_pos = q0 + shift, last_pos = first_pos + rows - 1;
    const int window = a.window > 0 ? a.window : 0x40000000;
    const VisibleTiles vis = visible_tiles(first_pos, last_pos, a.window, a.keep_first);
    float* const scores_lds = reinterpret_cast<float*>(lds);
    const int score_rows = rows_held(heads, HPW), score_tile = score_rows * kTile;
    unsigned char* vimg = lds + (PAIRS ? 2 : 1) * score_tile * 4;
    for (int i = heads * kTile + tid; i < score_tile; i += blockDim.x) {                                      // heads that do not exist
        scores_lds[i] = 0.f;
        if (PAIRS) scores_lds[score_tile + i] = 0.f;
    }

    // steps of 32 keys: the halves of the visible tiles, without those nobody sees
    auto step_key = [&](int it) { return vis.tile(it >> 1) * 64 + (it & 1) * KB; };
    auto next_step = [&](int it) {
        for (++it; it < 2 * vis.count; ++it) {
            const int k0 = step_key(it);
            if (k0 <= last_pos && (k0 + KB - 1 > first_pos - window || k0 < a.keep_first)) break;
        }
        return it;
    };
    const int head_elems = a.block_size * (DK + DV), tiles_per_page = a.block_size >> 6;
    const int64_t page_elems = (int64_t)a.kv_heads * head_elems;
    const int32_t* table = a.block_tables + (int64_t)b * a.bt_stride;
    // lane i holds where visible tile 64 block + i lies (elements before its first key, row of that key in the page): the loop finds it without waiting for memory
    int block = -1, key_lo = 0, key_hi = 0, first_row = 0;
    auto fetch = [&](int t) {
        if (t >> 6 == block) return;
        block = t >> 6;
        const int i = 64 * block + lane, tile = vis.tile(i < vis.count ? i : vis.count - 1), pg = tile / tiles_per_page;
        first_row = (tile - pg * tiles_per_page) * 64;
        const int64_t at = table[pg] * page_elems + first_row * DK;
        key_lo = (int)at;
        key_hi = (int)(at >> 32);
        asm volatile("" : "+v"(key_lo), "+v"(key_hi), "+v"(first_row));        // (waited for here, not at every use)
    };
    struct Place {                                   // of a step: keys of head 0 in the page, its first row there
        const uint16_t* keys;
        int row;
    };
    auto place = [&](int i) {
        const int t = (i >> 1) & 63, half = (i & 1) * KB;
        const uint32_t lo = __builtin_amdgcn_readlane(key_lo, t), hi = __builtin_amdgcn_readlane(key_hi, t);
        return Place{reinterpret_cast<const uint16_t*>(a.cache) + (int64_t)((uint64_t)hi << 32 | lo) + half * DK, __builtin_amdgcn_readlane(first_row, t) + half};
    };
    // (rows past the last key repeat it: not seen)
    auto load_k = [&](bf16x8 (&kf)[STEPS], int k0, const Place& at, int g, int half) {
        const int live = sk - k0, r = 16 * half + lq;
        const char* p = reinterpret_cast<const char*>(at.keys + g * head_elems);                              // (uniform base, 32-bit offset: one address register)
        const uint32_t off = ((r < live ? r : live - 1) * DK + 8 * lg) * 2;
#pragma unroll
        for (int st = 0; st < STEPS; ++st) kf[st] = *reinterpret_cast<const bf16x8*>(p + off + 64 * st);
    };
    auto stage_v = [&](int k0, const Place& at, int image) {
        const int live = sk - k0;
        const char* p = reinterpret_cast<const char*>(at.keys + (a.block_size * DK + at.row * (DV - DK)));
        unsigned char* to = vimg + image * a.kv_heads * VIMG;
        for (int i = wave; i < a.kv_heads * NV; i += waves) {
            const int g = (unsigned)i / NV, r = (unsigned)((i - g * NV) * 64 + lane) / VP, c = ((lane & (VP - 1)) ^ swz_v<DV>(r)) * 8;
            dma16(p + (uint32_t)(g * head_elems + (r < live ? r : live - 1) * DV + c) * 2u, to + i * 1024);
        }
    };
    const int end = 2 * vis.count;
    int it = next_step(-1);
    fetch(it >> 1);
    Place at = place(it);
    const int g0 = (s0 < heads ? s0 : heads - 1) / ratio, half0 = PAIRS ? wave & 1 : 0;
    bf16x8 ka[STEPS], kb[HALVES == 2 ? STEPS : 1];
    load_k(ka, step_key(it), at, g0, half0);
    if (images == 2) stage_v(step_key(it), at, 0);

    const int my_q = q0 + lq, q_row = q_beg + (my_q < sq ? my_q : sq - 1), my_pos = my_q + shift;
    bf16x8 qf[SH][STEPS];
#pragma unroll
    for (int j = 0; j < SH; ++j) {
        const int h = s0 + j < heads ? s0 + j : heads - 1;
        const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + (int64_t)q_row * a.q_stride + h * DK + 8 * lg;
#pragma unroll
        for (int st = 0; st < STEPS; ++st) qf[j][st] = *reinterpret_cast<const bf16x8*>(qp + 32 * st);
    }
    f32x4 o[HPW][DT];
    float m[HPW], l[HPW];                            // running maximum (log2 domain, scaled) and this lane's share of the sum
#pragma unroll
    for (int j = 0; j < HPW; ++j) {
#pragma unroll
        for (int t = 0; t < DT; ++t) o[j][t] = f32x4{0.f, 0.f, 0.f, 0.f};
        m[j] = -INFINITY;
        l[j] = 0.f;
        if (a.sink) {
            const int h = h0 + j < heads ? h0 + j : heads - 1;
            float row_sum = 0.f;
            for (int g = 0; g < heads; ++g) row_sum += a.talk[h * heads + g];
            m[j] = (a.sink[h] - a.softcap * row_sum) * (kLog2e / unscale);
            l[j] = lg == 0 ? 1.f : 0.f;
        }
    }
    // A operands: T[16 i + lq][16 c + 4 lg + (e & 3)], the parts of it, behind the images of values
    f16x8* mix = reinterpret_cast<f16x8*>(vimg + images * a.kv_heads * VIMG) + lane;
    for (int ic = wave; ic < MT * MT; ic += waves) {
        f16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int r = 16 * (ic / MT) + lq, h = 16 * (ic % MT) + 4 * lg + e;
            const float x = r < heads && h < heads ? a.talk[r * heads + h] * (-kLog2e * kMixGain) : 0.f;
            hi[e] = hi[e + 4] = (_Float16)x;
            lo[e] = lo[e + 4] = (_Float16)(x - (float)hi[e]);
        }
        mix[ic * 128] = hi;
        mix[ic * 128 + 64] = lo;
    }
    // place in an image of value tile 0 (rows R0 and R0 + 16 share a swizzle); the swizzle is even, so tile t lies at this ^ 32 t
    const int R0 = 4 * lg + (lq >> 2), vplace = R0 * VROW + (lq & 1) * 8 + ((lq & 2) >> 1) * 16 + swz_v<DV>(R0) * 16;
    int key_head[SH];
#pragma unroll
    for (int j = 0; j < SH; ++j) key_head[j] = (s0 + j < heads ? s0 + j : heads - 1) / ratio;
    const int at1 = score_at(s0, 4 * lane), at3 = score_at(h0, 4 * lane);      // the wave's heads share a swizzle in either step
    const bool held = HPW != 1 || 4 * lg < score_rows;
    const int row2 = held ? 4 * lg : 0;                                        // (its scores meet zeros where there are no heads 4 lg ..)
    float* ex = scores_lds;
    int image = 0;
    while (it < end) {
        const int k0 = step_key(it), next = next_step(it);
        const bool more = next < end;
        if (more) fetch(next >> 1);
        const int next_k0 = step_key(more ? next : it);                        // (behind the last step: that one again, not used)
        const Place next_at = place(more ? next : it);
        // ---- 1: scores
        if constexpr (HALVES == 2) load_k(kb, k0, at, g0, 1);
        auto product = [&](const auto& kf, int j) {
            f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int st = 0; st < STEPS; ++st) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[st], qf[j][st], s, 0, 0, 0);
            return s;
        };
        auto keep = [&](f32x4 s, int j, int half) {  // (heads that do not exist fill rows the matrix has zeros for)
#pragma unroll
            for (int i = 0; i < 4; ++i) s[i] = fast_rcp(fmaf(fast_exp2(s[i] * rate), 1.f / kScoreGain, 1.f / kScoreGain));
            *reinterpret_cast<f32x4*>(ex + at1 + j * kTile + 256 * half) = s;
        };
        auto scores = [&](auto& kf, int half) {
            int g = g0;
#pragma unroll
            for (int j = 0; j < SH; j += 2) {
                if (!PAIRS && key_head[j] != g) load_k(kf, k0, at, key_head[j], half);
                f32x4 u = product(kf, j);
                g = key_head[j];
                if constexpr (SH > 1) {
                    if (!PAIRS && key_head[j + 1] != g) load_k(kf, k0, at, key_head[j + 1], half);
                    f32x4 v = product(kf, j + 1);
                    g = key_head[j + 1];
                    settle(u, v);
                    keep(u, j, half);
                    keep(v, j + 1, half);
                } else {
                    settle(u, u);
                    keep(u, j, half);
                }
            }
        };
        scores(ka, half0);
        if constexpr (HALVES == 2) scores(kb, 1);
        if (images == 2) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // this step's values have landed
        load_k(ka, next_k0, next_at, g0, half0);
        lds_only_barrier();
        if (images == 1) stage_v(k0, at, 0);
        else if (more) stage_v(next_k0, next_at, image ^ 1);
        // ---- 2: mixing, 16 pairs at a time
        for (int p0 = wave; p0 < 32; p0 += PB * waves) {
            int p[PB];
            f16x8 c[PB][MT];
#pragma unroll
            for (int n = 0; n < PB; ++n) {
                p[n] = p0 + n * waves < 32 ? p0 + n * waves : p0;              // (the same ones again where there are no more)
#pragma unroll
                for (int i = 0; i < MT; ++i) {
                    float x[4];
#pragma unroll
                    for (int e = 0; e < 4; ++e) x[e] = ex[score_at(16 * i + row2 + e, p[n] * 16 + lq)];
                    c[n][i] = split4(x);
                }
            }
            __builtin_amdgcn_sched_barrier(0);       // (the matrix is read behind the splits: registers)
#pragma unroll
            for (int i = 0; i < MT; ++i) {
                f32x4 d[PB];
#pragma unroll
                for (int n = 0; n < PB; ++n) d[n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < MT; ++s) {
                    const f16x8 hi = mix[(i * MT + s) * 128], lo = mix[(i * MT + s) * 128 + 64];
#pragma unroll
                    for (int n = 0; n < PB; ++n) d[n] = __builtin_amdgcn_mfma_f32_16x16x32_f16(lo, c[n][s], d[n], 0, 0, 0);
#pragma unroll
                    for (int n = 0; n < PB; ++n) d[n] = __builtin_amdgcn_mfma_f32_16x16x32_f16(hi, c[n][s], d[n], 0, 0, 0);
                }
#pragma unroll
                for (int n = 0; n < PB; ++n)
                    if (held) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) ex[score_at(16 * i + row2 + r, p[n] * 16 + lq)] = d[n][r];        // (zero where there is no head)
                    }
            }
        }
        if (images == 1) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_only_barrier();
        // ---- 3: softmax and values of the wave's heads
        const bool masked = k0 + KB - 1 > first_pos || (k0 <= last_pos - window && k0 + KB > a.keep_first);
#pragma unroll
        for (int j = 0; j < HPW; ++j) {
            if (h0 + j >= heads) continue;
            f32x4 s[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) s[t] = *reinterpret_cast<const f32x4*>(ex + at3 + j * kTile + 256 * t);
            if (masked) {
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const int key = k0 + 16 * t + 4 * lg + r;
                        s[t][r] = key <= my_pos && (key > my_pos - window || key < a.keep_first) ? s[t][r] : -INFINITY;
                    }
            }
            float mx = max3f(s[0][0], s[0][1], s[0][2]);
            mx = max3f(mx, s[0][3], s[1][0]);
            mx = max3f(mx, s[1][1], s[1][2]);
            mx = max2(mx, s[1][3]);
            mx = max_xor16(mx);
            mx = max_xor32(mx);
            // (a maximum that grows by less than `slack` is left where it is: weights of up to 2^8, no sums to rescale)
            const float m_new = mx > m[j] + slack ? mx : m[j], m_use = m_new == -INFINITY ? 0.f : m_new, below = -m_use * unscale;
            float sum = 0.f;
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    s[t][r] = fast_exp2(s[t][r] * unscale + below);
                    sum += s[t][r];
                }
            if (__builtin_amdgcn_ballot_w64(m_new != m[j]) != 0) {
                const float alpha = fast_exp2((m[j] - m_use) * unscale);
                l[j] *= alpha;
#pragma unroll
                for (int t = 0; t < DT; ++t) o[j][t] *= alpha;
            }
            l[j] += sum;
            m[j] = m_new;
            u32x4 hraw, lraw;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float p0 = s[i >> 1][2 * (i & 1)], p1 = s[i >> 1][2 * (i & 1) + 1];
                hraw[i] = pack_bf16x2(p0, p1);
                asm volatile("" : "+v"(hraw[i]));    // (its halves are taken from here, not converted once more)
                lraw[i] = pack_bf16x2(p0 - bf16_lo(hraw[i]), p1 - bf16_hi(hraw[i]));
            }
            const bf16x8 p_hi = *reinterpret_cast<const bf16x8*>(&hraw), p_lo = *reinterpret_cast<const bf16x8*>(&lraw);
            const uint32_t vaddr = lds_addr_of(vimg + (image * a.kv_heads + (h0 + j) / ratio) * VIMG) + vplace;
#pragma unroll
            for (int t0 = 0; t0 < DT; t0 += 2) {
                bf16x8 v[2];
                read_v2<16 * VROW>(v[0], v[1], vaddr ^ 32 * t0, vaddr ^ 32 * (t0 + 1));
#pragma unroll
                for (int t = 0; t < 2; ++t) o[j][t0 + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[t], p_hi, o[j][t0 + t], 0, 0, 0);
#pragma unroll
                for (int t = 0; t < 2; ++t) o[j][t0 + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[t], p_lo, o[j][t0 + t], 0, 0, 0);
            }
        }
        image ^= images - 1;
        if (PAIRS) ex = scores_lds + (ex == scores_lds ? score_tile : 0);   // (a wave of the pair may be ahead)
        it = next;
        at = next_at;
    }
#pragma unroll
    for (int j = 0; j < HPW; ++j) {
        if (h0 + j >= heads) continue;
        const float sum = sum_xor32(sum_xor16(l[j]));
        if (my_q >= sq) continue;
        const float inv = sum > 0.f ? 1.f / sum : 0.f;
        uint16_t* out = reinterpret_cast<uint16_t*>(a.out) + (int64_t)q_row * a.out_stride + (h0 + j) * DV + 4 * lg;
#pragma unroll
        for (int t = 0; t < DT; ++t) act_st4(out + 16 * t, o[j][t] * inv);
    }
}

// heads per wave: one (sixteen waves of 128 registers), two where the heads are wide, four where there are more than sixteen of them; 0: not held
int heads_per_wave(int heads, int dk, int dv) {
    const bool narrow = dk <= 128 && dv <= 128;
    return heads <= 16 ? (narrow ? 1 : 2) : heads <= 32 && narrow ? 4 : 0;
}
bool in_pairs(int heads, int kv_heads, int hpw) { return hpw == 1 && heads / kv_heads % 2 == 0; }
size_t lds_bytes(int heads, int kv_heads, int hpw, int dv, int images) {
    const size_t mt = (heads + 15) / 16;
    return (size_t)(in_pairs(heads, kv_heads, hpw) ? 2 : 1) * rows_held(heads, hpw) * kTile * 4 + (size_t)images * kv_heads * 64 * dv + mt * mt * 2048;
}

template <int DK, int DV, int HPW, int MT, bool PAIRS>
int launch_one(const PagedAttendArgs& a, hipStream_t stream) {
    const int waves = (a.heads + HPW - 1) / HPW, q_tiles = (a.max_q + 15) / 16;
    // two images where they take no workgroup's place
    const size_t one = lds_bytes(a.heads, a.kv_heads, HPW, DV, 1), two = lds_bytes(a.heads, a.kv_heads, HPW, DV, 2);
    const int images = two <= kLdsBytes && (two <= kLdsBytes / 2 || one > kLdsBytes / 2 || waves > 8) ? 2 : 1;
    const size_t lds = images == 2 ? two : one;
    const float rate = 2.f * kLog2e * a.scale / a.softcap, unscale = 2.f * a.softcap / (kScoreGain * kMixGain);
    const auto kernel = talk_prompt_kernel<DK, DV, HPW, MT, PAIRS>;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    kernel<<<a.batch * q_tiles, 64 * waves, lds, stream>>>(a, q_tiles, images, rate, unscale, 8.f / unscale);
    return check_launch("talk_prompt");
}
template <int DK, int DV>
int launch_dims(const PagedAttendArgs& a, hipStream_t stream) {
    if constexpr (DK <= 128 && DV <= 128) {
        if (a.heads > 16) return launch_one<DK, DV, 4, 2, false>(a, stream);
        return in_pairs(a.heads, a.kv_heads, 1) ? launch_one<DK, DV, 1, 1, true>(a, stream) : launch_one<DK, DV, 1, 1, false>(a, stream);
    } else {
        return launch_one<DK, DV, 2, 1, false>(a, stream);
    }
}
template <int DK>
int launch_key(const PagedAttendArgs& a, hipStream_t stream) {
    if (a.dv == 64) return launch_dims<DK, 64>(a, stream);
    if (a.dv == 128) return launch_dims<DK, 128>(a, stream);
    return launch_dims<DK, 256>(a, stream);
}

}  // namespace

bool talk_prompt_supported(int heads, int kv_heads, int dk, int dv, int block_size) {
    const int hpw = heads_per_wave(heads, dk, dv);
    return block_size % 64 == 0 && (dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128 || dv == 256) && hpw > 0 &&
           lds_bytes(heads, kv_heads, hpw, dv, 1) <= kLdsBytes;
}

int launch_talk_prompt(const PagedAttendArgs& a, hipStream_t stream) {
    switch (a.dk) {
        case 64: return launch_key<64>(a, stream);
        case 128: return launch_key<128>(a, stream);
        case 192: return launch_key<192>(a, stream);
        default: return launch_key<256>(a, stream);
    }
}

}  // namespace nvh
