// Attention with mixed heads over prompt portions (gfx950 MFMA): scores are capped (tanh) and mixed across the heads before the softmax, so one workgroup holds all
// heads of 16 query rows and walks the visible keys 32 at a time:
//   1  every wave, for its own heads: S^T = K Q^T with the keys as fragments straight from the page, capped, to LDS as the register image it is
//   2  the mixing matrix times the heads' scores on the 32-bit matrix pipe, 16 (query, key) pairs per product, in place: a wave takes whole pairs, all heads of them
//   3  every wave, for its own heads: online softmax (log2 domain: the matrix carries log2 e), O^T = V^T P^T with the weights as bf16 hi + lo
// Two barriers per 32 keys.  Values reach LDS by DMA into an image of the wave's own, the keys of the next step are on their way into registers meanwhile.
// What no query of the tile sees is not read.  A sink starts the running maximum and sum.
// Algorithmic flops per launch: sum over sequences of (2 (DK + DV) + 2 heads) heads (visible pairs).
#include "attend_tile.h"
#include "talk.h"

namespace nvh {

namespace {

constexpr int kTalkRow = 512 + 16;                   // floats of a head's scores (16 queries x 32 keys); 16 more: four heads' rows start in different banks
constexpr size_t kLdsBytes = 160 * 1024;

// waves of HPW heads each; MT: tiles of 16 heads
template <int DK, int DV, int HPW, int MT>
__global__ __launch_bounds__(512) void talk_prompt_kernel(const PagedAttendArgs a, const int q_tiles) {
    constexpr int STEPS = DK / 32, DT = DV / 16, KB = 32, VROW = DV * 2, VIMG = KB * VROW, VP = DV / 8, NV = VIMG / 1024;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];        // [waves] images of values, [heads, padded to 4][kTalkRow] scores
    int b, qt;
    {
        // one XCD takes a run of neighbouring query tiles: what runs at once shares keys and values in its L2
        const int lin = blockIdx.x, total = gridDim.x, per = total >> 3, idx = lin < per * 8 ? (lin & 7) * per + (lin >> 3) : lin;
        b = idx / q_tiles;
        qt = idx - b * q_tiles;
    }
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b], q0 = qt * 16;
    if (q0 >= sq || sk < sq) return;
    const int shift = sk - sq;                       // query row r has position r + shift
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), waves = blockDim.x >> 6, lq = lane & 15, lg = lane >> 4;
    const int ratio = a.heads / a.kv_heads, heads = a.heads, h0 = wave * HPW;
    const int rows = sq - q0 < 16 ? sq - q0 : 16, first_pos = q0 + shift, last_pos = first_pos + rows - 1;
    const int window = a.window > 0 ? a.window : 0x40000000;
    const VisibleTiles vis = visible_tiles(first_pos, last_pos, a.window, a.keep_first);
    unsigned char* vimg = lds + wave * VIMG;
    float* ex = reinterpret_cast<float*>(lds + waves * VIMG);
    for (int i = heads * kTalkRow + tid; i < score_cols(heads) * kTalkRow; i += blockDim.x) ex[i] = 0.f;      // heads of the last product that do not exist

    // steps of 32 keys: the halves of the visible tiles, without those nobody sees
    auto step_key = [&](int it) { return vis.tile(it >> 1) * 64 + (it & 1) * KB; };
    auto next_step = [&](int it) {
        for (++it; it < 2 * vis.count; ++it) {
            const int k0 = step_key(it);
            if (k0 <= last_pos && (k0 + KB - 1 > first_pos - window || k0 < a.keep_first)) break;
        }
        return it;
    };
    const int64_t head_elems = (int64_t)a.block_size * (DK + DV), page_elems = a.kv_heads * head_elems;
    const int32_t* table = a.block_tables + (int64_t)b * a.bt_stride;
    // (rows past the last key repeat it: not seen)
    bf16x8 kf[2][STEPS];
    auto load_k = [&](int k0, int g) {
        const int off = k0 % a.block_size, live = sk - k0;
        const uint16_t* base = reinterpret_cast<const uint16_t*>(a.cache) + table[k0 / a.block_size] * page_elems + g * head_elems + (int64_t)off * DK + 8 * lg;
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const int r = 16 * t + lq;
            const uint16_t* p = base + (r < live ? r : live - 1) * DK;
#pragma unroll
            for (int st = 0; st < STEPS; ++st) kf[t][st] = *reinterpret_cast<const bf16x8*>(p + 32 * st);
        }
    };
    auto stage_v = [&](int k0, int g) {
        const int off = k0 % a.block_size, live = sk - k0;
        const uint16_t* base = reinterpret_cast<const uint16_t*>(a.cache) + table[k0 / a.block_size] * page_elems + g * head_elems + (int64_t)a.block_size * DK + (int64_t)off * DV;
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int s = j * 64 + lane, r = s / VP, c = ((s - r * VP) ^ swz_v<DV>(r)) * 8;
            dma16(base + (r < live ? r : live - 1) * DV + c, vimg + j * 1024);
        }
    };
    int it = next_step(-1);
    const int g0 = (h0 < heads ? h0 : heads - 1) / ratio;
    load_k(step_key(it), g0);
    stage_v(step_key(it), g0);

    const int my_q = q0 + lq, q_row = q_beg + (my_q < sq ? my_q : sq - 1), my_pos = my_q + shift;
    bf16x8 qf[HPW][STEPS];
    f32x4 o[HPW][DT];
    float m[HPW], l[HPW];                            // running maximum (log2 domain) and this lane's share of the sum
#pragma unroll
    for (int j = 0; j < HPW; ++j) {
        const int h = h0 + j < heads ? h0 + j : heads - 1;
        const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + (int64_t)q_row * a.q_stride + h * DK + 8 * lg;
#pragma unroll
        for (int st = 0; st < STEPS; ++st) qf[j][st] = *reinterpret_cast<const bf16x8*>(qp + 32 * st);
#pragma unroll
        for (int t = 0; t < DT; ++t) o[j][t] = f32x4{0.f, 0.f, 0.f, 0.f};
        m[j] = a.sink ? a.sink[h] * kLog2e : -INFINITY;
        l[j] = a.sink && lg == 0 ? 1.f : 0.f;
    }
    float tf[MT][4 * MT];                            // A operand: T[16 i + lq][4 s + lg]
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int s = 0; s < 4 * MT; ++s) {
            const int r = 16 * i + lq, c = 4 * s + lg;
            tf[i][s] = r < heads && c < heads ? a.talk[r * heads + c] * kLog2e : 0.f;
        }
    uint32_t vaddr[DT];
    {
        const int R0 = 4 * lg + (lq >> 2), p = lq & 3, swz = swz_v<DV>(R0);    // rows R0 and R0 + 16 share a swizzle
#pragma unroll
        for (int t = 0; t < DT; ++t) vaddr[t] = lds_addr_of(vimg + R0 * VROW + (p & 1) * 8 + (((2 * t + (p >> 1)) ^ swz) * 16));
    }
    const ScoreCap cap(a.scale, a.softcap);
    while (it < 2 * vis.count) {
        const int k0 = step_key(it);
        it = next_step(it);
        const bool more = it < 2 * vis.count;
        // ---- 1: scores of the wave's heads
        int g = g0;
#pragma unroll
        for (int j = 0; j < HPW; ++j) {
            if (h0 + j >= heads) continue;
            if (j && (h0 + j) / ratio != g) {
                g = (h0 + j) / ratio;
                load_k(k0, g);
            }
            f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int st = 0; st < STEPS; ++st)
#pragma unroll
                for (int t = 0; t < 2; ++t) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][st], qf[j][st], s[t], 0, 0, 0);
#pragma unroll
            for (int t = 0; t < 2; ++t) *reinterpret_cast<f32x4*>(ex + (h0 + j) * kTalkRow + (64 * t + lane) * 4) = cap(s[t]);
        }
        if (more) load_k(step_key(it), g0);
        lds_only_barrier();
        // ---- 2: mixing, 16 pairs at a time
        for (int p = wave; p < 32; p += waves) {
            float* at = ex + p * 16 + lq;
            float c[4 * MT];
#pragma unroll
            for (int s = 0; s < 4 * MT; ++s) c[s] = 4 * s < heads ? at[(4 * s + lg) * kTalkRow] : 0.f;
#pragma unroll
            for (int i = 0; i < MT; ++i) {
                f32x4 d = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < 4 * MT; ++s)
                    if (4 * s < heads) d = __builtin_amdgcn_mfma_f32_16x16x4f32(tf[i][s], c[s], d, 0, 0, 0);
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (16 * i + 4 * lg + r < heads) at[(16 * i + 4 * lg + r) * kTalkRow] = d[r];
            }
        }
        lds_only_barrier();
        // ---- 3: softmax and values of the wave's heads
        const bool masked = k0 + KB - 1 > first_pos || (k0 <= last_pos - window && k0 + KB > a.keep_first);
        g = g0;
#pragma unroll
        for (int j = 0; j < HPW; ++j) {
            if (h0 + j >= heads) continue;
            f32x4 s[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) s[t] = *reinterpret_cast<const f32x4*>(ex + (h0 + j) * kTalkRow + (64 * t + lane) * 4);
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
            const float m_new = max2(m[j], mx), m_use = m_new == -INFINITY ? 0.f : m_new;
            float sum = 0.f;
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    s[t][r] = fast_exp2(s[t][r] - m_use);
                    sum += s[t][r];
                }
            if (__builtin_amdgcn_ballot_w64(m_new != m[j]) != 0) {
                const float alpha = fast_exp2(m[j] - m_use);
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
                lraw[i] = pack_bf16x2(p0 - bf16_lo(hraw[i]), p1 - bf16_hi(hraw[i]));
            }
            const bf16x8 p_hi = *reinterpret_cast<const bf16x8*>(&hraw), p_lo = *reinterpret_cast<const bf16x8*>(&lraw);
            if (j && (h0 + j) / ratio != g) {        // (this wave's reads of the image are done: their results were waited for)
                g = (h0 + j) / ratio;
                stage_v(k0, g);
            }
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");                   // the image has landed (and the next keys, asked for long before)
            constexpr int TG = DT < 4 ? DT : 4;                                // value tiles read at a time
#pragma unroll
            for (int t0 = 0; t0 < DT; t0 += TG) {
                u32x2 vlo[TG], vhi[TG];
#pragma unroll
                for (int t = 0; t < TG; ++t) {
                    vlo[t] = ds_read_tr16<0>(vaddr[t0 + t]);
                    vhi[t] = ds_read_tr16<16 * VROW>(vaddr[t0 + t]);
                }
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int t = 0; t < TG; ++t) {
                    const u32x4 raw = {vlo[t][0], vlo[t][1], vhi[t][0], vhi[t][1]};
                    const bf16x8 vf = *reinterpret_cast<const bf16x8*>(&raw);
                    o[j][t0 + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_hi, o[j][t0 + t], 0, 0, 0);
                    o[j][t0 + t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_lo, o[j][t0 + t], 0, 0, 0);
                }
            }
        }
        if (more) stage_v(step_key(it), g0);
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

// heads per wave: two, or four where sixteen waves would be needed; 0: not held
int heads_per_wave(int heads, int dk, int dv) {
    const int hpw = heads <= 16 ? 2 : heads <= 32 && dk <= 128 && dv <= 128 ? 4 : 0;
    if (!hpw) return 0;
    const int waves = (heads + hpw - 1) / hpw;
    return (size_t)waves * 64 * dv + (size_t)score_cols(heads) * kTalkRow * 4 <= kLdsBytes ? hpw : 0;
}

template <int DK, int DV, int HPW, int MT>
int launch_one(const PagedAttendArgs& a, hipStream_t stream) {
    const int waves = (a.heads + HPW - 1) / HPW, q_tiles = (a.max_q + 15) / 16;
    const size_t lds = (size_t)waves * 64 * DV + (size_t)score_cols(a.heads) * kTalkRow * 4;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(talk_prompt_kernel<DK, DV, HPW, MT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    talk_prompt_kernel<DK, DV, HPW, MT><<<a.batch * q_tiles, 64 * waves, lds, stream>>>(a, q_tiles);
    return check_launch("talk_prompt");
}
template <int DK, int DV>
int launch_dims(const PagedAttendArgs& a, hipStream_t stream) {
    if constexpr (DK <= 128 && DV <= 128) {
        if (a.heads > 16) return launch_one<DK, DV, 4, 2>(a, stream);
    }
    return launch_one<DK, DV, 2, 1>(a, stream);
}
template <int DK>
int launch_key(const PagedAttendArgs& a, hipStream_t stream) {
    if (a.dv == 64) return launch_dims<DK, 64>(a, stream);
    if (a.dv == 128) return launch_dims<DK, 128>(a, stream);
    return launch_dims<DK, 256>(a, stream);
}

}  // namespace

bool talk_prompt_supported(int heads, int dk, int dv, int block_size) {
    return block_size % 64 == 0 && (dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128 || dv == 256) && heads_per_wave(heads, dk, dv) > 0;
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
