// Kernels over single query rows (decoding) that stream keys and values from pages, [page][kv head][block_size keys | block_size values], with windows, kept first
// tokens and sinks.  Where the scores of a unit of keys come from is a policy: the product of the query with the keys, or scores another launch left in memory.
// A sink is an entry of the softmax with score sink[head], no key and no value: it starts the running maximum and sum.
// Keys a window hides are not read: the walk covers the tiles of the kept first tokens, then those of the window.
#pragma once
#include <type_traits>

#include "mixers.h"

namespace nvh {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

// ------------------------------------------------------------------------------------------------ rows, any type and size
// one workgroup per (row, head); 64 keys at a time: 4 lanes per key for the scores, one thread per value column for the sums.
// TALK: a score is this head's row of the mixing matrix times the keys' scores of all heads in a.scores.
template <typename T, bool TALK = false>
__global__ __launch_bounds__(256) void paged_rows_generic_kernel(const PagedAttendArgs a) {
    constexpr int OC = 8;                            // value columns per thread: dv <= 2048
    extern __shared__ float q_lds[];                 // [dk] (TALK: [heads])
    __shared__ float p_lds[64];
    const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, g = head / (a.heads / a.kv_heads);
    const int seq = a.row_seq ? a.row_seq[row] : row;
    const int pos = (int)a.positions[row];
    const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)row * a.q_stride + head * a.dk;
    if constexpr (TALK) {
        for (int i = tid; i < a.heads; i += 256) q_lds[i] = a.talk[head * a.heads + i];
    } else {
        for (int i = tid; i < a.dk; i += 256) q_lds[i] = act_ld(q + i);
    }
    float o[OC], m = -INFINITY, l = 0.f;
    if (a.sink) {
        m = a.sink[head] * kLog2e;
        l = 1.f;
    }
#pragma unroll
    for (int j = 0; j < OC; ++j) o[j] = 0.f;
    const float sc = TALK ? kLog2e : a.scale * kLog2e;
    const int64_t head_elems = (int64_t)a.block_size * (a.dk + a.dv);
    __syncthreads();
    auto head_base = [&](int key) {
        const int64_t page = a.block_tables[seq * a.bt_stride + key / a.block_size];
        return reinterpret_cast<const T*>(a.cache) + (page * a.kv_heads + g) * head_elems;
    };
    const int lo = first_seen(pos, a.window, a.chunk);
    const VisibleTiles vis = visible_from(lo, pos, a.keep_first);
    for (int it = 0; it < vis.count; ++it) {
        const int t0 = vis.tile(it) * 64, key = t0 + (tid >> 2);
        const bool sees = key <= pos && (key >= lo || key < a.keep_first);
        float s = 0.f;
        if (TALK && sees && it * 64 < a.span) {
            const int cols = score_cols(a.heads);
            const float* r = a.scores + ((int64_t)row * a.span + it * 64 + (tid >> 2)) * cols;
            for (int i = tid & 3; i < a.heads; i += 4) s += r[i] * q_lds[i];
        } else if (!TALK && sees) {
            const T* r = head_base(key) + (int64_t)(key % a.block_size) * a.dk;
            for (int i = (tid & 3) * 4; i < a.dk; i += 16) {
                const f32x4 v = act_ld4(r + i);
                s += v[0] * q_lds[i] + v[1] * q_lds[i + 1] + v[2] * q_lds[i + 2] + v[3] * q_lds[i + 3];
            }
        }
        s += __shfl_xor(s, 1);
        s += __shfl_xor(s, 2);
        if ((tid & 3) == 0) p_lds[tid >> 2] = sees ? s * sc : -INFINITY;
        __syncthreads();
        float v = p_lds[tid & 63], mx = v;
        for (int d = 1; d < 64; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
        const float m_new = fmaxf(m, mx), m_use = m_new == -INFINITY ? 0.f : m_new, alpha = exp2f(m - m_use);
        v = exp2f(v - m_use);
        float sum = v;
        for (int d = 1; d < 64; d <<= 1) sum += __shfl_xor(sum, d);
        l = l * alpha + sum;
        m = m_new;
        __syncthreads();
        if (tid < 64) p_lds[tid] = v;
        __syncthreads();
#pragma unroll
        for (int j = 0; j < OC; ++j) o[j] *= alpha;
        for (int k = 0; k < 64; ++k) {
            const float p = p_lds[k];
            if (p == 0.f) continue;                  // (unseen, or a weight that vanished)
            const T* r = head_base(t0 + k) + (int64_t)a.block_size * a.dk + (int64_t)((t0 + k) % a.block_size) * a.dv;
#pragma unroll
            for (int j = 0; j < OC; ++j)
                if (tid + 256 * j < a.dv) o[j] += p * act_ld(r + tid + 256 * j);
        }
        __syncthreads();
    }
    const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
    for (int j = 0; j < OC; ++j) {
        const int c = tid + 256 * j;
        if (256 * j >= a.dv) continue;
        if (a.o_cos_sin) {                           // (pairs of columns lie in neighbouring lanes)
            const float other = __shfl_xor(o[j], 1);
            if (c < a.o_rot) {
                const float* cs = a.o_cos_sin + (int64_t)(pos < a.max_position ? pos : a.max_position - 1) * a.o_rot;
                const float co = cs[c / 2], si = cs[a.o_rot / 2 + c / 2];
                o[j] = c & 1 ? o[j] * co - other * si : o[j] * co + other * si;
            }
        }
        if (c >= a.dv) continue;
        if (a.out) act_st(reinterpret_cast<T*>(a.out) + (int64_t)row * a.out_stride + head * a.dv + c, o[j] * inv);
        if (a.out_packed) act_st(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(row, head * a.dv + c, a.heads * a.dv), o[j] * inv);
    }
}

// ------------------------------------------------------------------------------------------------ rows, streaming (bf16)
// grid (splits, kv heads x passes, rows), 4 waves.  A wave takes units of 32 keys: its keys come as MFMA fragments straight from the page (16 rows x 64 bytes
// per load), scores of all the pass's heads in one product (lane = head, 8 keys); weights go through a few LDS words to the lanes that hold the values'
// rows (16 bytes per lane), which sum them on the vector pipe.  Loads of the next unit's keys are issued behind the scores of this one, its values behind the
// sums, so about a unit per wave is always in flight.  Waves and splits are merged once.
// Split records (sums, maximum, sum of weights per head): 16-byte write-through stores, drained by every storing wave, then a ticket per (row, key/value
// head, pass); the last workgroup to arrive reads all records past the L1 and merges them in split order.
constexpr int kThroughAux = 16;                      // cache policy of the buffer accesses: sc1
typedef __amdgpu_buffer_rsrc_t RecordBuf;
__device__ __forceinline__ RecordBuf record_buffer(float* base, uint32_t bytes) { return __builtin_amdgcn_make_buffer_rsrc(base, 0, (int)bytes, 0x00020000); }
__device__ __forceinline__ void st16_through(RecordBuf rb, uint32_t byte_off, f32x4 v) {
    __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v), rb, (int)byte_off, 0, kThroughAux);
}
__device__ __forceinline__ f32x4 ld16_through(RecordBuf rb, uint32_t byte_off) {
    return __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(rb, (int)byte_off, 0, kThroughAux));
}

// Scores of a unit of 32 keys, left as s[t][r]: head lq of the pass, key 16 t + 4 lg + r; a softmax of base 2 takes them times factor().
// keys as MFMA fragments straight from the page
template <int DK>
struct KeyScores {
    static constexpr int STEPS = DK / 32;
    bf16x8_s q[STEPS];                               // B operand: column = head lq (past the last one: that one again, not used)
    bf16x8_s kd[2][STEPS];
    __device__ __forceinline__ KeyScores(const PagedAttendArgs& a, int row, int h0, int nh, int lq, int lg) {
        const uint16_t* qr = reinterpret_cast<const uint16_t*>(a.q) + (int64_t)row * a.q_stride + (int64_t)(h0 + (lq < nh ? lq : nh - 1)) * DK + 8 * lg;
#pragma unroll
        for (int st = 0; st < STEPS; ++st) q[st] = *reinterpret_cast<const bf16x8_s*>(qr + 32 * st);
    }
    static __device__ __forceinline__ int key_width(const PagedAttendArgs&) { return DK; }
    static __device__ __forceinline__ float factor(const PagedAttendArgs& a) { return a.scale * kLog2e; }
    // unit of the row's visible keys that starts at key k0; head: the page's rows of the key/value head; rows past the query's own position repeat it: not seen
    __device__ __forceinline__ void load(const PagedAttendArgs& a, int, int, int k0, int pos, const uint16_t* head, int lq, int lg) {
        const int o0 = k0 % a.block_size - k0;
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const int key = k0 + 16 * t + lq;
            const uint16_t* p = head + (int64_t)((key < pos ? key : pos) + o0) * DK + 8 * lg;
#pragma unroll
            for (int st = 0; st < STEPS; ++st) kd[t][st] = *reinterpret_cast<const bf16x8_s*>(p + 32 * st);
        }
    }
    __device__ __forceinline__ void product(f32x4 (&s)[2]) const {
#pragma unroll
        for (int st = 0; st < STEPS; ++st)
#pragma unroll
            for (int t = 0; t < 2; ++t)
                s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kd[t][st]), __builtin_bit_cast(bf16x8_t, q[st]), s[t], 0, 0, 0);
    }
};

template <typename Scores, int DV, int R>
__global__ __launch_bounds__(256) void paged_rows_kernel(const PagedAttendArgs a) {
    constexpr int UK = 32, LPR = DV / 8, SLOTS = 64 / LPR, NV = UK / SLOTS;      // lanes per row of values, rows per load, loads
    constexpr int RECW = DV + 4;                     // floats of one head's record in LDS: sums, max, sum
    __shared__ __attribute__((aligned(16))) float rec[4 * R * RECW];
    __shared__ __attribute__((aligned(16))) float weights[4][UK * R + R];      // per wave: [key][head], then the factors of the old sums
    __shared__ int last_flag;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4, ll = lane % LPR, ls = lane / LPR;
    const int split = blockIdx.x, row = blockIdx.z, ratio = a.heads / a.kv_heads, passes = (ratio + kRowsHeads - 1) / kRowsHeads;
    const int g = blockIdx.y / passes, h0 = g * ratio + (blockIdx.y - g * passes) * kRowsHeads;
    const int nh = (g + 1) * ratio - h0 < R ? (g + 1) * ratio - h0 : R;
    const int pos = (int)a.positions[row];
    const int lo = first_seen(pos, a.window, a.chunk);
    const VisibleTiles vis = visible_from(lo, pos, a.keep_first);
    const int per = (vis.count + a.splits - 1) / a.splits, t_beg = split * per, t_end = t_beg + per < vis.count ? t_beg + per : vis.count;
    const int units = t_end > t_beg ? (t_end - t_beg) * (64 / UK) : 0;

    Scores scores(a, row, h0, nh, lq, lg);
    float m = -INFINITY, l = 0.f, o[R][8];           // maximum of head lq; this lane's share of its sum; columns 8 ll .. of every head, keys of slot ls
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) o[r][e] = 0.f;
    const float sc = Scores::factor(a);
    const int dk = Scores::key_width(a);
    const int64_t head_elems = (int64_t)a.block_size * (dk + DV);
    const int32_t* table = a.block_tables + (int64_t)row * a.bt_stride;
    auto unit_key = [&](int u) { return vis.tile(t_beg + u / (64 / UK)) * 64 + (u % (64 / UK)) * UK; };
    u32x4 vd[NV];
    auto load_k = [&](int u, int k0, int page) {
        scores.load(a, row, t_beg * (64 / UK) + u, k0, pos, reinterpret_cast<const uint16_t*>(a.cache) + ((int64_t)page * a.kv_heads + g) * head_elems, lq, lg);
    };
    auto load_v = [&](int k0, int page) {
        const uint16_t* base = reinterpret_cast<const uint16_t*>(a.cache) + ((int64_t)page * a.kv_heads + g) * head_elems + (int64_t)a.block_size * dk + 8 * ll;
        const int o0 = k0 % a.block_size - k0;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int key = k0 + i * SLOTS + ls;
            vd[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(base + (int64_t)((key < pos ? key : pos) + o0) * DV));
        }
    };
    // a unit that starts past the query's position (the second half of its tile) holds nothing to see
    auto live = [&](int u) { return u < units && unit_key(u) <= pos; };
    auto page_of = [&](int u) { return table[unit_key(u < units ? u : 0) / a.block_size]; };
    float* wl = weights[wave];
    // one unit: scores, (the next unit's keys asked for,) softmax, sums, (its values asked for)
    auto take = [&](auto morec, int k0, int next, int next_key, int next_page) {
        constexpr bool MORE = decltype(morec)::value;
        f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        scores.product(s);
        if constexpr (MORE) load_k(next, next_key, next_page);
        float mx = m;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = k0 + 16 * t + 4 * lg + r;
                const float unseen = key <= pos && (key >= lo || key < a.keep_first) ? 0.f : -INFINITY;
                s[t][r] = s[t][r] * sc + unseen;
                mx = fmaxf(mx, s[t][r]);
            }
        mx = max_xor16(mx);
        mx = max_xor32(mx);
        const float m_use = mx == -INFINITY ? 0.f : mx, alpha = fast_exp2(m - m_use);
        float sum = 0.f;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                s[t][r] = fast_exp2(s[t][r] - m_use);
                sum += s[t][r];
            }
        l = l * alpha + sum;
        m = mx;
        if (lq < R) {
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) wl[(16 * t + 4 * lg + r) * R + lq] = s[t][r];
            if (lg == 0) wl[UK * R + lq] = alpha;
        }
        wave_lds_sync();
        float p[NV][R];
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float f = wl[UK * R + r];
#pragma unroll
            for (int e = 0; e < 8; ++e) o[r][e] *= f;
        }
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int r = 0; r < R; ++r) p[i][r] = wl[(i * SLOTS + ls) * R + r];
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int d = 0; d < 4; ++d) {
                const float v0 = bf16_lo(vd[i][d]), v1 = bf16_hi(vd[i][d]);
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    o[r][2 * d] += p[i][r] * v0;
                    o[r][2 * d + 1] += p[i][r] * v1;
                }
            }
        wave_lds_sync();                             // (the next unit's weights go to the same words)
        if constexpr (MORE) load_v(next_key, next_page);
    };
    int u = wave;
    if (live(u)) {
        {
            const int k0 = unit_key(u), page = page_of(u);
            load_k(u, k0, page);
            load_v(k0, page);
        }
        int next_page = page_of(u + 4);
        while (live(u + 4)) {
            const int page = next_page;
            next_page = page_of(u + 8);
            take(std::integral_constant<bool, true>{}, unit_key(u), u + 4, unit_key(u + 4), page);
            u += 4;
        }
        take(std::integral_constant<bool, false>{}, unit_key(u), 0, 0, 0);
    }
    // ---- merge the value slots of the wave, then the waves
    l = sum_xor16(l);
    l = sum_xor32(l);
#pragma unroll
    for (int r = 0; r < R; ++r) {
        float* dst = rec + (wave * R + r) * RECW;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float v = o[r][e];
            if constexpr (SLOTS >= 8) v += __shfl_xor(v, 8);
            if constexpr (SLOTS >= 4) v = sum_xor16(v);
            v = sum_xor32(v);
            if (ls == 0) dst[8 * ll + e] = v;
        }
        if (lane == r) {                             // (lane lq = r, lg = 0 holds head r's maximum and sum)
            dst[DV] = m;
            dst[DV + 1] = l;
        }
    }
    __syncthreads();
    constexpr int PIECES = DV / 4, RECB = (DV + 4) * 4;                        // 4-column pieces of a head; bytes of a split record
    auto finish = [&](int r, int c, f32x4 v) {       // 4 normalised columns of head h0 + r
        if (a.o_cos_sin) v = turn_back(v, a.o_cos_sin, pos, a.max_position, a.o_rot, c);
        const int col = (h0 + r) * DV + c;
        if (a.out) act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)row * a.out_stride + col, v);
        if (a.out_packed) act_st4(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(row, col, a.heads * DV), v);
    };
    const RecordBuf records = record_buffer(a.splits > 1 ? a.part + ((int64_t)row * a.heads + h0) * a.splits * (DV + 4) : nullptr, a.splits > 1 ? (uint32_t)nh * a.splits * RECB : 0u);
    for (int e = tid; e < nh * PIECES; e += 256) {
        const int r = e / PIECES, c = (e - r * PIECES) * 4;
        float mw[4], mx = -INFINITY, sum = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            mw[w] = rec[(w * R + r) * RECW + DV];
            mx = fmaxf(mx, mw[w]);
        }
        const float sink = a.splits == 1 && a.sink ? a.sink[h0 + r] * kLog2e : -INFINITY;
        mx = fmaxf(mx, sink);
        const float m_use = mx == -INFINITY ? 0.f : mx;
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float f = fast_exp2(mw[w] - m_use);
            v += *reinterpret_cast<const f32x4*>(rec + (w * R + r) * RECW + c) * f;
            sum += rec[(w * R + r) * RECW + DV + 1] * f;
        }
        if (a.splits == 1) {
            sum += fast_exp2(sink - m_use);
            finish(r, c, v * (sum > 0.f ? 1.f / sum : 0.f));
        } else {
            const uint32_t at = (uint32_t)(r * a.splits + split) * RECB;
            st16_through(records, at + c * 4, v);
            if (c == 0) st16_through(records, at + DV * 4, f32x4{mx, sum, 0.f, 0.f});
        }
    }
    if (a.splits == 1) return;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    uint32_t* ticket = a.tickets + ((int64_t)row * gridDim.y + blockIdx.y) * kAttendTicketWords;
    if (tid == 0) last_flag = __hip_atomic_fetch_add(ticket, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (uint32_t)a.splits - 1;
    __syncthreads();
    if (!last_flag) return;
    if (tid == 0) __hip_atomic_store(ticket, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    constexpr int SB = 4;                            // records asked for at a time
    for (int e = tid; e < nh * PIECES; e += 256) {
        const int r = e / PIECES, c = (e - r * PIECES) * 4;
        float mx = a.sink ? a.sink[h0 + r] * kLog2e : -INFINITY, sum = mx > -INFINITY ? 1.f : 0.f;
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < a.splits; s0 += SB) {
            f32x4 ml[SB], o4[SB];
#pragma unroll
            for (int s = 0; s < SB; ++s) {
                const uint32_t at = (uint32_t)(r * a.splits + (s0 + s < a.splits ? s0 + s : a.splits - 1)) * RECB;
                ml[s] = ld16_through(records, at + DV * 4);
                o4[s] = ld16_through(records, at + c * 4);
            }
            float top = mx;
#pragma unroll
            for (int s = 0; s < SB; ++s)
                if (s0 + s < a.splits) top = fmaxf(top, ml[s][0]);
            const float m_use = top == -INFINITY ? 0.f : top, old = fast_exp2(mx - m_use);
            v *= old;
            sum *= old;
            mx = top;
#pragma unroll
            for (int s = 0; s < SB; ++s)
                if (s0 + s < a.splits) {
                    const float f = fast_exp2(ml[s][0] - m_use);
                    v += o4[s] * f;
                    sum += ml[s][1] * f;
                }
        }
        finish(r, c, v * (sum > 0.f ? 1.f / sum : 0.f));
    }
}

}  // namespace nvh
