// Row ops of models that keep several copies of the residual stream (hyper-connections), and of those that look at the token before:
//   bigram_embed   x = embed[token] + bigram[row of (previous token, token)]
//   stream_mix     x_t <- sum_s mix[s][t] x_s + out[t] y, all streams at once from the old ones; u = sum_s in[s] x_s; RMS norm of u in equal groups of columns.
//                  y is a sublayer's output, or a scaled sum of two, each RMS-normed over the row first
//   token_shift    h + (h' - h) shift with h' the previous token's h, and mixes of that and ITS previous value, one per coefficient row (single tokens: inside stream_mix)
//   causal_conv    depthwise convolution over a sequence's last tokens, bias, silu
// Streams and sums are fp32.  HBM-bound row streams; one workgroup per row where a norm needs the whole row.
// What a later step needs of earlier rows lives in rings per state slot: row of position p at entry p % depth, one entry more than a step looks back, so the
// entry a single token writes is one nobody reads.  Portions of several tokens write theirs in a small launch behind.  Nothing is read before position 0: slots
// need no clearing when reused.
#include <type_traits>

#include "api_common.h"
#include "mixers.h"

namespace nvh {

namespace {

using BigramArgs = nvh_bigram_embed_desc;
using StreamMixArgs = nvh_stream_mix_desc;
using TokenShiftArgs = nvh_token_shift_desc;
using ConvArgs = nvh_causal_conv_desc;

// place of a row in its sequence's portion; null tables: row i is the one token of sequence i
struct RowPlace {
    int seq, first, last;                            // rows of the portion
};
__device__ __forceinline__ RowPlace row_place(const int32_t* row_seq, const int32_t* cu_rows, int row) {
    if (!cu_rows) return {row, row, row};
    const int s = row_seq[row];
    return {s, cu_rows[s], cu_rows[s + 1] - 1};
}

// one workgroup per row; the one of a portion's first row reads the sequence's last token and replaces it
template <typename T>
__global__ __launch_bounds__(256) void bigram_embed_kernel(const BigramArgs a) {
    const int row = blockIdx.x;
    const RowPlace at = row_place(a.row_seq, a.cu_rows, row);
    const int slot = a.state_slots[at.seq];
    const int64_t tok = a.tokens[row];
    int64_t prev = -1;
    if (row > at.first) prev = a.tokens[row - 1];
    else if (a.positions[row] > 0 && slot >= 0) prev = a.last_token[slot];
    __syncthreads();
    if (row == at.first && slot >= 0 && threadIdx.x == 0) a.last_token[slot] = a.tokens[at.last];
    const int64_t t = tok < 0 ? 0 : tok >= a.vocab ? a.vocab - 1 : tok;
    const int64_t b = prev < 0 ? a.buckets : (prev * a.mul_prev + tok * a.mul_cur) % a.buckets;
    const T* e = reinterpret_cast<const T*>(a.embed) + t * a.cols;
    const T* g = reinterpret_cast<const T*>(a.bigram) + (b < 0 ? b + a.buckets : b) * a.cols;
    for (int c = threadIdx.x * 8; c < a.cols; c += 2048) {
        const f32x8 u = act_ld8(e + c), v = act_ld8(g + c);
        act_st8(a.x + (int64_t)row * a.cols + c, f32x8{u.a + v.a, u.b + v.b});
    }
}

__device__ __forceinline__ f32x8 zero8() { return {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}; }
__device__ __forceinline__ void fma8(f32x8& acc, const f32x8& v, float w) {
    acc.a += v.a * w;
    acc.b += v.b * w;
}
__device__ __forceinline__ float sq8(const f32x8& v) { return sum4(v.a * v.a) + sum4(v.b * v.b); }

// sums of two values over the workgroup (up to 16 waves); lds: 32 floats
__device__ __forceinline__ void block_sum2(float& u, float& v, float* lds) {
    u = wave_sum64(u);
    v = wave_sum64(v);
    const int waves = blockDim.x >> 6;
    if ((threadIdx.x & 63) == 0) {
        lds[threadIdx.x >> 6] = u;
        lds[16 + (threadIdx.x >> 6)] = v;
    }
    __syncthreads();
    u = v = 0.f;
    for (int w = 0; w < waves; ++w) {
        u += lds[w];
        v += lds[16 + w];
    }
}

// row `back` tokens before `row` of a sequence (null: before position 0): this step's rows, or the ring
template <typename T>
__device__ __forceinline__ const T* earlier_row(const T* rows, int64_t stride, const T* ring, int depth, int cols, int row, int back, const RowPlace& at, int64_t pos, int slot) {
    if (row - back >= at.first) return rows + (int64_t)(row - back) * stride;
    if (pos < back || slot < 0) return nullptr;
    return ring + ((int64_t)slot * depth + (int)((pos - back) % depth)) * cols;
}
__device__ __forceinline__ f32x8 lerp8(const f32x8& h, const f32x8& before, const f32x8& mu) { return {h.a + (before.a - h.a) * mu.a, h.b + (before.b - h.b) * mu.b}; }

// a thread's 8-column pieces of all streams stay in registers from the update to the normed store.  S: streams held (the model's or the next size), CH: pieces
template <typename T, int S, int CH>
__global__ __launch_bounds__(1024) void stream_mix_kernel(const StreamMixArgs a) {
    extern __shared__ float lds[];                   // [32] sums, [groups] scales, sums of squares per unit of columns
    const int64_t row = blockIdx.x;
    const int threads = blockDim.x, n_str = a.streams;
    const float* xr = a.xin + row * a.xin_row;
    f32x8 x[CH][S], add[CH], u[CH];
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * threads) * 8;
        add[i] = zero8();
#pragma unroll
        for (int s = 0; s < S; ++s) x[i][s] = c < a.cols && s < n_str ? act_ld8(xr + s * a.xin_stream + c) : zero8();
        if (a.y && c < a.cols) add[i] = act_ld8(reinterpret_cast<const T*>(a.y) + row * a.y_stride + c);
    }
    if (a.y2) {
        f32x8 y2[CH];
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const int c = (threadIdx.x + i * threads) * 8;
            y2[i] = c < a.cols ? act_ld8(reinterpret_cast<const T*>(a.y2) + row * a.y2_stride + c) : zero8();
            sa += sq8(add[i]);
            sb += sq8(y2[i]);
        }
        block_sum2(sa, sb, lds);
        const float ia = a.y_scale / sqrtf(sa / a.n + a.eps), ib = a.y_scale / sqrtf(sb / a.n + a.eps);
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const int c = (threadIdx.x + i * threads) * 8;
            if (c >= a.cols) continue;
            const f32x8 wa = act_ld8(a.y_w + c), wb = act_ld8(a.y2_w + c);
            add[i] = {add[i].a * wa.a * ia + y2[i].a * wb.a * ib, add[i].b * wa.b * ia + y2[i].b * wb.b * ib};
        }
    }
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * threads) * 8;
        u[i] = zero8();
#pragma unroll
        for (int t = 0; t < S; ++t) {
            if (t >= n_str) continue;
            f32x8 v = x[i][t];
            if (a.y) {
                const float f = a.out[t];
                v = {add[i].a * f, add[i].b * f};
#pragma unroll
                for (int s = 0; s < S; ++s)
                    if (s < n_str) fma8(v, x[i][s], a.mix[s * n_str + t]);
                if (a.xout && c < a.cols) act_st8(a.xout + (row * n_str + t) * a.cols + c, v);
            }
            fma8(u[i], v, a.in ? a.in[t] : 1.f);
        }
        if (a.sum && c < a.cols) act_st8(a.sum + row * a.cols + c, u[i]);
    }
    if (!a.w) return;
    // ---- norm: every group of part columns by itself
    const int part = a.n / a.groups;
    float *inv = lds + 32, *unit = inv + a.groups;
    const bool whole = part % 8 == 0;                // a piece lies in one group
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int p = threadIdx.x + i * threads, c = p * 8;
        if (c >= a.cols) continue;
        if (whole) unit[p] = sq8(u[i]);
        else {
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                unit[c + k] = u[i].a[k] * u[i].a[k];
                unit[c + 4 + k] = u[i].b[k] * u[i].b[k];
            }
        }
    }
    __syncthreads();
    const int per = whole ? part / 8 : part;
    for (int g = threadIdx.x >> 6; g < a.groups; g += threads >> 6) {
        float s = 0.f;
        for (int e = threadIdx.x & 63; e < per; e += 64) s += unit[g * per + e];
        s = wave_sum64(s);
        if ((threadIdx.x & 63) == 0) inv[g] = 1.f / sqrtf(s / part + a.eps);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * threads) * 8;
        if (c >= a.cols) continue;
        const f32x8 w = act_ld8(a.w + c);            // (zero in the padding)
        f32x8 r;
        if (whole) {
            const int g = c / part;
            const float f = g < a.groups ? inv[g] : 0.f;
            r = {u[i].a * w.a * f, u[i].b * w.b * f};
        } else {
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const int g0 = (c + k) / part, g1 = (c + 4 + k) / part;
                r.a[k] = g0 < a.groups ? u[i].a[k] * w.a[k] * inv[g0] : 0.f;
                r.b[k] = g1 < a.groups ? u[i].b[k] * w.b[k] * inv[g1] : 0.f;
            }
        }
        if (a.h) act_st8(reinterpret_cast<T*>(a.h) + row * a.cols + c, r);
        if (a.packed) act_st8(reinterpret_cast<uint16_t*>(a.packed) + pack_index((int)row, c, a.cols), r);
        if (a.shift) {                               // single tokens: shift and mixes on the spot, the normed row goes to the ring
            const int slot = a.state_slots[row];
            const int64_t pos = a.positions[row];
            T* ring = reinterpret_cast<T*>(a.ring);
            const RowPlace at = {(int)row, (int)row, (int)row};
            const T* p1 = earlier_row((const T*)nullptr, 0, (const T*)ring, a.depth, a.cols, (int)row, 1, at, pos, slot);
            const T* p2 = a.mixes ? earlier_row((const T*)nullptr, 0, (const T*)ring, a.depth, a.cols, (int)row, 2, at, pos, slot) : nullptr;
#pragma unroll
            for (int k = 0; k < 4; ++k) {            // (the value the ring holds)
                r.a[k] = act_round(r.a[k], (const T*)nullptr);
                r.b[k] = act_round(r.b[k], (const T*)nullptr);
            }
            const f32x8 h1 = p1 ? act_ld8(p1 + c) : zero8(), h2 = p2 ? act_ld8(p2 + c) : zero8(), shift = act_ld8(a.shift + c);
            const f32x8 s0 = lerp8(r, h1, shift), s1 = lerp8(h1, h2, shift);
            uint16_t* dst = reinterpret_cast<uint16_t*>(a.shifted) + pack_index((int)row, c, a.cols);
            if (a.mixes == 0) act_st8(dst, s0);
            for (int k = 0; k < a.mixes; ++k) act_st8(dst + k * a.shifted_mix, lerp8(s0, s1, act_ld8(a.mu + (int64_t)k * a.cols + c)));
            if (slot >= 0) act_st8(ring + ((int64_t)slot * a.depth + (int)(pos % a.depth)) * a.cols + c, r);
        }
    }
}

// whether CNT rows from `row` on belong to one portion
template <int CNT>
__device__ __forceinline__ bool one_portion(const int32_t* row_seq, const int32_t* cu_rows, int row, int rows) {
    return CNT > 1 && cu_rows && row + CNT <= rows && row_seq[row] == row_seq[row + CNT - 1];
}

// grid (CNT rows each, column blocks of 2048).  Rows of one portion share the loads of coefficients and of each other; others go one by one
template <typename T, int CNT>
__global__ __launch_bounds__(256) void token_shift_kernel(const TokenShiftArgs a) {
    const int r0 = blockIdx.x * CNT, c = (blockIdx.y * 256 + threadIdx.x) * 8;
    if (c >= a.cols) return;
    const T* h = reinterpret_cast<const T*>(a.h);
    T* ring = reinterpret_cast<T*>(a.ring);
    const f32x8 shift = act_ld8(a.shift + c);
    auto put = [&](int row, int k, const f32x8& v) {
        if (a.packed) act_st8(reinterpret_cast<uint16_t*>(a.out) + k * a.out_mix + pack_index(row, c, a.cols), v);
        else act_st8(reinterpret_cast<T*>(a.out) + k * a.out_mix + (int64_t)row * a.cols + c, v);
    };
    auto run = [&](auto cnt, int row0) {             // decltype(cnt)::value rows of one portion
        constexpr int N = decltype(cnt)::value;
        const RowPlace at = row_place(a.row_seq, a.cu_rows, row0);
        const int slot = a.state_slots[at.seq];
        const int64_t pos = a.positions[row0];
        const T* p1 = earlier_row(h, a.h_stride, (const T*)ring, a.depth, a.cols, row0, 1, at, pos, slot);
        const T* p2 = a.mixes ? earlier_row(h, a.h_stride, (const T*)ring, a.depth, a.cols, row0, 2, at, pos, slot) : nullptr;
        f32x8 hv[N], before = p1 ? act_ld8(p1 + c) : zero8(), s1 = p2 ? act_ld8(p2 + c) : zero8();
#pragma unroll
        for (int i = 0; i < N; ++i) hv[i] = act_ld8(h + (int64_t)(row0 + i) * a.h_stride + c);
        s1 = lerp8(before, s1, shift);
        if (!a.cu_rows && slot >= 0) act_st8(ring + ((int64_t)slot * a.depth + (int)(pos % a.depth)) * a.cols + c, hv[0]);
        f32x8 sv[N];
#pragma unroll
        for (int i = 0; i < N; ++i) {
            sv[i] = lerp8(hv[i], before, shift);
            before = hv[i];
            if (a.mixes == 0) put(row0 + i, 0, sv[i]);
        }
        for (int k = 0; k < a.mixes; ++k) {
            const f32x8 mu = act_ld8(a.mu + (int64_t)k * a.cols + c);
#pragma unroll
            for (int i = 0; i < N; ++i) put(row0 + i, k, lerp8(sv[i], i ? sv[i ? i - 1 : 0] : s1, mu));
        }
    };
    if (one_portion<CNT>(a.row_seq, a.cu_rows, r0, a.rows)) {
        run(std::integral_constant<int, CNT>{}, r0);
    } else {
        for (int r = r0; r < r0 + CNT && r < a.rows; ++r) run(std::integral_constant<int, 1>{}, r);
    }
}

// grid (CNT rows each, column blocks of 2048).  TAPS: the kernel's size, 0: any (CNT 1)
template <typename T, int TAPS, int CNT>
__global__ __launch_bounds__(256) void causal_conv_kernel(const ConvArgs a) {
    const int r0 = blockIdx.x * CNT, c = (blockIdx.y * 256 + threadIdx.x) * 8, taps = TAPS ? TAPS : a.taps;
    if (c >= a.cols) return;
    const T* x = reinterpret_cast<const T*>(a.x);
    T* ring = reinterpret_cast<T*>(a.ring);
    const f32x8 bias = act_ld8(a.b + c);
    auto tap = [&](f32x8& acc, const f32x8& v, const f32x8& w) {
        acc.a += v.a * w.a;
        acc.b += v.b * w.b;
    };
    auto finish = [&](int row, f32x8 acc) {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            acc.a[k] = silu_f(acc.a[k]);
            acc.b[k] = silu_f(acc.b[k]);
        }
        if (a.packed) act_st8(reinterpret_cast<uint16_t*>(a.packed) + pack_index(row, c, a.cols), acc);
        if (a.out) act_st8(reinterpret_cast<T*>(a.out) + (int64_t)row * a.cols + c, acc);
    };
    auto before = [&](int row, int back, const RowPlace& at, int64_t pos, int slot) {
        const T* p = earlier_row(x, a.x_stride, (const T*)ring, a.taps, a.cols, row, back, at, pos, slot);
        return p ? act_ld8(p + c) : zero8();
    };
    if constexpr (TAPS > 0 && CNT > 1) {
        if (one_portion<CNT>(a.row_seq, a.cu_rows, r0, a.rows)) {
            const RowPlace at = row_place(a.row_seq, a.cu_rows, r0);
            const int slot = a.state_slots[at.seq];
            const int64_t pos = a.positions[r0];
            f32x8 v[CNT + TAPS - 1], w[TAPS];
#pragma unroll
            for (int i = 0; i < CNT; ++i) v[TAPS - 1 + i] = act_ld8(x + (int64_t)(r0 + i) * a.x_stride + c);
#pragma unroll
            for (int i = 0; i < TAPS - 1; ++i) v[i] = before(r0, TAPS - 1 - i, at, pos, slot);
#pragma unroll
            for (int j = 0; j < TAPS; ++j) w[j] = act_ld8(a.w + (int64_t)j * a.cols + c);
#pragma unroll
            for (int i = 0; i < CNT; ++i) {
                f32x8 acc = bias;
#pragma unroll
                for (int j = 0; j < TAPS; ++j) tap(acc, v[i + j], w[j]);
                finish(r0 + i, acc);
            }
            return;
        }
    }
    for (int row = r0; row < r0 + CNT && row < a.rows; ++row) {
        const RowPlace at = row_place(a.row_seq, a.cu_rows, row);
        const int slot = a.state_slots[at.seq];
        const int64_t pos = a.positions[row];
        f32x8 acc = bias;
        const f32x8 own = act_ld8(x + (int64_t)row * a.x_stride + c);
        if constexpr (TAPS > 0) {
            f32x8 v[TAPS > 1 ? TAPS - 1 : 1];
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) v[j] = before(row, TAPS - 1 - j, at, pos, slot);
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) tap(acc, v[j], act_ld8(a.w + (int64_t)j * a.cols + c));
        } else {
            for (int j = 0; j < taps - 1; ++j) tap(acc, before(row, taps - 1 - j, at, pos, slot), act_ld8(a.w + (int64_t)j * a.cols + c));
        }
        tap(acc, own, act_ld8(a.w + (int64_t)(taps - 1) * a.cols + c));
        finish(row, acc);
        if (!a.cu_rows && slot >= 0) act_st8(ring + ((int64_t)slot * a.taps + (int)(pos % a.taps)) * a.cols + c, own);
    }
}

// the last rows of every portion into its ring; grid (sequences, depth, column blocks)
template <typename T>
__global__ __launch_bounds__(256) void ring_store_kernel(T* __restrict__ ring, const T* __restrict__ rows, int64_t stride, int depth, int cols, const int32_t* __restrict__ cu_rows,
                                                         const int64_t* __restrict__ positions, const int32_t* __restrict__ state_slots) {
    const int seq = blockIdx.x, row = cu_rows[seq + 1] - 1 - blockIdx.y, slot = state_slots[seq], c = (blockIdx.z * 256 + threadIdx.x) * 8;
    if (row < cu_rows[seq] || slot < 0 || c >= cols) return;
    act_st8(ring + ((int64_t)slot * depth + (int)(positions[row] % depth)) * cols + c, act_ld8(rows + (int64_t)row * stride + c));
}

template <typename T>
void ring_store(void* ring, const void* rows, int64_t stride, int depth, int cols, int sequences, const int32_t* cu_rows, const int64_t* positions, const int32_t* slots,
                hipStream_t stream) {
    ring_store_kernel<T><<<dim3(sequences, depth, (cols + 2047) / 2048), 256, 0, stream>>>((T*)ring, (const T*)rows, stride, depth, cols, cu_rows, positions, slots);
}

template <typename T, int S>
int mix_s(const StreamMixArgs& a, hipStream_t stream) {
    const int pieces = a.cols / 8;
    const int threads = pieces <= 256 ? 256 : pieces <= 512 ? 512 : 1024;
    const size_t lds = (32 + a.groups + (a.w ? (a.n / a.groups % 8 == 0 ? a.cols / 8 : a.cols) : 0)) * 4;
    auto go = [&](auto ch) {
        auto* fn = stream_mix_kernel<T, S, decltype(ch)::value>;
        if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        fn<<<a.rows, threads, lds, stream>>>(a);
    };
    if (pieces <= 1024) go(std::integral_constant<int, 1>{});
    else go(std::integral_constant<int, 2>{});
    return check_launch("stream_mix");
}
template <typename T>
int mix_t(const StreamMixArgs& a, hipStream_t stream) {
    switch (a.streams) {
        case 1: return mix_s<T, 1>(a, stream);
        case 2: return mix_s<T, 2>(a, stream);
        case 3: return mix_s<T, 3>(a, stream);
        case 4: return mix_s<T, 4>(a, stream);
        default: return a.streams <= 8 ? mix_s<T, 8>(a, stream) : mix_s<T, 16>(a, stream);
    }
}

template <typename T>
int shift_t(const TokenShiftArgs& a, hipStream_t stream) {
    const unsigned blocks = (a.cols + 2047) / 2048;
    if (a.cu_rows && a.rows >= 1024) token_shift_kernel<T, 4><<<dim3((a.rows + 3) / 4, blocks), 256, 0, stream>>>(a);
    else token_shift_kernel<T, 1><<<dim3(a.rows, blocks), 256, 0, stream>>>(a);
    if (a.cu_rows) ring_store<T>(a.ring, a.h, a.h_stride, a.depth, a.cols, a.sequences, a.cu_rows, a.positions, a.state_slots, stream);
    return check_launch("token_shift");
}

template <typename T>
int conv_t(const ConvArgs& a, hipStream_t stream) {
    const unsigned blocks = (a.cols + 2047) / 2048;
    auto go = [&](auto taps) {
        if (a.cu_rows && a.rows >= 1024) causal_conv_kernel<T, decltype(taps)::value, 8><<<dim3((a.rows + 7) / 8, blocks), 256, 0, stream>>>(a);
        else causal_conv_kernel<T, decltype(taps)::value, 1><<<dim3(a.rows, blocks), 256, 0, stream>>>(a);
    };
    if (a.taps == 4) go(std::integral_constant<int, 4>{});
    else if (a.taps == 3) go(std::integral_constant<int, 3>{});
    else if (a.taps == 2) go(std::integral_constant<int, 2>{});
    else causal_conv_kernel<T, 0, 1><<<dim3(a.rows, blocks), 256, 0, stream>>>(a);
    if (a.cu_rows) ring_store<T>(a.ring, a.x, a.x_stride, a.taps, a.cols, a.sequences, a.cu_rows, a.positions, a.state_slots, stream);
    return check_launch("causal_conv");
}

}  // namespace

}  // namespace nvh

using namespace nvh;

extern "C" {

int nvh_bigram_embed(const nvh_bigram_embed_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "bigram_embed: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("bigram_embed");
    REQUIRE(d->x && d->tokens && d->positions && d->state_slots && d->embed && d->bigram && d->last_token && (!d->cu_rows == !d->row_seq), NVH_E_NULL, "bigram_embed: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->vocab > 0 && d->buckets > 0, NVH_E_SHAPE, "bigram_embed: rows %d cols %d (%%8) vocab %d buckets %lld", d->rows, d->cols,
            d->vocab, (long long)d->buckets);
    REQUIRE(aligned16(d->x) && aligned16(d->embed) && aligned16(d->bigram), NVH_E_ALIGN, "bigram_embed: pointers must be 16-byte aligned");
    if (dtype == NVH_F32) bigram_embed_kernel<float><<<d->rows, 256, 0, (hipStream_t)stream>>>(*d);
    else bigram_embed_kernel<uint16_t><<<d->rows, 256, 0, (hipStream_t)stream>>>(*d);
    return check_launch("bigram_embed");
}

int nvh_stream_mix(const nvh_stream_mix_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "stream_mix: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("stream_mix");
    REQUIRE(d->xin && (!d->y || (d->mix && d->out)) && (!d->y2 || (d->y && d->y_w && d->y2_w)) && (!d->xout || d->y) && (!d->w || d->h || d->packed || d->shift) && (d->w || d->sum || d->xout), NVH_E_NULL,
            "stream_mix: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->cols <= 16384 && d->n > 0 && d->n <= d->cols && d->streams > 0 && d->streams <= 16 && d->groups > 0 &&
            d->n % d->groups == 0, NVH_E_SHAPE, "stream_mix: cols %d (%%8, <= 16384), %d columns in %d groups, %d streams (<= 16)", d->cols, d->n, d->groups, d->streams);
    REQUIRE((!d->packed && !d->shift) || (dtype == NVH_BF16 && d->cols % 32 == 0), NVH_E_SHAPE, "stream_mix: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(!d->shift || (d->w && d->ring && d->shifted && d->positions && d->state_slots && d->mixes >= 0 && d->mixes <= 64 && (!d->mixes || d->mu) && d->depth == (d->mixes ? 3 : 2) &&
            d->shifted_mix % 8 == 0 && aligned16(d->shift) && aligned16(d->mu) && aligned16(d->ring) && aligned16(d->shifted)), NVH_E_SHAPE, "stream_mix: shift of %d mixes, ring of %d",
            d->mixes, d->depth);
    REQUIRE(d->xin_row % 8 == 0 && d->xin_stream % 8 == 0 && (!d->y || (d->y_stride % 8 == 0 && d->y_stride >= d->cols)) && (!d->y2 || (d->y2_stride % 8 == 0 && d->y2_stride >= d->cols)),
            NVH_E_STRIDE, "stream_mix: row strides");
    REQUIRE(aligned16(d->xin) && aligned16(d->xout) && aligned16(d->y) && aligned16(d->y2) && aligned16(d->y_w) && aligned16(d->y2_w) && aligned16(d->w) && aligned16(d->sum) && aligned16(d->h) &&
            aligned16(d->packed), NVH_E_ALIGN, "stream_mix: pointers must be 16-byte aligned");
    return dtype == NVH_F32 ? mix_t<float>(*d, (hipStream_t)stream) : mix_t<uint16_t>(*d, (hipStream_t)stream);
}

int nvh_token_shift(const nvh_token_shift_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "token_shift: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("token_shift");
    REQUIRE(d->h && d->shift && d->out && d->ring && d->positions && d->state_slots && (!d->mixes || d->mu) && (!d->cu_rows == !d->row_seq), NVH_E_NULL, "token_shift: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->mixes >= 0 && d->mixes <= 64 && d->depth == (d->mixes ? 3 : 2) && (!d->cu_rows || (d->sequences > 0 && d->sequences <= 65535)),
            NVH_E_SHAPE, "token_shift: cols %d (%%8), %d mixes, ring of %d", d->cols, d->mixes, d->depth);
    REQUIRE(!d->packed || (dtype == NVH_BF16 && d->cols % 32 == 0), NVH_E_SHAPE, "token_shift: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(d->h_stride % 8 == 0 && d->h_stride >= d->cols && d->out_mix % 8 == 0, NVH_E_STRIDE, "token_shift: strides");
    REQUIRE(aligned16(d->h) && aligned16(d->shift) && aligned16(d->mu) && aligned16(d->out) && aligned16(d->ring), NVH_E_ALIGN, "token_shift: pointers must be 16-byte aligned");
    return dtype == NVH_F32 ? shift_t<float>(*d, (hipStream_t)stream) : shift_t<uint16_t>(*d, (hipStream_t)stream);
}

int nvh_causal_conv(const nvh_causal_conv_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "causal_conv: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("causal_conv");
    REQUIRE(d->x && d->w && d->b && (d->out || d->packed) && d->ring && d->positions && d->state_slots && (!d->cu_rows == !d->row_seq), NVH_E_NULL, "causal_conv: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->taps > 0 && d->taps <= 65535 && (!d->cu_rows || (d->sequences > 0 && d->sequences <= 65535)), NVH_E_SHAPE,
            "causal_conv: cols %d (%%8), %d taps", d->cols, d->taps);
    REQUIRE(!d->packed || (dtype == NVH_BF16 && d->cols % 32 == 0), NVH_E_SHAPE, "causal_conv: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(d->x_stride % 8 == 0 && d->x_stride >= d->cols, NVH_E_STRIDE, "causal_conv: row stride");
    REQUIRE(aligned16(d->x) && aligned16(d->w) && aligned16(d->b) && aligned16(d->out) && aligned16(d->packed) && aligned16(d->ring), NVH_E_ALIGN, "causal_conv: pointers must be 16-byte aligned");
    return dtype == NVH_F32 ? conv_t<float>(*d, (hipStream_t)stream) : conv_t<uint16_t>(*d, (hipStream_t)stream);
}

}  // extern "C"
