// Real-gated linear recurrent unit with a causal depthwise convolution in front of it:
//   u = conv(x)           y-branch gate applied at the end
//   r = sigmoid(ra u), i = sigmoid(ri u)            block-diagonal maps (MFMA)
//   log a = -rate r ; S = a S + sqrt(1 - a^2) i u ; out = S gelu(y)
// The recurrence and everything that enters it besides u is fp32; u is rounded once to the activation type.
//
// Prompt portions (launch_rglru_chunks): a portion is cut into chunks of 64 tokens that are scanned in parallel —
//   gates kernel   one workgroup per (chunk, diagonal block): convolution into LDS, both gates on MFMA tiles, and the scan of the chunk IN the
//                  accumulator layout (a lane holds 4 consecutive tokens of one channel, the 4 lane groups 16 consecutive ones: compose 4 in
//                  the lane, two shuffles across the groups, a carry over the 16-token tiles).  Writes the scan from zero and the running
//                  product of the decays; a portion's first chunk starts from the sequence's state instead and is final.
//   apply kernel   carries the chunk totals of the earlier chunks of the portion, out = S gelu(y), and leaves state + convolution inputs.
// The state is read by the first kernel and written by the second only, so no workgroup can see a half-updated one.
// Decode (launch_rglru_step): one workgroup per 16 channels and 32 sequences does all of it in one launch.  Convolution inputs live in a ring of
// `taps` entries (input of position p at entry p % taps): the entry a step writes is the one no workgroup of that step reads.
// A sequence's first token (position 0) takes state and earlier inputs as zero instead of reading them: slots need no clearing when reused.
// Bytes per (token, channel), prompt form: 2 (x) + 8 (scan, decay out) + 8 (in) + 2 (y) + 2 (out).
#include "hybrid.h"

namespace nvh {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
constexpr int CH = kRglruChunk;

__device__ __forceinline__ void decay_and_input(float rate, float r, float ig, float u, float& a, float& b) {
    const float log_a = -rate * r;
    a = __expf(log_a);
    b = sqrtf(-expm1f(2.f * log_a)) * ig * u;
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

// ------------------------------------------------------------------------------------------------ prompt portions, MFMA form (bf16)
__global__ __launch_bounds__(256) void rglru_gates_kernel(const RglruArgs a) {
    extern __shared__ __attribute__((aligned(16))) uint16_t u_lds[];           // [CH][block + 8]
    const int chunk = blockIdx.x, blk = blockIdx.y;
    const int row0 = a.chunks[chunk * 4], n = a.chunks[chunk * 4 + 1], seq = a.chunks[chunk * 4 + 2], kth = a.chunks[chunk * 4 + 3];
    const int seq_row0 = row0 - kth * CH;
    const int slot = a.state_slots[seq];
    const int64_t pos0 = a.positions[seq_row0];
    const int ld = a.block + 8, oct = a.block / 8;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;

    // ---- u of the chunk into LDS: a thread owns 8 channels and a run of tokens, eight at a time
    for (int ob = 0; ob < oct; ob += 256) {
        const int width = oct - ob < 256 ? oct - ob : 256;
        const int segs = 256 / width, seg_len = (CH + segs - 1) / segs;
        const int o = ob + tid % width, seg = tid / width;
        if (seg >= segs) continue;
        const int ch = blk * a.block + o * 8;
        for (int t0 = seg * seg_len; t0 < (seg + 1) * seg_len && t0 < CH; t0 += 8) {
            const int cnt = (seg + 1) * seg_len - t0 < 8 ? (seg + 1) * seg_len - t0 : 8;
            float acc[8][8];
            const f32x4 b0 = *reinterpret_cast<const f32x4*>(a.conv_b + ch), b1 = *reinterpret_cast<const f32x4*>(a.conv_b + ch + 4);
#pragma unroll
            for (int i = 0; i < 8; ++i)
#pragma unroll
                for (int k = 0; k < 8; ++k) acc[i][k] = k < 4 ? b0[k] : b1[k - 4];
            for (int j = 0; j < a.taps; ++j) {
                const float* w = a.conv_w + (int64_t)j * a.width + ch;
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const int t = t0 + i;
                    if (i < cnt && t < n) {
                        const uint16_t* p = conv_input<uint16_t>(a, seq_row0, kth * CH + t - (a.taps - 1) + j, pos0, slot, ch);
                        if (p) fma8(acc[i], *reinterpret_cast<const u32x4*>(p), w);
                    }
                }
            }
#pragma unroll
            for (int i = 0; i < 8; ++i)
                if (i < cnt && t0 + i < CH)
                    *reinterpret_cast<u32x4*>(u_lds + (t0 + i) * ld + o * 8) = t0 + i < n ? pack8(acc[i]) : u32x4{0, 0, 0, 0};
        }
    }
    __syncthreads();

    const uint16_t* ra = reinterpret_cast<const uint16_t*>(a.ra) + (int64_t)blk * a.block * a.block;
    const uint16_t* ri = reinterpret_cast<const uint16_t*>(a.ri) + (int64_t)blk * a.block * a.block;
    const int ksteps = a.block / 32;
    const bool from_state = kth == 0;
    for (int nt = wave; nt < a.block / 16; nt += 4) {
        f32x4 gr[4], gi[4];
#pragma unroll
        for (int m = 0; m < 4; ++m) gr[m] = gi[m] = f32x4{0.f, 0.f, 0.f, 0.f};
        const uint16_t* wr = ra + (int64_t)(16 * nt + lq) * a.block + 8 * lg;
        const uint16_t* wi = ri + (int64_t)(16 * nt + lq) * a.block + 8 * lg;
        for (int ks = 0; ks < ksteps; ++ks) {
            const bf16x8 br = *reinterpret_cast<const bf16x8*>(wr + 32 * ks), bi = *reinterpret_cast<const bf16x8*>(wi + 32 * ks);
#pragma unroll
            for (int m = 0; m < 4; ++m) {
                const bf16x8 ua = *reinterpret_cast<const bf16x8*>(u_lds + (16 * m + lq) * ld + 32 * ks + 8 * lg);
                gr[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, br, gr[m], 0, 0, 0);
                gi[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, bi, gi[m], 0, 0, 0);
            }
        }
        // ---- decays, inputs and the scan: this lane holds tokens 16 m + 4 lg + i of channel ch
        const int cb = 16 * nt + lq, ch = blk * a.block + cb;
        const float rb = a.ra_b[ch], ib = a.ri_b[ch], rate = a.rate[ch];
        float ca = 1.f, cs = 0.f;                                              // carry into the tile: product of decays, scan value
        if (from_state) {
            ca = 0.f;
            if (pos0 > 0 && slot >= 0) cs = a.state[(int64_t)slot * a.width + ch];
        }
#pragma unroll
        for (int m = 0; m < 4; ++m) {
            float av[4], sv[4];
            float pa = 1.f, ps = 0.f;                                          // inclusive composition over the lane's 4 tokens
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * m + 4 * lg + i;
                float dec = 1.f, inp = 0.f;
                if (t < n) decay_and_input(rate, sigmoid_f(gr[m][i] + rb), sigmoid_f(gi[m][i] + ib), act_ld(u_lds + t * ld + cb), dec, inp);
                ps = dec * ps + inp;
                pa *= dec;
                av[i] = pa;
                sv[i] = ps;
            }
            // exclusive composition of the lane groups before this one
            float ga = pa, gs = ps;                                            // inclusive over the groups so far
            {
                const float oa = __shfl_up(ga, 16), os = __shfl_up(gs, 16);
                if (lg >= 1) { gs = ga * os + gs; ga *= oa; }
            }
            {
                const float oa = __shfl_up(ga, 32), os = __shfl_up(gs, 32);
                if (lg >= 2) { gs = ga * os + gs; ga *= oa; }
            }
            float xa = __shfl_up(ga, 16), xs = __shfl_up(gs, 16);
            if (lg == 0) { xa = 1.f; xs = 0.f; }
            const float ba = xa * ca, bs = xa * cs + xs;                       // everything before this lane's first token
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * m + 4 * lg + i;
                if (t < n) {
                    a.s_loc[(int64_t)(row0 + t) * a.width + ch] = av[i] * bs + sv[i];
                    if (!from_state) a.a_cum[(int64_t)(row0 + t) * a.width + ch] = av[i] * ba;
                }
            }
            const float ta = __shfl(ga, 48 + lq), ts = __shfl(gs, 48 + lq);    // the whole tile
            cs = ta * cs + ts;
            ca *= ta;
        }
    }
}

// ------------------------------------------------------------------------------------------------ prompt portions, any type and size
// one workgroup per (chunk, 64 channels of a diagonal block): gates by plain dot products over LDS tiles, scan by one thread per channel
template <typename T>
__global__ __launch_bounds__(256) void rglru_gates_generic_kernel(const RglruArgs a) {
    constexpr int KT = 32;
    __shared__ float u_t[CH][KT + 1];
    __shared__ float wr_t[64][KT + 1], wi_t[64][KT + 1];
    __shared__ float dec[CH][65], inp[CH][65];
    const int chunk = blockIdx.x;
    const int tiles = (a.block + 63) / 64, blk = blockIdx.y / tiles, n0 = (blockIdx.y % tiles) * 64;
    const int row0 = a.chunks[chunk * 4], n = a.chunks[chunk * 4 + 1], seq = a.chunks[chunk * 4 + 2], kth = a.chunks[chunk * 4 + 3];
    const int seq_row0 = row0 - kth * CH;
    const int slot = a.state_slots[seq];
    const int64_t pos0 = a.positions[seq_row0];
    const T* ra = reinterpret_cast<const T*>(a.ra) + (int64_t)blk * a.block * a.block;
    const T* ri = reinterpret_cast<const T*>(a.ri) + (int64_t)blk * a.block * a.block;
    const int tid = threadIdx.x, c = tid & 63, tq = tid >> 6;
    auto conv_at = [&](int t, int ch) {
        float s = a.conv_b[ch];
        for (int j = 0; j < a.taps; ++j) {
            const T* p = conv_input<T>(a, seq_row0, kth * CH + t - (a.taps - 1) + j, pos0, slot, ch);
            if (p) s += a.conv_w[(int64_t)j * a.width + ch] * act_ld(p);
        }
        return act_round(s, (const T*)nullptr);
    };
    float gr[16], gi[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) gr[i] = gi[i] = 0.f;
    for (int k0 = 0; k0 < a.block; k0 += KT) {
        for (int e = tid; e < CH * KT; e += 256) {
            const int t = e / KT, k = e % KT;
            u_t[t][k] = t < n ? conv_at(t, blk * a.block + k0 + k) : 0.f;
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
    const int ch = blk * a.block + n0 + c;
    const bool live = n0 + c < a.block;
    if (live) {
        const float rb = a.ra_b[ch], ib = a.ri_b[ch], rate = a.rate[ch];
        for (int i = 0; i < 16; ++i) {
            const int t = tq * 16 + i;
            float d = 1.f, b = 0.f;
            if (t < n) {
                // (accurate exponentials: this form also serves the true fp32 model)
                const float r = 1.f / (1.f + expf(-(gr[i] + rb))), ig = 1.f / (1.f + expf(-(gi[i] + ib)));
                const float log_a = -rate * r;
                d = expf(log_a);
                b = sqrtf(-expm1f(2.f * log_a)) * ig * conv_at(t, ch);
            }
            dec[t][c] = d;
            inp[t][c] = b;
        }
    }
    __syncthreads();
    if (tid < 64 && live) {
        float ca = 1.f, cs = 0.f;
        if (kth == 0) {
            ca = 0.f;
            if (pos0 > 0 && slot >= 0) cs = a.state[(int64_t)slot * a.width + ch];
        }
        for (int t = 0; t < n; ++t) {
            cs = dec[t][c] * cs + inp[t][c];
            ca *= dec[t][c];
            a.s_loc[(int64_t)(row0 + t) * a.width + ch] = cs;
            if (kth != 0) a.a_cum[(int64_t)(row0 + t) * a.width + ch] = ca;
        }
    }
}

// out = S gelu(y) with S = scan + decay product x carry; the portion's last chunk leaves the state.  256 threads = 64 x 4 channels, 4 token lanes
template <typename T>
__global__ __launch_bounds__(256) void rglru_apply_kernel(const RglruArgs a) {
    const int chunk = blockIdx.x;
    const int row0 = a.chunks[chunk * 4], n = a.chunks[chunk * 4 + 1], seq = a.chunks[chunk * 4 + 2], kth = a.chunks[chunk * 4 + 3];
    const int ch = (blockIdx.y * 64 + (threadIdx.x & 63)) * 4, tl = threadIdx.x >> 6;
    if (ch >= a.width) return;
    f32x4 carry = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < kth; ++k) {
        const int64_t last = (int64_t)(row0 - (kth - k) * CH + CH - 1) * a.width + ch;
        const f32x4 s = *reinterpret_cast<const f32x4*>(a.s_loc + last);
        if (k == 0) carry = s;
        else carry = *reinterpret_cast<const f32x4*>(a.a_cum + last) * carry + s;
    }
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    for (int t = tl; t < n; t += 4) {
        const int64_t at = (int64_t)(row0 + t) * a.width + ch;
        s = *reinterpret_cast<const f32x4*>(a.s_loc + at);
        if (kth) s += *reinterpret_cast<const f32x4*>(a.a_cum + at) * carry;
        const f32x4 y = act_ld4(reinterpret_cast<const T*>(a.yx) + (int64_t)(row0 + t) * a.yx_stride + ch);
        f32x4 o;
#pragma unroll
        for (int k = 0; k < 4; ++k) o[k] = s[k] * gelu_tanh_f(y[k]);
        act_st4(reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t) * a.out_stride + ch, o);
    }
    const bool last_chunk = chunk + 1 == a.n_chunks || a.chunks[(chunk + 1) * 4 + 2] != seq;
    const int slot = a.state_slots[seq];
    if (!last_chunk || slot < 0) return;
    if ((n - 1) % 4 == tl) *reinterpret_cast<f32x4*>(a.state + (int64_t)slot * a.width + ch) = s;
    const int portion = kth * CH + n;
    const int keep = portion < a.taps ? portion : a.taps;
    for (int j = tl; j < keep; j += 4) {
        const int row = row0 + n - 1 - j;
        const int e = (int)(a.positions[row] % a.taps);
        act_st4(reinterpret_cast<T*>(a.conv_state) + ((int64_t)slot * a.taps + e) * a.width + ch,
                act_ld4(reinterpret_cast<const T*>(a.yx) + (int64_t)row * a.yx_stride + a.width + ch));
    }
}

// ------------------------------------------------------------------------------------------------ one token per sequence (bf16)
// grid (width / 16 channel tiles, 32-row tiles); the 4 waves split the contraction over the diagonal block and add up through LDS
__global__ __launch_bounds__(256) void rglru_step_kernel(const RglruArgs a, const int rows) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int per = a.block / 16, blk = blockIdx.x / per, nt = blockIdx.x % per;
    const int r0 = blockIdx.y * 32, nr = rows - r0 < 32 ? rows - r0 : 32;
    const int ld = a.block + 8, oct = a.block / 8;
    uint16_t* u_lds = reinterpret_cast<uint16_t*>(smem);                        // [32][block + 8]
    f32x4* red = reinterpret_cast<f32x4*>(smem + 32 * ld * 2);                  // [wave][2 gates x 2 row tiles][64 lanes]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const uint16_t* yx = reinterpret_cast<const uint16_t*>(a.yx);
    for (int e = tid; e < 32 * oct; e += 256) {
        const int row = e / oct, o = e - row * oct;
        u32x4 packed = {0, 0, 0, 0};
        if (row < nr) {
            const int slot = a.state_slots[r0 + row], ch = blk * a.block + o * 8;
            const int64_t pos = a.positions[r0 + row];
            float acc[8];
#pragma unroll
            for (int k = 0; k < 8; ++k) acc[k] = a.conv_b[ch + k];
            for (int j = 0; j < a.taps; ++j) {
                const uint16_t* p = conv_input<uint16_t>(a, r0 + row, j - (a.taps - 1), pos, slot, ch);
                if (p) fma8(acc, *reinterpret_cast<const u32x4*>(p), a.conv_w + (int64_t)j * a.width + ch);
            }
            packed = pack8(acc);
        }
        *reinterpret_cast<u32x4*>(u_lds + row * ld + o * 8) = packed;
    }
    __syncthreads();
    f32x4 g[4];
#pragma unroll
    for (int m = 0; m < 4; ++m) g[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint16_t* wr = reinterpret_cast<const uint16_t*>(a.ra) + ((int64_t)blk * a.block + 16 * nt + lq) * a.block + 8 * lg;
    const uint16_t* wi = reinterpret_cast<const uint16_t*>(a.ri) + ((int64_t)blk * a.block + 16 * nt + lq) * a.block + 8 * lg;
    for (int ks = wave; ks < a.block / 32; ks += 4) {
        const bf16x8 br = *reinterpret_cast<const bf16x8*>(wr + 32 * ks), bi = *reinterpret_cast<const bf16x8*>(wi + 32 * ks);
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            const bf16x8 ua = *reinterpret_cast<const bf16x8*>(u_lds + (16 * m + lq) * ld + 32 * ks + 8 * lg);
            g[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, br, g[m], 0, 0, 0);
            g[2 + m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua, bi, g[2 + m], 0, 0, 0);
        }
    }
#pragma unroll
    for (int m = 0; m < 4; ++m) red[(wave * 4 + m) * 64 + lane] = g[m];
    __syncthreads();
    // thread -> (row tile, lane of the C layout, half of its 4 rows): 2 outputs each
    const int m = tid >> 7, cl = (tid >> 1) & 63, half = tid & 1;
    const int cb = 16 * nt + (cl & 15), ch = blk * a.block + cb;
    f32x4 sr = {0.f, 0.f, 0.f, 0.f}, si = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
        sr += red[(w * 4 + m) * 64 + cl];
        si += red[(w * 4 + 2 + m) * 64 + cl];
    }
    const float rb = a.ra_b[ch], ib = a.ri_b[ch], rate = a.rate[ch];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int row = 16 * m + 4 * (cl >> 4) + 2 * half + i;
        if (row >= nr) continue;
        const int slot = a.state_slots[r0 + row];
        const int64_t pos = a.positions[r0 + row];
        float dec, inp;
        decay_and_input(rate, sigmoid_f((half ? sr[2 + i] : sr[i]) + rb), sigmoid_f((half ? si[2 + i] : si[i]) + ib), act_ld(u_lds + row * ld + cb), dec, inp);
        float s = inp;
        if (slot >= 0) {
            float* sp = a.state + (int64_t)slot * a.width + ch;
            if (pos > 0) s += dec * *sp;
            *sp = s;
            reinterpret_cast<uint16_t*>(a.conv_state)[((int64_t)slot * a.taps + (int)(pos % a.taps)) * a.width + ch] =
                yx[(int64_t)(r0 + row) * a.yx_stride + a.width + ch];
        }
        const float o = s * gelu_tanh_f(act_ld(yx + (int64_t)(r0 + row) * a.yx_stride + ch));
        if (a.out) act_st(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(r0 + row) * a.out_stride + ch, o);
        if (a.out_packed) act_st(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(r0 + row, ch, a.width), o);
    }
}

constexpr size_t kMaxLds = 160 * 1024;
size_t gates_lds(int block) { return (size_t)CH * (block + 8) * 2; }
size_t step_lds(int block) { return (size_t)32 * (block + 8) * 2 + 16 * 64 * sizeof(f32x4); }

}  // namespace

bool rglru_step_supported(int block) { return step_lds(block) <= kMaxLds; }

int launch_rglru_chunks(const RglruArgs& a, int f32, int generic, hipStream_t stream) {
    if (a.n_chunks == 0) return 0;
    if (f32 || generic || gates_lds(a.block) > kMaxLds) {
        const dim3 grid(a.n_chunks, a.blocks * ((a.block + 63) / 64));
        if (f32) rglru_gates_generic_kernel<float><<<grid, 256, 0, stream>>>(a);
        else rglru_gates_generic_kernel<uint16_t><<<grid, 256, 0, stream>>>(a);
    } else {
        const size_t lds = gates_lds(a.block);
        if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rglru_gates_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
        rglru_gates_kernel<<<dim3(a.n_chunks, a.blocks), 256, lds, stream>>>(a);
    }
    int rc = check_launch("rglru_gates");
    if (rc) return rc;
    const dim3 grid(a.n_chunks, (a.width + 255) / 256);
    if (f32) rglru_apply_kernel<float><<<grid, 256, 0, stream>>>(a);
    else rglru_apply_kernel<uint16_t><<<grid, 256, 0, stream>>>(a);
    return check_launch("rglru_apply");
}

int launch_rglru_step(const RglruArgs& a, int rows, hipStream_t stream) {
    const size_t lds = step_lds(a.block);
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rglru_step_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
    rglru_step_kernel<<<dim3(a.blocks * (a.block / 16), (rows + 31) / 32), 256, lds, stream>>>(a, rows);
    return check_launch("rglru_step");
}

}  // namespace nvh
