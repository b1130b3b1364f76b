// Mixture of experts; the router's scores are sigmoids with choice corrections and expert groups, or a softmax over the chosen logits.
//   route     32-bit logits of a row tile against every expert (MFMA for bf16), group and expert choice, weights: one launch
//   dispatch  pairs (row, chosen expert) sorted by expert and cut into tiles of one expert each: two launches, no host round trip
//   gemm      expert products: gate | up with the gated unit in the epilogue, and down.  Large batches: 128 x 128 or 256 x 256 MFMA tiles over the
//             sorted pairs, the rows gathered by the DMA that fills LDS.  At most 64 rows: every wave streams 16 weight rows once for all the rows that chose the expert.
// Outputs stay per pair; the weighted sum over a row's experts belongs to the residual add (hybrid_ops.hip).
#include "attend_tile.h"
#include "mixers.h"

namespace nvh {

namespace {

// ------------------------------------------------------------------------------------------------ choice (one wave per row)
__device__ __forceinline__ float wave_max64(float v) {
    v = fmaxf(v, pair_in_row<1>(v));
    v = fmaxf(v, pair_in_row<2>(v));
    v = fmaxf(v, pair_in_row<4>(v));
    v = fmaxf(v, pair_in_row<8>(v));
    v = max_xor16(v);
    return max_xor32(v);
}
// lane that holds the wave's largest value (the first of equal ones)
__device__ __forceinline__ int wave_winner(float v) {
    const uint64_t b = __builtin_amdgcn_ballot_w64(v == wave_max64(v));
    return b ? __builtin_ctzll(b) : 0;               // (0 only where a router delivers no number)
}
__device__ __forceinline__ float lane_value(float v, int lane) { return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), lane)); }

__device__ __forceinline__ float group_score(const float* choice, int size) {
    float b0 = -INFINITY, b1 = -INFINITY;            // the two largest
    for (int k = 0; k < size; ++k) {
        const float c = choice[k];
        b1 = fmaxf(b1, fminf(b0, c));
        b0 = fmaxf(b0, c);
    }
    return size > 1 ? b0 + b1 : b0;
}

__device__ __forceinline__ void store_choice(const MoeRouteArgs& a, int row, int lane, int id, float score, float total) {
    if (lane < a.top) {
        a.ids[(int64_t)row * a.top + lane] = id;
        a.weights[(int64_t)row * a.top + lane] = score / (total + 1e-20f) * a.scale;
    }
}

// score of an expert from its logit
__device__ __forceinline__ float expert_score(const MoeRouteArgs& a, float z, int e) { return a.softmax ? z + a.correction[e] : 1.f / (1.f + expf(-z)); }
// its part of the weights, with `top` the score of the first choice (a softmax is taken relative to its largest entry)
__device__ __forceinline__ float expert_part(const MoeRouteArgs& a, float score, float top) { return a.softmax ? expf(score - top) : score; }

// z [E]: logits in, scores out; choice [E], gs [groups]: scratch in LDS.  Up to 64 experts: one per lane, LDS for the group scores only.
__device__ __forceinline__ void choose_experts(const MoeRouteArgs& a, int row, int lane, float* z, float* choice, float* gs) {
    const int size = a.experts / a.groups;
    float total = 0.f, mine = 0.f, top = 0.f;
    int my_id = 0;
    if (a.experts <= 64) {
        const bool ok = lane < a.experts;
        const float s = ok ? expert_score(a, z[lane], lane) : 0.f;
        float c = ok ? (a.softmax ? s : s + a.correction[lane]) : -INFINITY;
        if (a.keep < a.groups) {
            choice[lane] = c;
            wave_lds_sync();
            float g = lane < a.groups ? group_score(choice + lane * size, size) : -INFINITY;
            uint64_t open = 0;
            for (int k = 0; k < a.keep; ++k) {
                const int w = wave_winner(g);
                open |= 1ull << w;
                if (lane == w) g = -INFINITY;
            }
            if (!((open >> (lane / size)) & 1)) c = -INFINITY;
        }
        for (int k = 0; k < a.top; ++k) {
            const int w = wave_winner(c);
            const float score = lane_value(s, w);
            if (k == 0) top = score;
            const float sw = expert_part(a, score, top);
            total += sw;
            if (lane == k) {
                mine = sw;
                my_id = w < a.experts ? w : 0;
            }
            if (lane == w) c = -INFINITY;
        }
        store_choice(a, row, lane, my_id, mine, total);
        return;
    }
    for (int e = lane; e < a.experts; e += 64) {
        const float s = expert_score(a, z[e], e);
        z[e] = s;
        choice[e] = a.softmax ? s : s + a.correction[e];
    }
    wave_lds_sync();
    auto best = [&](const float* list, int n) {      // index of the list's largest value
        float v = -INFINITY;
        int i = 0;
        for (int e = lane; e < n; e += 64) {
            const float c = list[e];
            if (c > v) {
                v = c;
                i = e;
            }
        }
        return __builtin_amdgcn_readlane(i, wave_winner(v));
    };
    if (a.keep < a.groups) {
        for (int g = lane; g < a.groups; g += 64) gs[g] = group_score(choice + g * size, size);
        wave_lds_sync();
        for (int k = 0; k < a.keep; ++k) {           // an open group is marked by NaN: it loses every comparison
            const int g = best(gs, a.groups);
            if (lane == 0) gs[g] = NAN;
            wave_lds_sync();
        }
        for (int e = lane; e < a.experts; e += 64)
            if (gs[e / size] == gs[e / size]) choice[e] = -INFINITY;
        wave_lds_sync();
    }
    for (int k = 0; k < a.top; ++k) {
        const int e = best(choice, a.experts);
        if (k == 0) top = z[e];
        const float s = expert_part(a, z[e], top);
        total += s;
        if (lane == k) {
            mine = s;
            my_id = e;
        }
        wave_lds_sync();
        if (lane == 0) choice[e] = -INFINITY;
        wave_lds_sync();
    }
    store_choice(a, row, lane, my_id, mine, total);
}

// live rows (at most 16) per workgroup, the contraction shared by 8 waves, 64 experts at a time
__global__ __launch_bounds__(512) void moe_route_kernel(const MoeRouteArgs a, const int live) {
    extern __shared__ __attribute__((aligned(16))) float lds_r[];
    const int ez = (a.experts + 63) / 64 * 64;
    float *part = lds_r, *z = part + 8 * 16 * 68, *choice = z + 16 * ez, *gs = choice + 8 * ez;     // [8][16][64 + 4], [16][ez], per wave [ez], [groups]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const int r0 = blockIdx.x * live, rows = a.rows - r0 < live ? a.rows - r0 : live, row = r0 + (lq < rows ? lq : rows - 1);
    const int steps = a.cols / 32, per = (steps + 7) / 8, s0 = wave * per, s1 = s0 + per < steps ? s0 + per : steps;
    const uint16_t* x = reinterpret_cast<const uint16_t*>(a.x) + (int64_t)row * a.x_stride + 8 * lg;
    for (int e0 = 0; e0 < a.experts; e0 += 64) {
        const uint16_t* w[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            const int e = e0 + 16 * t + lq;
            w[t] = reinterpret_cast<const uint16_t*>(a.router) + (int64_t)(e < a.experts ? e : a.experts - 1) * a.cols + 8 * lg;
        }
        f32x4 acc[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
        auto walk = [&](auto ntc) {                  // (tiles that hold no expert are not read)
            constexpr int NT = decltype(ntc)::value;
            constexpr int UN = 4;
            int s = s0;
            for (; s + UN <= s1; s += UN) {
                bf16x8 xf[UN], wf[UN][NT];
#pragma unroll
                for (int i = 0; i < UN; ++i) {
                    xf[i] = *reinterpret_cast<const bf16x8*>(x + 32 * (s + i));
#pragma unroll
                    for (int t = 0; t < NT; ++t) wf[i][t] = *reinterpret_cast<const bf16x8*>(w[t] + 32 * (s + i));
                }
#pragma unroll
                for (int i = 0; i < UN; ++i)
#pragma unroll
                    for (int t = 0; t < NT; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[i][t], xf[i], acc[t], 0, 0, 0);
            }
            for (; s < s1; ++s) {
                const bf16x8 xf = *reinterpret_cast<const bf16x8*>(x + 32 * s);
#pragma unroll
                for (int t = 0; t < NT; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(w[t] + 32 * s), xf, acc[t], 0, 0, 0);
            }
        };
        switch ((a.experts - e0 + 15) / 16) {
            case 1: walk(std::integral_constant<int, 1>{}); break;
            case 2: walk(std::integral_constant<int, 2>{}); break;
            case 3: walk(std::integral_constant<int, 3>{}); break;
            default: walk(std::integral_constant<int, 4>{}); break;
        }
        // D: lane = row lq, experts 16 t + 4 lg ..
#pragma unroll
        for (int t = 0; t < 4; ++t) *reinterpret_cast<f32x4*>(part + (wave * 16 + lq) * 68 + 16 * t + 4 * lg) = acc[t];
        __syncthreads();
        for (int i = tid; i < rows * 64; i += 512) {
            const int r = i >> 6, e = i & 63;
            float s = 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k) s += part[(k * 16 + r) * 68 + e];
            z[r * ez + e0 + e] = s;
        }
        __syncthreads();
    }
    for (int r = wave; r < rows; r += 8) choose_experts(a, r0 + r, lane, z + r * ez, choice + wave * ez, gs + wave * a.groups);
}

// any type and width: one workgroup per row, a wave per expert in turn
template <typename T>
__global__ __launch_bounds__(256) void moe_route_generic_kernel(const MoeRouteArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds_r[];
    float *z = lds_r, *choice = z + a.experts, *gs = choice + a.experts;
    const int row = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const T* x = reinterpret_cast<const T*>(a.x) + (int64_t)row * a.x_stride;
    for (int e = wave; e < a.experts; e += 4) {
        const T* w = reinterpret_cast<const T*>(a.router) + (int64_t)e * a.cols;
        float s = 0.f;
        for (int c = lane * 4; c < a.cols; c += 256) s += sum4(act_ld4(x + c) * act_ld4(w + c));
        s = wave_sum64(s);
        if (lane == 0) z[e] = s;
    }
    __syncthreads();
    if (wave == 0) choose_experts(a, row, lane, z, choice, gs);
}

// ------------------------------------------------------------------------------------------------ dispatch
constexpr int DP = 2048;                             // pairs per workgroup

__global__ __launch_bounds__(256) void moe_count_kernel(int32_t* __restrict__ counts, const int32_t* __restrict__ ids, int pairs, int experts) {
    __shared__ int hist[kMoeMaxExperts];
    for (int e = threadIdx.x; e < experts; e += 256) hist[e] = 0;
    __syncthreads();
    const int p0 = blockIdx.x * DP;
    for (int p = p0 + threadIdx.x; p < p0 + DP && p < pairs; p += 256) atomicAdd(&hist[ids[p]], 1);
    __syncthreads();
    for (int e = threadIdx.x; e < experts; e += 256) counts[(int64_t)blockIdx.x * experts + e] = hist[e];
}

// every workgroup sums the counts in front of its own pairs; the first one also writes the tiles
__global__ __launch_bounds__(256) void moe_scatter_kernel(int32_t* __restrict__ slot_pair, int32_t* __restrict__ tiles, const int32_t* __restrict__ counts,
                                                          const int32_t* __restrict__ ids, int pairs, int experts, int tile_rows, int max_tiles) {
    __shared__ int at[kMoeMaxExperts], total[kMoeMaxExperts], start[kMoeMaxExperts], tile0[kMoeMaxExperts];
    __shared__ int n_tiles;
    for (int e = threadIdx.x; e < experts; e += 256) {
        int before = 0, all = 0;
        for (int b = 0; b < (int)gridDim.x; ++b) {
            const int c = counts[(int64_t)b * experts + e];
            if (b < (int)blockIdx.x) before += c;
            all += c;
        }
        at[e] = before;
        total[e] = all;
    }
    __syncthreads();
    if (threadIdx.x < 64) {                          // exclusive scans over the experts, 64 at a time
        int base = 0, tbase = 0;
        for (int e0 = 0; e0 < experts; e0 += 64) {
            const int e = e0 + threadIdx.x, n = e < experts ? total[e] : 0, t = (n + tile_rows - 1) / tile_rows;
            int s = n, u = t;
            for (int d = 1; d < 64; d <<= 1) {
                const int ps = __shfl_up(s, d), pu = __shfl_up(u, d);
                if ((int)threadIdx.x >= d) {
                    s += ps;
                    u += pu;
                }
            }
            if (e < experts) {
                start[e] = base + s - n;
                tile0[e] = tbase + u - t;
            }
            base += __shfl(s, 63);
            tbase += __shfl(u, 63);
        }
        if (threadIdx.x == 0) n_tiles = tbase;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < experts; e += 256) at[e] += start[e];
    __syncthreads();
    const int p0 = blockIdx.x * DP;
    for (int p = p0 + threadIdx.x; p < p0 + DP && p < pairs; p += 256) slot_pair[atomicAdd(&at[ids[p]], 1)] = p;
    if (blockIdx.x == 0) {
        for (int e = threadIdx.x; e < experts; e += 256)
            for (int t = 0; t * tile_rows < total[e]; ++t) {
                const int left = total[e] - t * tile_rows;
                reinterpret_cast<int4*>(tiles)[tile0[e] + t] = int4{e, start[e] + t * tile_rows, left < tile_rows ? left : tile_rows, n_tiles};
            }
        for (int t = n_tiles + threadIdx.x; t < max_tiles; t += 256) reinterpret_cast<int4*>(tiles)[t] = int4{0, 0, 0, n_tiles};
    }
}

// ------------------------------------------------------------------------------------------------ products, large batches (bf16)
// MW x NW waves of MT x NT tiles of 16 x 16: TM pairs by TN weight rows per workgroup, 32 of the contraction at a time, both operands by LDS-DMA through a
// ring of four images: three are on their way while the fourth is read into registers, and the one before it is multiplied from there.
// GLU: weight rows alternate 16 of gate, 16 of up, so a lane holds both halves of its outputs.
constexpr int TK = 32, kRing = 4;
// SiLU(g) u, or the clamped unit where the launch names an alpha
__device__ __forceinline__ float expert_unit(const MoeGemmArgs& a, float g, float u) { return a.alpha != 0.f ? clamped_glu(g, u, a.limit, a.alpha) : silu_f(g) * u; }
template <int MW, int NW, int MT, int NT>
struct GemmShape {
    static constexpr int WAVES = MW * NW, TM = MW * MT * 16, TN = NW * NT * 16, ROWS = TM + TN, IMG = ROWS * TK * 2, DMA = IMG / 1024 / WAVES;
    static constexpr size_t LDS = (size_t)kRing * IMG;
    static_assert(IMG % (1024 * WAVES) == 0 && NT % 2 == 0, "DMA instructions and gate/up tiles divide evenly");
};

template <bool GLU, int MW, int NW, int MT, int NT>
__global__ __launch_bounds__(64 * MW * NW) void moe_gemm_kernel(const MoeGemmArgs a) {
    using G = GemmShape<MW, NW, MT, NT>;
    constexpr int TN = G::TN, DMA = G::DMA, OUTS = GLU ? TN / 2 : TN;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];        // [ring][TN weight rows | TM pairs][64 bytes]
    int nt, mt;
    {
        // one XCD takes a run of the tiles, eight row tiles times the columns at a time, rows first: what runs at once shares rows and weights in its L2
        const int nx = gridDim.x, tiles = a.tiles[3], total = nx * tiles, lin = (int)(blockIdx.x + gridDim.x * blockIdx.y), per = total >> 3;
        if (lin >= total) return;
        const int idx = lin < per * 8 ? (lin & 7) * per + (lin >> 3) : lin;
        const int g = idx / (8 * nx), in = idx - g * 8 * nx, gm = tiles - 8 * g < 8 ? tiles - 8 * g : 8;
        nt = in / gm;
        mt = 8 * g + in - nt * gm;
    }
    const int expert = a.tiles[4 * mt], first = a.tiles[4 * mt + 1], live = a.tiles[4 * mt + 2];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4, wm = wave / NW, wn = wave % NW;
    const uint16_t* w = reinterpret_cast<const uint16_t*>(a.w) + (int64_t)expert * (GLU ? 2 : 1) * a.n * a.k;
    auto swz = [](int r) { return (r >> 2) & 3; };   // 16-byte pieces of a row are xor-ed: 16 rows read at one column spread over all banks
    // this lane's piece of each DMA instruction: 16 rows of 64 bytes
    const uint16_t* src[DMA];
#pragma unroll
    for (int j = 0; j < DMA; ++j) {
        const int R = (wave * DMA + j) * 16 + (lane >> 2), piece = ((lane & 3) ^ swz(R)) * 8;
        if (R < TN) {
            int col = nt * OUTS + (GLU ? (R >> 5) * 16 + (R & 15) : R);
            if (col >= a.n) col = a.n - 1;
            src[j] = w + (int64_t)(GLU && (R & 16) ? a.n + col : col) * a.k + piece;
        } else {
            const int r = R - TN, pair = a.slot_pair[first + (r < live ? r : live - 1)];
            src[j] = reinterpret_cast<const uint16_t*>(a.x) + (GLU ? (int64_t)(pair / a.top) * a.x_stride : (int64_t)pair * a.k) + piece;
        }
    }
    auto stage = [&](int it, int buf) {
#pragma unroll
        for (int j = 0; j < DMA; ++j) dma16(src[j] + it * TK, lds + buf * G::IMG + (wave * DMA + j) * 1024);
    };
    f32x4 acc[NT][MT];                               // D[weight row 16 i + 4 lg + r][pair 16 j + lq]
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int j = 0; j < MT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int iters = a.k / TK;                      // (k is a multiple of 64: even)
    // (images past the last one are asked for again: every iteration leaves the same number of loads in flight, without a branch)
    auto stage_next = [&](int it) { stage(it < iters ? it : iters - 1, it % kRing); };
#pragma unroll
    for (int it = 0; it < kRing; ++it) stage_next(it);
    struct Operands {
        bf16x8 w[NT], x[MT];
    };
    Operands even, odd;                              // of the image being multiplied and of the next one, read meanwhile
    auto read = [&](int it, Operands& f) {
        const int at = (it % kRing) * G::IMG + lq * 64 + (lg ^ swz(lq)) * 16;
        const unsigned char* wimg = lds + at + wn * NT * 16 * 64;
        const unsigned char* ximg = lds + at + (TN + wm * MT * 16) * 64;
#pragma unroll
        for (int t = 0; t < NT; ++t) f.w[t] = *reinterpret_cast<const bf16x8*>(wimg + t * 16 * 64);
#pragma unroll
        for (int t = 0; t < MT; ++t) f.x[t] = *reinterpret_cast<const bf16x8*>(ximg + t * 16 * 64);
    };
    // the oldest image in flight has landed (`younger` behind it), and everyone has read the one before it
    auto arrive = [&](auto younger) {
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"(decltype(younger)::value * DMA) : "memory");
        lds_only_barrier();
    };
    // reads and loads spread between the products
    auto spread = [] {
#pragma unroll
        for (int k = 0; k < NT + MT; ++k) {
            __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);                 // LDS read
            __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);                 // MFMA
        }
#pragma unroll
        for (int k = 0; k < DMA; ++k) {
            __builtin_amdgcn_sched_group_barrier(0x010, 1, 0);                 // load
            __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
        }
    };
    auto multiply = [&](const Operands& f) {
#pragma unroll
        for (int j = 0; j < MT; ++j)
#pragma unroll
            for (int i = 0; i < NT; ++i) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.w[i], f.x[j], acc[i][j], 0, 0, 0);
    };
    arrive(std::integral_constant<int, kRing - 1>{});
    read(0, even);
    constexpr std::integral_constant<int, kRing - 2> in_flight{};
    for (int it = 0; it < iters; it += 2) {
        arrive(in_flight);
        read(it + 1, odd);
        stage_next(it + kRing);
        multiply(even);
        spread();
        arrive(in_flight);
        read(it + 2, even);                          // (behind the last image: read and not used)
        stage_next(it + 1 + kRing);
        multiply(odd);
        spread();
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    // ---- results through LDS (the images are done with): a wave's MT * 16 pairs by CW columns, then whole rows of them to memory
    lds_only_barrier();
    constexpr int CW = GLU ? NT * 8 : NT * 16, CP = CW / 8;                    // columns of a wave, 16-byte pieces of a row
    unsigned char* tile = lds + wave * MT * 16 * CW * 2;
    auto put = [&](int r, int col, f32x4 v) {        // columns col .. + 3 of row r
        act_st4(reinterpret_cast<uint16_t*>(tile + r * CW * 2 + (((col >> 3) ^ (r & (CP - 1))) * 16 + (col & 4) * 2)), v);
    };
#pragma unroll
    for (int j = 0; j < MT; ++j) {
        if constexpr (GLU) {
#pragma unroll
            for (int i = 0; i < NT / 2; ++i) {
                f32x4 v;
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = expert_unit(a, acc[2 * i][j][r], acc[2 * i + 1][j][r]);
                put(16 * j + lq, 16 * i + 4 * lg, v);
            }
        } else {
#pragma unroll
            for (int i = 0; i < NT; ++i) put(16 * j + lq, 16 * i + 4 * lg, acc[i][j]);
        }
    }
    wave_lds_sync();
    const int col = nt * OUTS + wn * CW + (lane % CP) * 8;
    if (col < a.n) {                                 // (n is a multiple of 64: whole pieces)
#pragma unroll
        for (int k = 0; k < MT * 16 * CP / 64; ++k) {
            const int r = (k * 64 + lane) / CP, R = wm * MT * 16 + r;
            if (R < live)
                *reinterpret_cast<u32x4*>(reinterpret_cast<uint16_t*>(a.out) + (int64_t)a.slot_pair[first + R] * a.n + col) =
                    *reinterpret_cast<const u32x4*>(tile + r * CW * 2 + ((lane % CP) ^ (r & (CP - 1))) * 16);
        }
    }
}

template <bool GLU, int MW, int NW, int MT, int NT>
void gemm_shape(const MoeGemmArgs& a, hipStream_t stream) {
    using G = GemmShape<MW, NW, MT, NT>;
    const int outs = GLU ? G::TN / 2 : G::TN;
    if (G::LDS > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(moe_gemm_kernel<GLU, MW, NW, MT, NT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)G::LDS);
    moe_gemm_kernel<GLU, MW, NW, MT, NT><<<dim3((a.n + outs - 1) / outs, a.max_tiles), 64 * G::WAVES, G::LDS, stream>>>(a);
}

// ------------------------------------------------------------------------------------------------ products, at most 64 rows (bf16)
// grid (n / (16 x waves' tiles), experts): the pairs of the expert are found from the ids; an expert nobody chose costs one scan.
// SPLIT: the 4 waves share one 16-column tile and split the contraction; otherwise every wave owns a tile.
template <bool GLU, int MT, bool SPLIT>
__device__ __forceinline__ void moe_small_tile(const MoeGemmArgs& a, int expert, int n0, int s0, int s1, const int* list, int count, float* red, int wave, int lane) {
    const int lq = lane & 15, lg = lane >> 4;
    const uint16_t* w = reinterpret_cast<const uint16_t*>(a.w) + ((int64_t)expert * (GLU ? 2 : 1) * a.n + n0 + lq) * a.k + 8 * lg;
    const uint16_t* x[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int p = list[16 * m + lq < count ? 16 * m + lq : count - 1];
        x[m] = reinterpret_cast<const uint16_t*>(a.x) + (GLU ? (int64_t)(p / a.top) * a.x_stride : (int64_t)p * a.k) + 8 * lg;
    }
    f32x4 g[MT], u[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) g[m] = u[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int UN = GLU ? (MT > 2 ? 2 : 4) : (MT > 2 ? 4 : 8);
    const int64_t up = (int64_t)a.n * a.k;
    int s = s0;
    for (; s + UN <= s1; s += UN) {
        bf16x8 wg[UN], wu[UN], xf[UN][MT];
#pragma unroll
        for (int i = 0; i < UN; ++i) {
            wg[i] = *reinterpret_cast<const bf16x8*>(w + 32 * (s + i));    // (half of a 128-byte line: a streaming hint would drop the other half)
            if constexpr (GLU) wu[i] = *reinterpret_cast<const bf16x8*>(w + up + 32 * (s + i));
        }
#pragma unroll
        for (int i = 0; i < UN; ++i)
#pragma unroll
            for (int m = 0; m < MT; ++m) xf[i][m] = *reinterpret_cast<const bf16x8*>(x[m] + 32 * (s + i));
#pragma unroll
        for (int i = 0; i < UN; ++i)
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                g[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wg[i], xf[i][m], g[m], 0, 0, 0);
                if constexpr (GLU) u[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wu[i], xf[i][m], u[m], 0, 0, 0);
            }
    }
    for (; s < s1; ++s) {
        const bf16x8 wg = *reinterpret_cast<const bf16x8*>(w + 32 * s);
        bf16x8 wu = wg;
        if constexpr (GLU) wu = *reinterpret_cast<const bf16x8*>(w + up + 32 * s);
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            const bf16x8 xf = *reinterpret_cast<const bf16x8*>(x[m] + 32 * s);
            g[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wg, xf, g[m], 0, 0, 0);
            if constexpr (GLU) u[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wu, xf, u[m], 0, 0, 0);
        }
    }
    if constexpr (SPLIT) {                           // red [4 waves][2][MT][64 lanes][4]
        constexpr int W = 2 * MT * 256;
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            *reinterpret_cast<f32x4*>(red + wave * W + m * 256 + lane * 4) = g[m];
            if constexpr (GLU) *reinterpret_cast<f32x4*>(red + wave * W + (MT + m) * 256 + lane * 4) = u[m];
        }
        __syncthreads();
        if (wave) return;
#pragma unroll
        for (int k = 1; k < 4; ++k)
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                g[m] += *reinterpret_cast<const f32x4*>(red + k * W + m * 256 + lane * 4);
                if constexpr (GLU) u[m] += *reinterpret_cast<const f32x4*>(red + k * W + (MT + m) * 256 + lane * 4);
            }
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        if (16 * m + lq >= count) continue;
        f32x4 v = g[m];
        if constexpr (GLU) {
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = expert_unit(a, g[m][r], u[m][r]);
        }
        act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)list[16 * m + lq] * a.n + n0 + 4 * lg, v);
    }
}

template <bool GLU, bool SPLIT>
__global__ __launch_bounds__(256) void moe_small_kernel(const MoeGemmArgs a) {
    __shared__ int list[64];
    __shared__ int count_s;
    __shared__ __attribute__((aligned(16))) float red[SPLIT ? 4 * 2 * 4 * 256 : 4];
    const int expert = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    if (wave == 0) {                                 // (an expert is chosen at most once per row: at most 64 pairs)
        int n = 0;
        for (int p0 = 0; p0 < a.pairs; p0 += 64) {
            const bool mine = p0 + lane < a.pairs && a.ids[p0 + lane] == expert;
            const uint64_t ball = __builtin_amdgcn_ballot_w64(mine);
            const int at = n + __popcll(ball & ((1ull << lane) - 1));
            if (mine && at < 64) list[at] = p0 + lane;
            n += __popcll(ball);
        }
        if (lane == 0) count_s = n < 64 ? n : 64;
    }
    __syncthreads();
    const int count = __builtin_amdgcn_readfirstlane(count_s);
    if (count == 0) return;
    const int tile = SPLIT ? blockIdx.x : blockIdx.x * 4 + wave, steps = a.k / 32;
    if (tile * 16 >= a.n) return;                    // (whole waves; only the form without a later barrier has such tiles)
    const int per = (steps + 3) / 4, s0 = SPLIT ? wave * per : 0, s1 = SPLIT ? (s0 + per < steps ? s0 + per : steps) : steps;
    if (count <= 16) moe_small_tile<GLU, 1, SPLIT>(a, expert, tile * 16, s0, s1, list, count, red, wave, lane);
    else if (count <= 32) moe_small_tile<GLU, 2, SPLIT>(a, expert, tile * 16, s0, s1, list, count, red, wave, lane);
    else moe_small_tile<GLU, 4, SPLIT>(a, expert, tile * 16, s0, s1, list, count, red, wave, lane);
}

// ------------------------------------------------------------------------------------------------ products in 32-bit
// 64 pairs x 64 outputs per workgroup, 16 of the contraction at a time through LDS, 4 x 4 outputs per thread
constexpr int FM = 64;

template <bool GLU>
__global__ __launch_bounds__(256) void moe_gemm_f32_kernel(const MoeGemmArgs a) {
    __shared__ __attribute__((aligned(16))) float xs[16][FM + 4], ws[2][16][64 + 4];
    const int mt = blockIdx.y, n0 = blockIdx.x * 64, tid = threadIdx.x;
    const int expert = a.tiles[4 * mt], first = a.tiles[4 * mt + 1], live = a.tiles[4 * mt + 2];
    if (live <= 0) return;
    const float* w = reinterpret_cast<const float*>(a.w) + (int64_t)expert * (GLU ? 2 : 1) * a.n * a.k;
    const int lr = tid >> 2, lc = (tid & 3) * 4;     // staging: row lr, 4 of the contraction
    const int pair = a.slot_pair[first + (lr < live ? lr : live - 1)];
    const float* x = reinterpret_cast<const float*>(a.x) + (GLU ? (int64_t)(pair / a.top) * a.x_stride : (int64_t)pair * a.k) + lc;
    const float* wr = w + (int64_t)(n0 + lr) * a.k + lc;
    const int tm = (tid >> 4) * 4, tn = (tid & 15) * 4;
    float g[4][4] = {}, u[4][4] = {};
    for (int k0 = 0; k0 < a.k; k0 += 16) {
        const f32x4 xv = *reinterpret_cast<const f32x4*>(x + k0), gv = *reinterpret_cast<const f32x4*>(wr + k0);
        f32x4 uv = gv;
        if constexpr (GLU) uv = *reinterpret_cast<const f32x4*>(wr + (int64_t)a.n * a.k + k0);
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            xs[lc + i][lr] = xv[i];
            ws[0][lc + i][lr] = gv[i];
            if constexpr (GLU) ws[1][lc + i][lr] = uv[i];
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            const f32x4 m = *reinterpret_cast<const f32x4*>(&xs[k][tm]), n = *reinterpret_cast<const f32x4*>(&ws[0][k][tn]);
            f32x4 n2 = n;
            if constexpr (GLU) n2 = *reinterpret_cast<const f32x4*>(&ws[1][k][tn]);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    g[i][j] += m[i] * n[j];
                    if constexpr (GLU) u[i][j] += m[i] * n2[j];
                }
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        if (tm + i >= live) continue;
        f32x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            v[j] = g[i][j];
            if constexpr (GLU) {
                if (a.alpha != 0.f) {
                    const float gate = fminf(g[i][j], a.limit);
                    v[j] = gate / (1.f + expf(-a.alpha * gate)) * (fminf(fmaxf(u[i][j], -a.limit), a.limit) + 1.f);
                } else {
                    v[j] = g[i][j] / (1.f + expf(-g[i][j])) * u[i][j];
                }
            }
        }
        *reinterpret_cast<f32x4*>(reinterpret_cast<float*>(a.out) + (int64_t)a.slot_pair[first + tm + i] * a.n + n0 + tn) = v;
    }
}

}  // namespace

int launch_moe_route(const MoeRouteArgs& a, int f32, hipStream_t stream) {
    if (!f32 && a.cols % 32 == 0) {
        const int ez = (a.experts + 63) / 64 * 64;
        const size_t lds = (size_t)(8 * 16 * 68 + 24 * ez + 8 * a.groups) * 4;
        if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(moe_route_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        const int live = a.rows <= 256 ? 2 : a.rows <= 2048 ? 8 : 16;           // few rows: more workgroups, shorter choice
        moe_route_kernel<<<(a.rows + live - 1) / live, 512, lds, stream>>>(a, live);
    } else {
        const size_t lds = (size_t)(2 * a.experts + a.groups) * 4;
        if (f32) moe_route_generic_kernel<float><<<a.rows, 256, lds, stream>>>(a);
        else moe_route_generic_kernel<uint16_t><<<a.rows, 256, lds, stream>>>(a);
    }
    return check_launch("moe_route");
}

int moe_dispatch_blocks(int pairs) { return (pairs + DP - 1) / DP; }

int launch_moe_dispatch(int32_t* slot_pair, int32_t* tiles, int32_t* counts, const int32_t* ids, int pairs, int experts, int tile_rows, int max_tiles,
                        hipStream_t stream) {
    const int grid = moe_dispatch_blocks(pairs);
    moe_count_kernel<<<grid, 256, 0, stream>>>(counts, ids, pairs, experts);
    const int rc = check_launch("moe_count");
    if (rc) return rc;
    moe_scatter_kernel<<<grid, 256, 0, stream>>>(slot_pair, tiles, counts, ids, pairs, experts, tile_rows, max_tiles);
    return check_launch("moe_scatter");
}

int moe_tile_rows(int pairs, int experts, int f32) { return f32 ? FM : pairs / experts >= 256 ? 256 : 128; }

int launch_moe_gemm(const MoeGemmArgs& a, int f32, hipStream_t stream) {
    if (f32) {
        const dim3 grid(a.n / 64, a.max_tiles);
        if (a.glu) moe_gemm_f32_kernel<true><<<grid, 256, 0, stream>>>(a);
        else moe_gemm_f32_kernel<false><<<grid, 256, 0, stream>>>(a);
    } else if (!a.tiles) {
        const int tiles = a.n / 16, busy = a.pairs < a.experts ? a.pairs : a.experts;
        const bool split = a.k >= 2048 || (int64_t)busy * tiles < 4 * 512;     // a long contraction, or too few waves with a tile each: four share one
        const dim3 grid(split ? tiles : (tiles + 3) / 4, a.experts);
        if (a.glu && split) moe_small_kernel<true, true><<<grid, 256, 0, stream>>>(a);
        else if (a.glu) moe_small_kernel<true, false><<<grid, 256, 0, stream>>>(a);
        else if (split) moe_small_kernel<false, true><<<grid, 256, 0, stream>>>(a);
        else moe_small_kernel<false, false><<<grid, 256, 0, stream>>>(a);
    } else {
        if (a.tile_rows == 256) {
            if (a.glu) gemm_shape<true, 2, 4, 8, 4>(a, stream);
            else gemm_shape<false, 2, 4, 8, 4>(a, stream);
        } else {
            if (a.glu) gemm_shape<true, 2, 2, 4, 4>(a, stream);
            else gemm_shape<false, 2, 2, 4, 4>(a, stream);
        }
    }
    return check_launch("moe_gemm");
}

}  // namespace nvh
