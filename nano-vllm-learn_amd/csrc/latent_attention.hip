// Latent attention over a paged cache of one shared row per token: [normed latent c (kv_cols) | rotated key part (rot_cols)].
//   prep     query latent norm, key latent norm, interleaved rotation of the shared key part, cache store: one launch over the projection's rows
//   absorb   per head  q_lat = W_uk^T q_unrotated  and the rotation of the rotated part: queries in the cache's own space
//   attend   softmax(scale q_lat . row) over the rows a query sees, un-normalised sums of c per split of the context
//   value    combine the splits, per head  W_uv (latent sum)
// A query's score against a key needs the cache row only, so one stream over the context serves every head (the decode form; prompts use the
// expanded form of latent_prefill.hip).  Scores, weights and sums are fp32; the weights enter the MFMA as bf16 hi + lo halves.
// Every step exists for bf16 on MFMA tiles and in a plain form for any size and for fp32 activations.
#include "attend_tile.h"

namespace nvh {

namespace {

// ------------------------------------------------------------------------------------------------ prep
__device__ __forceinline__ float wave_sum(float v) {
    v = group_sum<16>(v);
    v = sum_xor16(v);
    return sum_xor32(v);
}
__device__ __forceinline__ float dot4(f32x4 v) { return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]; }

// one wave norms one row part: out(column, 4 values).  Pieces of 4 columns, the first RC per lane kept in registers between the two passes
template <typename T, typename Out>
__device__ __forceinline__ void norm_part(const T* x, int cols, int n, float eps, const float* w, int lane, Out out) {
    constexpr int RC = 6;
    f32x4 keep[RC];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < RC; ++i) {
        const int c = (lane + 64 * i) * 4;
        keep[i] = c < cols ? act_ld4(x + c) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int i = 0; i < RC; ++i) ss += dot4(keep[i]);
    for (int c = (lane + 64 * RC) * 4; c < cols; c += 256) ss += dot4(act_ld4(x + c));
    const float inv = 1.f / sqrtf(wave_sum(ss) / n + eps);
#pragma unroll
    for (int i = 0; i < RC; ++i) {
        const int c = (lane + 64 * i) * 4;
        if (c < cols) out(c, keep[i] * inv * *reinterpret_cast<const f32x4*>(w + c));
    }
    for (int c = (lane + 64 * RC) * 4; c < cols; c += 256) out(c, act_ld4(x + c) * inv * *reinterpret_cast<const f32x4*>(w + c));
}

// one wave per row part (query latent, cache row), four per workgroup: no barrier
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(const LatentPrepArgs a) {
    const int parts = a.kv_cols ? 2 : 1, unit = blockIdx.x * 4 + (threadIdx.x >> 6), row = unit / parts, lane = threadIdx.x & 63;
    if (row >= a.rows) return;
    const T* x = reinterpret_cast<const T*>(a.a) + (int64_t)row * a.a_stride;
    const T* c = x + a.q_cols;
    if (unit - row * parts == 0) {
        norm_part<T>(x, a.q_cols, a.q_rank, a.eps, a.q_w, lane, [&](int i, f32x4 v) {
            if (a.cq_packed) act_st4(reinterpret_cast<uint16_t*>(a.cq_packed) + pack_index(row, i, a.q_cols), v);
            else act_st4(reinterpret_cast<T*>(a.cq) + (int64_t)row * a.q_cols + i, v);
        });
        return;
    }
    const int slot = a.slots[row];
    if (slot < 0) return;
    T* out = reinterpret_cast<T*>(a.cache) + (int64_t)slot * (a.kv_cols + a.rot_cols);
    norm_part<T>(c, a.kv_cols, a.kv_rank, a.eps, a.kv_w, lane, [&](int i, f32x4 v) { act_st4(out + i, v); });
    int64_t pos = a.positions[row];
    if (pos >= a.max_position) pos = a.max_position - 1;
    const float* cs = a.cos_sin + pos * a.rot;
    for (int i = lane; i < a.rot / 2; i += 64) {
        const float u = act_ld(c + a.kv_cols + 2 * i), v = act_ld(c + a.kv_cols + 2 * i + 1), co = cs[i], si = cs[a.rot / 2 + i];
        act_st(out + a.kv_cols + 2 * i, u * co - v * si);
        act_st(out + a.kv_cols + 2 * i + 1, v * co + u * si);
    }
}

// ------------------------------------------------------------------------------------------------ absorb
// rotated part of this workgroup's (row, head): qa[kv_cols ..] = rotate(q[dim_cols ..]); columns past `rot` are zero
template <typename T>
__device__ __forceinline__ void rotate_query(const LatentAttnArgs& a, int row, int head, int first, int step) {
    const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)row * a.q_stride + head * (a.dim_cols + a.qrot_cols) + a.dim_cols;
    T* o = reinterpret_cast<T*>(a.qa) + ((int64_t)row * a.heads + head) * (a.kv_cols + a.rot_cols) + a.kv_cols;
    int64_t pos = a.positions[row];
    if (pos >= a.max_position) pos = a.max_position - 1;
    const float* cs = a.cos_sin + pos * a.rot;
    for (int i = first; i < a.rot_cols / 2; i += step) {
        float r0 = 0.f, r1 = 0.f;
        if (i < a.rot / 2) {
            const float u = act_ld(q + 2 * i), v = act_ld(q + 2 * i + 1), co = cs[i], si = cs[a.rot / 2 + i];
            r0 = u * co - v * si;
            r1 = v * co + u * si;
        }
        act_st(o + 2 * i, r0);
        act_st(o + 2 * i + 1, r1);
    }
}

// grid (heads, kv_cols / 64, row tiles of 16), 4 waves x 16 latent columns
__global__ __launch_bounds__(256) void latent_absorb_kernel(const LatentAttnArgs a) {
    const int head = blockIdx.x, r0 = blockIdx.z * 16;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const int n0 = blockIdx.y * 64 + wave * 16, cols = a.kv_cols + a.rot_cols;
    const int row = r0 + lq < a.rows ? r0 + lq : a.rows - 1;
    const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + (int64_t)row * a.q_stride + head * (a.dim_cols + a.qrot_cols) + 8 * lg;
    const uint16_t* w = reinterpret_cast<const uint16_t*>(a.w_uk) + ((int64_t)head * a.kv_cols + n0 + lq) * a.dim_cols + 8 * lg;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < a.dim_cols; k += 32)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(w + k), *reinterpret_cast<const bf16x8*>(q + k), acc, 0, 0, 0);
    // C^T layout: lane = query row lq, latent columns n0 + 4 lg ..
    if (r0 + lq < a.rows)
        act_st4(reinterpret_cast<uint16_t*>(a.qa) + ((int64_t)(r0 + lq) * a.heads + head) * cols + n0 + 4 * lg, acc);
    if (blockIdx.y == 0 && r0 + (tid >> 4) < a.rows) rotate_query<uint16_t>(a, r0 + (tid >> 4), head, tid & 15, 16);
}

template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_generic_kernel(const LatentAttnArgs a) {
    extern __shared__ float q_lds[];
    const int row = blockIdx.x, head = blockIdx.y;
    const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)row * a.q_stride + head * (a.dim_cols + a.qrot_cols);
    for (int i = threadIdx.x; i < a.dim_cols; i += 256) q_lds[i] = act_ld(q + i);
    __syncthreads();
    T* o = reinterpret_cast<T*>(a.qa) + ((int64_t)row * a.heads + head) * (a.kv_cols + a.rot_cols);
    for (int n = threadIdx.x; n < a.kv_cols; n += 256) {
        const T* w = reinterpret_cast<const T*>(a.w_uk) + ((int64_t)head * a.kv_cols + n) * a.dim_cols;
        float s = 0.f;
        for (int k = 0; k < a.dim_cols; k += 4) {
            const f32x4 v = act_ld4(w + k);
            s += v[0] * q_lds[k] + v[1] * q_lds[k + 1] + v[2] * q_lds[k + 2] + v[3] * q_lds[k + 3];
        }
        act_st(o + n, s);
    }
    rotate_query<T>(a, row, head, threadIdx.x, 256);
}

// ------------------------------------------------------------------------------------------------ attend, any type and size
// one workgroup per (row, head, split); 64 keys at a time: 4 lanes per key for the scores, one thread per latent column for the sums
__device__ __forceinline__ void split_range(int ctx, int splits, int split, int& k0, int& k1) {
    const int tiles = (ctx + 63) / 64, per = (tiles + splits - 1) / splits;
    k0 = split * per * 64;
    k1 = k0 + per * 64 < ctx ? k0 + per * 64 : ctx;
}

template <typename T>
__global__ __launch_bounds__(256) void latent_attend_generic_kernel(const LatentAttnArgs a) {
    constexpr int OC = 8;                            // latent columns per thread: kv_cols <= 2048
    extern __shared__ float q_lds[];                 // [kv_cols + rot_cols]
    __shared__ float p_lds[64];
    const int row = blockIdx.x, head = blockIdx.y, split = blockIdx.z, cols = a.kv_cols + a.rot_cols, tid = threadIdx.x;
    const int seq = a.row_seq ? a.row_seq[row] : row;
    const int ctx = (int)a.positions[row] + 1;
    int k0, k1;
    split_range(ctx, a.splits, split, k0, k1);
    const T* q = reinterpret_cast<const T*>(a.qa) + ((int64_t)row * a.heads + head) * cols;
    for (int i = tid; i < cols; i += 256) q_lds[i] = act_ld(q + i);
    float o[OC], m = -INFINITY, l = 0.f;
#pragma unroll
    for (int j = 0; j < OC; ++j) o[j] = 0.f;
    const float sc = a.scale * kLog2e;
    __syncthreads();
    auto cache_row = [&](int key) {
        const int64_t page = a.block_tables[seq * a.bt_stride + key / a.block_size];
        return reinterpret_cast<const T*>(a.cache) + (page * a.block_size + key % a.block_size) * cols;
    };
    for (int t0 = k0; t0 < k1; t0 += 64) {
        const int key = t0 + (tid >> 2);
        float s = 0.f;
        if (key < k1) {
            const T* r = cache_row(key);
            for (int i = (tid & 3) * 4; i < cols; i += 16) {
                const f32x4 v = act_ld4(r + i);
                s += v[0] * q_lds[i] + v[1] * q_lds[i + 1] + v[2] * q_lds[i + 2] + v[3] * q_lds[i + 3];
            }
        }
        s += __shfl_xor(s, 1);
        s += __shfl_xor(s, 2);
        if ((tid & 3) == 0) p_lds[tid >> 2] = key < k1 ? s * sc : -INFINITY;
        __syncthreads();
        float v = p_lds[tid & 63], mx = v;
        for (int d = 1; d < 64; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
        const float m_new = fmaxf(m, mx), alpha = exp2f(m - m_new);
        v = exp2f(v - m_new);
        float sum = v;
        for (int d = 1; d < 64; d <<= 1) sum += __shfl_xor(sum, d);
        l = l * alpha + sum;
        m = m_new;
        __syncthreads();
        if (tid < 64) p_lds[tid] = v;
        __syncthreads();
#pragma unroll
        for (int j = 0; j < OC; ++j) o[j] *= alpha;
        const int cnt = k1 - t0 < 64 ? k1 - t0 : 64;
        for (int k = 0; k < cnt; ++k) {
            const T* r = cache_row(t0 + k);
            const float p = p_lds[k];
#pragma unroll
            for (int j = 0; j < OC; ++j)
                if (tid + 256 * j < a.kv_cols) o[j] += p * act_ld(r + tid + 256 * j);
        }
        __syncthreads();
    }
    const int64_t rec = ((int64_t)row * a.splits + split) * a.heads + head;
#pragma unroll
    for (int j = 0; j < OC; ++j)
        if (tid + 256 * j < a.kv_cols) a.part_o[rec * a.kv_cols + tid + 256 * j] = o[j];
    if (tid == 0) {
        a.part_ml[rec * 2] = m;
        a.part_ml[rec * 2 + 1] = l;
    }
}

// ------------------------------------------------------------------------------------------------ attend, MFMA (bf16, one row per sequence)
// grid (splits, rows, groups of HT head tiles of 16), 4 waves per head tile.  64 keys at a time in ONE LDS image that serves as K (row reads) and as V (hardware-transposed
// reads): wave w scores keys 16 w .. + 15 for all 16 heads (queries in registers), the waves agree on the tile's maxima through LDS, weights go to
// LDS as bf16 hi + lo in the order the transposed reads deliver keys, and wave w sums its quarter of the latent columns.
// Two images, refilled as soon as a tile has been summed: up to two tiles travel at once, so the stream does not pause for a round trip per tile.
constexpr int kAttendTileBytes = 2 * 16 * 72 * 2 + 4 * 16 * 4;                 // weights and maxima of one head tile

template <int NT, int HT>                            // kv_cols = 64 * NT, rot_cols = 64
__global__ __launch_bounds__(256 * HT) void latent_attend_kernel(const LatentAttnArgs a) {
    constexpr int COLS = 64 * NT + 64, ROWB = COLS * 2, CPR = COLS / 8, KS = COLS / 32, NI = CPR / (4 * HT);   // NI: DMA instructions per wave
    constexpr bool kOdd = ((ROWB / 128) & 1) != 0;
    constexpr int IMG = 64 * ROWB;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];       // [2 images][64][ROWB], 16-byte pieces swizzled inside groups of 8
    const int tid = threadIdx.x, lane = tid & 63, all_wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const int ht = all_wave >> 2, wave = all_wave & 3;                         // head tile of this workgroup, wave of the tile
    uint16_t* p_lds = reinterpret_cast<uint16_t*>(smem + 2 * IMG + ht * kAttendTileBytes);     // [hi | lo][16 heads][64 + 8]
    float* mx_lds = reinterpret_cast<float*>(p_lds + 2 * 16 * 72);                              // [4 waves][16]
    const int split = blockIdx.x, row = blockIdx.y, h0 = (blockIdx.z * HT + ht) * 16;
    const int ctx = (int)a.positions[row] + 1;
    const bool head_ok = h0 + lq < a.heads;
    int k0, k1;
    split_range(ctx, a.splits, split, k0, k1);
    const int64_t rec = ((int64_t)row * a.splits + split) * a.heads + h0 + lq;
    if (k0 >= k1) {
        if (wave == 0 && lg == 0 && head_ok) {
            a.part_ml[rec * 2] = -INFINITY;
            a.part_ml[rec * 2 + 1] = 0.f;
        }
        return;
    }
    auto swz = [](int r) { return kOdd ? ((r >> 1) & 7) : (r & 7); };
    const uint16_t* cache = reinterpret_cast<const uint16_t*>(a.cache);
    // staging: piece s of the image -> (row s / CPR, place s % CPR); the source piece is the place with its low three bits xor-ed
    auto stage = [&](int t0, int buf) {
        unsigned char* img = smem + buf * IMG;
        const int64_t page = a.block_tables[row * a.bt_stride + t0 / a.block_size];          // 64 divides the page: one page per tile
        const uint16_t* base = cache + (page * a.block_size + t0 % a.block_size) * COLS;
        const int live = k1 - t0 < 64 ? k1 - t0 : 64;
#pragma unroll
        for (int j = 0; j < NI; ++j) {
            const int s = (all_wave * NI + j) * 64 + lane;
            const int r = s / CPR, place = s - r * CPR, piece = place ^ swz(r);
            const int rc = r < live ? r : live - 1;                                           // (rows past the context repeat its last one: masked)
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(base + rc * COLS + piece * 8),
                                             (__attribute__((address_space(3))) void*)(img + (all_wave * NI + j) * 1024), 16, 0, 0);
        }
    };
    bf16x8 qf[KS];                                   // B operand: column = head lq, 8 consecutive columns
    {
        const uint16_t* q = reinterpret_cast<const uint16_t*>(a.qa) + ((int64_t)row * a.heads + (head_ok ? h0 + lq : a.heads - 1)) * COLS + 8 * lg;
#pragma unroll
        for (int s = 0; s < KS; ++s) qf[s] = *reinterpret_cast<const bf16x8*>(q + 32 * s);
    }
    // (the queries' loads are issued in front of the tiles': vector-memory operations complete in order)
    stage(k0, 0);
    if (k0 + 64 < k1) stage(k0 + 64, 1);
    f32x4 o[NT];                                     // latent columns 64 t' .. : tile index 4 t + wave -> columns 16 (4 t + wave) + 4 lg, head lq
#pragma unroll
    for (int t = 0; t < NT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    const float sc = a.scale * kLog2e;
    // transposed reads: lane 4 q + p of a 16-lane group addresses key row 4 lg + q (+ 16), columns 4 p .. of the 16-column tile
    const int vr = 4 * lg + (lq >> 2), vp = lq & 3;
    auto tile_body = [&](auto bufc, const int t0) {
        constexpr int buf = decltype(bufc)::value;
        const unsigned char* img = smem + buf * IMG;
        if (t0 + 64 < k1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(NI) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_only_barrier();                          // this tile is in LDS, the next one travels
        const int R = 16 * wave + lq;
        f32x4 s4 = {0.f, 0.f, 0.f, 0.f}, s4b = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const bf16x8 kf = *reinterpret_cast<const bf16x8*>(img + R * ROWB + ((4 * s + lg) ^ swz(R)) * 16);
            if (s & 1) s4b = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], s4b, 0, 0, 0);
            else s4 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], s4, 0, 0, 0);
        }
        s4 += s4b;
        float mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            s4[r] = t0 + 16 * wave + 4 * lg + r < k1 ? s4[r] * sc : -INFINITY;
            mx = fmaxf(mx, s4[r]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        if (lg == 0) mx_lds[wave * 16 + lq] = mx;
        lds_only_barrier();
        mx = fmaxf(fmaxf(mx_lds[lq], mx_lds[16 + lq]), fmaxf(mx_lds[32 + lq], mx_lds[48 + lq]));   // finite: the tile holds a visible key
        const float m_new = fmaxf(m, mx), alpha = fast_exp2(m - m_new);
        m = m_new;
        float p[4], hi[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            p[r] = fast_exp2(s4[r] - m_new);
            hi[r] = (float)(__bf16)p[r];
        }
        l = l * alpha + (p[0] + p[1] + p[2] + p[3]);
        // key 16 w + 4 lg + r -> 32-key half w / 2, slot 8 lg + 4 (w & 1) + r
        const int at = lq * 72 + 32 * (wave >> 1) + 8 * lg + 4 * (wave & 1);
        *reinterpret_cast<u32x2*>(p_lds + at) = u32x2{pack_bf16x2(p[0], p[1]), pack_bf16x2(p[2], p[3])};
        *reinterpret_cast<u32x2*>(p_lds + 16 * 72 + at) = u32x2{pack_bf16x2(p[0] - hi[0], p[1] - hi[1]), pack_bf16x2(p[2] - hi[2], p[3] - hi[3])};
        lds_only_barrier();
#pragma unroll
        for (int t = 0; t < NT; ++t) o[t] *= alpha;
#pragma unroll
        for (int hh = 0; hh < 2; ++hh) {
            const bf16x8 ph = *reinterpret_cast<const bf16x8*>(p_lds + lq * 72 + 32 * hh + 8 * lg);
            const bf16x8 pl = *reinterpret_cast<const bf16x8*>(p_lds + 16 * 72 + lq * 72 + 32 * hh + 8 * lg);
            u32x2 v0[NT], v1[NT];
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int tile = 4 * t + wave, ra = 32 * hh + vr, rb = ra + 16;
                v0[t] = ds_read_tr16<0>(lds_addr_of(img + ra * ROWB + ((2 * tile + (vp >> 1)) ^ swz(ra)) * 16 + (vp & 1) * 8));
                v1[t] = ds_read_tr16<0>(lds_addr_of(img + rb * ROWB + ((2 * tile + (vp >> 1)) ^ swz(rb)) * 16 + (vp & 1) * 8));
            }
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const u32x4 raw = {v0[t][0], v0[t][1], v1[t][0], v1[t][1]};
                const bf16x8 vf = *reinterpret_cast<const bf16x8*>(&raw);
                o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, o[t], 0, 0, 0);
                o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, o[t], 0, 0, 0);
            }
        }
        if (t0 + 128 < k1) {
            lds_only_barrier();                      // every wave is done with this image: the tile after the next may have it
            stage(t0 + 128, buf);
        }
    };
    for (int t0 = k0; t0 < k1; t0 += 128) {
        tile_body(std::integral_constant<int, 0>{}, t0);
        if (t0 + 64 < k1) tile_body(std::integral_constant<int, 1>{}, t0 + 64);
    }
    if (head_ok) {
#pragma unroll
        for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(a.part_o + rec * a.kv_cols + 16 * (4 * t + wave) + 4 * lg) = o[t];
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (lg == 0) mx_lds[wave * 16 + lq] = l;
    __syncthreads();
    if (wave == 0 && lg == 0 && head_ok) {
        a.part_ml[rec * 2] = m;
        a.part_ml[rec * 2 + 1] = mx_lds[lq] + mx_lds[16 + lq] + mx_lds[32 + lq] + mx_lds[48 + lq];
    }
}

// ------------------------------------------------------------------------------------------------ value
// normalised latent sum of (row, head) at columns c .. c + 3 from the split records
__device__ __forceinline__ f32x4 combine_splits(const LatentAttnArgs& a, int row, int head, int c, float m, float inv) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.splits; ++s) {
        const int64_t rec = ((int64_t)row * a.splits + s) * a.heads + head;
        const float ms = a.part_ml[rec * 2];
        if (ms == -INFINITY) continue;               // an empty split wrote no sums
        acc += *reinterpret_cast<const f32x4*>(a.part_o + rec * a.kv_cols + c) * (fast_exp2(ms - m) * inv);
    }
    return acc;
}
__device__ __forceinline__ void split_totals(const LatentAttnArgs& a, int row, int head, float& m, float& inv) {
    m = -INFINITY;
    for (int s = 0; s < a.splits; ++s) m = fmaxf(m, a.part_ml[(((int64_t)row * a.splits + s) * a.heads + head) * 2]);
    float l = 0.f;
    for (int s = 0; s < a.splits; ++s) {
        const int64_t rec = ((int64_t)row * a.splits + s) * a.heads + head;
        const float ms = a.part_ml[rec * 2];
        if (ms != -INFINITY) l += a.part_ml[rec * 2 + 1] * fast_exp2(ms - m);
    }
    inv = l > 0.f ? 1.f / l : 0.f;
}

// grid (heads, row tiles of RW), 8 waves: weights of the splits into LDS, latent sums of the rows into LDS as the second operand, waves share the
// value columns.  The first value columns' weights are asked for before anything else.
template <int RW>
__global__ __launch_bounds__(512) void latent_value_kernel(const LatentAttnArgs a) {
    extern __shared__ __attribute__((aligned(16))) uint16_t lat[];             // [RW][kv_cols + 8]
    __shared__ float wsp[RW][64];
    constexpr int PRE = 16;
    const int head = blockIdx.x, r0 = blockIdx.y * RW, ld = a.kv_cols + 8, pieces = a.kv_cols / 4, ksteps = a.kv_cols / 32;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const uint16_t* w_head = reinterpret_cast<const uint16_t*>(a.w_uv) + ((int64_t)head * a.v_cols + lq) * a.kv_cols + 8 * lg;
    // everything this workgroup reads is asked for at once: maxima and sums of its rows' splits (lane = split; places past the live ones are dropped)
    constexpr int RPW = (RW + 7) / 8;
    float ms_all[RPW], ls_all[RPW];
#pragma unroll
    for (int i = 0; i < RPW; ++i) {
        const int r = wave + 8 * i, row = r < RW && r0 + r < a.rows ? r0 + r : r0;
        const int64_t rec = ((int64_t)row * a.splits + (lane < a.splits ? lane : 0)) * a.heads + head;
        ms_all[i] = a.part_ml[rec * 2];
        ls_all[i] = a.part_ml[rec * 2 + 1];
    }
    // this thread's first piece: the sums of the first PS splits, asked for before their weights are known (places past the live splits are dropped)
    constexpr int PS = 8;
    f32x4 first[PS];
    {
        const int r = tid / pieces, row = r0 + r < a.rows && r < RW ? r0 + r : r0;
        const float* p = a.part_o + ((int64_t)row * a.splits * a.heads + head) * a.kv_cols + (tid - r * pieces) * 4;
#pragma unroll
        for (int s = 0; s < PS; ++s) first[s] = *reinterpret_cast<const f32x4*>(p + (s < a.splits ? s : 0) * (int64_t)a.heads * a.kv_cols);
    }
    bf16x8 pre[PRE];
    {
        const uint16_t* w = w_head + (int64_t)(16 * wave < a.v_cols ? 16 * wave : 0) * a.kv_cols;
#pragma unroll
        for (int k = 0; k < PRE; ++k) pre[k] = *reinterpret_cast<const bf16x8*>(w + 32 * (k < ksteps ? k : 0));
    }
    auto live_splits = [&](int row) {                // splits that hold keys of this row
        const int tiles = ((int)a.positions[row] + 64) / 64, per = (tiles + a.splits - 1) / a.splits;
        return (tiles + per - 1) / per;
    };
#pragma unroll
    for (int i = 0; i < RPW; ++i) {
        const int r = wave + 8 * i;
        if (r >= RW || r0 + r >= a.rows) break;
        const bool ok = lane < live_splits(r0 + r);
        const float ms = ok ? ms_all[i] : -INFINITY, ls = ok ? ls_all[i] : 0.f;
        float m = ms;
        for (int d = 1; d < 64; d <<= 1) m = fmaxf(m, __shfl_xor(m, d));
        const float e = fast_exp2(ms - m);
        float l = ls * e;
        for (int d = 1; d < 64; d <<= 1) l += __shfl_xor(l, d);
        wsp[r][lane] = e * (l > 0.f ? 1.f / l : 0.f);
    }
    __syncthreads();
    for (int e = tid; e < RW * pieces; e += 512) {
        const int r = e / pieces, c = (e - r * pieces) * 4;
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r0 + r < a.rows) {
            const int n = live_splits(r0 + r);
            const float* p = a.part_o + ((int64_t)(r0 + r) * a.splits * a.heads + head) * a.kv_cols + c;
            const int64_t step = (int64_t)a.heads * a.kv_cols;
            if (e == tid) {
#pragma unroll
                for (int s = 0; s < PS; ++s)
                    if (s < n) v += first[s] * wsp[r][s];
            }
#pragma unroll 4
            for (int s = e == tid ? PS : 0; s < n; ++s) v += *reinterpret_cast<const f32x4*>(p + s * step) * wsp[r][s];
        }
        act_st4(lat + r * ld + c, v);
    }
    __syncthreads();
    const uint16_t* l_row = lat + (lq < RW ? lq : 0) * ld + 8 * lg;            // (columns past RW are computed and dropped)
    for (int nt = wave; nt < a.v_cols / 16; nt += 8) {
        const uint16_t* w = w_head + (int64_t)16 * nt * a.kv_cols;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if (nt == wave) {
            f32x4 acc2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < PRE; ++k)
                if (k < ksteps) {
                    f32x4& c = k & 1 ? acc2 : acc;
                    c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pre[k], *reinterpret_cast<const bf16x8*>(l_row + 32 * k), c, 0, 0, 0);
                }
            acc += acc2;
        }
        for (int k = nt == wave ? PRE : 0; k < ksteps; ++k)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(w + 32 * k), *reinterpret_cast<const bf16x8*>(l_row + 32 * k), acc, 0, 0, 0);
        if (lq < RW && r0 + lq < a.rows) {           // C^T: lane = row lq, value columns 16 nt + 4 lg ..
            const int col = head * a.v_cols + 16 * nt + 4 * lg;
            if (a.out) act_st4(reinterpret_cast<uint16_t*>(a.out) + (int64_t)(r0 + lq) * a.out_stride + col, acc);
            if (a.out_packed) act_st4(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(r0 + lq, col, a.heads * a.v_cols), acc);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_value_generic_kernel(const LatentAttnArgs a) {
    extern __shared__ float latf[];
    const int row = blockIdx.x, head = blockIdx.y;
    float m, inv;
    split_totals(a, row, head, m, inv);
    for (int c = threadIdx.x * 4; c < a.kv_cols; c += 1024) {
        const f32x4 v = combine_splits(a, row, head, c, m, inv);
#pragma unroll
        for (int k = 0; k < 4; ++k) latf[c + k] = act_round(v[k], (const T*)nullptr);
    }
    __syncthreads();
    for (int n = threadIdx.x; n < a.v_cols; n += 256) {
        const T* w = reinterpret_cast<const T*>(a.w_uv) + ((int64_t)head * a.v_cols + n) * a.kv_cols;
        float s = 0.f;
        for (int k = 0; k < a.kv_cols; k += 4) {
            const f32x4 v = act_ld4(w + k);
            s += v[0] * latf[k] + v[1] * latf[k + 1] + v[2] * latf[k + 2] + v[3] * latf[k + 3];
        }
        act_st(reinterpret_cast<T*>(a.out) + (int64_t)row * a.out_stride + head * a.v_cols + n, s);
    }
}

// ------------------------------------------------------------------------------------------------ gather
// cache rows of every key of the sequences, packed: out[cu_k[b] + j] = row of key j of sequence b.  One 16-byte piece per thread
__global__ __launch_bounds__(256) void latent_gather_kernel(u32x4* __restrict__ out, const u32x4* __restrict__ cache, const int32_t* __restrict__ cu_k,
                                                             const int32_t* __restrict__ block_tables, int64_t bt_stride, int batch, int total, int pieces,
                                                             int block_size) {
    const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int row = (int)(e / pieces), p = (int)(e - (int64_t)row * pieces);
    if (row >= total) return;
    int lo = 0, hi = batch;                          // sequence of this row: the last b with cu_k[b] <= row
    while (hi - lo > 1) {
        const int mid = (lo + hi) / 2;
        if (cu_k[mid] <= row) lo = mid;
        else hi = mid;
    }
    const int key = row - cu_k[lo];
    const int64_t page = block_tables[lo * bt_stride + key / block_size];
    out[e] = cache[(page * block_size + key % block_size) * pieces + p];
}

template <int NT, int HT>
void attend_ht(const LatentAttnArgs& a, hipStream_t stream) {
    constexpr size_t lds = 2 * 64 * (64 * NT + 64) * 2 + HT * kAttendTileBytes;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(latent_attend_kernel<NT, HT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    latent_attend_kernel<NT, HT><<<dim3(a.splits, a.rows, (a.heads + 16 * HT - 1) / (16 * HT)), 256 * HT, lds, stream>>>(a);
}
template <int NT>
void attend_nt(const LatentAttnArgs& a, hipStream_t stream) {
    if (a.heads > 16) attend_ht<NT, 2>(a, stream);   // two head tiles share the images: one stream over the cache for 32 heads
    else attend_ht<NT, 1>(a, stream);
}

}  // namespace

int launch_latent_prep(const LatentPrepArgs& a, int f32, hipStream_t stream) {
    const int grid = (a.rows * (a.kv_cols ? 2 : 1) + 3) / 4;
    if (f32) latent_prep_kernel<float><<<grid, 256, 0, stream>>>(a);
    else latent_prep_kernel<uint16_t><<<grid, 256, 0, stream>>>(a);
    return check_launch("latent_prep");
}

int launch_latent_absorb(const LatentAttnArgs& a, int f32, hipStream_t stream) {
    if (!f32 && a.dim_cols % 32 == 0 && a.kv_cols % 64 == 0) {
        latent_absorb_kernel<<<dim3(a.heads, a.kv_cols / 64, (a.rows + 15) / 16), 256, 0, stream>>>(a);
    } else {
        const dim3 grid(a.rows, a.heads);
        if (f32) latent_absorb_generic_kernel<float><<<grid, 256, a.dim_cols * 4, stream>>>(a);
        else latent_absorb_generic_kernel<uint16_t><<<grid, 256, a.dim_cols * 4, stream>>>(a);
    }
    return check_launch("latent_absorb");
}

bool latent_mfma_supported(int kv_cols, int rot_cols, int block_size) {
    if (rot_cols != 64 || block_size % 64) return false;
    switch (kv_cols) {
        case 64: case 128: case 192: case 256: case 384: case 512: return true;
        default: return false;
    }
}

int launch_latent_attend(const LatentAttnArgs& a, int f32, int generic, hipStream_t stream) {
    if (!f32 && !generic && !a.row_seq && latent_mfma_supported(a.kv_cols, a.rot_cols, a.block_size)) {
        switch (a.kv_cols) {
            case 64: attend_nt<1>(a, stream); break;
            case 128: attend_nt<2>(a, stream); break;
            case 192: attend_nt<3>(a, stream); break;
            case 256: attend_nt<4>(a, stream); break;
            case 384: attend_nt<6>(a, stream); break;
            default: attend_nt<8>(a, stream); break;
        }
    } else {
        const dim3 grid(a.rows, a.heads, a.splits);
        const size_t lds = (size_t)(a.kv_cols + a.rot_cols) * 4;
        if (f32) latent_attend_generic_kernel<float><<<grid, 256, lds, stream>>>(a);
        else latent_attend_generic_kernel<uint16_t><<<grid, 256, lds, stream>>>(a);
    }
    return check_launch("latent_attend");
}

int launch_latent_value(const LatentAttnArgs& a, int f32, hipStream_t stream) {
    if (!f32 && a.v_cols % 16 == 0 && a.kv_cols % 32 == 0 && a.splits <= 64) {
        if (a.rows <= 128) latent_value_kernel<4><<<dim3(a.heads, (a.rows + 3) / 4), 512, (size_t)4 * (a.kv_cols + 8) * 2, stream>>>(a);
        else latent_value_kernel<16><<<dim3(a.heads, (a.rows + 15) / 16), 512, (size_t)16 * (a.kv_cols + 8) * 2, stream>>>(a);
    } else {
        const dim3 grid(a.rows, a.heads);
        if (f32) latent_value_generic_kernel<float><<<grid, 256, a.kv_cols * 4, stream>>>(a);
        else latent_value_generic_kernel<uint16_t><<<grid, 256, a.kv_cols * 4, stream>>>(a);
    }
    return check_launch("latent_value");
}

int launch_latent_gather(void* out, const void* cache, const int32_t* cu_k, const int32_t* block_tables, int64_t bt_stride, int batch, int total, int cols,
                         int block_size, int f32, hipStream_t stream) {
    const int pieces = cols * (f32 ? 4 : 2) / 16;
    const int64_t grid = ((int64_t)total * pieces + 255) / 256;
    latent_gather_kernel<<<(unsigned)grid, 256, 0, stream>>>((u32x4*)out, (const u32x4*)cache, cu_k, block_tables, bt_stride, batch, total, pieces, block_size);
    return check_launch("latent_gather");
}

}  // namespace nvh
