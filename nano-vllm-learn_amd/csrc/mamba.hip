// Selective scan: per channel c and state n, with a step size per (token, channel) and input and output vectors per token,
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n        y_c = sum_n S[c, n] C_n + D_c x_c        out = y silu(z)
// dt = softplus(projection + bias).  Everything but the projections and x is fp32.
//
// Prompt portions (launch_scan_chunks): a workgroup owns one (segment, CHN channels) and takes TT tokens at a time.  dt and dt x are computed once per (token,
// channel) on 16-byte pieces of the rows and left in LDS, next to B and C of the tokens; then NL lanes per channel walk the tokens with NS states each in
// registers; a last pass adds D x, gates and writes 16-byte pieces.  The next tile's rows are fetched while this one is scanned.
// A portion of several segments: a SUMMARY walk leaves every segment's own contribution and its sum of dt (the product of its decays is exp(A sum dt)), a small
// launch turns those into states at segment starts, and the second walk begins there.
// Decoding (launch_scan_step): four states per lane, dt from the projection's low-rank row on the spot, several rows per workgroup so that its weights are read
// once for all of them.
// Per (token, channel, state): one transcendental and four vector instructions: issue-bound, not HBM-bound.
// A sequence's first token (position 0) takes the state as zero instead of reading it: slots need no clearing when reused.
#include <type_traits>

#include "api_common.h"
#include "mixers.h"

namespace nvh {

namespace {

using ScanArgs = nvh_scan_desc;
constexpr int TILE = 2048;                           // (token, channel) pairs a workgroup stages at a time
constexpr int min3(int x, int y, int z) { return x < y ? (x < z ? x : z) : (y < z ? y : z); }

// log(1 + e^z); by the series of log(1 + e) where 1 + e would round
__device__ __forceinline__ float softplus_f(float z) {
    const float e = __expf(z);
    const float small = e * (1.f - e * (1.f / 2 - e * (1.f / 3 - e * (1.f / 4 - e * (1.f / 5)))));
    return z > 20.f ? z : e < 0.0625f ? small : __logf(1.f + e);
}

__device__ __forceinline__ float gate_f(float z) { return z * fast_rcp(1.f + fast_exp2(-kLog2e * z)); }         // silu

template <int LANES>
__device__ __forceinline__ float sum_lanes(float v) {        // over aligned groups of LANES lanes
    if constexpr (LANES >= 2) v += pair_in_row<1>(v);
    if constexpr (LANES >= 4) v += pair_in_row<2>(v);
    if constexpr (LANES >= 8) v += pair_in_row<4>(v);
    if constexpr (LANES >= 16) v += pair_in_row<8>(v);
    if constexpr (LANES >= 32) v = sum_xor16(v);
    if constexpr (LANES >= 64) v = sum_xor32(v);
    return v;
}

template <typename T, int NS, int NL, bool SUMMARY>
__global__ __launch_bounds__(256) void scan_walk_kernel(const ScanArgs a) {
    constexpr int NP = NS * NL, CHN = 256 / NL, TT = min3(TILE / CHN, 64, 4096 / NP), PIECES = TT * CHN / 8;     // (PIECES <= 256)
    constexpr int BCP = (TT * 2 * NP / 8 + 255) / 256;                         // pieces of B | C per thread
    __shared__ __attribute__((aligned(16))) float dt_s[TT * CHN], dx_s[TT * CHN], y_s[SUMMARY ? 8 : TT * CHN], bc_s[TT * 2 * NP];
    const int32_t* ch = a.chunks + 4 * blockIdx.x;
    const int row0 = ch[0], n_rows = ch[1], seq = ch[2];
    const bool last = blockIdx.x + 1 == (unsigned)a.n_chunks || a.chunks[4 * (blockIdx.x + 1) + 3] == 0;
    if (SUMMARY && last) return;                     // (nothing follows it)
    const int tid = threadIdx.x, c0 = blockIdx.y * CHN, lane_ch = tid / NL, sl = tid % NL;
    const int my = c0 + lane_ch < a.inner ? c0 + lane_ch : a.inner - 1;        // channel this lane scans (a last group may be short)
    const int64_t slot = a.state_slots[seq];
    float A[NS], S[NS], dt_sum = 0.f;
#pragma unroll
    for (int s = 0; s < NS; s += 4) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(a.a_log2 + (int64_t)my * NP + sl * NS + s);
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            A[s + k] = v[k];
            S[s + k] = 0.f;
        }
    }
    if constexpr (!SUMMARY) {
        const float* src = nullptr;
        if (a.summaries) src = a.seg_state + ((int64_t)blockIdx.x * a.inner + my) * NP;
        else if (slot >= 0 && a.positions[row0] > 0) src = a.state + (slot * a.inner + my) * NP;
        if (src) {
#pragma unroll
            for (int s = 0; s < NS; s += 4) {
                const f32x4 v = *reinterpret_cast<const f32x4*>(src + sl * NS + s);
#pragma unroll
                for (int k = 0; k < 4; ++k) S[s + k] = v[k];
            }
        }
    }
    // ---- this thread's piece of the tile: token pt, channels pc .. pc + 7
    const int pt = tid / (CHN / 8), pc = c0 + tid % (CHN / 8) * 8;
    const bool piece = tid < PIECES && pc < a.inner;
    const f32x8 bias = piece ? act_ld8(a.dt_bias + pc) : f32x8{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    f32x8 D = bias;
    if (!SUMMARY && piece) D = act_ld8(a.d + pc);
    f32x8 xr, dr, zr, bc[BCP];
    const f32x8 zero = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    auto fetch = [&](int t0) {
        const bool ok = piece && t0 + pt < n_rows;
        const int64_t r = row0 + t0 + pt;
        xr = ok ? act_ld8(reinterpret_cast<const T*>(a.x) + r * a.x_stride + pc) : zero;
        dr = ok ? act_ld8(reinterpret_cast<const T*>(a.dt) + r * a.dt_stride + pc) : zero;
        if constexpr (!SUMMARY) zr = ok ? act_ld8(reinterpret_cast<const T*>(a.z) + r * a.z_stride + pc) : zero;
#pragma unroll
        for (int j = 0; j < BCP; ++j) {
            const int e = j * 256 + tid, t = e / (2 * NP / 8), p = e - t * (2 * NP / 8);
            bc[j] = e < TT * 2 * NP / 8 && t0 + t < n_rows ? act_ld8(reinterpret_cast<const T*>(a.bc) + (int64_t)(row0 + t0 + t) * a.bc_stride + p * 8) : zero;
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < n_rows; t0 += TT) {
        const int n = n_rows - t0 < TT ? n_rows - t0 : TT;
        const f32x8 xk = xr, zk = zr;
        if (tid < PIECES) {
            f32x8 dt;
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                dt.a[k] = pt < n ? softplus_f(dr.a[k] + bias.a[k]) : 0.f;      // (a token past the end leaves the state alone)
                dt.b[k] = pt < n ? softplus_f(dr.b[k] + bias.b[k]) : 0.f;
            }
            act_st8(dt_s + tid * 8, dt);
            act_st8(dx_s + tid * 8, f32x8{dt.a * xk.a, dt.b * xk.b});
        }
#pragma unroll
        for (int j = 0; j < BCP; ++j)
            if (j * 256 + tid < TT * 2 * NP / 8) act_st8(bc_s + (j * 256 + tid) * 8, bc[j]);
        __syncthreads();
        if (t0 + TT < n_rows) fetch(t0 + TT);
        for (int tb = 0; tb < n; tb += 4) {
#pragma unroll
            for (int t = tb; t < tb + 4; ++t) {
                const float dt = dt_s[t * CHN + lane_ch], dx = dx_s[t * CHN + lane_ch];
                const float* b = bc_s + t * 2 * NP + sl * NS;
                float y = 0.f;
#pragma unroll
                for (int s = 0; s < NS; s += 4) {
                    const f32x4 bv = *reinterpret_cast<const f32x4*>(b + s);
                    f32x4 cv = bv;
                    if constexpr (!SUMMARY) cv = *reinterpret_cast<const f32x4*>(b + NP + s);
#pragma unroll
                    for (int k = 0; k < 4; ++k) {
                        S[s + k] = fast_exp2(dt * A[s + k]) * S[s + k] + dx * bv[k];
                        if constexpr (!SUMMARY) y += S[s + k] * cv[k];
                    }
                }
                if constexpr (SUMMARY) {
                    dt_sum += dt;
                } else {
                    y = sum_lanes<NL>(y);
                    if (sl == 0) y_s[t * CHN + lane_ch] = y;
                }
            }
        }
        __syncthreads();
        if constexpr (!SUMMARY) {
            if (piece && pt < n) {
                f32x8 y = act_ld8(y_s + tid * 8);
                y.a += D.a * xk.a;
                y.b += D.b * xk.b;
#pragma unroll
                for (int k = 0; k < 4; ++k) {
                    y.a[k] *= gate_f(zk.a[k]);
                    y.b[k] *= gate_f(zk.b[k]);
                }
                act_st8(reinterpret_cast<T*>(a.out) + (int64_t)(row0 + t0 + pt) * a.out_stride + pc, y);
            }
        }
        // (the next tile's y is written behind the barrier that follows its staging)
    }
    if (c0 + lane_ch >= a.inner) return;
    float* dst = nullptr;
    if constexpr (SUMMARY) {
        dst = a.seg_state + ((int64_t)blockIdx.x * a.inner + my) * NP;
        if (sl == 0) a.seg_dt[(int64_t)blockIdx.x * a.inner + my] = dt_sum;
    } else if (last && slot >= 0) {
        dst = a.state + (slot * a.inner + my) * NP;
    }
    if (dst) {
#pragma unroll
        for (int s = 0; s < NS; s += 4) *reinterpret_cast<f32x4*>(dst + sl * NS + s) = f32x4{S[s], S[s + 1], S[s + 2], S[s + 3]};
    }
}

// contributions of the segments -> states at their starts, in place; one thread per state, walking the segments of every portion
__global__ __launch_bounds__(256) void scan_starts_kernel(const ScanArgs a) {
    const int64_t per = (int64_t)a.inner * a.n, e = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int first = blockIdx.y;                    // only a portion's first segment starts a walk
    if (e >= per || a.chunks[4 * first + 3] != 0) return;
    const float A = a.a_log2[e];
    const int64_t c = e / a.n, slot = a.state_slots[a.chunks[4 * first + 2]];
    float cur = slot >= 0 && a.positions[a.chunks[4 * first]] > 0 ? a.state[slot * per + e] : 0.f;
    for (int k = first; k < a.n_chunks && (k == first || a.chunks[4 * k + 3] != 0); ++k) {
        const bool more = k + 1 < a.n_chunks && a.chunks[4 * (k + 1) + 3] != 0;        // (the last segment left no contribution)
        const float own = more ? a.seg_state[k * per + e] : 0.f;
        a.seg_state[k * per + e] = cur;
        if (more) cur = fast_exp2(A * a.seg_dt[k * a.inner + c]) * cur + own;
    }
}

// one new token per sequence (bf16): grid (channel groups, groups of R rows), LN = n / 4 lanes per channel
template <int LN, int R>
__global__ __launch_bounds__(256) void scan_step_kernel(const ScanArgs a) {
    constexpr int CHN = 256 / LN, NP = 4 * LN;
    const int tid = threadIdx.x, sl = tid % LN, c = blockIdx.x * CHN + tid / LN;
    const bool ok = c < a.inner;
    const int my = ok ? c : a.inner - 1;
    const uint16_t* w = reinterpret_cast<const uint16_t*>(a.w_dt) + (int64_t)my * a.rank;
    const int r0 = blockIdx.y * R;
    f32x4 s[R];
    float xv[R], zv[R];
#pragma unroll
    for (int i = 0; i < R; ++i) {                    // asked for before anything is computed
        const int row = r0 + i < a.rows ? r0 + i : a.rows - 1;
        const int64_t slot = a.state_slots[row];
        s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (slot >= 0 && a.positions[row] > 0) s[i] = *reinterpret_cast<const f32x4*>(a.state + (slot * a.inner + my) * NP + 4 * sl);
        xv[i] = act_ld(reinterpret_cast<const uint16_t*>(a.x) + (int64_t)row * a.x_stride + my);
        zv[i] = act_ld(reinterpret_cast<const uint16_t*>(a.z) + (int64_t)row * a.z_stride + my);
    }
    const f32x4 A = *reinterpret_cast<const f32x4*>(a.a_log2 + (int64_t)my * NP + 4 * sl);
    float acc[R];
#pragma unroll
    for (int i = 0; i < R; ++i) acc[i] = 0.f;
    for (int p = sl * 8; p < a.rank; p += LN * 8) {
        const u32x4 wv = *reinterpret_cast<const u32x4*>(w + p);
#pragma unroll
        for (int i = 0; i < R; ++i) {
            const int row = r0 + i < a.rows ? r0 + i : a.rows - 1;
            const u32x4 v = *reinterpret_cast<const u32x4*>(reinterpret_cast<const uint16_t*>(a.dt) + (int64_t)row * a.dt_stride + p);
#pragma unroll
            for (int k = 0; k < 4; ++k) acc[i] = dot2_bf16(wv[k], v[k], acc[i]);
        }
    }
    const float bias = a.dt_bias[my], D = a.d[my];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int row = r0 + i;
        if (row >= a.rows) continue;                 // (workgroup-uniform)
        const float dt = softplus_f(sum_lanes<LN>(acc[i]) + bias), dx = dt * xv[i];
        const uint16_t* bc = reinterpret_cast<const uint16_t*>(a.bc) + (int64_t)row * a.bc_stride + 4 * sl;
        const f32x4 b = act_ld4(bc), cv = act_ld4(bc + NP);
        f32x4 n;
        float y = 0.f;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            n[k] = fast_exp2(dt * A[k]) * s[i][k] + dx * b[k];
            y += n[k] * cv[k];
        }
        const int64_t slot = a.state_slots[row];
        if (ok && slot >= 0) *reinterpret_cast<f32x4*>(a.state + (slot * a.inner + my) * NP + 4 * sl) = n;
        y = (sum_lanes<LN>(y) + D * xv[i]) * gate_f(zv[i]);
        if (ok && sl == 0) {
            if (a.out) act_st(reinterpret_cast<uint16_t*>(a.out) + (int64_t)row * a.out_stride + c, y);
            if (a.out_packed) act_st(reinterpret_cast<uint16_t*>(a.out_packed) + pack_index(row, c, a.inner), y);
        }
    }
}

template <typename T, int NS, int NL>
int walk_ns(const ScanArgs& a, hipStream_t stream) {
    constexpr int CHN = 256 / NL;
    const dim3 grid(a.n_chunks, (a.inner + CHN - 1) / CHN);
    if (a.summaries) {
        scan_walk_kernel<T, NS, NL, true><<<grid, 256, 0, stream>>>(a);
        int rc = check_launch("scan summary");
        if (rc) return rc;
        const int64_t per = (int64_t)a.inner * a.n;
        scan_starts_kernel<<<dim3((unsigned)((per + 255) / 256), a.n_chunks), 256, 0, stream>>>(a);
        rc = check_launch("scan starts");
        if (rc) return rc;
    }
    scan_walk_kernel<T, NS, NL, false><<<grid, 256, 0, stream>>>(a);
    return check_launch("scan walk");
}

template <typename T>
int walk_t(const ScanArgs& a, hipStream_t stream) {
    // states per lane: fewer lanes per channel cost less, but two waves per SIMD of the 256 CUs should be there
    const int64_t waves = (int64_t)a.n_chunks * ((a.inner + 63) / 64);
    switch (a.n) {
        case 8: return waves >= 2048 ? walk_ns<T, 8, 1>(a, stream) : walk_ns<T, 4, 2>(a, stream);
        case 16: return waves >= 2048 ? walk_ns<T, 16, 1>(a, stream) : waves >= 1024 ? walk_ns<T, 8, 2>(a, stream) : walk_ns<T, 4, 4>(a, stream);
        case 32: return waves >= 1024 ? walk_ns<T, 16, 2>(a, stream) : walk_ns<T, 8, 4>(a, stream);
        case 64: return walk_ns<T, 16, 4>(a, stream);
        case 128: return walk_ns<T, 16, 8>(a, stream);
        default: return walk_ns<T, 16, 16>(a, stream);
    }
}

template <int LN>
void step_ln(const ScanArgs& a, hipStream_t stream) {
    constexpr int CHN = 256 / LN;
    const unsigned groups = (a.inner + CHN - 1) / CHN;
    if ((int64_t)groups * a.rows >= 2048) scan_step_kernel<LN, 4><<<dim3(groups, (a.rows + 3) / 4), 256, 0, stream>>>(a);
    else scan_step_kernel<LN, 1><<<dim3(groups, a.rows), 256, 0, stream>>>(a);
}

int check_scan(const char* fn, const nvh_scan_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->x && d->dt && d->dt_bias && d->bc && d->z && d->a_log2 && d->d && d->positions && d->state_slots && d->state && (d->out || d->out_packed), NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->rows > 0 && d->inner > 0 && d->inner % 8 == 0 && nvh_scan_states(d->n) == d->n, NVH_E_SHAPE, "%s: %d channels (%%8), %d states", fn, d->inner, d->n);
    REQUIRE(d->x_stride % 8 == 0 && d->x_stride >= d->inner && d->z_stride % 8 == 0 && d->z_stride >= d->inner && d->bc_stride % 8 == 0 && d->bc_stride >= 2 * d->n &&
            d->dt_stride % 8 == 0 && (!d->out || (d->out_stride % 8 == 0 && d->out_stride >= d->inner)), NVH_E_STRIDE, "%s: row strides", fn);
    REQUIRE(aligned16(d->x) && aligned16(d->dt) && aligned16(d->dt_bias) && aligned16(d->bc) && aligned16(d->z) && aligned16(d->a_log2) && aligned16(d->d) && aligned16(d->state) &&
            aligned16(d->seg_state) && aligned16(d->out) && aligned16(d->out_packed), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

}  // namespace

}  // namespace nvh

using namespace nvh;

extern "C" {

int nvh_scan_states(int n) {
    for (int p = 8; p <= 256; p *= 2)
        if (n > 0 && n <= p) return p;
    return 0;
}

int nvh_scan_chunks(const nvh_scan_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "scan_chunks: null descriptor");
    if (d->n_chunks == 0) return 0;
    const int rc = check_scan("scan_chunks", d, dtype);
    if (rc) return rc;
    REQUIRE(d->chunks && d->n_chunks > 0 && d->n_chunks <= 65535 && d->out && d->dt_stride >= d->inner && (!d->summaries || (d->seg_state && d->seg_dt)), NVH_E_NULL,
            "scan_chunks: %d segments or null pointer", d->n_chunks);
    return dtype == NVH_F32 ? walk_t<float>(*d, (hipStream_t)stream) : walk_t<uint16_t>(*d, (hipStream_t)stream);
}

int nvh_scan_step(const nvh_scan_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "scan_step: null descriptor");
    if (d->rows == 0) return 0;
    const int rc = check_scan("scan_step", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16 && d->w_dt && aligned16(d->w_dt) && d->rank > 0 && d->rank % 8 == 0 && d->dt_stride >= d->rank && d->rows <= 65535 && (!d->out_packed || d->inner % 32 == 0),
            NVH_E_SHAPE, "scan_step: bf16, rank %d (%%8), rows %d", d->rank, d->rows);
    switch (d->n / 4) {
        case 2: step_ln<2>(*d, (hipStream_t)stream); break;
        case 4: step_ln<4>(*d, (hipStream_t)stream); break;
        case 8: step_ln<8>(*d, (hipStream_t)stream); break;
        case 16: step_ln<16>(*d, (hipStream_t)stream); break;
        case 32: step_ln<32>(*d, (hipStream_t)stream); break;
        default: step_ln<64>(*d, (hipStream_t)stream); break;
    }
    return check_launch("scan_step");
}

}  // extern "C"
