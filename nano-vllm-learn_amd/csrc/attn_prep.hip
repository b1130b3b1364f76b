// Row ops between a q | k | v projection and attention over pages: norm of queries and keys (over all columns of the projection at once, or per head with one
// weight for all heads), rotation of interleaved pairs (of values too, where they are stored turned), store of keys and values: one launch over the projection's rows.
#include <type_traits>

#include "api_common.h"
#include "mixers.h"

namespace nvh {

namespace {

// interleaved pairs of 8 elements from dimension d on, turned by a table row (cos | sin of `rot` / 2 angles); dimensions past `rot` pass
__device__ __forceinline__ f32x8 turn8(const f32x8& r, const float* cs, int rot, int d) {
    float e[8] = {r.a[0], r.a[1], r.a[2], r.a[3], r.b[0], r.b[1], r.b[2], r.b[3]};
    float co[4], si[4];
    if ((rot & 7) == 0) {                            // (whole pieces turn or pass)
        const bool turns = d < rot;
        const f32x4 cv = turns ? *reinterpret_cast<const f32x4*>(cs + d / 2) : f32x4{1.f, 1.f, 1.f, 1.f};
        const f32x4 sv = turns ? *reinterpret_cast<const f32x4*>(cs + rot / 2 + d / 2) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int p = 0; p < 4; ++p) {
            co[p] = cv[p];
            si[p] = sv[p];
        }
    } else {
#pragma unroll
        for (int p = 0; p < 4; ++p) {
            const bool turns = d / 2 + p < rot / 2;
            co[p] = turns ? cs[d / 2 + p] : 1.f;
            si[p] = turns ? cs[rot / 2 + d / 2 + p] : 0.f;
        }
    }
#pragma unroll
    for (int p = 0; p < 4; ++p) {
        const float u = e[2 * p], w = e[2 * p + 1];
        e[2 * p] = u * co[p] - w * si[p];
        e[2 * p + 1] = w * co[p] + u * si[p];
    }
    return {f32x4{e[0], e[1], e[2], e[3]}, f32x4{e[4], e[5], e[6], e[7]}};
}

// one workgroup per row; a thread keeps its 8-element pieces of [q | k | v] in registers between the sums and the second pass
// HEADS: the norm runs over every head of queries and keys by itself
template <typename T, int CH, bool HEADS>
__global__ __launch_bounds__(256) void attn_prep_kernel(const AttnPrepArgs a) {
    __shared__ __attribute__((aligned(16))) float lds[HEADS ? CH * 256 : 8];
    const int64_t row = blockIdx.x;
    T* x = reinterpret_cast<T*>(a.qkv) + row * a.qkv_stride;
    const int nq = a.heads * a.dk, nk = a.kv_heads * a.dk, total = nq + nk + a.kv_heads * a.dv;
    int64_t pos = a.positions[row];
    if ((a.rot > 0 || a.v_cos_sin) && pos >= a.max_position) pos = a.max_position - 1;
    const float* cs = a.cos_sin + pos * a.rot;
    const int slot = a.slots[row];
    const int page = slot >= 0 ? slot / a.block_size : 0, off = slot >= 0 ? slot - page * a.block_size : 0;
    T* cache = reinterpret_cast<T*>(a.cache) + (int64_t)page * a.kv_heads * a.block_size * (a.dk + a.dv);
    f32x8 v[CH];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        v[i] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (c < total) v[i] = act_ld8(x + c);
    }
    float head_inv[CH];
    if constexpr (HEADS) {
        const int pieces = a.dk / 8;                 // of a head; heads of 8, 16 or 32 pieces lie in aligned lanes of one wave
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            float ss = sum4(v[i].a * v[i].a) + sum4(v[i].b * v[i].b);
            if (pieces == 8) ss = group_sum<8>(ss);
            else if (pieces == 16) ss = group_sum<16>(ss);
            else if (pieces == 32) ss = sum_xor16(group_sum<16>(ss));
            else lds[threadIdx.x + i * 256] = ss;
            head_inv[i] = ss;
        }
        const bool through_lds = pieces != 8 && pieces != 16 && pieces != 32;
        if (through_lds) __syncthreads();
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const int c = (threadIdx.x + i * 256) * 8;
            if (c >= nq + nk) continue;
            if (through_lds) {
                const float* part = lds + c / a.dk * pieces;
                float ss = 0.f;
                for (int p = 0; p < pieces; ++p) ss += part[p];
                head_inv[i] = ss;
            }
            head_inv[i] = 1.f / sqrtf(head_inv[i] / (c < nq ? a.q_n : a.k_n) + a.eps);
        }
    } else if (a.q_w) {
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const int c = (threadIdx.x + i * 256) * 8;
            const float ss = sum4(v[i].a * v[i].a) + sum4(v[i].b * v[i].b);
            if (c < nq) sq += ss;
            else if (c < nq + nk) sk += ss;
        }
        block_sum256x2(sq, sk, lds);
        sq = 1.f / sqrtf(sq / a.q_n + a.eps);
        sk = 1.f / sqrtf(sk / a.k_n + a.eps);
    }
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= total) continue;
        f32x8 r = v[i];
        if (c < nq + nk) {
            const bool is_q = c < nq;
            const int h = is_q ? c / a.dk : (c - nq) / a.dk, d = (is_q ? c : c - nq) - h * a.dk;
            if (a.q_w) {
                const float* w = HEADS ? (is_q ? a.q_w : a.k_w) + d : is_q ? a.q_w + c : a.k_w + (c - nq);
                const float inv = HEADS ? head_inv[i] : is_q ? sq : sk;
                r.a *= inv * *reinterpret_cast<const f32x4*>(w);
                r.b *= inv * *reinterpret_cast<const f32x4*>(w + 4);
            }
            if (a.rot > 0) r = turn8(r, cs, a.rot, d);
            if (is_q) act_st8(x + c, r);
            else if (slot >= 0) act_st8(cache + (int64_t)h * a.block_size * (a.dk + a.dv) + off * a.dk + d, r);
        } else if (slot >= 0) {
            const int h = (c - nq - nk) / a.dv, d = c - nq - nk - h * a.dv;
            if (a.v_cos_sin) r = turn8(r, a.v_cos_sin + pos * a.v_rot, a.v_rot, d);
            act_st8(cache + (int64_t)h * a.block_size * (a.dk + a.dv) + (int64_t)a.block_size * a.dk + (int64_t)off * a.dv + d, r);
        }
    }
}

template <typename T, int CH>
void prep_ch(const AttnPrepArgs& a, hipStream_t stream) {
    if (a.head_norm) attn_prep_kernel<T, CH, true><<<a.rows, 256, 0, stream>>>(a);
    else attn_prep_kernel<T, CH, false><<<a.rows, 256, 0, stream>>>(a);
}
template <typename T>
void prep_t(const AttnPrepArgs& a, hipStream_t stream) {
    const int ch = (a.heads * a.dk + a.kv_heads * (a.dk + a.dv) + 2047) / 2048;
    if (ch <= 1) prep_ch<T, 1>(a, stream);
    else if (ch <= 2) prep_ch<T, 2>(a, stream);
    else if (ch <= 4) prep_ch<T, 4>(a, stream);
    else if (ch <= 8) prep_ch<T, 8>(a, stream);
    else prep_ch<T, kRowPieces>(a, stream);
}

}  // namespace

int launch_attn_prep(const AttnPrepArgs& a, int f32, hipStream_t stream) {
    if (f32) prep_t<float>(a, stream);
    else prep_t<uint16_t>(a, stream);
    return check_launch("attn_prep");
}

}  // namespace nvh

using namespace nvh;

extern "C" int nvh_attn_prep(const nvh_attn_prep_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "attn_prep: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("attn_prep");
    REQUIRE(d->qkv && d->positions && (d->cos_sin || d->rot == 0) && d->cache && d->slots && (!d->q_w == !d->k_w), NVH_E_NULL, "attn_prep: null pointer");
    const int64_t cols = (int64_t)d->heads * d->dk + (int64_t)d->kv_heads * (d->dk + d->dv);
    REQUIRE(d->rows > 0 && d->heads > 0 && d->kv_heads > 0 && d->dk > 0 && d->dk % 8 == 0 && d->dv > 0 && d->dv % 8 == 0 && cols <= kMaxRowCols && d->rot >= 0 && d->rot % 2 == 0 &&
            d->rot <= d->dk && ((d->rot == 0 && !d->v_cos_sin) || d->max_position > 0) && (!d->v_cos_sin || (d->v_rot > 0 && d->v_rot % 2 == 0 && d->v_rot <= d->dv)) && d->block_size > 0 && (!d->q_w || (d->q_n > 0 && d->k_n > 0)) && (!d->head_norm || d->q_w), NVH_E_SHAPE,
            "attn_prep: heads %d/%d widths %d/%d rot %d (row of at most %d)", d->heads, d->kv_heads, d->dk, d->dv, d->rot, kMaxRowCols);
    REQUIRE(d->qkv_stride % 8 == 0 && d->qkv_stride >= cols, NVH_E_STRIDE, "attn_prep: row stride");
    REQUIRE(aligned16(d->qkv) && aligned16(d->cache) && aligned16(d->q_w) && aligned16(d->k_w), NVH_E_ALIGN, "attn_prep: pointers must be 16-byte aligned");
    return launch_attn_prep(*d, dtype == NVH_F32, (hipStream_t)stream);
}
