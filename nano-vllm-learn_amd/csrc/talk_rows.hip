// Attention with mixed heads, single query rows: a softmax over scores that are capped (tanh) and then mixed across the heads, so that every weight needs
// all heads' scores.  Two launches:
//   scores  q . k of every visible key, capped, to memory: [row][key in the order of the row's visible tiles][head]
//   rows    the streaming kernel of paged_rows.h; a unit's scores come from memory, and the mixing matrix is a 32-bit MFMA operand (16 keys x 4 heads at a time)
#include "paged_rows.h"
#include "talk.h"

namespace nvh {

namespace {

// ------------------------------------------------------------------------------------------------ scores
// one workgroup per (row, head, visible tile of 64 keys), 4 lanes per key
template <typename T>
__global__ __launch_bounds__(256) void talk_scores_generic_kernel(const PagedAttendArgs a) {
    const int row = blockIdx.x, head = blockIdx.y, it = blockIdx.z, tid = threadIdx.x, g = head / (a.heads / a.kv_heads);
    const int pos = (int)a.positions[row];
    const VisibleTiles vis = visible_tiles(pos, pos, a.window, a.keep_first);
    if (it >= vis.count) return;
    const int key = vis.tile(it) * 64 + (tid >> 2);
    float s = 0.f;
    if (key <= pos) {
        const int seq = a.row_seq ? a.row_seq[row] : row;
        const int64_t page = a.block_tables[seq * a.bt_stride + key / a.block_size];
        const T* r = reinterpret_cast<const T*>(a.cache) + (page * a.kv_heads + g) * a.block_size * (a.dk + a.dv) + (int64_t)(key % a.block_size) * a.dk;
        const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)row * a.q_stride + head * a.dk;
        for (int i = (tid & 3) * 4; i < a.dk; i += 16) s += sum4(act_ld4(r + i) * act_ld4(q + i));
    }
    s += __shfl_xor(s, 1);
    s += __shfl_xor(s, 2);
    if ((tid & 3) == 0 && key <= pos)
        a.scores[((int64_t)row * a.span + it * 64 + (tid >> 2)) * score_cols(a.heads) + head] = ScoreCap(a.scale, a.softcap).exact(s);
}

constexpr int kScoreHeads = 16;                      // query heads of one key/value head per pass: the columns of a product

// grid (units of 128 keys, kv heads x passes, rows): a wave takes 32 keys
template <int DK>
__global__ __launch_bounds__(256) void talk_scores_kernel(const PagedAttendArgs a) {
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lq = lane & 15, lg = lane >> 4;
    const int row = blockIdx.z, ratio = a.heads / a.kv_heads, passes = (ratio + kScoreHeads - 1) / kScoreHeads;
    const int g = blockIdx.y / passes, h0 = g * ratio + (blockIdx.y - g * passes) * kScoreHeads, left = (g + 1) * ratio - h0, nh = left < kScoreHeads ? left : kScoreHeads;
    const int pos = (int)a.positions[row];
    const VisibleTiles vis = visible_tiles(pos, pos, a.window, a.keep_first);
    const int u = blockIdx.x * 4 + wave;
    if (u >= vis.count * 2 || u * 32 >= a.span) return;
    const int k0 = vis.tile(u >> 1) * 64 + (u & 1) * 32;
    if (k0 > pos) return;
    KeyScores<DK> ks(a, row, h0, nh, lq, lg);
    const int page = a.block_tables[(int64_t)row * a.bt_stride + k0 / a.block_size];
    ks.load(a, row, u, k0, pos, reinterpret_cast<const uint16_t*>(a.cache) + ((int64_t)page * a.kv_heads + g) * a.block_size * (DK + a.dv), lq, lg);
    f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    ks.product(s);
    const ScoreCap cap(a.scale, a.softcap);
    const int cols = score_cols(a.heads);
    float* out = a.scores + ((int64_t)row * a.span + u * 32 + 4 * lg) * cols + h0 + lq;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const f32x4 c = cap(s[t]);
        if (lq < nh) {
#pragma unroll
            for (int r = 0; r < 4; ++r) out[(16 * t + r) * cols] = c[r];
        }
    }
}

// ------------------------------------------------------------------------------------------------ rows
// MS: groups of 16 heads.  Step e of group m takes head 16 m + 4 lg + e of both operands: a lane's scores of a key are one 16-byte piece.
template <int MS>
struct MixedScores {
    f32x4 t[MS];                                     // B operand: T[head lq of the pass][16 m + 4 lg + e]
    f32x4 c[2][MS];                                  // A operand: scores of key 16 t + lq
    __device__ __forceinline__ MixedScores(const PagedAttendArgs& a, int, int h0, int nh, int lq, int lg) {
        const float* tr = a.talk + (int64_t)(h0 + (lq < nh ? lq : nh - 1)) * a.heads;
#pragma unroll
        for (int m = 0; m < MS; ++m)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int h = 16 * m + 4 * lg + e;
                t[m][e] = h < a.heads ? tr[h] : 0.f;
            }
    }
    static __device__ __forceinline__ int key_width(const PagedAttendArgs& a) { return a.dk; }
    static __device__ __forceinline__ float factor(const PagedAttendArgs&) { return kLog2e; }
    __device__ __forceinline__ void load(const PagedAttendArgs& a, int row, int u, int k0, int pos, const uint16_t*, int lq, int lg) {
        const int cols = score_cols(a.heads);
#pragma unroll
        for (int t2 = 0; t2 < 2; ++t2) {
            const int off = 16 * t2 + lq, last = pos - k0;                     // keys past the query's own position were not written
            const float* r = a.scores + ((int64_t)row * a.span + (u * 32 < a.span ? u * 32 : a.span - 32) + (off < last ? off : last)) * cols;
#pragma unroll
            for (int m = 0; m < MS; ++m) {
                const int h = 16 * m + 4 * lg;
                c[t2][m] = *reinterpret_cast<const f32x4*>(r + (h < cols ? h : 0));
#pragma unroll
                for (int e = 0; e < 4; ++e) c[t2][m][e] = h + e < a.heads ? c[t2][m][e] : 0.f;
            }
        }
    }
    __device__ __forceinline__ void product(f32x4 (&s)[2]) const {
#pragma unroll
        for (int m = 0; m < MS; ++m)
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int t2 = 0; t2 < 2; ++t2) s[t2] = __builtin_amdgcn_mfma_f32_16x16x4f32(c[t2][m][e], t[m][e], s[t2], 0, 0, 0);
    }
};

template <int DV, int MS>
void rows_heads(const PagedAttendArgs& a, hipStream_t stream) {
    const int ratio = a.heads / a.kv_heads;
    const dim3 grid(a.splits, a.kv_heads * paged_attend_groups(a.heads, a.kv_heads), a.rows);
    if (ratio == 1) paged_rows_kernel<MixedScores<MS>, DV, 1><<<grid, 256, 0, stream>>>(a);
    else if (ratio == 2) paged_rows_kernel<MixedScores<MS>, DV, 2><<<grid, 256, 0, stream>>>(a);
    else if (ratio <= 4) paged_rows_kernel<MixedScores<MS>, DV, 4><<<grid, 256, 0, stream>>>(a);
    else paged_rows_kernel<MixedScores<MS>, DV, 8><<<grid, 256, 0, stream>>>(a);
}
template <int DV>
void rows_width(const PagedAttendArgs& a, hipStream_t stream) {
    if (a.heads <= 16) rows_heads<DV, 1>(a, stream);
    else if (a.heads <= 32) rows_heads<DV, 2>(a, stream);
    else rows_heads<DV, 4>(a, stream);
}

template <typename T>
int rows_generic(const PagedAttendArgs& a, hipStream_t stream) {
    talk_scores_generic_kernel<T><<<dim3(a.rows, a.heads, a.span / 64), 256, 0, stream>>>(a);
    const int rc = check_launch("talk_scores");
    if (rc) return rc;
    paged_rows_generic_kernel<T, true><<<dim3(a.rows, a.heads), 256, a.heads * 4, stream>>>(a);
    return check_launch("talk_rows");
}

}  // namespace

bool talk_rows_supported(int heads, int dk, int dv, int block_size) {
    return block_size % 64 == 0 && heads <= 64 && (dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128 || dv == 256);
}

int launch_talk_rows(const PagedAttendArgs& a, int f32, int generic, hipStream_t stream) {
    if (f32) return rows_generic<float>(a, stream);
    if (generic || a.row_seq || !talk_rows_supported(a.heads, a.dk, a.dv, a.block_size)) return rows_generic<uint16_t>(a, stream);
    const int ratio = a.heads / a.kv_heads;
    const dim3 grid((a.span + 127) / 128, a.kv_heads * ((ratio + kScoreHeads - 1) / kScoreHeads), a.rows);
    switch (a.dk) {
        case 64: talk_scores_kernel<64><<<grid, 256, 0, stream>>>(a); break;
        case 128: talk_scores_kernel<128><<<grid, 256, 0, stream>>>(a); break;
        case 192: talk_scores_kernel<192><<<grid, 256, 0, stream>>>(a); break;
        default: talk_scores_kernel<256><<<grid, 256, 0, stream>>>(a); break;
    }
    const int rc = check_launch("talk_scores");
    if (rc) return rc;
    if (a.dv == 64) rows_width<64>(a, stream);
    else if (a.dv == 128) rows_width<128>(a, stream);
    else rows_width<256>(a, stream);
    return check_launch("talk_rows");
}

}  // namespace nvh
