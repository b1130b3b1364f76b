// Attention of prompt portions over the pages of one layer (gfx950 MFMA, tile scheme of attend_tile.h): keys and values come straight from the pages,
// 64 rows of one (page, key/value head) per tile by LDS-DMA, double-buffered.  A query tile walks the tiles of the kept first tokens, then the window's:
// what no query of the tile sees is not read.  A sink starts the running maximum and sum.
// Algorithmic flops per launch: sum over sequences of 2 (DK + DV) heads (visible pairs).
#include "attend_tile.h"
#include "mixers.h"

namespace nvh {

namespace {

template <int DK, int DV, int QT>
__global__ __launch_bounds__(256, DK + DV <= 320 ? 2 : 1) void paged_prompt_kernel(const PagedAttendArgs a) {
    using Images = TileImages<DK, DV>;
    constexpr int BM = 64 * QT, WR = 16 * QT, BN = Images::BN, KP = Images::KP, VP = Images::VP, NK = Images::NK, NV = Images::NV;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    int qt, head, b;
    attend_unit(a.heads, qt, head, b);
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b];
    const int q0 = qt * BM;
    if (q0 >= sq || sk < sq) return;
    const int shift = sk - sq;                       // query row r has position r + shift
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    const int g = head / (a.heads / a.kv_heads);
    const int rows = sq - q0 < BM ? sq - q0 : BM;
    const VisibleTiles vis = visible_from(first_seen(q0 + shift, a.window, a.chunk), q0 + rows - 1 + shift, a.keep_first);
    const int n_tiles = vis.count;
    const int wave_first = q0 + wave * WR + shift, wave_last = wave_first + WR - 1;       // positions of this wave's rows
    const int lo_first = first_seen(wave_first, a.window, a.chunk), lo_last = first_seen(wave_last, a.window, a.chunk);

    // ---- staging: this lane's piece of each DMA instruction: row of the tile and offset inside it
    const uint16_t* cache = reinterpret_cast<const uint16_t*>(a.cache) + (int64_t)g * a.block_size * (DK + DV);
    const int64_t page_elems = (int64_t)a.kv_heads * a.block_size * (DK + DV);
    const int32_t* table = a.block_tables + (int64_t)b * a.bt_stride;
    int kr[NK], kc[NK], vr[NV], vc[NV];
#pragma unroll
    for (int j = 0; j < NK; ++j) {
        const int s = (wave * NK + j) * 64 + lane, R = s / KP;
        kr[j] = R;
        kc[j] = ((s - R * KP) ^ swz_k<DK>(R)) * 8;
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int s = (wave * NV + j) * 64 + lane, R = s / VP;
        vr[j] = R;
        vc[j] = ((s - R * VP) ^ swz_v<DV>(R)) * 8;
    }
    auto page_of = [&](int it) { return it < n_tiles ? table[vis.tile(it) * BN / a.block_size] : 0; };
    int page = page_of(0);                           // of the tile that is staged next
    auto stage = [&](int it, int buf) {
        unsigned char* kimg = Images::k(lds, buf);
        unsigned char* vimg = Images::v(lds, buf);
        const int kv0 = vis.tile(it) * BN, off = kv0 % a.block_size, live = sk - kv0 < BN ? sk - kv0 : BN;
        const uint16_t* kb = cache + page * page_elems + (int64_t)off * DK;
        const uint16_t* vb = cache + page * page_elems + (int64_t)a.block_size * DK + (int64_t)off * DV;
#pragma unroll
        for (int j = 0; j < NK; ++j) dma16(kb + (kr[j] < live ? kr[j] : live - 1) * DK + kc[j], kimg + (wave * NK + j) * 1024);   // rows past the end repeat the last key: masked
#pragma unroll
        for (int j = 0; j < NV; ++j) dma16(vb + (vr[j] < live ? vr[j] : live - 1) * DV + vc[j], vimg + (wave * NV + j) * 1024);
        page = page_of(it + 1);
    };
    int my_q[QT], lo[QT];
    bool q_ok[QT];
    const uint16_t* qp[QT];
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        my_q[qs] = q0 + wave * WR + 16 * qs + lq;
        q_ok[qs] = my_q[qs] < sq;
        lo[qs] = first_seen(my_q[qs] + shift, a.window, a.chunk);
        qp[qs] = reinterpret_cast<const uint16_t*>(a.q) + (int64_t)(q_beg + (q_ok[qs] ? my_q[qs] : sq - 1)) * a.q_stride + (int64_t)head * DK + lg * 8;
    }
    attend_walk<DK, DV, QT>(
        lds, n_tiles, a.scale * kLog2e, a.sink ? a.sink[head] * kLog2e : -INFINITY, lane, stage,
        [&](int qs, int st) { return *reinterpret_cast<const bf16x8*>(qp[qs] + st * 32); }, [&](int it) { return vis.tile(it) * BN; },
        [&](int kv0) { return kv0 <= wave_last && (kv0 + BN > lo_first || kv0 < a.keep_first); },
        [&](int kv0) { return kv0 + BN - 1 > wave_first || kv0 + BN > sk || (kv0 < lo_last && kv0 + BN > a.keep_first); },
        [&](int kv0, int qs, int off) {
            const int pos = my_q[qs] + shift, at = kv0 + 4 * lg + off;
            return at <= (pos < sk - 1 ? pos : sk - 1) && (at >= lo[qs] || at < a.keep_first);
        },
        [&](int qs) { return q_ok[qs] ? reinterpret_cast<uint16_t*>(a.out) + (int64_t)(q_beg + my_q[qs]) * a.out_stride + head * DV : nullptr; },
        [&](int qs, int d, f32x4 v) { return a.o_cos_sin ? turn_back(v, a.o_cos_sin, my_q[qs] + shift, a.max_position, a.o_rot, d) : v; });
}

template <int DK, int DV, int QT>
int launch_one(const PagedAttendArgs& a, hipStream_t stream) {
    constexpr size_t lds = TileImages<DK, DV>::BYTES;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(paged_prompt_kernel<DK, DV, QT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    paged_prompt_kernel<DK, DV, QT><<<dim3(a.heads, a.batch, (a.max_q + 64 * QT - 1) / (64 * QT)), 256, lds, stream>>>(a);
    return check_launch("paged_attend_prompt");
}
template <int DK, int DV>
int launch_dims(const PagedAttendArgs& a, hipStream_t stream) {
    if constexpr (DV <= 128) {
        if (a.max_q > 256) return launch_one<DK, DV, 2>(a, stream);
    }
    return launch_one<DK, DV, 1>(a, stream);
}

}  // namespace

int launch_paged_attend_prompt(const PagedAttendArgs& a, hipStream_t stream) {
    switch (a.dk * 1000 + a.dv) {
        case 64064: return launch_dims<64, 64>(a, stream);
        case 64128: return launch_dims<64, 128>(a, stream);
        case 128064: return launch_dims<128, 64>(a, stream);
        case 128128: return launch_dims<128, 128>(a, stream);
        case 192064: return launch_dims<192, 64>(a, stream);
        case 192128: return launch_dims<192, 128>(a, stream);
        case 256064: return launch_dims<256, 64>(a, stream);
        case 256128: return launch_dims<256, 128>(a, stream);
        case 256256: return launch_dims<256, 256>(a, stream);
        default: set_error("paged_attend_prompt: key width %d / value width %d", a.dk, a.dv); return -2;
    }
}

}  // namespace nvh
