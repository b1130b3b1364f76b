// Causal attention of prompt portions in expanded latent form (gfx950 MFMA): the keys and values of every visible token have been expanded from the
// cached latents by two projections; a head's key is [its own unrotated part | the rotated part all heads share], key width DK != value width DV.
// Tile scheme of attend_tile.h, images double-buffered by LDS-DMA; what is special:
//   * a key row in LDS is gathered from two sources: each 16-byte piece comes from the expanded rows or from the shared rotated rows
//   * the query's rotated part is turned in registers while the fragments are loaded, so no launch of its own rotates queries
//   * unequal widths: DK in {64, 128, 192, 256}, DV in {64, 128}
// Algorithmic flops per launch: sum over sequences of 2 (DK + DV) heads (causal pairs).
#include "attend_tile.h"

namespace nvh {

namespace {

template <int DK, int DV, int QT>
__global__ __launch_bounds__(256, DK + DV <= 320 ? 2 : 1) void latent_prefill_kernel(const LatentPrefillArgs a) {
    using Images = TileImages<DK, DV>;
    constexpr int BM = 64 * QT, WR = 16 * QT, BN = Images::BN, KP = Images::KP, VP = Images::VP, NK = Images::NK, NV = Images::NV;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    int qt, head, b;
    attend_unit(a.heads, qt, head, b);
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, k_beg = a.cu_k[b], sk = a.cu_k[b + 1] - k_beg;
    const int q0 = qt * BM;
    if (q0 >= sq || sk <= 0) return;
    const int shift = sk - sq;                       // query r sees keys <= r + shift
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lq = lane & 15, lg = lane >> 4;
    int kv_end = q0 + BM + shift;
    if (kv_end > sk) kv_end = sk;
    const int n_tiles = (kv_end + BN - 1) / BN;
    const int wave_first_key = q0 + wave * WR + shift, wave_last_key = wave_first_key + WR - 1;

    // ---- staging: this lane's piece of each DMA instruction: LDS row, source pointer of the sequence's first key, row stride
    const uint16_t *kp[NK], *vp_[NV];
    int64_t ks[NK];
    int kr[NK], vr_[NV];
#pragma unroll
    for (int j = 0; j < NK; ++j) {
        const int s = (wave * NK + j) * 64 + lane, R = s / KP, piece = (s - R * KP) ^ swz_k<DK>(R);
        const bool own = piece * 8 < a.dim_cols;
        kr[j] = R;
        ks[j] = own ? a.k_stride : a.kr_stride;
        kp[j] = own ? a.k + (int64_t)k_beg * a.k_stride + head * a.dim_cols + piece * 8 : a.k_rot + (int64_t)k_beg * a.kr_stride + (piece * 8 - a.dim_cols);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int s = (wave * NV + j) * 64 + lane, R = s / VP, piece = (s - R * VP) ^ swz_v<DV>(R);
        vr_[j] = R;
        vp_[j] = a.v + (int64_t)k_beg * a.v_stride + head * DV + piece * 8;
    }
    auto stage = [&](int it, int buf) {
        unsigned char* kimg = Images::k(lds, buf);
        unsigned char* vimg = Images::v(lds, buf);
        const int kv0 = it * BN;
#pragma unroll
        for (int j = 0; j < NK; ++j) {
            const int row = kv0 + kr[j] < sk ? kv0 + kr[j] : sk - 1;           // rows past the end repeat the last key: masked
            dma16(kp[j] + row * ks[j], kimg + (wave * NK + j) * 1024);
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int row = kv0 + vr_[j] < sk ? kv0 + vr_[j] : sk - 1;
            dma16(vp_[j] + row * a.v_stride, vimg + (wave * NV + j) * 1024);
        }
    };
    // ---- queries, the rotated part turned while the fragments are loaded
    int my_q[QT];
    bool q_ok[QT];
    const uint16_t* qp[QT];
    const float* cs[QT];
#pragma unroll
    for (int qs = 0; qs < QT; ++qs) {
        my_q[qs] = q0 + wave * WR + 16 * qs + lq;
        q_ok[qs] = my_q[qs] < sq;
        const int64_t qrow = q_beg + (q_ok[qs] ? my_q[qs] : sq - 1);
        qp[qs] = a.q + qrow * a.q_stride + (int64_t)head * DK + lg * 8;
        int64_t pos = a.positions[qrow];
        if (pos >= a.max_position) pos = a.max_position - 1;
        cs[qs] = a.cos_sin + pos * a.rot;
    }
    auto query = [&](int qs, int st) {
        u32x4 raw = *reinterpret_cast<const u32x4*>(qp[qs] + st * 32);
        const int i0 = (32 * st + 8 * lg - a.dim_cols) / 2;                   // first pair of this piece (dim_cols is a multiple of 32)
        if (32 * st >= a.dim_cols) {
#pragma unroll
            for (int k = 0; k < 4; ++k)
                if (i0 + k < a.rot / 2) {
                    const float u = bf16_lo(raw[k]), v = bf16_hi(raw[k]), co = cs[qs][i0 + k], si = cs[qs][a.rot / 2 + i0 + k];
                    raw[k] = pack_bf16x2(u * co - v * si, v * co + u * si);
                }
        }
        return *reinterpret_cast<const bf16x8*>(&raw);
    };
    attend_walk<DK, DV, QT>(
        lds, n_tiles, a.scale_log2, -INFINITY, lane, stage, query, [&](int it) { return it * BN; }, [&](int kv0) { return kv0 <= wave_last_key; },
        [&](int kv0) { return kv0 + BN - 1 > wave_first_key || kv0 + BN > sk; },
        [&](int kv0, int qs, int off) { return off <= (my_q[qs] + shift < sk - 1 ? my_q[qs] + shift : sk - 1) - kv0 - 4 * lg; },
        [&](int qs) { return q_ok[qs] ? a.out + (int64_t)(q_beg + my_q[qs]) * a.out_stride + head * DV : nullptr; }, [](int, int, f32x4 v) { return v; });
}

template <int DK, int DV, int QT>
int launch_one(const LatentPrefillArgs& a, hipStream_t stream) {
    constexpr size_t lds = TileImages<DK, DV>::BYTES;
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(latent_prefill_kernel<DK, DV, QT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    latent_prefill_kernel<DK, DV, QT><<<dim3(a.heads, a.batch, (a.max_q + 64 * QT - 1) / (64 * QT)), 256, lds, stream>>>(a);
    return check_launch("latent_prefill");
}
template <int DK, int DV>
int launch_dims(const LatentPrefillArgs& a, hipStream_t stream) {
    return a.max_q > 256 ? launch_one<DK, DV, 2>(a, stream) : launch_one<DK, DV, 1>(a, stream);
}

}  // namespace

bool latent_prefill_supported(int dk, int dv) { return (dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128); }

int launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t stream) {
    if (a.batch == 0 || a.max_q <= 0) return 0;
    switch (a.dk * 1000 + a.dv) {
        case 64064: return launch_dims<64, 64>(a, stream);
        case 64128: return launch_dims<64, 128>(a, stream);
        case 128064: return launch_dims<128, 64>(a, stream);
        case 128128: return launch_dims<128, 128>(a, stream);
        case 192064: return launch_dims<192, 64>(a, stream);
        case 192128: return launch_dims<192, 128>(a, stream);
        case 256064: return launch_dims<256, 64>(a, stream);
        case 256128: return launch_dims<256, 128>(a, stream);
        default: set_error("latent_prefill: key width %d / value width %d", a.dk, a.dv); return -2;
    }
}

}  // namespace nvh
