// What the kernels of attention with mixed heads share: capped scores, and the mixing matrix T, score_h <- sum over g of T[h][g] score_g.
#pragma once
#include "mixers.h"

namespace nvh {

// cap * tanh(scale * s / cap); cap == 0: scale * s
struct ScoreCap {
    float scale, cap, rate;
    __device__ __forceinline__ ScoreCap(float scale_, float cap_) : scale(scale_), cap(cap_), rate(cap_ > 0.f ? 2.f * kLog2e * scale_ / cap_ : 0.f) {}
    __device__ __forceinline__ f32x4 operator()(f32x4 s) const {
        f32x4 r;
        if (cap > 0.f) {
#pragma unroll
            for (int i = 0; i < 4; ++i) r[i] = cap - 2.f * cap * fast_rcp(1.f + fast_exp2(s[i] * rate));     // tanh(t) = 1 - 2 / (1 + exp(2 t))
        } else {
            r = s * scale;
        }
        return r;
    }
    __device__ __forceinline__ float exact(float s) const { return cap > 0.f ? cap * tanhf(s * scale / cap) : s * scale; }
};

}  // namespace nvh
