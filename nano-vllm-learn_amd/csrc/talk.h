// What the kernels of attention with mixed heads share: capped scores, and the mixing matrix T, score_h <- sum over g of T[h][g] score_g.
#pragma once
#include "mixers.h"

namespace nvh {

// cap * tanh(scale * s / cap); cap == 0: scale * s
struct ScoreCap {
    float scale, cap, rate;
    // gain: the result is this many times the score
    __device__ __forceinline__ ScoreCap(float scale_, float cap_, float gain = 1.f) : scale(scale_ * gain), cap(cap_ * gain), rate(cap_ > 0.f ? 2.f * kLog2e * scale_ / cap_ : 0.f) {}
    __device__ __forceinline__ f32x4 capped(f32x4 s) const {                   // (cap > 0)
        f32x4 r;
#pragma unroll
        for (int i = 0; i < 4; ++i) r[i] = cap - 2.f * cap * fast_rcp(1.f + fast_exp2(s[i] * rate));         // tanh(t) = 1 - 2 / (1 + exp(2 t))
        return r;
    }
    __device__ __forceinline__ f32x4 operator()(f32x4 s) const { return cap > 0.f ? capped(s) : s * scale; }
    __device__ __forceinline__ float exact(float s) const { return cap > 0.f ? cap * tanhf(s * scale / cap) : s * scale; }
};

}  // namespace nvh
