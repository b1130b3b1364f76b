// Row-wise ops of the models that keep their residual stream in fp32:
//   embed_rows     x = embed[token] * scale (+ a learned row per position), as the fp32 stream (twice, where the embedding is needed again) and in the activation type
//   norm_residual  x += rmsnorm(y) * w and the new stream in the activation type (what the next projection reads), or rmsnorm(x) * w
//   residual_norm  x += y + weighted expert outputs (or mult times the layer norm of that sum), x += rows of another stream, x += one row for all, and the layer
//                  norm of the new row (what the next sublayers read)
//   poly_norm      a N(z) + b N(z^2) + c N(z^3) + e, powers by element, N(v) = v / sqrt(mean(v^2) + eps) over the row
//   softcap        cap * tanh(x / cap)
//   clamped_glu    g * sigmoid(alpha g) * (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit);  gelu_glu  gelu_tanh(gate) * up
// HBM-bound row streams; one workgroup per row where a norm needs the whole row.  Every op exists for bf16 and for fp32 activations.
#include <type_traits>

#include "mixers.h"

namespace nvh {

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(float* __restrict__ x, T* __restrict__ xb, uint16_t* __restrict__ packed, const int64_t* __restrict__ tokens,
                                                          const T* __restrict__ embed, float scale, int cols, int vocab, float* __restrict__ copy,
                                                          const int64_t* __restrict__ positions, const float* __restrict__ table, int max_position) {
    const int64_t row = blockIdx.x;
    int64_t tok = tokens[row], pos = table ? positions[row] : 0;
    tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
    pos = pos < 0 ? 0 : (pos >= max_position ? max_position - 1 : pos);
    for (int c = threadIdx.x * 4; c < cols; c += 1024) {
        f32x4 v = act_ld4(embed + tok * cols + c) * scale;
        if (table) v += *reinterpret_cast<const f32x4*>(table + pos * cols + c);
        *reinterpret_cast<f32x4*>(x + row * cols + c) = v;
        if (copy) *reinterpret_cast<f32x4*>(copy + row * cols + c) = v;
        if (xb) act_st4(xb + row * cols + c, v);
        if (packed) act_st4(packed + pack_index((int)row, c, cols), v);
    }
}

// CH: 4-element pieces per thread held in registers between the two passes over the row
template <typename T, int CH>
__global__ __launch_bounds__(256) void norm_residual_kernel(const NormResidualArgs a) {
    __shared__ float lds[4];
    const int64_t row = blockIdx.x;
    float* xr = a.x + row * a.cols;
    const T* yr = a.y ? reinterpret_cast<const T*>(a.y) + row * a.y_stride : nullptr;
    f32x4 v[CH], xv[CH];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        v[i] = xv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (c < a.cols) {
            xv[i] = *reinterpret_cast<const f32x4*>(xr + c);
            v[i] = yr ? act_ld4(yr + c) : xv[i];
        }
        ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
    const float inv = 1.f / sqrtf(block_sum256(ss, lds) / a.n + a.eps);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        if (c >= a.cols) continue;
        f32x4 r = v[i] * inv * *reinterpret_cast<const f32x4*>(a.w + c);
        if (yr) {
            r += xv[i];
            *reinterpret_cast<f32x4*>(xr + c) = r;
        }
        if (a.xb) act_st4(reinterpret_cast<T*>(a.xb) + row * a.cols + c, r);
        if (a.packed) act_st4(reinterpret_cast<uint16_t*>(a.packed) + pack_index((int)row, c, a.cols), r);
    }
}

template <typename T, bool GELU>
__global__ __launch_bounds__(256) void clamped_glu_kernel(T* __restrict__ out, const T* __restrict__ gu, int rows, int inter, int64_t gu_stride,
                                                           int64_t out_stride, float limit, float alpha) {
    const int pieces = inter / 4;
    const int64_t total = (int64_t)rows * pieces;
    for (int64_t idx = blockIdx.x * (int64_t)256 + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * 256) {
        const int64_t row = idx / pieces;
        const int c = (int)(idx - row * pieces) * 4;
        const f32x4 g = act_ld4(gu + row * gu_stride + c), u = act_ld4(gu + row * gu_stride + inter + c);
        f32x4 r;
#pragma unroll
        for (int k = 0; k < 4; ++k) r[k] = GELU ? gelu_tanh_f(g[k]) * u[k] : clamped_glu(g[k], u[k], limit, alpha);
        act_st4(out + row * out_stride + c, r);
    }
}

// mean and 1 / sqrt(variance + eps) over n columns of a row held as 8-element pieces, padding columns zero; v becomes v - mean (0 in the padding)
template <int CH>
__device__ __forceinline__ float centre_row(f32x8 (&v)[CH], int cols, int n, float eps, float* lds) {
    float s[1] = {0.f}, ss[1] = {0.f};
#pragma unroll
    for (int i = 0; i < CH; ++i) s[0] += sum4(v[i].a) + sum4(v[i].b);
    block_sums256(s, lds);
    const float mean = s[0] / n;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= cols) continue;
        float d[8];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            d[k] = c + k < n ? v[i].a[k] - mean : 0.f;
            d[4 + k] = c + 4 + k < n ? v[i].b[k] - mean : 0.f;
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) ss[0] += d[k] * d[k];
        v[i] = {f32x4{d[0], d[1], d[2], d[3]}, f32x4{d[4], d[5], d[6], d[7]}};
    }
    block_sums256(ss, lds + 4);
    return 1.f / sqrtf(ss[0] / n + eps);
}
__device__ __forceinline__ f32x8 scale_shift(const f32x8& v, float inv, const float* w, const float* b) {
    return {v.a * inv * *reinterpret_cast<const f32x4*>(w) + *reinterpret_cast<const f32x4*>(b),
            v.b * inv * *reinterpret_cast<const f32x4*>(w + 4) + *reinterpret_cast<const f32x4*>(b + 4)};
}

// a thread's 8-element pieces stay in registers from the additions to the normed store.  POST: what is added goes through a norm of its own first
template <typename T, int CH, bool POST>
__global__ __launch_bounds__(256) void residual_norm_kernel(const ResidualNormArgs a) {
    __shared__ float lds[8], lds_post[8];
    const int64_t row = blockIdx.x;
    float* xr = a.x + row * a.cols;
    const T* yr = a.y ? reinterpret_cast<const T*>(a.y) + row * a.y_stride : nullptr;
    const T* er = a.e ? reinterpret_cast<const T*>(a.e) + row * a.top * a.cols : nullptr;
    f32x8 v[CH], add[CH];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        v[i] = add[i] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (c >= a.cols) continue;
        v[i] = act_ld8(xr + c);
        if (er) {
#pragma unroll 4
            for (int k = 0; k < a.top; ++k) {
                const f32x8 e = act_ld8(er + (int64_t)k * a.cols + c);
                const float w = a.ew[row * a.top + k];
                add[i].a += e.a * w;
                add[i].b += e.b * w;
            }
        }
        if (yr) {
            const f32x8 y = act_ld8(yr + c);
            add[i].a += y.a;
            add[i].b += y.b;
        }
    }
    float post = 0.f;
    if constexpr (POST) {
        if (a.post_w) post = centre_row(add, a.cols, a.n, a.eps, lds_post);
    }
    const bool changed = yr || er || (POST && (a.base || a.shift));
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= a.cols) continue;
        if constexpr (POST) {
            if (a.post_w) add[i] = scale_shift(add[i], post, a.post_w + c, a.post_b + c);
            v[i].a += add[i].a * a.mult;
            v[i].b += add[i].b * a.mult;
            if (a.base) {
                const f32x8 t = act_ld8(a.base + row * a.cols + c);
                v[i].a += t.a;
                v[i].b += t.b;
            }
            if (a.shift) {
                const f32x8 t = act_ld8(a.shift + c);
                v[i].a += t.a;
                v[i].b += t.b;
            }
        } else {
            v[i].a += add[i].a;
            v[i].b += add[i].b;
        }
        if (changed) act_st8(xr + c, v[i]);
    }
    if (!a.w) return;
    const float inv = centre_row(v, a.cols, a.n, a.eps, lds);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= a.cols) continue;
        const f32x8 r = scale_shift(v[i], inv, a.w + c, a.b + c);
        if (a.xb) act_st8(reinterpret_cast<T*>(a.xb) + row * a.cols + c, r);
        if (a.packed) act_st8(reinterpret_cast<uint16_t*>(a.packed) + pack_index((int)row, c, a.cols), r);
    }
}

template <typename T, int CH>
__global__ __launch_bounds__(256) void poly_norm_kernel(T* __restrict__ out, uint16_t* __restrict__ packed, const T* __restrict__ z, const float* __restrict__ coef, float eps,
                                                         int cols, int n, int64_t z_stride, int64_t out_stride) {
    __shared__ float lds[12];
    const int64_t row = blockIdx.x;
    const T* zr = z + row * z_stride;
    f32x8 v[CH];
    float s[3] = {0.f, 0.f, 0.f};                    // sums of z^2, z^4, z^6 (padding columns are zero)
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        v[i] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (c < cols) v[i] = act_ld8(zr + c);
        const f32x4 qa = v[i].a * v[i].a, qb = v[i].b * v[i].b, fa = qa * qa, fb = qb * qb;
        s[0] += sum4(qa) + sum4(qb);
        s[1] += sum4(fa) + sum4(fb);
        s[2] += sum4(fa * qa) + sum4(fb * qb);
    }
    block_sums256(s, lds);
    const float k1 = coef[0] / sqrtf(s[0] / n + eps), k2 = coef[1] / sqrtf(s[1] / n + eps), k3 = coef[2] / sqrtf(s[2] / n + eps), k0 = coef[3];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= cols) continue;
        f32x8 r = {((v[i].a * k3 + k2) * v[i].a + k1) * v[i].a + k0, ((v[i].b * k3 + k2) * v[i].b + k1) * v[i].b + k0};
        if (c + 8 > n) {
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                if (c + k >= n) r.a[k] = 0.f;
                if (c + 4 + k >= n) r.b[k] = 0.f;
            }
        }
        if (out) act_st8(out + row * out_stride + c, r);
        if (packed) act_st8(packed + pack_index((int)row, c, cols), r);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, float cap, int cols, int64_t stride) {
    T* r = x + (int64_t)blockIdx.y * stride;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < cols; c += gridDim.x * 256) act_st(r + c, cap * tanhf(act_ld(r + c) / cap));
}

}  // namespace

int launch_embed_rows(float* x, void* xb, void* packed, const int64_t* tokens, const void* embed, float scale, int rows, int cols, int vocab, float* copy,
                      const int64_t* positions, const float* table, int max_position, int f32, hipStream_t stream) {
    if (f32) embed_rows_kernel<float><<<rows, 256, 0, stream>>>(x, (float*)xb, nullptr, tokens, (const float*)embed, scale, cols, vocab, copy, positions, table, max_position);
    else embed_rows_kernel<uint16_t><<<rows, 256, 0, stream>>>(x, (uint16_t*)xb, (uint16_t*)packed, tokens, (const uint16_t*)embed, scale, cols, vocab, copy, positions, table,
                                                               max_position);
    return check_launch("embed_rows");
}

template <typename T>
static void norm_residual_t(const NormResidualArgs& a, hipStream_t stream) {
    const int ch = (a.cols + 1023) / 1024;
    if (ch <= 1) norm_residual_kernel<T, 1><<<a.rows, 256, 0, stream>>>(a);
    else if (ch <= 2) norm_residual_kernel<T, 2><<<a.rows, 256, 0, stream>>>(a);
    else if (ch <= 4) norm_residual_kernel<T, 4><<<a.rows, 256, 0, stream>>>(a);
    else if (ch <= 8) norm_residual_kernel<T, 8><<<a.rows, 256, 0, stream>>>(a);
    else norm_residual_kernel<T, 16><<<a.rows, 256, 0, stream>>>(a);
}

int launch_norm_residual(const NormResidualArgs& a, int f32, hipStream_t stream) {
    if (f32) norm_residual_t<float>(a, stream);
    else norm_residual_t<uint16_t>(a, stream);
    return check_launch("norm_residual");
}

template <bool GELU>
static void glu_go(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, float limit, float alpha, int f32, hipStream_t stream) {
    const int64_t work = ((int64_t)rows * (inter / 4) + 255) / 256;
    const int grid = (int)(work < 8192 ? (work < 1 ? 1 : work) : 8192);
    if (f32) clamped_glu_kernel<float, GELU><<<grid, 256, 0, stream>>>((float*)out, (const float*)gate_up, rows, inter, gu_stride, out_stride, limit, alpha);
    else clamped_glu_kernel<uint16_t, GELU><<<grid, 256, 0, stream>>>((uint16_t*)out, (const uint16_t*)gate_up, rows, inter, gu_stride, out_stride, limit, alpha);
}

int launch_clamped_glu(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, float limit, float alpha, int f32,
                       hipStream_t stream) {
    glu_go<false>(out, gate_up, rows, inter, gu_stride, out_stride, limit, alpha, f32, stream);
    return check_launch("clamped_glu");
}

int launch_gelu_glu(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, int f32, hipStream_t stream) {
    glu_go<true>(out, gate_up, rows, inter, gu_stride, out_stride, 0.f, 0.f, f32, stream);
    return check_launch("gelu_glu");
}

template <typename T>
static void residual_norm_t(const ResidualNormArgs& a, hipStream_t stream) {
    const int ch = (a.cols + 2047) / 2048;
    auto go = [&](auto k) {
        if (a.post_w || a.base || a.shift || a.mult != 1.f) residual_norm_kernel<T, decltype(k)::value, true><<<a.rows, 256, 0, stream>>>(a);
        else residual_norm_kernel<T, decltype(k)::value, false><<<a.rows, 256, 0, stream>>>(a);
    };
    if (ch <= 1) go(std::integral_constant<int, 1>{});
    else if (ch <= 2) go(std::integral_constant<int, 2>{});
    else if (ch <= 4) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, 8>{});
}

int launch_residual_norm(const ResidualNormArgs& a, int f32, hipStream_t stream) {
    if (f32) residual_norm_t<float>(a, stream);
    else residual_norm_t<uint16_t>(a, stream);
    return check_launch("residual_norm");
}

template <typename T>
static void poly_norm_t(void* out, void* packed, const void* z, const float* coef, float eps, int rows, int cols, int n, int64_t z_stride, int64_t out_stride, hipStream_t stream) {
    const int ch = (cols + 2047) / 2048;
    auto go = [&](auto k) {
        poly_norm_kernel<T, decltype(k)::value><<<rows, 256, 0, stream>>>((T*)out, (uint16_t*)packed, (const T*)z, coef, eps, cols, n, z_stride, out_stride);
    };
    if (ch <= 1) go(std::integral_constant<int, 1>{});
    else if (ch <= 2) go(std::integral_constant<int, 2>{});
    else if (ch <= 4) go(std::integral_constant<int, 4>{});
    else if (ch <= 8) go(std::integral_constant<int, 8>{});
    else go(std::integral_constant<int, kRowPieces>{});
}

int launch_poly_norm(void* out, void* packed, const void* z, const float* coef, float eps, int rows, int cols, int n, int64_t z_stride, int64_t out_stride, int f32,
                     hipStream_t stream) {
    if (f32) poly_norm_t<float>(out, packed, z, coef, eps, rows, cols, n, z_stride, out_stride, stream);
    else poly_norm_t<uint16_t>(out, packed, z, coef, eps, rows, cols, n, z_stride, out_stride, stream);
    return check_launch("poly_norm");
}

int launch_softcap(void* x, float cap, int rows, int cols, int64_t stride, int f32, hipStream_t stream) {
    const dim3 grid((unsigned)((cols + 1023) / 1024), rows);
    if (f32) softcap_kernel<float><<<grid, 256, 0, stream>>>((float*)x, cap, cols, stride);
    else softcap_kernel<uint16_t><<<grid, 256, 0, stream>>>((uint16_t*)x, cap, cols, stride);
    return check_launch("softcap");
}

}  // namespace nvh
