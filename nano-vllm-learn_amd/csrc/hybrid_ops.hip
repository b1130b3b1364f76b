// Row-wise ops of the models that keep their residual stream in fp32:
//   embed_rows     x = embed[token] * scale, as the fp32 stream and in the activation type
//   norm_residual  x += rmsnorm(y) * w and the new stream in the activation type (what the next projection reads), or rmsnorm(x) * w
//   residual_norm  x += y + weighted expert outputs, and the layer norm of the new row (what the next layer's sublayers read)
//   softcap        cap * tanh(x / cap)
//   clamped_glu    g * sigmoid(alpha g) * (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit)
// HBM-bound row streams; one workgroup per row where a norm needs the whole row.  Every op exists for bf16 and for fp32 activations.
#include <type_traits>

#include "mixers.h"

namespace nvh {

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(float* __restrict__ x, T* __restrict__ xb, uint16_t* __restrict__ packed, const int64_t* __restrict__ tokens,
                                                          const T* __restrict__ embed, float scale, int cols, int vocab) {
    const int64_t row = blockIdx.x;
    int64_t tok = tokens[row];
    tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
    for (int c = threadIdx.x * 4; c < cols; c += 1024) {
        const f32x4 v = act_ld4(embed + tok * cols + c) * scale;
        *reinterpret_cast<f32x4*>(x + row * cols + c) = v;
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

template <typename T>
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
        for (int k = 0; k < 4; ++k) r[k] = clamped_glu(g[k], u[k], limit, alpha);
        act_st4(out + row * out_stride + c, r);
    }
}

// a thread's 8-element pieces stay in registers from the additions to the normed store
template <typename T, int CH>
__global__ __launch_bounds__(256) void residual_norm_kernel(const ResidualNormArgs a) {
    __shared__ float lds[8];
    const int64_t row = blockIdx.x;
    float* xr = a.x + row * a.cols;
    const T* yr = a.y ? reinterpret_cast<const T*>(a.y) + row * a.y_stride : nullptr;
    const T* er = a.e ? reinterpret_cast<const T*>(a.e) + row * a.top * a.cols : nullptr;
    f32x8 v[CH];
    float s = 0.f, unused = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        v[i] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (c >= a.cols) continue;
        v[i] = act_ld8(xr + c);
        f32x8 add = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        if (er) {
#pragma unroll 4
            for (int k = 0; k < a.top; ++k) {
                const f32x8 e = act_ld8(er + (int64_t)k * a.cols + c);
                const float w = a.ew[row * a.top + k];
                add.a += e.a * w;
                add.b += e.b * w;
            }
        }
        if (yr) {
            const f32x8 y = act_ld8(yr + c);
            add.a += y.a;
            add.b += y.b;
        }
        v[i].a += add.a;
        v[i].b += add.b;
        if (yr || er) act_st8(xr + c, v[i]);
        s += sum4(v[i].a) + sum4(v[i].b);            // (padding columns are zero)
    }
    if (!a.w) return;
    block_sum256x2(s, unused, lds);
    const float mean = s / a.n;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= a.cols) continue;
        float d[8];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            d[k] = c + k < a.n ? v[i].a[k] - mean : 0.f;
            d[4 + k] = c + 4 + k < a.n ? v[i].b[k] - mean : 0.f;
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) ss += d[k] * d[k];
        v[i] = {f32x4{d[0], d[1], d[2], d[3]}, f32x4{d[4], d[5], d[6], d[7]}};
    }
    __syncthreads();
    block_sum256x2(ss, unused, lds);
    const float inv = 1.f / sqrtf(ss / a.n + a.eps);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (threadIdx.x + i * 256) * 8;
        if (c >= a.cols) continue;
        const f32x8 r = {v[i].a * inv * *reinterpret_cast<const f32x4*>(a.w + c) + *reinterpret_cast<const f32x4*>(a.b + c),
                         v[i].b * inv * *reinterpret_cast<const f32x4*>(a.w + c + 4) + *reinterpret_cast<const f32x4*>(a.b + c + 4)};
        if (a.xb) act_st8(reinterpret_cast<T*>(a.xb) + row * a.cols + c, r);
        if (a.packed) act_st8(reinterpret_cast<uint16_t*>(a.packed) + pack_index((int)row, c, a.cols), r);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, float cap, int cols, int64_t stride) {
    T* r = x + (int64_t)blockIdx.y * stride;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < cols; c += gridDim.x * 256) act_st(r + c, cap * tanhf(act_ld(r + c) / cap));
}

}  // namespace

int launch_embed_rows(float* x, void* xb, void* packed, const int64_t* tokens, const void* embed, float scale, int rows, int cols, int vocab, int f32, hipStream_t stream) {
    if (f32) embed_rows_kernel<float><<<rows, 256, 0, stream>>>(x, (float*)xb, nullptr, tokens, (const float*)embed, scale, cols, vocab);
    else embed_rows_kernel<uint16_t><<<rows, 256, 0, stream>>>(x, (uint16_t*)xb, (uint16_t*)packed, tokens, (const uint16_t*)embed, scale, cols, vocab);
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

int launch_clamped_glu(void* out, const void* gate_up, int rows, int inter, int64_t gu_stride, int64_t out_stride, float limit, float alpha, int f32,
                       hipStream_t stream) {
    const int64_t work = ((int64_t)rows * (inter / 4) + 255) / 256;
    const int grid = (int)(work < 8192 ? (work < 1 ? 1 : work) : 8192);
    if (f32) clamped_glu_kernel<float><<<grid, 256, 0, stream>>>((float*)out, (const float*)gate_up, rows, inter, gu_stride, out_stride, limit, alpha);
    else clamped_glu_kernel<uint16_t><<<grid, 256, 0, stream>>>((uint16_t*)out, (const uint16_t*)gate_up, rows, inter, gu_stride, out_stride, limit, alpha);
    return check_launch("clamped_glu");
}

template <typename T>
static void residual_norm_t(const ResidualNormArgs& a, hipStream_t stream) {
    const int ch = (a.cols + 2047) / 2048;
    auto go = [&](auto k) { residual_norm_kernel<T, decltype(k)::value><<<a.rows, 256, 0, stream>>>(a); };
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

int launch_softcap(void* x, float cap, int rows, int cols, int64_t stride, int f32, hipStream_t stream) {
    const dim3 grid((unsigned)((cols + 1023) / 1024), rows);
    if (f32) softcap_kernel<float><<<grid, 256, 0, stream>>>((float*)x, cap, cols, stride);
    else softcap_kernel<uint16_t><<<grid, 256, 0, stream>>>((uint16_t*)x, cap, cols, stride);
    return check_launch("softcap");
}

}  // namespace nvh
