// C ABI of the row ops of models with an fp32 residual stream (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

extern "C" {

int nvh_embed_rows(float* x, void* xb, void* packed, const int64_t* tokens, const void* embed, float scale, int rows, int cols, int vocab, float* copy,
                   const int64_t* positions, const float* table, int max_position, int dtype, void* stream) {
    if (rows == 0) return 0;
    DTYPE("embed_rows");
    REQUIRE(x && tokens && embed && (!table || (positions && max_position > 0)), NVH_E_NULL, "embed_rows: null pointer");
    REQUIRE(rows > 0 && cols > 0 && cols % 8 == 0 && vocab > 0, NVH_E_SHAPE, "embed_rows: rows %d cols %d (%%8) vocab %d", rows, cols, vocab);
    REQUIRE(!packed || (dtype == NVH_BF16 && cols % 32 == 0), NVH_E_SHAPE, "embed_rows: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(aligned16(x) && aligned16(embed) && aligned16(xb) && aligned16(packed) && aligned16(copy) && aligned16(table), NVH_E_ALIGN, "embed_rows: pointers must be 16-byte aligned");
    return launch_embed_rows(x, xb, packed, tokens, embed, scale, rows, cols, vocab, copy, positions, table, max_position, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_norm_residual(const nvh_norm_residual_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "norm_residual: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("norm_residual");
    REQUIRE(d->x && d->w && (d->y || d->xb || d->packed), NVH_E_NULL, "norm_residual: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->cols <= 16384 && d->n > 0 && d->n <= d->cols, NVH_E_SHAPE,
            "norm_residual: cols %d (%%8, <= 16384), mean over %d", d->cols, d->n);
    REQUIRE(!d->packed || (dtype == NVH_BF16 && d->cols % 32 == 0), NVH_E_SHAPE, "norm_residual: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(!d->y || (d->y_stride % 4 == 0 && d->y_stride >= d->cols), NVH_E_STRIDE, "norm_residual: y row stride");
    REQUIRE(aligned16(d->x) && aligned16(d->w) && (!d->y || aligned16(d->y)) && (!d->xb || aligned16(d->xb)) && (!d->packed || aligned16(d->packed)), NVH_E_ALIGN,
            "norm_residual: pointers must be 16-byte aligned");
    return launch_norm_residual(*d, dtype == NVH_F32, (hipStream_t)stream);
}

namespace {

int check_glu(const char* fn, void* out, const void* gate_up, int rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride, int dtype) {
    DTYPE(fn);
    REQUIRE(out && gate_up, NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(rows > 0 && inter > 0 && inter % 8 == 0 && gate_up_row_stride >= 2 * (int64_t)inter && gate_up_row_stride % 8 == 0 && out_row_stride >= inter && out_row_stride % 8 == 0,
            NVH_E_SHAPE, "%s: inter %d (%%8) / row strides", fn, inter);
    REQUIRE(aligned16(out) && aligned16(gate_up), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

}  // namespace

int nvh_clamped_glu(void* out, const void* gate_up, int rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride, float limit, float alpha,
                    int dtype, void* stream) {
    if (rows == 0) return 0;
    const int rc = check_glu("clamped_glu", out, gate_up, rows, inter, gate_up_row_stride, out_row_stride, dtype);
    return rc ? rc : launch_clamped_glu(out, gate_up, rows, inter, gate_up_row_stride, out_row_stride, limit, alpha, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_gelu_glu(void* out, const void* gate_up, int rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride, int dtype, void* stream) {
    if (rows == 0) return 0;
    const int rc = check_glu("gelu_glu", out, gate_up, rows, inter, gate_up_row_stride, out_row_stride, dtype);
    return rc ? rc : launch_gelu_glu(out, gate_up, rows, inter, gate_up_row_stride, out_row_stride, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_residual_norm(const nvh_residual_norm_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "residual_norm: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("residual_norm");
    REQUIRE(d->x && (d->y || d->e || d->w || d->base || d->shift) && (!d->post_w || (d->post_b && (d->y || d->e))) && (!d->e || d->ew) &&
            (!d->w || (d->b && (d->xb || d->packed))), NVH_E_NULL, "residual_norm: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->cols <= 16384 && d->n > 0 && d->n <= d->cols && (!d->e || d->top > 0), NVH_E_SHAPE,
            "residual_norm: cols %d (%%8, <= 16384), mean over %d, top %d", d->cols, d->n, d->top);
    REQUIRE(!d->packed || (dtype == NVH_BF16 && d->cols % 32 == 0), NVH_E_SHAPE, "residual_norm: packed rows are bf16, cols %% 32 == 0");
    REQUIRE(!d->y || (d->y_stride % 8 == 0 && d->y_stride >= d->cols), NVH_E_STRIDE, "residual_norm: y row stride");
    REQUIRE(aligned16(d->x) && aligned16(d->y) && aligned16(d->e) && aligned16(d->w) && aligned16(d->b) && aligned16(d->xb) && aligned16(d->packed), NVH_E_ALIGN,
            "residual_norm: pointers must be 16-byte aligned");
    REQUIRE(aligned16(d->post_w) && aligned16(d->post_b) && aligned16(d->base) && aligned16(d->shift), NVH_E_ALIGN, "residual_norm: pointers must be 16-byte aligned");
    return launch_residual_norm(*d, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_poly_norm(void* out, void* packed, const void* z, const float* coef, float eps, int rows, int cols, int n, int64_t z_stride, int64_t out_stride, int dtype,
                  void* stream) {
    if (rows == 0) return 0;
    DTYPE("poly_norm");
    REQUIRE((out || packed) && z && coef, NVH_E_NULL, "poly_norm: null pointer");
    REQUIRE(rows > 0 && cols > 0 && cols % 8 == 0 && cols <= kMaxRowCols && n > 0 && n <= cols && (!packed || (dtype == NVH_BF16 && cols % 32 == 0)), NVH_E_SHAPE,
            "poly_norm: cols %d (%%8, <= %d), means over %d", cols, kMaxRowCols, n);
    REQUIRE(z_stride % 8 == 0 && z_stride >= cols && (!out || (out_stride % 8 == 0 && out_stride >= cols)), NVH_E_STRIDE, "poly_norm: row strides");
    REQUIRE(aligned16(out) && aligned16(packed) && aligned16(z), NVH_E_ALIGN, "poly_norm: pointers must be 16-byte aligned");
    return launch_poly_norm(out, packed, z, coef, eps, rows, cols, n, z_stride, out_stride, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_softcap(void* x, float cap, int rows, int cols, int64_t stride, int dtype, void* stream) {
    if (rows == 0) return 0;
    DTYPE("softcap");
    REQUIRE(x, NVH_E_NULL, "softcap: null pointer");
    REQUIRE(rows > 0 && rows <= 65535 && cols > 0 && stride >= cols && cap > 0.f, NVH_E_SHAPE, "softcap: rows %d cols %d cap %g", rows, cols, (double)cap);
    return launch_softcap(x, cap, rows, cols, stride, dtype == NVH_F32, (hipStream_t)stream);
}

}  // extern "C"
