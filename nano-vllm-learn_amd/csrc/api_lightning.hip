// C ABI of lightning attention (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

namespace {

int check_lightning(const char* fn, const nvh_lightning_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->qkv && d->decay && d->positions && d->state_slots && d->state && d->out, NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->rows > 0 && d->heads > 0 && d->heads <= 65535 && d->dk > 0 && d->dk % 8 == 0 && d->dk <= 1024 && d->dv > 0 && d->dv % 8 == 0, NVH_E_SHAPE,
            "%s: heads %d widths %d (<= 1024) / %d", fn, d->heads, d->dk, d->dv);
    REQUIRE(d->qkv_stride % 8 == 0 && d->qkv_stride >= (int64_t)d->heads * (2 * d->dk + d->dv) && d->out_stride % 4 == 0 && d->out_stride >= (int64_t)d->heads * d->dv,
            NVH_E_STRIDE, "%s: row strides", fn);
    REQUIRE(aligned16(d->qkv) && aligned16(d->state) && aligned16(d->seg_state) && aligned16(d->out), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

}  // namespace

extern "C" {

int nvh_lightning_supported(int dk, int dv) { return lightning_supported(dk, dv); }

int nvh_lightning_chunks(const nvh_lightning_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "lightning_chunks: null descriptor");
    if (d->n_chunks == 0) return 0;
    const int rc = check_lightning("lightning_chunks", d, dtype);
    if (rc) return rc;
    REQUIRE(d->chunks && d->n_chunks > 0 && d->n_chunks <= 65535 && (!d->summaries || d->seg_state), NVH_E_NULL, "lightning_chunks: %d segments or null pointer", d->n_chunks);
    return launch_lightning_chunks(*d, dtype == NVH_F32, generic, (hipStream_t)stream);
}

int nvh_lightning_step(const nvh_lightning_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "lightning_step: null descriptor");
    if (d->rows == 0) return 0;
    const int rc = check_lightning("lightning_step", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16 && lightning_supported(d->dk, d->dv) && d->rows <= 65535, NVH_E_SHAPE, "lightning_step: bf16, widths %d/%d", d->dk, d->dv);
    return launch_lightning_step(*d, (hipStream_t)stream);
}

int nvh_norm_gate(void* out, void* packed, const void* x, const void* gate, const float* w, float eps, int rows, int cols, int n, int64_t x_stride,
                  int64_t gate_stride, int64_t out_stride, int dtype, void* stream) {
    if (rows == 0) return 0;
    DTYPE("norm_gate");
    REQUIRE((out || packed) && x && gate && w, NVH_E_NULL, "norm_gate: null pointer");
    REQUIRE(rows > 0 && cols > 0 && cols % 8 == 0 && cols <= kMaxRowCols && n > 0 && n <= cols && (!packed || (dtype == NVH_BF16 && cols % 32 == 0)), NVH_E_SHAPE,
            "norm_gate: cols %d (%%8, <= %d), mean over %d", cols, kMaxRowCols, n);
    REQUIRE(x_stride % 8 == 0 && x_stride >= cols && gate_stride % 8 == 0 && gate_stride >= cols && (!out || (out_stride % 8 == 0 && out_stride >= cols)), NVH_E_STRIDE,
            "norm_gate: row strides");
    REQUIRE(aligned16(out) && aligned16(packed) && aligned16(x) && aligned16(gate) && aligned16(w), NVH_E_ALIGN, "norm_gate: pointers must be 16-byte aligned");
    return launch_norm_gate(out, packed, x, gate, w, eps, rows, cols, n, x_stride, gate_stride, out_stride, dtype == NVH_F32, (hipStream_t)stream);
}

}  // extern "C"
