// C ABI of attention over pages (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

extern "C" {

int nvh_paged_attend_supported(int dk, int dv, int block_size) { return paged_attend_supported(dk, dv, block_size); }

size_t nvh_paged_attend_ticket_bytes(int rows, int kv_heads, int heads) {
    if (rows <= 0 || kv_heads <= 0 || heads % kv_heads) return 0;
    return (size_t)rows * kv_heads * paged_attend_groups(heads, kv_heads) * kAttendTicketWords * 4;
}

int nvh_paged_attend_rows(const nvh_paged_attend_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d && !d->talk, NVH_E_NULL, "paged_attend_rows: null descriptor, or one with mixed heads");
    if (d->rows == 0) return 0;
    const int rc = check_attend("paged_attend_rows", d, dtype);
    if (rc) return rc;
    REQUIRE(d->positions && d->rows > 0 && d->splits >= 1 && d->splits <= 64 && (d->splits == 1 || (d->part && aligned16(d->part) && d->tickets)), NVH_E_NULL,
            "paged_attend_rows: rows %d splits %d or null pointer", d->rows, d->splits);
    REQUIRE(!d->out_packed || (dtype == NVH_BF16 && (d->heads * d->dv) % 32 == 0), NVH_E_SHAPE, "paged_attend_rows: packed output is bf16, width %% 32 == 0");
    return launch_paged_attend_rows(*d, dtype == NVH_F32, generic, (hipStream_t)stream);
}

int nvh_paged_attend_prompt(const nvh_paged_attend_desc* d, int dtype, void* stream) {
    REQUIRE(d && !d->talk, NVH_E_NULL, "paged_attend_prompt: null descriptor, or one with mixed heads");
    if (d->batch == 0 || d->max_q == 0) return 0;
    const int rc = check_attend("paged_attend_prompt", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16, NVH_E_DTYPE, "paged_attend_prompt: bf16 only");
    REQUIRE(d->cu_q && d->cu_k && d->out && !d->out_packed, NVH_E_NULL, "paged_attend_prompt: null pointer or packed output");
    REQUIRE(paged_attend_supported(d->dk, d->dv, d->block_size) && d->batch > 0 && d->batch <= 65535 && d->max_q > 0 && d->scale > 0.f, NVH_E_SHAPE,
            "paged_attend_prompt: widths %d/%d page %d scale %g", d->dk, d->dv, d->block_size, (double)d->scale);
    return launch_paged_attend_prompt(*d, (hipStream_t)stream);
}

}  // extern "C"
