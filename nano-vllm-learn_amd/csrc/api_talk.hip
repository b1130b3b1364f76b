// C ABI of attention over pages with scores mixed across the heads (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

namespace {

int check_talk(const char* fn, const nvh_paged_attend_desc* d, int dtype) {
    REQUIRE(d && d->talk, NVH_E_NULL, "%s: null descriptor or no mixing matrix", fn);
    REQUIRE(d->softcap >= 0.f, NVH_E_SHAPE, "%s: softcap %g", fn, (double)d->softcap);
    return check_attend(fn, d, dtype);
}

}  // namespace

extern "C" {

int nvh_talk_rows_supported(int heads, int dk, int dv, int block_size) { return talk_rows_supported(heads, dk, dv, block_size); }

int nvh_talk_score_cols(int heads) { return heads > 0 ? score_cols(heads) : 0; }

size_t nvh_talk_ticket_bytes(int rows, int kv_heads, int heads) {
    if (rows <= 0 || kv_heads <= 0 || heads % kv_heads) return 0;
    return (size_t)rows * kv_heads * paged_attend_groups(heads, kv_heads) * kAttendTicketWords * 4;
}

int nvh_talk_rows(const nvh_paged_attend_desc* d, int generic, int dtype, void* stream) {
    if (d && d->rows == 0) return 0;
    const int rc = check_talk("talk_rows", d, dtype);
    if (rc) return rc;
    REQUIRE(d->positions && d->rows > 0 && d->splits >= 1 && d->splits <= 64 && (d->splits == 1 || (d->part && aligned16(d->part) && d->tickets)), NVH_E_NULL,
            "talk_rows: rows %d splits %d or null pointer", d->rows, d->splits);
    REQUIRE(d->scores && aligned16(d->scores) && d->span > 0 && d->span % 64 == 0 && d->span / 64 <= 65535, NVH_E_NULL, "talk_rows: scores of %d keys (a multiple of 64)", d->span);
    REQUIRE(d->heads <= 4096 && (dtype == NVH_F32 || generic || d->row_seq || d->rows <= 65535), NVH_E_SHAPE, "talk_rows: %d heads, %d rows", d->heads, d->rows);
    REQUIRE(!d->out_packed || (dtype == NVH_BF16 && (d->heads * d->dv) % 32 == 0), NVH_E_SHAPE, "talk_rows: packed output is bf16, width %% 32 == 0");
    return launch_talk_rows(*d, dtype == NVH_F32, generic, (hipStream_t)stream);
}

int nvh_talk_prompt_supported(int heads, int kv_heads, int dk, int dv, int block_size, float softcap) {
    return heads > 0 && kv_heads > 0 && softcap > 0.f && softcap <= kTalkPromptCap && talk_prompt_supported(heads, kv_heads, dk, dv, block_size);
}

int nvh_talk_prompt(const nvh_paged_attend_desc* d, int dtype, void* stream) {
    if (d && (d->batch == 0 || d->max_q == 0)) return 0;
    const int rc = check_talk("talk_prompt", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16, NVH_E_DTYPE, "talk_prompt: bf16 only");
    REQUIRE(d->cu_q && d->cu_k && d->out && !d->out_packed, NVH_E_NULL, "talk_prompt: null pointer or packed output");
    REQUIRE(nvh_talk_prompt_supported(d->heads, d->kv_heads, d->dk, d->dv, d->block_size, d->softcap) && d->batch > 0 &&
            d->max_q > 0 && (int64_t)d->batch * ((d->max_q + 15) / 16) <= 0x7fffffff, NVH_E_SHAPE,
            "talk_prompt: heads %d/%d, widths %d/%d page %d cap %g", d->heads, d->kv_heads, d->dk, d->dv, d->block_size, (double)d->softcap);
    return launch_talk_prompt(*d, (hipStream_t)stream);
}

}  // extern "C"
