// C ABI of paged sink/window attention, lightning attention and the mixture of experts (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

namespace {

int check_attend(const char* fn, const nvh_paged_attend_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->q && d->cache && d->block_tables && (d->out || d->out_packed), NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->heads > 0 && d->kv_heads > 0 && d->heads % d->kv_heads == 0 && d->dk > 0 && d->dk % 8 == 0 && d->dk <= 4096 && d->dv > 0 && d->dv % 8 == 0 && d->dv <= 2048 &&
            d->block_size > 0 && d->window >= 0 && d->keep_first >= 0, NVH_E_SHAPE, "%s: heads %d/%d widths %d/%d page %d window %d/%d", fn, d->heads, d->kv_heads,
            d->dk, d->dv, d->block_size, d->window, d->keep_first);
    REQUIRE(d->q_stride % 8 == 0 && d->q_stride >= (int64_t)d->heads * d->dk && d->bt_stride > 0 &&
            (!d->out || (d->out_stride % 4 == 0 && d->out_stride >= (int64_t)d->heads * d->dv)), NVH_E_STRIDE, "%s: row strides", fn);
    REQUIRE(aligned16(d->q) && aligned16(d->cache) && aligned16(d->out) && aligned16(d->out_packed), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

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

int nvh_attn_prep(const nvh_attn_prep_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "attn_prep: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("attn_prep");
    REQUIRE(d->qkv && d->positions && (d->cos_sin || d->rot == 0) && d->cache && d->slots && (!d->q_w == !d->k_w), NVH_E_NULL, "attn_prep: null pointer");
    const int64_t cols = (int64_t)d->heads * d->dk + (int64_t)d->kv_heads * (d->dk + d->dv);
    REQUIRE(d->rows > 0 && d->heads > 0 && d->kv_heads > 0 && d->dk > 0 && d->dk % 8 == 0 && d->dv > 0 && d->dv % 8 == 0 && cols <= kMaxRowCols && d->rot >= 0 && d->rot % 2 == 0 &&
            d->rot <= d->dk && d->max_position > 0 && d->block_size > 0 && (!d->q_w || (d->q_n > 0 && d->k_n > 0)), NVH_E_SHAPE,
            "attn_prep: heads %d/%d widths %d/%d rot %d (row of at most %d)", d->heads, d->kv_heads, d->dk, d->dv, d->rot, kMaxRowCols);
    REQUIRE(d->qkv_stride % 8 == 0 && d->qkv_stride >= cols, NVH_E_STRIDE, "attn_prep: row stride");
    REQUIRE(aligned16(d->qkv) && aligned16(d->cache) && aligned16(d->q_w) && aligned16(d->k_w), NVH_E_ALIGN, "attn_prep: pointers must be 16-byte aligned");
    return launch_attn_prep(*d, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_paged_attend_supported(int dk, int dv, int block_size) { return paged_attend_supported(dk, dv, block_size); }

size_t nvh_paged_attend_ticket_bytes(int rows, int kv_heads, int heads) {
    if (rows <= 0 || kv_heads <= 0 || heads % kv_heads) return 0;
    return (size_t)rows * kv_heads * paged_attend_groups(heads, kv_heads) * kAttendTicketWords * 4;
}

int nvh_paged_attend_rows(const nvh_paged_attend_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "paged_attend_rows: null descriptor");
    if (d->rows == 0) return 0;
    const int rc = check_attend("paged_attend_rows", d, dtype);
    if (rc) return rc;
    REQUIRE(d->positions && d->rows > 0 && d->splits >= 1 && d->splits <= 64 && (d->splits == 1 || (d->part && aligned16(d->part) && d->tickets)), NVH_E_NULL,
            "paged_attend_rows: rows %d splits %d or null pointer", d->rows, d->splits);
    REQUIRE(!d->out_packed || (dtype == NVH_BF16 && (d->heads * d->dv) % 32 == 0), NVH_E_SHAPE, "paged_attend_rows: packed output is bf16, width %% 32 == 0");
    return launch_paged_attend_rows(*d, dtype == NVH_F32, generic, (hipStream_t)stream);
}

int nvh_paged_attend_prompt(const nvh_paged_attend_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "paged_attend_prompt: null descriptor");
    if (d->batch == 0 || d->max_q == 0) return 0;
    const int rc = check_attend("paged_attend_prompt", d, dtype);
    if (rc) return rc;
    REQUIRE(dtype == NVH_BF16, NVH_E_DTYPE, "paged_attend_prompt: bf16 only");
    REQUIRE(d->cu_q && d->cu_k && d->out && !d->out_packed, NVH_E_NULL, "paged_attend_prompt: null pointer or packed output");
    REQUIRE(paged_attend_supported(d->dk, d->dv, d->block_size) && d->batch > 0 && d->batch <= 65535 && d->max_q > 0 && d->scale > 0.f, NVH_E_SHAPE,
            "paged_attend_prompt: widths %d/%d page %d scale %g", d->dk, d->dv, d->block_size, (double)d->scale);
    return launch_paged_attend_prompt(*d, (hipStream_t)stream);
}

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

int nvh_moe_route(const nvh_moe_route_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "moe_route: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("moe_route");
    REQUIRE(d->x && d->router && d->correction && d->ids && d->weights, NVH_E_NULL, "moe_route: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->experts > 0 && d->experts <= kMoeMaxExperts && d->groups > 0 && d->experts % d->groups == 0 && d->keep > 0 &&
            d->keep <= d->groups && d->top > 0 && d->top <= 64 && d->top <= d->keep * (d->experts / d->groups), NVH_E_SHAPE,
            "moe_route: %d experts (<= %d) in %d groups, %d kept, top %d (<= 64)", d->experts, kMoeMaxExperts, d->groups, d->keep, d->top);
    REQUIRE(d->x_stride % 8 == 0 && d->x_stride >= d->cols, NVH_E_STRIDE, "moe_route: row stride");
    REQUIRE(aligned16(d->x) && aligned16(d->router), NVH_E_ALIGN, "moe_route: pointers must be 16-byte aligned");
    return launch_moe_route(*d, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_moe_dispatch_blocks(int pairs) { return pairs > 0 ? moe_dispatch_blocks(pairs) : 0; }

int nvh_moe_dispatch(int32_t* slot_pair, int32_t* tiles, int32_t* counts, const int32_t* ids, int pairs, int experts, int tile_rows, int max_tiles, void* stream) {
    if (pairs == 0) return 0;
    REQUIRE(slot_pair && tiles && counts && ids, NVH_E_NULL, "moe_dispatch: null pointer");
    REQUIRE(pairs > 0 && experts > 0 && experts <= kMoeMaxExperts && tile_rows > 0 && max_tiles >= pairs / tile_rows + experts, NVH_E_SHAPE,
            "moe_dispatch: %d pairs %d experts: room for %d tiles of %d", pairs, experts, max_tiles, tile_rows);
    REQUIRE(aligned16(tiles), NVH_E_ALIGN, "moe_dispatch: tiles must be 16-byte aligned");
    return launch_moe_dispatch(slot_pair, tiles, counts, ids, pairs, experts, tile_rows, max_tiles, (hipStream_t)stream);
}

int nvh_moe_tile_rows(int pairs, int experts, int dtype) { return pairs > 0 && experts > 0 ? moe_tile_rows(pairs, experts, dtype == NVH_F32) : 0; }

int nvh_moe_gemm(const nvh_moe_gemm_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "moe_gemm: null descriptor");
    if (d->pairs == 0) return 0;
    DTYPE("moe_gemm");
    REQUIRE(d->out && d->x && d->w && (d->tiles ? d->slot_pair != nullptr : d->ids != nullptr), NVH_E_NULL, "moe_gemm: null pointer");
    REQUIRE(d->pairs > 0 && d->top > 0 && d->pairs % d->top == 0 && d->experts > 0 && d->experts <= kMoeMaxExperts && d->n > 0 && d->n % 64 == 0 && d->k > 0 && d->k % 64 == 0,
            NVH_E_SHAPE, "moe_gemm: %d pairs of top %d, n %d k %d (%%64)", d->pairs, d->top, d->n, d->k);
    REQUIRE(!d->tiles || d->tile_rows == (dtype == NVH_F32 ? 64 : 128) || (dtype == NVH_BF16 && d->tile_rows == 256), NVH_E_SHAPE, "moe_gemm: tiles of %d rows", d->tile_rows);
    REQUIRE(d->tiles ? d->max_tiles > 0 && d->max_tiles <= 65535 : dtype == NVH_BF16 && d->pairs / d->top <= 64, NVH_E_SHAPE,
            "moe_gemm: %d tiles, or the small form with more than 64 rows", d->max_tiles);
    REQUIRE(!d->glu || (d->x_stride % 8 == 0 && d->x_stride >= d->k), NVH_E_STRIDE, "moe_gemm: row stride");
    REQUIRE(aligned16(d->out) && aligned16(d->x) && aligned16(d->w) && aligned16(d->tiles), NVH_E_ALIGN, "moe_gemm: pointers must be 16-byte aligned");
    return launch_moe_gemm(*d, dtype == NVH_F32, (hipStream_t)stream);
}

}  // extern "C"
