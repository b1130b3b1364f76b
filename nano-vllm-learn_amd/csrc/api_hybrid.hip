// C ABI of the recurrent and latent-attention layers (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "hybrid.h"

using namespace nvh;

namespace {

int check_rglru(const char* fn, const nvh_rglru_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->yx && d->conv_w && d->conv_b && d->ra && d->ri && d->ra_b && d->ri_b && d->rate && d->positions && d->state_slots && d->state && d->conv_state,
            NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->block > 0 && d->block % 32 == 0 && d->blocks > 0 && d->width == d->block * d->blocks && d->width % 64 == 0 && d->taps >= 1 && d->taps <= 64, NVH_E_SHAPE,
            "%s: width %d must be blocks %d x block %d (%%32), a multiple of 64; taps %d in 1..64", fn, d->width, d->blocks, d->block, d->taps);
    REQUIRE(d->yx_stride % 8 == 0 && d->yx_stride >= 2 * (int64_t)d->width && (!d->out || (d->out_stride % 8 == 0 && d->out_stride >= d->width)), NVH_E_STRIDE,
            "%s: row strides", fn);
    REQUIRE(aligned16(d->yx) && aligned16(d->ra) && aligned16(d->ri) && aligned16(d->state) && aligned16(d->conv_state) && aligned16(d->conv_w) &&
            aligned16(d->conv_b) && (!d->out || aligned16(d->out)), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

}  // namespace

extern "C" {

int nvh_rglru_chunk_tokens(void) { return kRglruChunk; }
int nvh_rglru_step_supported(int block) { return block > 0 && block % 32 == 0 && rglru_step_supported(block); }

int nvh_rglru_chunks(const nvh_rglru_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "rglru_chunks: null descriptor");
    if (d->n_chunks == 0) return 0;
    const int rc = check_rglru("rglru_chunks", d, dtype);
    if (rc) return rc;
    REQUIRE(d->chunks && d->s_loc && d->a_cum && d->out && d->n_chunks > 0, NVH_E_NULL, "rglru_chunks: null pointer");
    REQUIRE(d->segment > 0 && d->segment % kRglruChunk == 0, NVH_E_SHAPE, "rglru_chunks: segment %d must be a positive multiple of %d", d->segment, kRglruChunk);
    REQUIRE(!d->out_packed, NVH_E_SHAPE, "rglru_chunks: packed output belongs to the step form");
    REQUIRE(aligned16(d->s_loc) && aligned16(d->a_cum), NVH_E_ALIGN, "rglru_chunks: scratch must be 16-byte aligned");
    return launch_rglru_chunks(*d, dtype == NVH_F32, generic, (hipStream_t)stream);
}

int nvh_rglru_step(const nvh_rglru_desc* d, int rows, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "rglru_step: null descriptor");
    if (rows == 0) return 0;
    REQUIRE(dtype == NVH_BF16, NVH_E_DTYPE, "rglru_step: bf16 only");
    const int rc = check_rglru("rglru_step", d, dtype);
    if (rc) return rc;
    REQUIRE(rows > 0 && (d->out || d->out_packed), NVH_E_NULL, "rglru_step: no output");
    REQUIRE(rglru_step_supported(d->block), NVH_E_SHAPE, "rglru_step: block %d too large", d->block);
    return launch_rglru_step(*d, rows, (hipStream_t)stream);
}

int nvh_latent_prep(const nvh_latent_prep_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "latent_prep: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("latent_prep");
    REQUIRE(d->a && d->q_w && (d->cq || d->cq_packed), NVH_E_NULL, "latent_prep: null pointer");
    REQUIRE(d->kv_cols == 0 || (d->kv_w && d->cache && d->slots && d->positions && d->cos_sin), NVH_E_NULL, "latent_prep: null cache pointer");
    REQUIRE(d->rows > 0 && d->q_cols > 0 && d->q_cols % 32 == 0 && d->q_rank > 0 && d->q_rank <= d->q_cols && d->kv_cols % 8 == 0 && d->kv_rank <= d->kv_cols &&
            d->rot % 2 == 0 && d->rot <= d->rot_cols && d->rot_cols % 8 == 0 && (d->kv_cols == 0 || (d->kv_rank > 0 && d->max_position > 0)), NVH_E_SHAPE,
            "latent_prep: q %d/%d kv %d/%d rot %d/%d", d->q_rank, d->q_cols, d->kv_rank, d->kv_cols, d->rot, d->rot_cols);
    REQUIRE(!d->cq_packed || dtype == NVH_BF16, NVH_E_DTYPE, "latent_prep: packed rows are bf16");
    REQUIRE(d->a_stride % 8 == 0 && d->a_stride >= d->q_cols + d->kv_cols + (d->kv_cols ? d->rot_cols : 0), NVH_E_STRIDE, "latent_prep: row stride");
    REQUIRE(aligned16(d->a) && aligned16(d->q_w) && (!d->cq || aligned16(d->cq)) && (!d->cq_packed || aligned16(d->cq_packed)) &&
            (d->kv_cols == 0 || (aligned16(d->kv_w) && aligned16(d->cache))), NVH_E_ALIGN, "latent_prep: pointers must be 16-byte aligned");
    return launch_latent_prep(*d, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_latent_attend_mfma(int kv_cols, int rot_cols, int block_size) { return latent_mfma_supported(kv_cols, rot_cols, block_size); }

int nvh_latent_attention(const nvh_latent_attn_desc* d, int generic, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "latent_attention: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("latent_attention");
    REQUIRE(d->q && d->cache && d->block_tables && d->positions && d->cos_sin && d->w_uk && d->w_uv && d->qa && d->part_o && d->part_ml && (d->out || d->out_packed),
            NVH_E_NULL, "latent_attention: null pointer");
    REQUIRE(d->rows > 0 && d->heads > 0 && d->dim_cols % 8 == 0 && d->dim_cols > 0 && d->qrot_cols >= d->rot && d->qrot_cols % 8 == 0 && d->kv_cols > 0 && d->kv_cols % 8 == 0 &&
            d->kv_cols <= 2048 && d->rot % 2 == 0 && d->rot <= d->rot_cols && d->rot_cols % 8 == 0 && d->v_cols > 0 && d->v_cols % 8 == 0 && d->block_size > 0 &&
            d->splits >= 1 && d->splits <= 64 && d->max_position > 0 && d->max_blocks > 0, NVH_E_SHAPE,
            "latent_attention: heads %d dim %d rot %d/%d/%d latent %d value %d page %d splits %d", d->heads, d->dim_cols, d->rot, d->qrot_cols, d->rot_cols, d->kv_cols,
            d->v_cols, d->block_size, d->splits);
    REQUIRE(!d->out_packed || (dtype == NVH_BF16 && d->v_cols % 16 == 0 && d->kv_cols % 32 == 0 && (d->heads * d->v_cols) % 32 == 0), NVH_E_SHAPE,
            "latent_attention: packed output is bf16, value width %% 16 == 0");
    REQUIRE(d->q_stride % 8 == 0 && d->q_stride >= (int64_t)d->heads * (d->dim_cols + d->qrot_cols) && d->bt_stride >= d->max_blocks &&
            (!d->out || (d->out_stride % 4 == 0 && d->out_stride >= (int64_t)d->heads * d->v_cols)), NVH_E_STRIDE, "latent_attention: row strides");
    REQUIRE(aligned16(d->q) && aligned16(d->cache) && aligned16(d->w_uk) && aligned16(d->w_uv) && aligned16(d->qa) && aligned16(d->part_o) && (!d->out || aligned16(d->out)),
            NVH_E_ALIGN, "latent_attention: pointers must be 16-byte aligned");
    const int f32 = dtype == NVH_F32;
    int rc = launch_latent_absorb(*d, f32, (hipStream_t)stream);
    if (!rc) rc = launch_latent_attend(*d, f32, generic, (hipStream_t)stream);
    if (!rc) rc = launch_latent_value(*d, f32, (hipStream_t)stream);
    return rc;
}

int nvh_latent_gather(void* out, const void* cache, const int32_t* cu_k, const int32_t* block_tables, int64_t bt_stride, int batch, int total, int cols,
                      int block_size, int dtype, void* stream) {
    if (total == 0 || batch == 0) return 0;
    DTYPE("latent_gather");
    REQUIRE(out && cache && cu_k && block_tables, NVH_E_NULL, "latent_gather: null pointer");
    REQUIRE(batch > 0 && total > 0 && cols > 0 && cols % 8 == 0 && block_size > 0, NVH_E_SHAPE, "latent_gather: cols %d (%%8) page %d", cols, block_size);
    REQUIRE(aligned16(out) && aligned16(cache), NVH_E_ALIGN, "latent_gather: pointers must be 16-byte aligned");
    return launch_latent_gather(out, cache, cu_k, block_tables, bt_stride, batch, total, cols, block_size, dtype == NVH_F32, (hipStream_t)stream);
}

int nvh_latent_prefill_supported(int dk, int dv) { return latent_prefill_supported(dk, dv); }

int nvh_latent_prefill(const nvh_latent_prefill_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "latent_prefill: null descriptor");
    if (d->batch == 0 || d->max_q == 0) return 0;
    REQUIRE(dtype == NVH_BF16, NVH_E_DTYPE, "latent_prefill: bf16 only");
    REQUIRE(d->q && d->k && d->k_rot && d->v && d->out && d->cu_q && d->cu_k && d->positions && d->cos_sin, NVH_E_NULL, "latent_prefill: null pointer");
    REQUIRE(latent_prefill_supported(d->dk, d->dv) && d->dim_cols > 0 && d->dim_cols % 32 == 0 && d->dim_cols < d->dk && d->rot % 2 == 0 && d->rot <= d->dk - d->dim_cols &&
            d->heads > 0 && d->batch > 0 && d->max_q > 0 && d->max_position > 0 && d->scale_log2 > 0.f, NVH_E_SHAPE,
            "latent_prefill: key width %d (own part %d, rotated %d) value width %d heads %d scale %g", d->dk, d->dim_cols, d->rot, d->dv, d->heads, (double)d->scale_log2);
    REQUIRE(d->q_stride % 8 == 0 && d->k_stride % 8 == 0 && d->kr_stride % 8 == 0 && d->v_stride % 8 == 0 && d->out_stride % 4 == 0 &&
            d->q_stride >= (int64_t)d->heads * d->dk && d->k_stride >= (int64_t)d->heads * d->dim_cols && d->kr_stride >= d->dk - d->dim_cols &&
            d->v_stride >= (int64_t)d->heads * d->dv && d->out_stride >= (int64_t)d->heads * d->dv, NVH_E_STRIDE, "latent_prefill: row strides");
    REQUIRE(aligned16(d->q) && aligned16(d->k) && aligned16(d->k_rot) && aligned16(d->v) && aligned16(d->out), NVH_E_ALIGN, "latent_prefill: pointers must be 16-byte aligned");
    return launch_latent_prefill(*d, (hipStream_t)stream);
}

}  // extern "C"
