// C ABI of the mixture of experts (declared in include/nvh_attn.h): argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include "api_common.h"
#include "mixers.h"

using namespace nvh;

extern "C" {

int nvh_moe_route(const nvh_moe_route_desc* d, int dtype, void* stream) {
    REQUIRE(d, NVH_E_NULL, "moe_route: null descriptor");
    if (d->rows == 0) return 0;
    DTYPE("moe_route");
    REQUIRE(d->x && d->router && d->correction && d->ids && d->weights, NVH_E_NULL, "moe_route: null pointer");
    REQUIRE(d->rows > 0 && d->cols > 0 && d->cols % 8 == 0 && d->experts > 0 && d->experts <= kMoeMaxExperts && d->groups > 0 && d->experts % d->groups == 0 && d->keep > 0 &&
            d->keep <= d->groups && (!d->softmax || d->groups == 1) && d->top > 0 && d->top <= 64 && d->top <= d->keep * (d->experts / d->groups), NVH_E_SHAPE,
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
