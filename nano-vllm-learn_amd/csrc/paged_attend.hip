// Softmax attention over pages of one layer, single query rows (paged_rows.h): the scores are the query's products with the keys.
#include "paged_rows.h"

namespace nvh {

namespace {

template <int DK, int DV>
void rows_dims(const PagedAttendArgs& a, hipStream_t stream) {
    const int ratio = a.heads / a.kv_heads;
    const dim3 grid(a.splits, a.kv_heads * paged_attend_groups(a.heads, a.kv_heads), a.rows);
    if (ratio == 1) paged_rows_kernel<KeyScores<DK>, DV, 1><<<grid, 256, 0, stream>>>(a);
    else if (ratio == 2) paged_rows_kernel<KeyScores<DK>, DV, 2><<<grid, 256, 0, stream>>>(a);
    else if (ratio <= 4) paged_rows_kernel<KeyScores<DK>, DV, 4><<<grid, 256, 0, stream>>>(a);
    else paged_rows_kernel<KeyScores<DK>, DV, 8><<<grid, 256, 0, stream>>>(a);
}

}  // namespace

bool paged_attend_supported(int dk, int dv, int block_size) {
    if (block_size % 64) return false;
    return ((dk == 64 || dk == 128 || dk == 192 || dk == 256) && (dv == 64 || dv == 128)) || (dk == 256 && dv == 256);
}

int launch_paged_attend_rows(const PagedAttendArgs& a, int f32, int generic, hipStream_t stream) {
    if (!f32 && !generic && !a.row_seq && paged_attend_supported(a.dk, a.dv, a.block_size)) {
        switch (a.dk * 1000 + a.dv) {
            case 64064: rows_dims<64, 64>(a, stream); break;
            case 64128: rows_dims<64, 128>(a, stream); break;
            case 128064: rows_dims<128, 64>(a, stream); break;
            case 128128: rows_dims<128, 128>(a, stream); break;
            case 192064: rows_dims<192, 64>(a, stream); break;
            case 192128: rows_dims<192, 128>(a, stream); break;
            case 256064: rows_dims<256, 64>(a, stream); break;
            case 256128: rows_dims<256, 128>(a, stream); break;
            default: rows_dims<256, 256>(a, stream); break;
        }
    } else {
        const dim3 grid(a.rows, a.heads);
        if (f32) paged_rows_generic_kernel<float><<<grid, 256, a.dk * 4, stream>>>(a);
        else paged_rows_generic_kernel<uint16_t><<<grid, 256, a.dk * 4, stream>>>(a);
    }
    return check_launch("paged_attend_rows");
}

}  // namespace nvh
