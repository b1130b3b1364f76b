// Shared by the C ABI files: argument checks, validation of descriptors several of them take.
#pragma once
#include <stdint.h>

#include "../../include/nvh_attn.h"
#include "common.h"
#include "kernels.h"

namespace nvh {

// diagnostic builds (-DNVH_STAMPS) set this through nvh_debug_set_stamps; always null in the shipped library
extern unsigned long long* g_stamps;

inline bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

#define REQUIRE(cond, code, ...) do { if (!(cond)) { set_error(__VA_ARGS__); return code; } } while (0)

inline int check_dtype(const char* fn, int dtype) {
    REQUIRE(dtype == NVH_BF16 || dtype == NVH_F32, NVH_E_DTYPE, "%s: dtype %d unsupported (bf16 or f32)", fn, dtype);
    return 0;
}
#define DTYPE(fn) do { const int rc_ = check_dtype(fn, dtype); if (rc_) return rc_; } while (0)

// what every form of attention over pages asks of its descriptor
inline int check_attend(const char* fn, const nvh_paged_attend_desc* d, int dtype) {
    DTYPE(fn);
    REQUIRE(d->q && d->cache && d->block_tables && (d->out || d->out_packed), NVH_E_NULL, "%s: null pointer", fn);
    REQUIRE(d->heads > 0 && d->kv_heads > 0 && d->heads % d->kv_heads == 0 && d->dk > 0 && d->dk % 8 == 0 && d->dk <= 4096 && d->dv > 0 && d->dv % 8 == 0 && d->dv <= 2048 &&
            d->block_size > 0 && d->window >= 0 && d->keep_first >= 0 && d->chunk >= 0 && (!d->chunk || !d->window), NVH_E_SHAPE, "%s: heads %d/%d widths %d/%d page %d window %d/%d", fn, d->heads, d->kv_heads,
            d->dk, d->dv, d->block_size, d->window, d->keep_first);
    REQUIRE(d->q_stride % 8 == 0 && d->q_stride >= (int64_t)d->heads * d->dk && d->bt_stride > 0 &&
            (!d->out || (d->out_stride % 4 == 0 && d->out_stride >= (int64_t)d->heads * d->dv)), NVH_E_STRIDE, "%s: row strides", fn);
    REQUIRE(!d->o_cos_sin || (d->o_rot > 0 && d->o_rot % 2 == 0 && d->o_rot <= d->dv && d->max_position > 0), NVH_E_SHAPE, "%s: outputs turned back by %d of %d dimensions", fn,
            d->o_rot, d->dv);
    REQUIRE(!d->talk || (!d->chunk && !d->o_cos_sin), NVH_E_SHAPE, "%s: mixed heads know windows only", fn);
    REQUIRE(aligned16(d->q) && aligned16(d->cache) && aligned16(d->out) && aligned16(d->out_packed), NVH_E_ALIGN, "%s: pointers must be 16-byte aligned", fn);
    return 0;
}

// validates the descriptor and fills `a`; returns 1 when there is nothing to do (m == 0), 0 when `a` is ready, < 0 on rejection
int linear_args(LinearArgs& a, const nvh_linear_desc* d, int dtype);

}  // namespace nvh
