// Shared by the C ABI files: argument checks and the linear descriptor's validation.
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

// validates the descriptor and fills `a`; returns 1 when there is nothing to do (m == 0), 0 when `a` is ready, < 0 on rejection
int linear_args(LinearArgs& a, const nvh_linear_desc* d, int dtype);

}  // namespace nvh
