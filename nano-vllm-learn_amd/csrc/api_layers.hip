// C ABI of the layer ops and the small-batch linear layer (declared in include/nvh_attn.h): error strings, argument validation, dispatch.
// Nothing here allocates, synchronises or reads device memory: every entry point is capture-safe.
#include <stdarg.h>
#include <stdio.h>
#include <string.h>

#include "api_common.h"

namespace nvh {

static thread_local char g_err[512] = "";

void set_error(const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
}

int check_launch(const char* what) {
    hipError_t e = hipGetLastError();
    if (e != hipSuccess) {
        set_error("%s: launch failed: %s", what, hipGetErrorString(e));
        return (int)e;
    }
    return 0;
}

unsigned long long* g_stamps = nullptr;

}  // namespace nvh

using namespace nvh;

extern "C" {

int nvh_version(void) { return NVH_VERSION; }

#ifdef NVH_STAMPS
void nvh_debug_set_stamps(void* p) { g_stamps = (unsigned long long*)p; }
#endif

const char* nvh_last_error(void) { return g_err; }

int nvh_add_rmsnorm(void* out, const void* x, void* residual, const void* weight, float eps, int n_rows, int hidden,
                    int64_t x_row_stride, int64_t out_row_stride, int64_t residual_row_stride, int dtype, void* stream) {
    if (n_rows == 0) return 0;
    if (dtype != NVH_BF16) { set_error("add_rmsnorm: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!out || !x || !weight) { set_error("add_rmsnorm: null pointer"); return NVH_E_NULL; }
    if (n_rows < 0 || hidden <= 0 || hidden % 8 || hidden > max_rmsnorm_hidden()) { set_error("add_rmsnorm: hidden %d unsupported", hidden); return NVH_E_SHAPE; }
    if (x_row_stride % 8 || out_row_stride % 8 || (residual && residual_row_stride % 8) || x_row_stride < hidden || out_row_stride < hidden) {
        set_error("add_rmsnorm: row strides must be multiples of 8 and >= hidden");
        return NVH_E_STRIDE;
    }
    if (!aligned16(out) || !aligned16(x) || !aligned16(weight) || (residual && !aligned16(residual))) { set_error("add_rmsnorm: pointers must be 16-byte aligned"); return NVH_E_ALIGN; }
    return launch_add_rmsnorm(out, x, residual, weight, eps, n_rows, hidden, x_row_stride, out_row_stride, residual_row_stride, (hipStream_t)stream);
}

int nvh_residual_add_pack(void* residual, const void* y, void* packed, int n_rows, int hidden, int64_t residual_row_stride,
                          int64_t y_row_stride, int dtype, void* stream) {
    if (n_rows == 0) return 0;
    if (dtype != NVH_BF16) { set_error("residual_add_pack: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!residual || !y) { set_error("residual_add_pack: null pointer"); return NVH_E_NULL; }
    if (n_rows < 0 || hidden <= 0 || hidden % 32) { set_error("residual_add_pack: hidden %d must be a positive multiple of 32", hidden); return NVH_E_SHAPE; }
    if (residual_row_stride % 8 || y_row_stride % 8 || residual_row_stride < hidden || y_row_stride < hidden) { set_error("residual_add_pack: bad row strides"); return NVH_E_STRIDE; }
    if (!aligned16(residual) || !aligned16(y) || (packed && !aligned16(packed))) { set_error("residual_add_pack: pointers must be 16-byte aligned"); return NVH_E_ALIGN; }
    return launch_residual_add_pack(residual, y, packed, n_rows, hidden, residual_row_stride, y_row_stride, (hipStream_t)stream);
}

int nvh_silu_mul(void* out, const void* gate_up, int n_rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride,
                 int dtype, void* stream) {
    if (n_rows == 0) return 0;
    if (dtype != NVH_BF16) { set_error("silu_mul: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!out || !gate_up) { set_error("silu_mul: null pointer"); return NVH_E_NULL; }
    if (n_rows < 0 || inter <= 0 || inter % 8) { set_error("silu_mul: inter %d must be a positive multiple of 8", inter); return NVH_E_SHAPE; }
    if (gate_up_row_stride % 8 || out_row_stride % 8 || gate_up_row_stride < 2 * (int64_t)inter || out_row_stride < inter) {
        set_error("silu_mul: bad row strides");
        return NVH_E_STRIDE;
    }
    if (!aligned16(out) || !aligned16(gate_up)) { set_error("silu_mul: pointers must be 16-byte aligned"); return NVH_E_ALIGN; }
    return launch_silu_mul(out, gate_up, n_rows, inter, gate_up_row_stride, out_row_stride, (hipStream_t)stream);
}

int nvh_argmax_rows(int64_t* out, const void* x, int n_rows, int n, int64_t x_row_stride, int dtype, void* stream) {
    if (n_rows == 0) return 0;
    if (dtype != NVH_BF16) { set_error("argmax_rows: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!out || !x) { set_error("argmax_rows: null pointer"); return NVH_E_NULL; }
    if (n_rows < 0 || n <= 0) { set_error("argmax_rows: bad shape"); return NVH_E_SHAPE; }
    if (x_row_stride % 8 || x_row_stride < n) { set_error("argmax_rows: row stride must be a multiple of 8 and >= n"); return NVH_E_STRIDE; }
    if (!aligned16(x)) { set_error("argmax_rows: x must be 16-byte aligned"); return NVH_E_ALIGN; }
    return launch_argmax_rows(out, x, n_rows, n, x_row_stride, AdvanceArgs{}, (hipStream_t)stream);
}

int nvh_greedy_advance(const void* logits, int n_rows, int n, int64_t logits_row_stride,
                       int64_t* input_ids, int64_t* positions, int32_t* context_lens, int32_t* slot_mapping,
                       const int32_t* block_tables, int64_t bt_row_stride, int block_size,
                       int64_t* tokens_log, int64_t log_row_stride, int64_t* row_steps, int dtype, void* stream) {
    if (n_rows == 0) return 0;
    if (dtype != NVH_BF16) { set_error("greedy_advance: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!logits || !input_ids || !positions || !context_lens || !slot_mapping || !block_tables || !tokens_log || !row_steps) { set_error("greedy_advance: null pointer"); return NVH_E_NULL; }
    if (n_rows < 0 || n <= 0 || block_size <= 0 || log_row_stride < n_rows) { set_error("greedy_advance: bad shape"); return NVH_E_SHAPE; }
    if (logits_row_stride % 8 || logits_row_stride < n) { set_error("greedy_advance: logits row stride must be a multiple of 8 and >= n"); return NVH_E_STRIDE; }
    if (!aligned16(logits)) { set_error("greedy_advance: logits must be 16-byte aligned"); return NVH_E_ALIGN; }
    AdvanceArgs adv{input_ids, positions, context_lens, slot_mapping, block_tables, bt_row_stride, block_size, tokens_log, log_row_stride, row_steps};
    return launch_argmax_rows(nullptr, logits, n_rows, n, logits_row_stride, adv, (hipStream_t)stream);
}

int nvh_linear_small_m(void* out, const void* x, const void* w, const void* bias, int m, int n, int k, int silu_inter,
                       int64_t x_row_stride, int64_t out_row_stride, int dtype, void* stream) {
    if (m == 0) return 0;
    if (dtype != NVH_BF16) { set_error("linear_small_m: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    if (!out || !x || !w) { set_error("linear_small_m: null pointer"); return NVH_E_NULL; }
    if (m < 0 || m > 64 || n <= 0 || k <= 0 || k % 32 || n % 16) { set_error("linear_small_m: m=%d (<=64) n=%d (%%16) k=%d (%%32)", m, n, k); return NVH_E_SHAPE; }
    if (silu_inter && (silu_inter * 2 != n || silu_inter % 16 || bias)) { set_error("linear_small_m: silu mode needs n == 2*inter, inter %% 16 == 0, no bias"); return NVH_E_SHAPE; }
    const int out_cols = silu_inter ? silu_inter : n;
    if (x_row_stride % 8 || x_row_stride < k || out_row_stride < out_cols) { set_error("linear_small_m: bad row strides"); return NVH_E_STRIDE; }
    if (!aligned16(x) || !aligned16(w)) { set_error("linear_small_m: x and w must be 16-byte aligned"); return NVH_E_ALIGN; }
    nvh_linear_desc d = {};
    d.out = out; d.x = x; d.w = w; d.bias = bias; d.m = m; d.n = n; d.k = k; d.silu_inter = silu_inter;
    d.x_row_stride = x_row_stride; d.out_row_stride = out_row_stride;
    d.epilogue = silu_inter ? NVH_EPI_SILU_MUL : NVH_EPI_NONE;
    return nvh_linear_small_m_ex(&d, dtype, stream);
}

}  // extern "C"

// validates the descriptor and fills `a`; returns 1 when there is nothing to do (m == 0), 0 when `a` is ready, < 0 on rejection
int nvh::linear_args(LinearArgs& a, const nvh_linear_desc* d, int dtype) {
    if (!d) { set_error("linear_small_m_ex: null descriptor"); return NVH_E_NULL; }
    if (d->m == 0) return 1;
    if (dtype != NVH_BF16) { set_error("linear_small_m_ex: dtype %d unsupported (bf16 only)", dtype); return NVH_E_DTYPE; }
    const bool out_optional = (d->out_packed && (d->epilogue == NVH_EPI_NONE || d->epilogue == NVH_EPI_SILU_MUL)) ||
                              (d->candidate_val && d->epilogue == NVH_EPI_NONE);
    if ((d->candidate_val != nullptr) != (d->candidate_idx != nullptr) || (d->candidate_val && d->candidate_stride < d->m)) {
        set_error("linear_small_m_ex: candidate_val / candidate_idx come together, candidate_stride >= m");
        return NVH_E_NULL;
    }
    if ((!d->out && !out_optional) || !d->x || !d->w) { set_error("linear_small_m_ex: null pointer"); return NVH_E_NULL; }
    if (d->m < 0 || d->m > 64 || d->n <= 0 || d->k <= 0 || d->k % 64 || d->n % 16) {
        set_error("linear_small_m_ex: m=%d (<=64) n=%d (%%16) k=%d (%%64)", d->m, d->n, d->k);
        return NVH_E_SHAPE;
    }
    int out_cols = d->n;
    switch (d->epilogue) {
        case NVH_EPI_NONE: break;
        case NVH_EPI_SILU_MUL:
            if (d->silu_inter * 2 != d->n || d->silu_inter % 16 || d->bias) { set_error("linear_small_m_ex: silu needs n == 2*inter, inter %% 16 == 0, no bias"); return NVH_E_SHAPE; }
            out_cols = d->silu_inter;
            break;
        case NVH_EPI_RESIDUAL_ADD:
            if (d->bias) { set_error("linear_small_m_ex: residual-add epilogue takes no bias"); return NVH_E_SHAPE; }
            break;
        case NVH_EPI_ROPE_STORE:
            if ((d->hd != 64 && d->hd != 128) || d->h <= 0 || d->kvh <= 0 || (d->h + 2 * d->kvh) * d->hd != d->n) {
                set_error("linear_small_m_ex: rope epilogue needs n == (h + 2*kvh) * hd, hd in {64,128}");
                return NVH_E_SHAPE;
            }
            if (!d->positions || !d->cos_sin || !d->k_cache || !d->v_cache || !d->slot_mapping) { set_error("linear_small_m_ex: rope epilogue pointers"); return NVH_E_NULL; }
            out_cols = d->h * d->hd;
            break;
        default: set_error("linear_small_m_ex: unknown epilogue %d", d->epilogue); return NVH_E_SHAPE;
    }
    if ((!d->x_packed && (d->x_row_stride % 8 || d->x_row_stride < d->k)) || (d->out && d->out_row_stride < out_cols)) { set_error("linear_small_m_ex: bad row strides"); return NVH_E_STRIDE; }
    if (d->out_packed && (!aligned16(d->out_packed) || out_cols % 32)) { set_error("linear_small_m_ex: out_packed needs 16-byte alignment and cols %% 32 == 0"); return NVH_E_ALIGN; }
    if (d->workspace && !aligned16(d->workspace)) { set_error("linear_small_m_ex: workspace must be 16-byte aligned"); return NVH_E_ALIGN; }
    if (!aligned16(d->x) || !aligned16(d->w) || (d->norm_weight && !aligned16(d->norm_weight))) { set_error("linear_small_m_ex: x, w, norm_weight must be 16-byte aligned"); return NVH_E_ALIGN; }
    a.out = d->out; a.x = (const uint16_t*)d->x; a.w = (const uint16_t*)d->w; a.bias = (const uint16_t*)d->bias;
    a.M = d->m; a.N = d->n; a.K = d->k; a.inter = d->silu_inter; a.x_stride = d->x_row_stride; a.out_stride = d->out_row_stride;
    if (d->norm_folded && d->norm_weight) { set_error("linear_small_m_ex: norm_folded excludes norm_weight"); return NVH_E_NULL; }
    a.norm_w = (const uint16_t*)d->norm_weight; a.norm_eps = d->norm_eps; a.epi = d->epilogue;
    a.glu_limit = d->glu_limit; a.glu_alpha = d->glu_alpha; a.glu_gelu = d->glu_gelu;
    a.x_groups = 0;
    a.norm_mode = d->norm_folded ? 2 : (d->norm_weight ? 1 : 0);
    a.positions = d->positions; a.cos_sin = d->cos_sin; a.k_cache = (uint16_t*)d->k_cache; a.v_cache = (uint16_t*)d->v_cache;
    a.slots = d->slot_mapping; a.h = d->h; a.kvh = d->kvh; a.hd = d->hd;
    if (d->epilogue == NVH_EPI_NONE) a.inter = a.hd = 0;
    if (d->x_groups > 1) {
        if (d->epilogue != NVH_EPI_NONE || !d->x_packed || d->candidate_val || d->x_group_rows <= 0 || d->x_group_rows % 16 ||
            (int64_t)d->x_group_rows * (d->x_groups - 1) >= d->n || d->x_group_stride < (d->m + 15) / 16 * 16 * d->k || d->x_group_stride % 8) {
            set_error("linear_small_m_ex: x groups need packed activations, the NONE epilogue, rows %% 16 == 0 and a stride of whole packed rows");
            return NVH_E_SHAPE;
        }
        a.x_groups = d->x_groups; a.inter = d->x_group_rows; a.hd = d->x_group_stride;
    }
    a.stamps = g_stamps;
    a.x_packed = d->x_packed; a.out_packed = (uint16_t*)d->out_packed; a.ws_raw = d->workspace; a.ws_bytes = d->workspace_bytes;
    a.ws = nullptr; a.counters = nullptr; a.ksplit = 1; a.tiles = 0;
    a.cand_val = d->candidate_val; a.cand_idx = d->candidate_idx; a.cand_stride = d->candidate_stride;
    // prefetch hint: whole 128-byte lines inside [prefetch, prefetch + prefetch_bytes) only (reads never leave the caller's range)
    // Ranges above 4 MiB are ignored: the hint pays for operands whose FIRST-BYTE latency dominates their consumer (a few MB read by a
    // few dozen workgroups); 8.7 and 17.4 MB ranges measured +-0 and +1.3 % on the decode step (the prefetching workgroups outlive the launch)
    a.pf_ptr = nullptr; a.pf_bytes = 0;
    a.pf_kv = {};
#ifndef NVH_PF_MAX_MB
#define NVH_PF_MAX_MB 4                      // (A/B builds lift it)
#endif
    if (d->prefetch && d->prefetch_bytes >= 256 && d->prefetch_bytes <= ((size_t)NVH_PF_MAX_MB << 20)) {
        const uintptr_t p0 = ((uintptr_t)d->prefetch + 127) & ~(uintptr_t)127, p1 = ((uintptr_t)d->prefetch + d->prefetch_bytes) & ~(uintptr_t)127;
        if (p1 > p0) { a.pf_ptr = (const void*)p0; a.pf_bytes = (int64_t)(p1 - p0); }
    }
    return 0;
}

extern "C" {

int nvh_linear_small_m_ex(const nvh_linear_desc* d, int dtype, void* stream) {
    LinearArgs a;
    const int rca = linear_args(a, d, dtype);
    if (rca) return rca > 0 ? 0 : rca;
    const int rc = launch_linear_stream(a, (hipStream_t)stream);
    if (rc != -100) return rc;
    if (d->x_packed || d->out_packed || d->candidate_val) {
        set_error("linear_small_m_ex: packed activations / candidates need the streaming kernel (k %% 64 == 0, no exact-norm prologue, workspace when k > 1024)");
        return NVH_E_SHAPE;
    }
    return launch_linear_small_m(a, (hipStream_t)stream);
}

size_t nvh_linear_small_m_workspace(int m, int n, int k, int epilogue) { return linear_stream_workspace_bytes(m, n, k, epilogue); }
int nvh_linear_small_m_candidate_groups(int n, int k) { return linear_stream_candidate_groups(n, k); }

}  // extern "C"
