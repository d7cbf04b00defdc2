// kf_ctx.h -- the context object behind the C ABI and the argument-check plumbing shared by the files that define ABI entries.
#pragma once
#include <hip/hip_runtime.h>

#include <vector>

#include "../../include/kf_abi.h"

struct kf_ctx {
    int device;
    hipStream_t stream;
    bool own_stream;
    bool capturing;
    float* amax_val; /* per-workgroup partial maxima for kf_lm_head when the caller passes no scratch */
    int* amax_idx;
    int canonical;    /* 1: the decode kernels sum in the canonical order of oracle/kf_oracle.c sections 4c / 6 (bit-exact against the oracle; the default); 0: v_dot2c / fp32 forms */
    void* scratch;    /* caller-owned workspace of kf_linear (kf_set_scratch): AWQ slice partials, or a weight dequantised to bf16 */
    size_t scratch_bytes;
    // resident GetDataX copies for token batches (kf_set_dequant_arena): caller-owned memory, filled on first use, keyed by the data pointers of the matrices a route
    // multiplies in one launch and the form they are laid out in (DEQ_STACK: back to back; DEQ_ILV: gate | up interleaved in blocks of 16 rows)
    struct DeqCopy {
        const void* key[3];
        int form;
        size_t off;
    };
    void* arena;
    size_t arena_bytes, arena_used;
    std::vector<DeqCopy> copies;
};
enum { DEQ_STACK = 0, DEQ_ILV = 1 };

namespace kf {
int abi_fail(int code, const char* fmt, ...); /* records the text kf_last_error() returns, gives `code` back (kf_abi.hip) */
}

#define HIPCHK(expr)                                                                                   \
    do {                                                                                               \
        hipError_t e_ = (expr);                                                                        \
        if (e_ != hipSuccess) return kf::abi_fail(KF_HIP_CHECK, "%s: %s (%s:%d)", #expr, hipGetErrorString(e_), __FILE__, __LINE__); \
    } while (0)
#define CHKCTX(c) \
    if (!(c)) return kf::abi_fail(KF_INVALID_ARGS, "%s: null kf_ctx", __func__)
#define RET(code) \
    do {          \
        int c_ = (code); \
        if (c_ != KF_OK) return kf::abi_fail(c_, "%s failed with %d", __func__, c_); \
        return KF_OK;    \
    } while (0)

static inline bool al16(const void* p) { return (((uintptr_t)p) & 15) == 0; }
