// kf_rb_ops.hip -- the row-batch operators around the products: embedding, RMS norm of the 32-bit residual (with the alpha-scaled residual sum over experts), the router
// and its pair list, the greedy pick.  One workgroup per row, float4 columns; widths are padded (kf_rb.h), so there are no column tails.
#include <math.h>

#include "kf_ctx.h"
#include "kf_rb_common.h"

namespace kf {

template <class T>
__device__ __forceinline__ void embed_row(const T* __restrict__ table, int tok, int vocab, int dim, long long ld, float* __restrict__ x, T* __restrict__ h) {
    tok = tok < 0 ? 0 : (tok < vocab ? tok : vocab - 1);
    const T* src = table + (size_t)tok * ld;
    for (int i = 4 * (int)threadIdx.x; i < ld; i += 4 * (int)blockDim.x) {
        f32x4 v = rb_ld4(src + i);
        if (i + 3 >= dim) {
#pragma unroll
            for (int j = 0; j < 4; j++)
                if (i + j >= dim) v[j] = 0.f;
        }
        rb_st4(x + i, v);
        rb_st4(h + i, v);
    }
}
template <class T>
__global__ void rb_embed_kernel(const T* table, int vocab, int dim, long long ld, const int32_t* tokens, float* x, T* h) {
    const size_t r = blockIdx.x;
    embed_row(table, tokens[r], vocab, dim, ld, x + r * ld, h + r * ld);
}
template <class T>
__global__ void rb_embed_state_kernel(const T* table, int vocab, int dim, long long ld, int32_t* state, const int32_t* forced, int forced_stride, int max_pos, float* x, T* h,
                                      int32_t* meta) {
    const int s = blockIdx.x;
    const int pos = state[4 * s + 1], parked = state[4 * s + 2];
    const bool in = pos >= 0 && pos < max_pos, on = !parked && in;
    int tok = state[4 * s];
    if (on && forced) {
        const int f = forced[(size_t)s * forced_stride + pos];
        tok = f >= 0 ? f : tok;
    }
    if (threadIdx.x == 0) {
        *reinterpret_cast<u32x4*>(meta + KF_RB_META * s) = u32x4{(uint32_t)(on ? pos : -1), (uint32_t)s, (uint32_t)pos, (uint32_t)pos};
        if (!parked && !in) state[4 * s + 3] |= 64;
    }
    embed_row(table, tok, vocab, dim, ld, x + (size_t)s * ld, h + (size_t)s * ld);
}

struct RbNorm {
    const void* z;
    const float* res;
    const int32_t* rows;
    const void* w;
    float* x_out;
    void* h_out;
    long long ld;
    float alpha, eps;
    int dim, top;
};
// VPT float4 columns per thread held in registers (ld <= 4 VPT blockDim); in place on z / res is fine: a thread reads its columns before it writes them
template <class T, int VPT>
__global__ void __launch_bounds__(256) rb_norm_kernel(const RbNorm a) {
    const int t = blockIdx.x, src = a.rows ? a.rows[t] : t, nt = blockDim.x;
    f32x4 v[VPT];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * ((int)threadIdx.x + i * nt);
        v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (c < a.ld) {
            if (a.res) {
                const f32x4 r = rb_ld4(a.res + (size_t)src * a.ld + c);
                f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
                for (int j = 0; j < a.top; j++) s += rb_ld4(reinterpret_cast<const T*>(a.z) + ((size_t)src * a.top + j) * a.ld + c);
#pragma unroll
                for (int j = 0; j < 4; j++) v[i][j] = fmaf(a.alpha, r[j], s[j]);
            } else {
                v[i] = rb_ld4(reinterpret_cast<const float*>(a.z) + (size_t)src * a.ld + c);
            }
#pragma unroll
            for (int j = 0; j < 4; j++) { /* pad columns do not count, whatever they hold */
                if (c + j >= a.dim) v[i][j] = 0.f;
                ss = fmaf(v[i][j], v[i][j], ss);
            }
        }
    }
    __shared__ float red[4];
    ss = wave_sum(ss);
    if (nt > 64) {
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        __syncthreads();
        ss = 0.f;
        for (int w = 0; w < nt / 64; w++) ss += red[w];
    }
    const float rs = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
    const T* w = reinterpret_cast<const T*>(a.w);
    T* h = reinterpret_cast<T*>(a.h_out);
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * ((int)threadIdx.x + i * nt);
        if (c < a.ld) {
            const f32x4 g = rb_ld4(w + c);
            f32x4 o;
#pragma unroll
            for (int j = 0; j < 4; j++) o[j] = v[i][j] * rs * g[j];
            if (a.x_out) rb_st4(a.x_out + (size_t)t * a.ld + c, o);
            rb_st4(h + (size_t)t * a.ld + c, o);
        }
    }
}
template <class T>
static int norm_go(hipStream_t st, const RbNorm& a, int n) {
    const int quads = (int)(a.ld / 4);
    int nt = (quads + 63) / 64 * 64;
    nt = nt > 256 ? 256 : nt;
    const int vpt = (quads + nt - 1) / nt;
    if (vpt <= 1) hipLaunchKernelGGL((rb_norm_kernel<T, 1>), dim3(n), dim3(nt), 0, st, a);
    else if (vpt <= 2) hipLaunchKernelGGL((rb_norm_kernel<T, 2>), dim3(n), dim3(nt), 0, st, a);
    else if (vpt <= 4) hipLaunchKernelGGL((rb_norm_kernel<T, 4>), dim3(n), dim3(nt), 0, st, a);
    else if (vpt <= 8) hipLaunchKernelGGL((rb_norm_kernel<T, 8>), dim3(n), dim3(nt), 0, st, a);
    else if (vpt <= 16) hipLaunchKernelGGL((rb_norm_kernel<T, 16>), dim3(n), dim3(nt), 0, st, a);
    else return 1;
    return KF_OK;
}

// the sum over a workgroup of up to 256 threads; red: 4 floats of LDS that no earlier sum still uses
__device__ __forceinline__ float group_sum(float v, float* red, int nt) {
    v = wave_sum(v);
    if (nt > 64) {
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
        __syncthreads();
        v = 0.f;
        for (int w = 0; w < nt / 64; w++) v += red[w];
    }
    return v;
}
// kf_rb_norm_rows: VPT float4 columns per thread in registers, as above; the LAYER kind takes the mean off first (two sums, no difference of large numbers)
template <class T, int VPT>
__global__ void __launch_bounds__(256) rb_norm_rows_kernel(const kf_rb_norming a) {
    __shared__ float red[2][4];
    const int t = blockIdx.x, src = a.rows ? a.rows[t] : t, nt = blockDim.x;
    f32x4 v[VPT];
    float s = 0.f;
    const float *hi = nullptr, *lo = nullptr;
    if (a.pos_hi) {
        const int p = a.meta[KF_RB_META * src], pos = p > 0 ? p : 0; /* (an inactive row: whatever) */
        hi = a.pos_hi + (size_t)(pos >> 6) * a.ld, lo = a.pos_lo + (size_t)(pos & 63) * a.ld;
    }
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * ((int)threadIdx.x + i * nt);
        v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (c < a.ld) {
            v[i] = rb_ld4(a.z + (size_t)src * a.ld + c);
            if (hi) { /* two (sin, cos) pairs of each factor */
                const f32x4 p = rb_ld4(hi + c), q = rb_ld4(lo + c);
                v[i].x += p.x * q.y + p.y * q.x, v[i].y += p.y * q.y - p.x * q.x;
                v[i].z += p.z * q.w + p.w * q.z, v[i].w += p.w * q.w - p.z * q.z;
            }
#pragma unroll
            for (int j = 0; j < 4; j++) {
                if (c + j >= a.dim) v[i][j] = 0.f;
                s += v[i][j];
            }
        }
    }
    float mean = 0.f, ss = 0.f;
    if (a.kind == KF_RB_LAYER) mean = group_sum(s, red[0], nt) / (float)a.dim;
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * ((int)threadIdx.x + i * nt);
#pragma unroll
        for (int j = 0; j < 4; j++) {
            v[i][j] = c + j < a.dim ? v[i][j] - mean : 0.f;
            ss = fmaf(v[i][j], v[i][j], ss);
        }
    }
    const float rs = 1.0f / sqrtf(group_sum(ss, red[1], nt) / (float)a.dim + a.eps);
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * ((int)threadIdx.x + i * nt);
        if (c < a.ld) {
            const f32x4 g = rb_ld4(reinterpret_cast<const T*>(a.w) + c);
            f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
            if (a.add) o = rb_ld4(a.add + (size_t)src * a.ld + c);
#pragma unroll
            for (int j = 0; j < 4; j++) o[j] = c + j < a.dim ? o[j] + v[i][j] * rs * g[j] : 0.f;
            if (a.x_out) rb_st4(a.x_out + (size_t)t * a.ld + c, o);
            if (a.h_out) rb_st4(reinterpret_cast<T*>(a.h_out) + (size_t)t * a.ld + c, o);
        }
    }
}
template <class T>
static int norm_rows_go(hipStream_t st, const kf_rb_norming& a) {
    const int quads = (int)(a.ld / 4);
    int nt = (quads + 63) / 64 * 64;
    nt = nt > 256 ? 256 : nt;
    const int vpt = (quads + nt - 1) / nt;
    if (vpt <= 1) hipLaunchKernelGGL((rb_norm_rows_kernel<T, 1>), dim3(a.n), dim3(nt), 0, st, a);
    else if (vpt <= 2) hipLaunchKernelGGL((rb_norm_rows_kernel<T, 2>), dim3(a.n), dim3(nt), 0, st, a);
    else if (vpt <= 4) hipLaunchKernelGGL((rb_norm_rows_kernel<T, 4>), dim3(a.n), dim3(nt), 0, st, a);
    else if (vpt <= 8) hipLaunchKernelGGL((rb_norm_rows_kernel<T, 8>), dim3(a.n), dim3(nt), 0, st, a);
    else if (vpt <= 16) hipLaunchKernelGGL((rb_norm_rows_kernel<T, 16>), dim3(a.n), dim3(nt), 0, st, a);
    else return 1;
    return KF_OK;
}

// ---- router: one wave per row; expert e sits in lane e % 64, register e / 64
constexpr int RB_MAX_EXPERTS = 1024;
struct RbRoute {
    const float* logits;
    const void* bias;
    const int32_t* meta;
    int32_t *ids, *tile_expert, *list;
    float* weight;
    long long ld;
    int n, n_expert, top, tile, n_tile;
};
template <class T, int NV> /* NV registers of 64 experts */
__device__ __forceinline__ void rb_topk_row(const RbRoute& a, int t, int lane) {
    const float* logits = a.logits;
    const T* bias = reinterpret_cast<const T*>(a.bias);
    const int32_t* meta = a.meta;
    int32_t* ids = a.ids;
    float* weight = a.weight;
    const long long ld = a.ld;
    const int n_expert = a.n_expert, top = a.top;
    if (meta && meta[KF_RB_META * t] < 0) {
        for (int j = lane; j < top; j += 64) ids[(size_t)t * top + j] = -1, weight[(size_t)t * top + j] = 0.f;
        return;
    }
    float v[NV];
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const int e = lane + 64 * i;
        v[i] = -__builtin_inff();
        if (e < n_expert) v[i] = logits[(size_t)t * ld + e] + (bias ? rb_ld(bias + e) : 0.f);
    }
    float best0 = 0.f, sum = 0.f, my_p = 0.f;
    int my_id = -1; /* choice j sits in lane j % 64 */
    auto flush = [&](int j0, int j1, float scale) {
        if (lane < j1 - j0) ids[(size_t)t * top + j0 + lane] = my_id, weight[(size_t)t * top + j0 + lane] = my_p * scale;
    };
    for (int j = 0; j < top; j++) {
        float m = v[0];
#pragma unroll
        for (int i = 1; i < NV; i++) m = fmaxf(m, v[i]);
        const float wm = wave_max(m);
        int cand = -1; /* ties: the lower expert.  NaN logits: none */
#pragma unroll
        for (int i = NV - 1; i >= 0; i--) {
            const unsigned long long on = __ballot(v[i] == wm && lane + 64 * i < n_expert);
            if (on) cand = 64 * i + __ffsll((long long)on) - 1;
        }
        if (j == 0) best0 = wm;
        const float p = expf(wm - best0);
        sum += p;
        if (lane == (j & 63)) my_p = p, my_id = cand;
#pragma unroll
        for (int i = 0; i < NV; i++)
            if (lane + 64 * i == cand) v[i] = -__builtin_inff();
        if ((j & 63) == 63 && j + 1 < top) flush(j - 63, j + 1, 1.f);
    }
    const float inv = 1.0f / sum;
    flush((top - 1) & ~63, top, inv);
    for (int j = lane; j < ((top - 1) & ~63); j += 64) weight[(size_t)t * top + j] *= inv; /* (more than 64 choices: a lane reads back what it wrote) */
}
template <class T, int NV>
__global__ void __launch_bounds__(256) rb_topk_kernel(const RbRoute a) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < a.n) rb_topk_row<T, NV>(a, t, threadIdx.x & 63);
}
// ---- pairs grouped by expert, one workgroup: count, tile-aligned offsets, fill
__device__ __forceinline__ void rb_list(const RbRoute& a) {
    __shared__ int cnt[RB_MAX_EXPERTS], off[RB_MAX_EXPERTS];
    const int32_t* ids = a.ids;
    int32_t *tile_expert = a.tile_expert, *list = a.list;
    const int n_pair = a.n * a.top, n_expert = a.n_expert, tile = a.tile, n_tile = a.n_tile;
    const int tid = threadIdx.x, nt = blockDim.x;
    for (int e = tid; e < n_expert; e += nt) cnt[e] = 0;
    for (int i = tid; i < n_tile; i += nt) tile_expert[i] = -1;
    for (int i = tid; i < n_tile * tile; i += nt) list[i] = -1;
    __syncthreads();
    for (int i = tid; i < n_pair; i += nt) {
        const int e = ids[i];
        if (e >= 0) atomicAdd(&cnt[e], 1);
    }
    __syncthreads();
    if (tid < 64) { /* exclusive scan of the tile counts, 64 experts at a time */
        int base = 0;
        for (int e0 = 0; e0 < n_expert; e0 += 64) {
            const int e = e0 + tid, nte = e < n_expert ? (cnt[e] + tile - 1) / tile : 0;
            int inc = nte;
            for (int o = 1; o < 64; o <<= 1) {
                const int u = __shfl_up(inc, o, 64);
                if (tid >= o) inc += u;
            }
            if (e < n_expert) off[e] = base + inc - nte;
            base += __shfl(inc, 63, 64);
        }
    }
    __syncthreads();
    for (int e = tid; e < n_expert; e += nt) {
        const int nte = (cnt[e] + tile - 1) / tile;
        for (int i = 0; i < nte; i++)
            if (off[e] + i < n_tile) tile_expert[off[e] + i] = e;
        cnt[e] = 0;
    }
    __syncthreads();
    for (int i = tid; i < n_pair; i += nt) {
        const int e = ids[i];
        if (e < 0) continue;
        const int p = off[e] * tile + atomicAdd(&cnt[e], 1);
        if (p < n_tile * tile) list[p] = i;
    }
}
__global__ void __launch_bounds__(1024) rb_list_kernel(const RbRoute a) { rb_list(a); }
/* a decode batch: both in one workgroup */
template <class T, int NV>
__global__ void __launch_bounds__(1024) rb_route_kernel(const RbRoute a) {
    for (int t = threadIdx.x >> 6; t < a.n; t += (int)blockDim.x >> 6) rb_topk_row<T, NV>(a, t, threadIdx.x & 63);
    __threadfence_block();
    __syncthreads();
    rb_list(a);
}
template <class T, int NV>
static void route_nv(hipStream_t st, const RbRoute& a) {
    if (a.n <= KF_RB_DECODE_MAX) {
        hipLaunchKernelGGL((rb_route_kernel<T, NV>), dim3(1), dim3(a.n <= 4 ? 256 : 1024), 0, st, a);
        return;
    }
    hipLaunchKernelGGL((rb_topk_kernel<T, NV>), dim3((a.n + 3) / 4), dim3(256), 0, st, a);
    hipLaunchKernelGGL(rb_list_kernel, dim3(1), dim3(1024), 0, st, a);
}
template <class T>
static void route_go(hipStream_t st, const RbRoute& a) {
    if (a.n_expert <= 64) route_nv<T, 1>(st, a);
    else if (a.n_expert <= 128) route_nv<T, 2>(st, a);
    else if (a.n_expert <= 256) route_nv<T, 4>(st, a);
    else route_nv<T, RB_MAX_EXPERTS / 64>(st, a);
}

// ---- greedy pick: maxima of PICK_SPAN-wide pieces, then the first maximum over the pieces
constexpr int PICK_SPAN = 4096, PICK_PIECES = 256;
__global__ void __launch_bounds__(256) rb_pick_part_kernel(const float* __restrict__ logits, long long ld, int vocab, int span, float* __restrict__ pv, int* __restrict__ pi) {
    const float* row = logits + (size_t)blockIdx.y * ld;
    const int lo = blockIdx.x * span, hi = lo + span < vocab ? lo + span : vocab;
    float m = -__builtin_inff();
    int idx = 0x7fffffff;
    for (int i = lo + (int)threadIdx.x; i < hi; i += 256) {
        const float v = row[i];
        if (v > m || idx == 0x7fffffff) m = v, idx = i;
    }
    for (int o = 32; o > 0; o >>= 1) {
        const float om = __shfl_xor(m, o, 64);
        const int oi = __shfl_xor(idx, o, 64);
        if (om > m || (om == m && oi < idx)) m = om, idx = oi;
    }
    __shared__ float sm[4];
    __shared__ int si[4];
    if ((threadIdx.x & 63) == 0) sm[threadIdx.x >> 6] = m, si[threadIdx.x >> 6] = idx;
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 4; w++)
            if (sm[w] > m || (sm[w] == m && si[w] < idx)) m = sm[w], idx = si[w];
        pv[blockIdx.y * PICK_PIECES + blockIdx.x] = m, pi[blockIdx.y * PICK_PIECES + blockIdx.x] = idx;
    }
}
__global__ void __launch_bounds__(64) rb_pick_finish_kernel(const float* __restrict__ pv, const int* __restrict__ pi, int pieces, int vocab, const int32_t* __restrict__ meta,
                                                            int32_t* __restrict__ state, int32_t* __restrict__ tokens_out, int tokens_stride) {
    const int r = blockIdx.x, pos = meta[KF_RB_META * r];
    if (pos < 0) return;
    float m = -__builtin_inff();
    int idx = 0x7fffffff;
    for (int i = threadIdx.x; i < pieces; i += 64) {
        const float v = pv[r * PICK_PIECES + i];
        const int j = pi[r * PICK_PIECES + i];
        if (v > m || (v == m && j < idx)) m = v, idx = j;
    }
    for (int o = 32; o > 0; o >>= 1) {
        const float om = __shfl_xor(m, o, 64);
        const int oi = __shfl_xor(idx, o, 64);
        if (om > m || (om == m && oi < idx)) m = om, idx = oi;
    }
    if (threadIdx.x == 0) {
        idx = idx < vocab ? idx : 0; /* every logit NaN: id 0 */
        const int s = meta[KF_RB_META * r + 1];
        if (tokens_out) tokens_out[(size_t)s * tokens_stride + pos] = idx;
        state[4 * s] = idx, state[4 * s + 1] = pos + 1;
    }
}
__global__ void __launch_bounds__(256) rb_to_bf16_kernel(const float* __restrict__ src, uint16_t* __restrict__ dst, size_t n) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) dst[i] = f2bf(src[i]);
}

template <class T>
__global__ void __launch_bounds__(256) rb_pack_kernel(const uint16_t* __restrict__ src, int cols, T* __restrict__ dst, long long ld, int row0, int half, int tiled) {
    const int r = blockIdx.x;
    const size_t d = half < 0 ? (size_t)row0 + r : (size_t)(32 * (r / 16) + 16 * half + r % 16);
    for (int i = threadIdx.x; i < cols; i += 256) {
        const size_t at = tiled ? ((d / 16) * (ld / 32) + i / 32) * 512 + (d % 16 + 16 * ((i % 32) / 8)) * 8 + i % 8 : d * ld + i;
        rb_st(dst + at, bf2f(src[(size_t)r * cols + i]));
    }
}

}  // namespace kf

using namespace kf;
static bool type_ok(int type) { return type == KF_BF16 || type == KF_F32; }
static int launched(const char* who) { return hipGetLastError() == hipSuccess ? KF_OK : abi_fail(KF_HIP_CHECK, "%s: launch failed", who); }

extern "C" {

int kf_rb_embed(kf_ctx* c, int type, const void* table, int vocab, int dim, int64_t ldx, const int32_t* tokens, int n, float* x, void* h) {
    CHKCTX(c);
    if (!type_ok(type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_embed: storage %d", type);
    if (!table || !tokens || !x || !h || vocab < 1 || dim < 1 || ldx < dim || ldx % KF_RB_PAD || n < 1) return abi_fail(KF_INVALID_ARGS, "kf_rb_embed: bad arguments");
    if (!al16(table) || !al16(x) || !al16(h)) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_embed: unaligned pointer");
    const int nt = ldx >= 1024 ? 256 : 64;
    if (type == KF_BF16) hipLaunchKernelGGL(rb_embed_kernel<uint16_t>, dim3(n), dim3(nt), 0, c->stream, (const uint16_t*)table, vocab, dim, (long long)ldx, tokens, x, (uint16_t*)h);
    else hipLaunchKernelGGL(rb_embed_kernel<float>, dim3(n), dim3(nt), 0, c->stream, (const float*)table, vocab, dim, (long long)ldx, tokens, x, (float*)h);
    return launched("kf_rb_embed");
}
int kf_rb_embed_state(kf_ctx* c, int type, const void* table, int vocab, int dim, int64_t ldx, int32_t* d_state, const int32_t* d_forced, int forced_stride, int max_pos, int n,
                      float* x, void* h, int32_t* meta) {
    CHKCTX(c);
    if (!type_ok(type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_embed_state: storage %d", type);
    if (!table || !d_state || !x || !h || !meta || vocab < 1 || dim < 1 || ldx < dim || ldx % KF_RB_PAD || n < 1 || max_pos < 1 || (d_forced && n > 1 && forced_stride < max_pos))
        return abi_fail(KF_INVALID_ARGS, "kf_rb_embed_state: bad arguments");
    if (!al16(table) || !al16(x) || !al16(h) || !al16(meta)) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_embed_state: unaligned pointer");
    const int nt = ldx >= 1024 ? 256 : 64;
    if (type == KF_BF16)
        hipLaunchKernelGGL(rb_embed_state_kernel<uint16_t>, dim3(n), dim3(nt), 0, c->stream, (const uint16_t*)table, vocab, dim, (long long)ldx, d_state, d_forced, forced_stride, max_pos, x,
                           (uint16_t*)h, meta);
    else
        hipLaunchKernelGGL(rb_embed_state_kernel<float>, dim3(n), dim3(nt), 0, c->stream, (const float*)table, vocab, dim, (long long)ldx, d_state, d_forced, forced_stride, max_pos, x,
                           (float*)h, meta);
    return launched("kf_rb_embed_state");
}
int kf_rb_norm(kf_ctx* c, int type, const void* z, const float* res, float alpha, int top, const void* w, float eps, int dim, int64_t ld, int n, const int32_t* rows, float* x_out,
               void* h_out) {
    CHKCTX(c);
    if (!type_ok(type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_norm: storage %d", type);
    if (!z || !w || !h_out || dim < 1 || ld < dim || ld % KF_RB_PAD || n < 1 || (res && top < 1)) return abi_fail(KF_INVALID_ARGS, "kf_rb_norm: bad arguments");
    if (!al16(z) || (res && !al16(res)) || !al16(w) || (x_out && !al16(x_out)) || !al16(h_out)) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_norm: unaligned pointer");
    RbNorm a{z, res, rows, w, x_out, h_out, (long long)ld, alpha, eps, dim, top};
    const int rc = type == KF_BF16 ? norm_go<uint16_t>(c->stream, a, n) : norm_go<float>(c->stream, a, n);
    if (rc) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_norm: rows of %d columns (served: up to 16384)", dim);
    return launched("kf_rb_norm");
}
int kf_rb_norm_rows(kf_ctx* c, const kf_rb_norming* a) {
    CHKCTX(c);
    if (!a || !a->z || !a->w || (!a->x_out && !a->h_out) || a->dim < 1 || a->ld < a->dim || a->ld % KF_RB_PAD || a->n < 1 || a->kind < KF_RB_RMS || a->kind > KF_RB_LAYER)
        return abi_fail(KF_INVALID_ARGS, "kf_rb_norm_rows: bad arguments");
    if (!type_ok(a->type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_norm_rows: storage %d", a->type);
    if (a->pos_hi && (!a->pos_lo || !a->meta || !al16(a->pos_hi) || !al16(a->pos_lo))) return abi_fail(KF_INVALID_ARGS, "kf_rb_norm_rows: positions");
    if (!al16(a->z) || (a->add && !al16(a->add)) || !al16(a->w) || (a->x_out && !al16(a->x_out)) || (a->h_out && !al16(a->h_out))) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_norm_rows: unaligned pointer");
    const int rc = a->type == KF_BF16 ? norm_rows_go<uint16_t>(c->stream, *a) : norm_rows_go<float>(c->stream, *a);
    if (rc) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_norm_rows: rows of %d columns (served: up to 16384)", a->dim);
    return launched("kf_rb_norm_rows");
}
int kf_rb_sinusoid_tables_host(float* hi, float* lo, int n_pos, int width, int64_t ld, double base) {
    if (!hi || !lo || n_pos < 1 || width < 1 || ld < width || (ld & 1) || !(base > 0)) return abi_fail(KF_INVALID_ARGS, "kf_rb_sinusoid_tables_host: bad arguments");
    for (int64_t i = 0; i < ld / 2; i++) {
        const double f = 2 * i < width ? pow(base, -2.0 * (double)i / width) : 0.0;
        for (int j = 0; j < (n_pos + 63) / 64; j++) hi[j * ld + 2 * i] = (float)sin(64.0 * j * f), hi[j * ld + 2 * i + 1] = (float)cos(64.0 * j * f);
        for (int j = 0; j < 64; j++) lo[j * ld + 2 * i] = (float)sin(j * f), lo[j * ld + 2 * i + 1] = (float)cos(j * f);
    }
    return KF_OK;
}
int kf_rb_list_tiles(int n, int top, int n_expert, int tile) {
    if (n < 1 || top < 1 || n_expert < 1 || tile < 1) return 0;
    const long long pairs = (long long)n * top, part = pairs < n_expert ? pairs : n_expert;
    return (int)(pairs / tile + part);
}
int kf_rb_route(kf_ctx* c, int type, const float* logits, int64_t ld, const void* bias, int n, const int32_t* meta, const kf_rb_experts* e) {
    CHKCTX(c);
    if (!type_ok(type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_route: storage %d", type);
    if (!logits || !e || n < 1 || e->n_expert < 1 || ld < e->n_expert || e->top < 1 || e->top > e->n_expert || e->tile < 1 || !e->tile_expert || !e->list || !e->ids || !e->weight)
        return abi_fail(KF_INVALID_ARGS, "kf_rb_route: bad arguments");
    if (e->n_expert > RB_MAX_EXPERTS) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_route: %d experts (served: up to %d)", e->n_expert, RB_MAX_EXPERTS);
    if (e->n_tile < kf_rb_list_tiles(n, e->top, e->n_expert, e->tile)) return abi_fail(KF_INVALID_ARGS, "kf_rb_route: the list has %d tiles", e->n_tile);
    RbRoute a{logits, bias, meta, const_cast<int32_t*>(e->ids), const_cast<int32_t*>(e->tile_expert), const_cast<int32_t*>(e->list), const_cast<float*>(e->weight), (long long)ld, n,
              e->n_expert, e->top, e->tile, e->n_tile};
    if (type == KF_BF16) route_go<uint16_t>(c->stream, a);
    else route_go<float>(c->stream, a);
    return launched("kf_rb_route");
}
size_t kf_rb_pick_scratch(int n) { return n < 1 ? 0 : (size_t)n * PICK_PIECES * 8; }
int kf_rb_pick(kf_ctx* c, const float* logits, int64_t ld, int vocab, int n, const int32_t* meta, int32_t* d_state, int32_t* d_tokens_out, int tokens_stride, void* scratch) {
    CHKCTX(c);
    if (!logits || !meta || !d_state || !scratch || vocab < 1 || ld < vocab || n < 1) return abi_fail(KF_INVALID_ARGS, "kf_rb_pick: bad arguments");
    int span = PICK_SPAN;
    while ((vocab + span - 1) / span > PICK_PIECES) span *= 2;
    const int pieces = (vocab + span - 1) / span;
    float* pv = (float*)scratch;
    int* pi = (int*)(pv + (size_t)n * PICK_PIECES);
    hipLaunchKernelGGL(rb_pick_part_kernel, dim3(pieces, n), dim3(256), 0, c->stream, logits, (long long)ld, vocab, span, pv, pi);
    hipLaunchKernelGGL(rb_pick_finish_kernel, dim3(n), dim3(64), 0, c->stream, pv, pi, pieces, vocab, meta, d_state, d_tokens_out, tokens_stride);
    return launched("kf_rb_pick");
}
int kf_rb_pack(kf_ctx* c, int type, const kf_bf16* src, int rows, int cols, void* dst, int64_t ld, int row0, int half, int tiled) {
    CHKCTX(c);
    if (!type_ok(type)) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_pack: storage %d", type);
    if (!src || !dst || rows < 1 || cols < 1 || ld < cols || row0 < 0 || half > 1 || (tiled && (type != KF_BF16 || ld % KF_RB_PAD))) return abi_fail(KF_INVALID_ARGS, "kf_rb_pack: bad arguments");
    if (type == KF_BF16) hipLaunchKernelGGL(rb_pack_kernel<uint16_t>, dim3(rows), dim3(256), 0, c->stream, src, cols, (uint16_t*)dst, (long long)ld, row0, half, tiled);
    else hipLaunchKernelGGL(rb_pack_kernel<float>, dim3(rows), dim3(256), 0, c->stream, src, cols, (float*)dst, (long long)ld, row0, half, 0);
    return launched("kf_rb_pack");
}
int kf_rb_to_bf16(kf_ctx* c, const float* src, kf_bf16* dst, size_t n) {
    CHKCTX(c);
    if (!src || !dst || n < 1) return abi_fail(KF_INVALID_ARGS, "kf_rb_to_bf16: bad arguments");
    const size_t blocks = (n + 255) / 256;
    hipLaunchKernelGGL(rb_to_bf16_kernel, dim3((unsigned)(blocks < 1024 ? blocks : 1024)), dim3(256), 0, c->stream, src, dst, n);
    return launched("kf_rb_to_bf16");
}
int kf_rb_rope_table_host(float* t, int n_pos, int dims, double base, double factor, double low, double high, double original) {
    if (!t || n_pos < 1 || dims < 2 || (dims & 1) || !(base > 0) || !(factor > 0)) return abi_fail(KF_INVALID_ARGS, "kf_rb_rope_table_host: bad arguments");
    const double two_pi = 6.283185307179586476925286766559;
    const int half = dims / 2;
    for (int i = 0; i < half; i++) {
        double f = pow(base, -2.0 * i / dims);
        if (factor != 1.0) {
            const double turns = original * f / two_pi;
            const double t = turns >= high ? 1.0 : (turns <= low ? 0.0 : (turns - low) / (high - low));
            f *= t + (1.0 - t) / factor;
        }
        for (int p = 0; p < n_pos; p++) t[((size_t)p * half + i) * 2] = (float)cos(p * f), t[((size_t)p * half + i) * 2 + 1] = (float)sin(p * f);
    }
    return KF_OK;
}

}  // extern "C"
