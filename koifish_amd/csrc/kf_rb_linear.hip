// kf_rb_linear.hip -- row-batch products y[t][m] = W[m] . x[t] for few rows (decode batches) and in 32-bit, and the ABI entry that picks the form.
//
// Decode batches stream the weights: a workgroup owns 16 weight rows (GATED: 16 gate and the 16 up rows that follow them), its waves take the 32-deep k-steps round robin --
// a wave instruction reads 16 rows x 64 contiguous bytes -- and multiply them against up to 64 token columns by v_mfma_f32_16x16x32_bf16 (A = weight rows, B = token rows,
// straight from global memory: the activations of a decode batch are a few KB and stay in L2).  The waves' partial tiles meet in LDS, one thread per output finishes it.
// With experts a workgroup's columns are the pairs of one expert (UP), or it walks every chosen expert with the columns that did not choose it held at zero (SUM): an
// expert's rows are read once per workgroup whoever chose them.
#include "kf_ctx.h"
#include "kf_rb_common.h"

namespace kf {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x4 rb_mfma16(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// k-steps wid, wid + NW, ... of the MG 16-row blocks at w (row stride k) against NT column blocks; xp[nt] = this lane's token row + 8 (lane >> 4), NULL: a zero column
template <int NT, int MG, int NW>
__device__ __forceinline__ void rb_stream_k(const uint16_t* __restrict__ w, int k, const uint16_t* const (&xp)[NT], f32x4 (&acc)[MG][NT], int wid, int lane) {
    const int r16 = lane & 15, q4 = lane >> 4, nstep = k / 32;
    const uint16_t* wr = w + (size_t)r16 * k + 8 * q4;
    constexpr int U = NT >= 4 ? 2 : 4; /* steps in flight */
    for (int s0 = wid; s0 < nstep; s0 += NW * U) {
        u32x4 a[U][MG], b[U][NT];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int s = s0 + u * NW;
            const bool on = s < nstep; /* wave-uniform */
#pragma unroll
            for (int g = 0; g < MG; g++) {
                a[u][g] = u32x4{0, 0, 0, 0};
                if (on) a[u][g] = ld_nt(reinterpret_cast<const u32x4*>(wr + (size_t)g * 16 * k + 32 * s));
            }
#pragma unroll
            for (int t = 0; t < NT; t++) {
                b[u][t] = u32x4{0, 0, 0, 0};
                if (on && xp[t]) b[u][t] = *reinterpret_cast<const u32x4*>(xp[t] + 32 * s);
            }
        }
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int g = 0; g < MG; g++)
#pragma unroll
                for (int t = 0; t < NT; t++) acc[g][t] = rb_mfma16(a[u][g], b[u][t], acc[g][t]);
    }
}

template <int NT, bool GATED, int NW>
__global__ void __launch_bounds__(64 * NW) rb_stream_kernel(const RbProduct q) {
    const kf_rb_product& p = q.p;
    constexpr int MG = GATED ? 2 : 1, COLS = 16 * NT;
    __shared__ float red[NW][MG][COLS][17]; /* [wave][block][column][row], padded */
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r16 = lane & 15, q4 = lane >> 4;
    const int m0 = blockIdx.x * (16 * MG);
    const uint16_t* W = reinterpret_cast<const uint16_t*>(p.w);
    const uint16_t* X = reinterpret_cast<const uint16_t*>(p.x);
    f32x4 acc[MG][NT];
#pragma unroll
    for (int g = 0; g < MG; g++)
#pragma unroll
        for (int t = 0; t < NT; t++) acc[g][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint16_t* xp[NT];
    const int32_t* list = nullptr;
    if (p.mode == KF_RB_SUM) {
        int last = -1;
        for (int i = 0; i < q.e.n_tile; i++) {
            const int ex = q.e.tile_expert[i];
            if (ex < 0) break;
            if (ex == last) continue; /* an expert with more pairs than a tile holds: its tiles follow each other */
            last = ex;
#pragma unroll
            for (int t = 0; t < NT; t++) {
                const int row = t * 16 + r16;
                xp[t] = nullptr;
                if (row < p.n)
                    for (int j = 0; j < q.e.top; j++)
                        if (q.e.ids[row * q.e.top + j] == ex) xp[t] = X + (size_t)(row * q.e.top + j) * p.ldx + 8 * q4;
            }
            rb_stream_k<NT, MG, NW>(W + (size_t)ex * q.e.w_stride + (size_t)m0 * p.k, p.k, xp, acc, wid, lane);
        }
    } else {
        if (p.mode != KF_RB_ALL) {
            const int ex = q.e.tile_expert[blockIdx.y];
            if (ex < 0) return;
            W += (size_t)ex * q.e.w_stride;
            list = q.e.list + (size_t)blockIdx.y * q.e.tile;
        }
#pragma unroll
        for (int t = 0; t < NT; t++) {
            const int col = t * 16 + r16;
            xp[t] = nullptr;
            if (list) {
                const int pair = list[col];
                if (pair >= 0) xp[t] = X + (size_t)(p.mode == KF_RB_UP ? pair / q.e.top : pair) * p.ldx + 8 * q4;
            } else if (col < p.n) {
                xp[t] = X + (size_t)col * p.ldx + 8 * q4;
            }
        }
        rb_stream_k<NT, MG, NW>(W + (size_t)m0 * p.k, p.k, xp, acc, wid, lane);
    }
#pragma unroll
    for (int g = 0; g < MG; g++)
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int j = 0; j < 4; j++) red[wid][g][t * 16 + r16][4 * q4 + j] = acc[g][t][j];
    __syncthreads();
    for (int i = tid; i < COLS * 16; i += 64 * NW) {
        const int row = i & 15, col = i >> 4;
        int yr = col;
        float scale = 1.f;
        if (list) {
            yr = list[col];
            if (yr < 0) continue;
            if (p.mode == KF_RB_UP) scale = q.e.weight[yr];
        } else if (col >= p.n) {
            continue;
        }
        float d = 0.f;
#pragma unroll
        for (int w = 0; w < NW; w++) d += red[w][0][col][row];
        if constexpr (GATED) {
            float u = 0.f;
#pragma unroll
            for (int w = 0; w < NW; w++) u += red[w][MG - 1][col][row];
            reinterpret_cast<uint16_t*>(p.y)[(size_t)yr * p.ldy + (m0 >> 1) + row] = f2bf(scale * (rb_activate(p.act, d) * u));
        } else if (p.epilogue == KF_RB_STORE) {
            reinterpret_cast<uint16_t*>(p.y)[(size_t)yr * p.ldy + m0 + row] = f2bf(d);
        } else if (p.epilogue == KF_RB_STORE_F32) {
            reinterpret_cast<float*>(p.y)[(size_t)yr * p.ldy + m0 + row] = d;
        } else {
            reinterpret_cast<float*>(p.y)[(size_t)yr * p.ldy + m0 + row] = fmaf(p.alpha, p.res[(size_t)yr * p.ldr + m0 + row], d);
        }
    }
}
template <int NT, int NW>
static void stream_go(hipStream_t st, const RbProduct& q, dim3 grid) {
    if (q.p.epilogue == KF_RB_GATED) hipLaunchKernelGGL((rb_stream_kernel<NT, true, NW>), grid, dim3(64 * NW), 0, st, q);
    else hipLaunchKernelGGL((rb_stream_kernel<NT, false, NW>), grid, dim3(64 * NW), 0, st, q);
}
int rb_stream_launch(hipStream_t st, const RbProduct& q) {
    const kf_rb_product& p = q.p;
    const bool tiles = p.mode == KF_RB_UP || p.mode == KF_RB_DOWN;
    const int cols = tiles ? q.e.tile : p.n, nt = (cols + 15) / 16;
    if (nt > 4 || (tiles && q.e.tile % 16)) return 1;
    dim3 grid(p.m / (p.epilogue == KF_RB_GATED ? 32 : 16), tiles ? q.e.n_tile : 1);
    const bool wide = (long)grid.x * grid.y < 768 && p.k >= 512; /* few workgroups: more waves each, more loads in flight per CU */
    switch (nt) {
        case 1: wide ? stream_go<1, 8>(st, q, grid) : stream_go<1, 4>(st, q, grid); break;
        case 2: wide ? stream_go<2, 8>(st, q, grid) : stream_go<2, 4>(st, q, grid); break;
        case 3: stream_go<3, 4>(st, q, grid); break;
        default: stream_go<4, 4>(st, q, grid); break;
    }
    return KF_OK;
}

// ---- the 32-bit product: 64 x 64 outputs per workgroup, k in steps of 16 through LDS, 4 x 4 outputs per thread, fp32 fma chains in k order
__global__ void __launch_bounds__(256) rb_f32_kernel(const RbProduct q) {
    const kf_rb_product& p = q.p;
    constexpr int KT = 16;
    __shared__ float sw[KT][68], sx[KT][68];
    __shared__ int srow[64], sdst[64];
    const int tid = threadIdx.x, m0 = blockIdx.x * 64, c0 = blockIdx.y * 64;
    const float* W = reinterpret_cast<const float*>(p.w);
    const float* X = reinterpret_cast<const float*>(p.x);
    const bool ex_mode = p.mode != KF_RB_ALL;
    if (ex_mode) {
        const int ex = q.e.tile_expert[blockIdx.y];
        if (ex < 0) return;
        W += (size_t)ex * q.e.w_stride;
    }
    if (tid < 64) {
        int src, dst;
        if (ex_mode) {
            dst = q.e.list[(size_t)blockIdx.y * 64 + tid];
            src = dst < 0 ? -1 : (p.mode == KF_RB_UP ? dst / q.e.top : dst);
        } else {
            dst = src = c0 + tid < p.n ? c0 + tid : -1;
        }
        srow[tid] = src, sdst[tid] = dst;
    }
    __syncthreads();
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) acc[i][j] = 0.f;
    const int lr = tid >> 2, lk = (tid & 3) * 4; /* staging: row lr, four k */
    const int tm = (tid & 15) * 4, tc = (tid >> 4) * 4;
    const int xr = srow[lr];
    for (int k0 = 0; k0 < p.k; k0 += KT) {
        const f32x4 wv = *reinterpret_cast<const f32x4*>(W + (size_t)(m0 + lr) * p.k + k0 + lk);
        f32x4 xv = f32x4{0.f, 0.f, 0.f, 0.f};
        if (xr >= 0) xv = *reinterpret_cast<const f32x4*>(X + (size_t)xr * p.ldx + k0 + lk);
        __syncthreads();
#pragma unroll
        for (int j = 0; j < 4; j++) sw[lk + j][lr] = wv[j], sx[lk + j][lr] = xv[j];
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < KT; kk++) {
            const f32x4 a = *reinterpret_cast<const f32x4*>(&sw[kk][tm]), b = *reinterpret_cast<const f32x4*>(&sx[kk][tc]);
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
        }
    }
    __shared__ float sout[64][65]; /* [column][row]: GATED pairs rows 16 apart */
    if (p.epilogue == KF_RB_GATED) {
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
            for (int j = 0; j < 4; j++) sout[tc + j][tm + i] = acc[i][j];
        __syncthreads();
        for (int i = tid; i < 64 * 32; i += 256) {
            const int f = i & 31, col = i >> 5, yr = sdst[col];
            if (yr < 0) continue;
            const int row = (f >> 4) * 32 + (f & 15);
            const float scale = p.mode == KF_RB_UP ? q.e.weight[yr] : 1.f;
            reinterpret_cast<float*>(p.y)[(size_t)yr * p.ldy + (m0 >> 1) + f] = scale * (rb_activate(p.act, sout[col][row]) * sout[col][row + 16]);
        }
        return;
    }
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int yr = sdst[tc + j];
        if (yr < 0) continue;
        f32x4 d = f32x4{acc[0][j], acc[1][j], acc[2][j], acc[3][j]};
        if (p.epilogue == KF_RB_RESIDUAL) {
            const f32x4 r = *reinterpret_cast<const f32x4*>(p.res + (size_t)yr * p.ldr + m0 + tm);
#pragma unroll
            for (int i = 0; i < 4; i++) d[i] = fmaf(p.alpha, r[i], d[i]);
        }
        *reinterpret_cast<f32x4*>(reinterpret_cast<float*>(p.y) + (size_t)yr * p.ldy + m0 + tm) = d;
    }
}
int rb_f32_launch(hipStream_t st, const RbProduct& q) {
    const kf_rb_product& p = q.p;
    if (p.mode == KF_RB_SUM || (p.mode != KF_RB_ALL && q.e.tile != 64)) return 1;
    dim3 grid(p.m / 64, p.mode == KF_RB_ALL ? (p.n + 63) / 64 : q.e.n_tile);
    hipLaunchKernelGGL(rb_f32_kernel, grid, dim3(256), 0, st, q);
    return KF_OK;
}

}  // namespace kf

using namespace kf;
extern "C" int kf_rb_linear(kf_ctx* c, const kf_rb_product* p) {
    CHKCTX(c);
    if (!p || !p->w || !p->x || !p->y) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: null pointer");
    if (p->type != KF_BF16 && p->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_linear: storage %d", p->type);
    if (p->m < 1 || p->k < 1 || p->n < 1 || p->m % KF_RB_PAD || p->k % KF_RB_PAD) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: %d x %d weight, %d rows", p->m, p->k, p->n);
    if (p->ldx < p->k || p->ldy < (p->epilogue == KF_RB_GATED ? p->m / 2 : p->m) || p->ldx % 8 || p->ldy % 4) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: row strides");
    if (!al16(p->w) || !al16(p->x) || !al16(p->y)) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_linear: unaligned pointer");
    if (p->epilogue < KF_RB_STORE || p->epilogue > KF_RB_GATED || p->mode < KF_RB_ALL || p->mode > KF_RB_SUM) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: epilogue or mode");
    if (p->epilogue == KF_RB_RESIDUAL && (!p->res || !al16(p->res) || p->ldr < p->m || p->ldr % 4)) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: residual");
    RbProduct q;
    q.p = *p;
    q.e = kf_rb_experts{};
    if (p->mode != KF_RB_ALL) {
        const kf_rb_experts* e = p->experts;
        if (!e || e->n_expert < 1 || e->top < 1 || e->tile < 1 || e->n_tile < 1 || !e->tile_expert || !e->list || !e->ids || !e->weight) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: experts");
        if (e->w_stride < (int64_t)p->m * p->k || e->w_stride % 8) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: expert stride");
        if ((p->mode == KF_RB_UP) != (p->epilogue == KF_RB_GATED) || (p->mode == KF_RB_DOWN && p->epilogue != KF_RB_STORE_F32) || (p->mode == KF_RB_SUM && p->epilogue != KF_RB_RESIDUAL))
            return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: this mode has another epilogue");
        q.e = *e;
    }
    int rc;
    if (p->type == KF_F32) rc = rb_f32_launch(c->stream, q);
    else {
        rc = 1;
        if (p->n <= KF_RB_DECODE_MAX) rc = rb_stream_launch(c->stream, q);
        if (rc == 1 && p->mode != KF_RB_SUM) rc = rb_gemm_launch(c->stream, q);
    }
    if (rc == 1) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_linear: no kernel for mode %d, %d rows, tiles of %d, storage %d", p->mode, p->n, q.e.tile, p->type);
    if (rc != KF_OK) return abi_fail(rc, "kf_rb_linear: launch failed");
    return hipGetLastError() == hipSuccess ? KF_OK : abi_fail(KF_HIP_CHECK, "kf_rb_linear: launch failed");
}
