// kf_rb_gemm.hip -- row-batch products on MFMA tiles: the 64-deep tile of kf_gemm3_tile.h (both operands global -> LDS by global_load_lds, swizzled at the source) with the
// row-batch epilogues (fp32 residual with alpha, gated activation of interleaved rows, fp32 store) and, for experts, a gathered token operand: the rows of a token tile are
// the pairs of one expert, each lane's source pointer is set up once from the pair list, so routed rows are never copied together.
#include <string.h>

#include "kf_gemm3_tile.h"
#include "kf_rb_common.h"

namespace kf {

using RbBig = G3Cfg<256, 256, 8>;
using RbSmall = G3Cfg<128, 128, 4>;
using RbMid = G3Cfg<64, 128, 4>;
using RbTiny = G3Cfg<64, 64, 4>;
using RbPairs = G3Cfg<128, 64, 4>; /* experts of about a hundred pairs: half the padding of 128-pair tiles, each weight tile read about once */

template <class C, bool EXPERTS>
__global__ void __launch_bounds__(C::NTH, C::WGS_PER_CU * C::NW / 4) rb_gemm_kernel(const RbProduct q) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    __shared__ int32_t s_src[EXPERTS ? C::BN : 1], s_dst[EXPERTS ? C::BN : 1];
    const kf_rb_product& p = q.p;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int nbx = (p.m + C::BM - 1) / C::BM, wg = g3_remap(blockIdx.x, gridDim.x), bx = wg % nbx, by = wg / nbx;
    const int m0 = bx * C::BM, t0 = by * C::BN;
    GemmArgs a; /* what the main loop reads */
    a.w = reinterpret_cast<const unsigned char*>(p.w), a.M = p.m, a.K = p.k, a.x = reinterpret_cast<const uint16_t*>(p.x), a.ldx = p.ldx, a.n = p.n, a.ldr = 0;
    f32x4 acc[C::MT][C::NT];
#pragma unroll
    for (int i = 0; i < C::MT; i++)
#pragma unroll
        for (int j = 0; j < C::NT; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if constexpr (EXPERTS) {
        const int ex = q.e.tile_expert[by];
        if (ex < 0) return; /* workgroup-uniform */
        a.w += (size_t)ex * q.e.w_stride * 2;
        for (int i = tid; i < C::BN; i += C::NTH) {
            const int pair = q.e.list[(size_t)by * C::BN + i];
            s_dst[i] = pair, s_src[i] = pair < 0 ? 0 : (p.mode == KF_RB_UP ? pair / q.e.top : pair);
        }
        __syncthreads();
        g3_mainloop<false, false, G3_BK, C, G3GatherTiled>(a, m0, 0, 0, p.k / G3_BK, acc, smem_raw, wid, lane, G3GatherTiled{s_src});
    } else {
        g3_mainloop<false, false, G3_BK, C, G3Tiled>(a, m0, t0, 0, p.k / G3_BK, acc, smem_raw, wid, lane);
    }
    const int wm = wid / C::WN, wn = wid % C::WN, r16 = lane & 15, q4 = lane >> 4;
#pragma unroll
    for (int nt = 0; nt < C::NT; nt++) {
        const int col = wn * (16 * C::NT) + nt * 16 + r16;
        int row = t0 + col;
        float scale = 1.f;
        if constexpr (EXPERTS) {
            row = s_dst[col];
            if (row < 0) continue;
            if (p.mode == KF_RB_UP) scale = q.e.weight[row];
        } else {
            if (row >= p.n) continue;
        }
        if (p.epilogue == KF_RB_GATED) {
#pragma unroll
            for (int mt = 0; mt < C::MT; mt += 2) {
                const int m = m0 + wm * (16 * C::MT) + mt * 16;
                if (m >= p.m) continue;
                const f32x4 g = acc[mt][nt], u = acc[mt + 1][nt];
                f32x4 o;
#pragma unroll
                for (int j = 0; j < 4; j++) o[j] = scale * (rb_activate(p.act, g[j]) * u[j]);
                rb_st4(reinterpret_cast<uint16_t*>(p.y) + (size_t)row * p.ldy + (m >> 1) + 4 * q4, o);
            }
        } else {
#pragma unroll
            for (int mt = 0; mt < C::MT; mt++) {
                const int m = m0 + wm * (16 * C::MT) + mt * 16 + 4 * q4;
                if (m >= p.m) continue;
                f32x4 d = acc[mt][nt];
                if (p.epilogue == KF_RB_STORE) {
                    if (m + 3 >= p.act_lo && m < p.act_hi) {
#pragma unroll
                        for (int j = 0; j < 4; j++)
                            if (m + j >= p.act_lo && m + j < p.act_hi) d[j] = rb_activate(p.act, d[j]);
                    }
                    rb_st4(reinterpret_cast<uint16_t*>(p.y) + (size_t)row * p.ldy + m, d);
                } else {
                    if (p.epilogue == KF_RB_RESIDUAL) {
                        const f32x4 r = rb_ld4(p.res + (size_t)row * p.ldr + m);
#pragma unroll
                        for (int j = 0; j < 4; j++) d[j] = fmaf(p.alpha, r[j], d[j]);
                    }
                    rb_st4(reinterpret_cast<float*>(p.y) + (size_t)row * p.ldy + m, d);
                }
            }
        }
    }
}
template <class C, bool EXPERTS>
static int rb_go(hipStream_t st, const RbProduct& q, long nwg) {
    constexpr int SMEM = 2 * C::STAGE;
    static int attr_set = 0;
    if (!attr_set && SMEM + 2 * 4 * C::BN > 64 * 1024) { /* the pair rows of the experts form sit in static LDS */
        if (hipFuncSetAttribute((const void*)rb_gemm_kernel<C, EXPERTS>, hipFuncAttributeMaxDynamicSharedMemorySize, SMEM) != hipSuccess) return KF_HIP_CHECK;
        attr_set = 1;
    }
    hipLaunchKernelGGL((rb_gemm_kernel<C, EXPERTS>), dim3((unsigned)nwg), dim3(C::NTH), SMEM, st, q);
    return KF_OK;
}
int rb_gemm_launch(hipStream_t st, const RbProduct& q) {
    const kf_rb_product& p = q.p;
    auto tiles = [&](int bm, int bn) { return (long)((p.m + bm - 1) / bm) * ((p.n + bn - 1) / bn); };
    if (p.mode != KF_RB_ALL) {
        if (q.e.tile == 128) return rb_go<RbSmall, true>(st, q, (long)((p.m + 127) / 128) * q.e.n_tile);
        if (q.e.tile == 64) return rb_go<RbPairs, true>(st, q, (long)((p.m + 127) / 128) * q.e.n_tile);
        return 1;
    }
    // the measured thresholds of gemm3_launch: big tiles from 160 of them, then smaller ones that fill the chip
    if (p.m >= 256 && p.n >= 256 && tiles(256, 256) >= 160) return rb_go<RbBig, false>(st, q, tiles(256, 256));
    if (tiles(128, 128) >= 256) return rb_go<RbSmall, false>(st, q, tiles(128, 128));
    if (tiles(64, 128) >= 192) return rb_go<RbMid, false>(st, q, tiles(64, 128));
    return rb_go<RbTiny, false>(st, q, tiles(64, 64));
}

}  // namespace kf
