// kf_rb_linear.hip -- row-batch products y[t][m] = W[m] . x[t] for few rows (decode batches) and in 32-bit, and the ABI entry that picks the form.
//
// Decode batches stream the weights: a workgroup owns 16 weight rows (GATED: 16 gate and the 16 up rows that follow them), its waves take runs of 32-deep k-steps -- a
// step's 16 x 32 weights are one stored tile, a contiguous kilobyte -- and multiply them against up to 64 token columns by v_mfma_f32_16x16x32_bf16 (A = weight rows, B = token rows, straight
// from global memory: the activations of a decode batch are a few KB and stay in L2), the next run's weights in flight.  The waves' partial tiles meet in LDS, one thread
// per output finishes it.  The RMS norm in front of a product (NORM: few rows of the 32-bit residual sum) costs no pass: the product that formed the sum left its squares
// per 16 columns, every wave adds them up for itself and norms its token fragments as it reads them.  With experts a workgroup's columns are the pairs of one expert (UP, DOWN), or it walks all chosen experts' k-steps as one list dealt to its waves,
// columns that did not choose an expert held at zero (SUM): an expert's rows are read once per workgroup whoever chose them.
#include "kf_ctx.h"
#include "kf_rb_common.h"

namespace kf {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x4 rb_mfma16(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// the run of U k-steps from step s of the MG 16-row blocks at wr (this lane's piece of the first block's first tile; a tile per step)
template <int MG, int U>
__device__ __forceinline__ void rb_load_w(u32x4 (&a)[U][MG], const uint16_t* __restrict__ wr, int k, int s, int s_end) {
#pragma unroll
    for (int u = 0; u < U; u++)
#pragma unroll
        for (int g = 0; g < MG; g++) {
            a[u][g] = u32x4{0, 0, 0, 0};
            if (s + u < s_end) a[u][g] = ld_nt(reinterpret_cast<const u32x4*>(wr + (size_t)g * 16 * k + 512 * (s + u))); /* wave-uniform */
        }
}
// token fragments of the same steps; xp[t]: this lane's token row + its k octet (NULLABLE: NULL is a zero column), steps past s_end read step s_end - 1 against zero weights
template <int NT, int U, bool NULLABLE>
__device__ __forceinline__ void rb_load_x(u32x4 (&b)[U][NT], const uint16_t* const (&xp)[NT], int s, int s_end) {
#pragma unroll
    for (int u = 0; u < U; u++) {
        const int st = s + u < s_end ? s + u : s_end - 1;
#pragma unroll
        for (int t = 0; t < NT; t++) {
            if (NULLABLE) {
                b[u][t] = u32x4{0, 0, 0, 0};
                if (xp[t]) b[u][t] = *reinterpret_cast<const u32x4*>(xp[t] + 32 * st);
            } else {
                b[u][t] = *reinterpret_cast<const u32x4*>(xp[t] + 32 * st);
            }
        }
    }
}
template <int NT, int MG, int U>
__device__ __forceinline__ void rb_multiply(const u32x4 (&a)[U][MG], const u32x4 (&b)[U][NT], f32x4 (&acc)[MG][NT]) {
#pragma unroll
    for (int u = 0; u < U; u++)
#pragma unroll
        for (int g = 0; g < MG; g++)
#pragma unroll
            for (int t = 0; t < NT; t++) acc[g][t] = rb_mfma16(a[u][g], b[u][t], acc[g][t]);
}
// the waves' partial tiles -> outputs; list: the columns are pairs
template <int NT, int MG, int NW>
__device__ __forceinline__ void rb_stream_finish(const RbProduct& q, const f32x4 (&acc)[MG][NT], float (&red)[NW][MG][16 * NT][17], const int32_t* list, int m0, int tid) {
    const kf_rb_product& p = q.p;
    const int lane = tid & 63, wid = tid >> 6, r16 = lane & 15, q4 = lane >> 4;
#pragma unroll
    for (int g = 0; g < MG; g++)
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int j = 0; j < 4; j++) red[wid][g][t * 16 + r16][4 * q4 + j] = acc[g][t][j];
    __syncthreads();
    const int cols = list ? 16 * NT : p.n;
    for (int i = tid; i < cols * 16; i += 64 * NW) {
        const int row = i & 15, col = i >> 4;
        int yr = col;
        float scale = 1.f;
        if (list) {
            yr = list[col];
            if (yr < 0) continue;
            if (p.mode == KF_RB_UP) scale = q.e.weight[yr];
        }
        float d = 0.f;
#pragma unroll
        for (int w = 0; w < NW; w++) d += red[w][0][col][row];
        if constexpr (MG == 2) {
            float u = 0.f;
#pragma unroll
            for (int w = 0; w < NW; w++) u += red[w][MG - 1][col][row];
            reinterpret_cast<uint16_t*>(p.y)[(size_t)yr * p.ldy + (m0 >> 1) + row] = f2bf(scale * (rb_activate(p.act, d) * u));
        } else if (p.epilogue == KF_RB_STORE) {
            const int m = m0 + row;
            reinterpret_cast<uint16_t*>(p.y)[(size_t)yr * p.ldy + m] = f2bf(m >= p.act_lo && m < p.act_hi ? rb_activate(p.act, d) : d);
        } else if (p.epilogue == KF_RB_STORE_F32) {
            reinterpret_cast<float*>(p.y)[(size_t)yr * p.ldy + m0 + row] = d;
        } else {
            const float z = fmaf(p.alpha, p.res[(size_t)yr * p.ldr + m0 + row], d);
            reinterpret_cast<float*>(p.y)[(size_t)yr * p.ldy + m0 + row] = z;
            if (NT == 1 && p.ssq) { /* 16 lanes = the 16 columns of one row */
                float ss = z * z;
                ss += dpp_f<0xB1>(ss);
                ss += dpp_f<0x4E>(ss);
                ss += dpp_f<0x141>(ss);
                ss += dpp_f<0x140>(ss);
                if (row == 0) p.ssq[(size_t)(m0 / 16) * KF_RB_NORM_ROWS + yr] = ss;
            }
        }
    }
}

template <int NT, bool GATED, int NW, bool NORM>
__global__ void __launch_bounds__(64 * NW) rb_stream_kernel(const RbProduct q) {
    const kf_rb_product& p = q.p;
    constexpr int MG = GATED ? 2 : 1, U = NT >= 4 ? 2 : 4;
    __shared__ float red[NW][MG][16 * NT][17]; /* [wave][block][column][row], padded */
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r16 = lane & 15, q4 = lane >> 4;
    const int m0 = blockIdx.x * (16 * MG), nstep = p.k / 32;
    const uint16_t* W = reinterpret_cast<const uint16_t*>(p.w);
    const uint16_t* X = reinterpret_cast<const uint16_t*>(p.x);
    const int32_t* list = nullptr;
    if (p.mode != KF_RB_ALL) {
        const int ex = q.e.tile_expert[blockIdx.y];
        if (ex < 0) return;
        W += (size_t)ex * q.e.w_stride;
        list = q.e.list + (size_t)blockIdx.y * q.e.tile;
    }
    const uint16_t* wr = W + (size_t)m0 * p.k + 8 * lane;
    u32x4 a[U][MG], b[U][NT];
    int s = wid * U;
    rb_load_w<MG, U>(a, wr, p.k, s, nstep);
    const uint16_t* xp[NT];
    const float* zp = nullptr;   /* NORM: this lane's row of the residual sum, and 1 / its root mean square */
    const uint16_t* gp = nullptr;
    float rs = 0.f;
    if constexpr (NORM) {
        static_assert(NT == 1, "a few rows");
        const int row = r16 < p.n ? r16 : p.n - 1, parts = p.k / 16;
        zp = p.norm_z + (size_t)row * p.ldx + 8 * q4, gp = reinterpret_cast<const uint16_t*>(p.norm_w) + 8 * q4;
        for (int t = 0; t < p.n; t++) { /* the sums of squares the product in front left per 16 columns: no barrier, every wave for itself */
            float ss = 0.f;
            for (int i = lane; i < parts; i += 64) ss += p.norm_ssq[(size_t)i * KF_RB_NORM_ROWS + t];
            ss = wave_sum(ss);
            if (row == t) rs = 1.0f / sqrtf(ss / (float)p.norm_dim + p.norm_eps);
        }
        xp[0] = nullptr;
    } else {
#pragma unroll
        for (int t = 0; t < NT; t++) { /* columns past the end repeat a row: their outputs are not stored */
            const int col = t * 16 + r16;
            int row = col < p.n ? col : p.n - 1;
            if (list) {
                const int pair = list[col];
                row = pair < 0 ? 0 : (p.mode == KF_RB_UP ? pair / q.e.top : pair);
            }
            xp[t] = X + (size_t)row * p.ldx + 8 * q4;
        }
    }
    f32x4 acc[MG][NT];
#pragma unroll
    for (int g = 0; g < MG; g++)
#pragma unroll
        for (int t = 0; t < NT; t++) acc[g][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (; s < nstep; s += NW * U) {
        u32x4 an[U][MG];
        if constexpr (NORM) {
            f32x4 z0[U], z1[U];
            u32x4 g[U];
#pragma unroll
            for (int u = 0; u < U; u++) {
                const int k0 = 32 * (s + u < nstep ? s + u : nstep - 1);
                z0[u] = rb_ld4(zp + k0), z1[u] = rb_ld4(zp + k0 + 4), g[u] = *reinterpret_cast<const u32x4*>(gp + k0);
            }
            rb_load_w<MG, U>(an, wr, p.k, s + NW * U, nstep);
#pragma unroll
            for (int u = 0; u < U; u++) {
                const f32x4 o0 = f32x4{z0[u].x * rs * bf_lo(g[u].x), z0[u].y * rs * bf_hi(g[u].x), z0[u].z * rs * bf_lo(g[u].y), z0[u].w * rs * bf_hi(g[u].y)};
                const f32x4 o1 = f32x4{z1[u].x * rs * bf_lo(g[u].z), z1[u].y * rs * bf_hi(g[u].z), z1[u].z * rs * bf_lo(g[u].w), z1[u].w * rs * bf_hi(g[u].w)};
                b[u][0] = u32x4{pack_bf16x2(o0.x, o0.y), pack_bf16x2(o0.z, o0.w), pack_bf16x2(o1.x, o1.y), pack_bf16x2(o1.z, o1.w)};
                if (blockIdx.x == 0 && r16 < p.n && s + u < nstep) { /* the normed rows themselves, once */
                    const size_t at = (size_t)r16 * p.ldx + 32 * (s + u) + 8 * q4;
                    rb_st4(p.norm_x + at, o0), rb_st4(p.norm_x + at + 4, o1);
                    *reinterpret_cast<u32x4*>(reinterpret_cast<uint16_t*>(const_cast<void*>(p.x)) + at) = b[u][0];
                }
            }
        } else {
            rb_load_x<NT, U, false>(b, xp, s, nstep);
            rb_load_w<MG, U>(an, wr, p.k, s + NW * U, nstep);
        }
        rb_multiply<NT, MG, U>(a, b, acc);
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int g = 0; g < MG; g++) a[u][g] = an[u][g];
    }
    rb_stream_finish<NT, MG, NW>(q, acc, red, list, m0, tid);
}

// RESIDUAL with the rows' experts summed: (chosen expert, k-step) pairs as one list, cut evenly over the waves
template <int NT, int NW>
__global__ void __launch_bounds__(64 * NW) rb_stream_sum_kernel(const RbProduct q) {
    const kf_rb_product& p = q.p;
    constexpr int U = NT >= 4 ? 2 : 4;
    __shared__ float red[NW][1][16 * NT][17];
    __shared__ int32_t s_ex[KF_RB_SUM_PAIRS], s_ids[KF_RB_SUM_PAIRS];
    __shared__ int s_n;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r16 = lane & 15, q4 = lane >> 4;
    const int m0 = blockIdx.x * 16, nstep = p.k / 32, pairs = p.n * q.e.top;
    const uint16_t* X = reinterpret_cast<const uint16_t*>(p.x);
    for (int i = tid; i < pairs; i += 64 * NW) s_ids[i] = q.e.ids[i];
    if (wid == 0) { /* the chosen experts, each once: a tile per expert (a tile holds as many pairs as the batch has rows) */
        int cnt = 0;
        for (int i0 = 0; i0 < q.e.n_tile; i0 += 64) {
            const int ex = i0 + lane < q.e.n_tile ? q.e.tile_expert[i0 + lane] : -1;
            const unsigned long long on = __ballot(ex >= 0);
            if (ex >= 0) s_ex[cnt + __popcll(on & ((1ull << lane) - 1))] = ex;
            cnt += __popcll(on);
        }
        if (lane == 0) s_n = cnt;
    }
    __syncthreads();
    const int total = s_n * nstep, span = (total + NW - 1) / NW;
    int at = wid * span;
    const int end = at + span < total ? at + span : total;
    f32x4 acc[1][NT];
#pragma unroll
    for (int t = 0; t < NT; t++) acc[0][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    while (at < end) { /* an expert's part of this wave's range (wave-uniform) */
        const int i = at / nstep, s0 = at - i * nstep, s1 = s0 + (end - at) < nstep ? s0 + (end - at) : nstep;
        const int ex = s_ex[i];
        const uint16_t* wr = reinterpret_cast<const uint16_t*>(p.w) + (size_t)ex * q.e.w_stride + (size_t)m0 * p.k + 8 * lane;
        u32x4 a[U][1], b[U][NT];
        rb_load_w<1, U>(a, wr, p.k, s0, s1);
        const uint16_t* xp[NT];
#pragma unroll
        for (int t = 0; t < NT; t++) {
            const int row = t * 16 + r16;
            xp[t] = nullptr;
            if (row < p.n)
                for (int j = 0; j < q.e.top; j++)
                    if (s_ids[row * q.e.top + j] == ex) xp[t] = X + (size_t)(row * q.e.top + j) * p.ldx + 8 * q4;
        }
        for (int s = s0; s < s1; s += U) {
            u32x4 an[U][1];
            rb_load_x<NT, U, true>(b, xp, s, s1);
            rb_load_w<1, U>(an, wr, p.k, s + U, s1);
            rb_multiply<NT, 1, U>(a, b, acc);
#pragma unroll
            for (int u = 0; u < U; u++) a[u][0] = an[u][0];
        }
        at += s1 - s0;
    }
    rb_stream_finish<NT, 1, NW>(q, acc, red, nullptr, m0, tid);
}
template <int NT, int NW>
static void stream_go(hipStream_t st, const RbProduct& q, dim3 grid) {
    if (q.p.mode == KF_RB_SUM) hipLaunchKernelGGL((rb_stream_sum_kernel<NT, NW>), grid, dim3(64 * NW), 0, st, q);
    else if (q.p.epilogue == KF_RB_GATED) hipLaunchKernelGGL((rb_stream_kernel<NT, true, NW, false>), grid, dim3(64 * NW), 0, st, q);
    else hipLaunchKernelGGL((rb_stream_kernel<NT, false, NW, false>), grid, dim3(64 * NW), 0, st, q);
}
template <int NW>
static void norm_stream_go(hipStream_t st, const RbProduct& q, dim3 grid) {
    if (q.p.epilogue == KF_RB_GATED) hipLaunchKernelGGL((rb_stream_kernel<1, true, 4, true>), grid, dim3(256), 0, st, q);
    else hipLaunchKernelGGL((rb_stream_kernel<1, false, NW, true>), grid, dim3(64 * NW), 0, st, q);
}
int rb_stream_launch(hipStream_t st, const RbProduct& q) {
    const kf_rb_product& p = q.p;
    const bool tiles = p.mode == KF_RB_UP || p.mode == KF_RB_DOWN;
    const int cols = tiles ? q.e.tile : p.n, nt = (cols + 15) / 16;
    if (nt > 4 || (tiles && q.e.tile % 16)) return 1;
    if (p.mode == KF_RB_SUM && ((long)p.n * q.e.top > KF_RB_SUM_PAIRS || q.e.tile < p.n)) return 1;
    dim3 grid(p.m / (p.epilogue == KF_RB_GATED ? 32 : 16), tiles ? q.e.n_tile : 1);
    const bool wide = (long)grid.x * grid.y < 768 && p.k >= 512; /* few workgroups: more waves each, more loads in flight per CU */
    if (p.norm_z) {
        wide ? norm_stream_go<8>(st, q, grid) : norm_stream_go<4>(st, q, grid);
        return KF_OK;
    }
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
        } else if (p.epilogue == KF_RB_STORE && m0 + tm + 3 >= p.act_lo && m0 + tm < p.act_hi) {
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (m0 + tm + i >= p.act_lo && m0 + tm + i < p.act_hi) d[i] = rb_activate(p.act, d[i]);
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
extern "C" int kf_rb_linear_norms(int type, int n, int k) { return type == KF_BF16 && n >= 1 && n <= KF_RB_NORM_ROWS && k % KF_RB_PAD == 0; }
extern "C" int kf_rb_linear(kf_ctx* c, const kf_rb_product* p) {
    CHKCTX(c);
    if (!p || !p->w || !p->x || !p->y) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: null pointer");
    if (p->type != KF_BF16 && p->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "kf_rb_linear: storage %d", p->type);
    if (p->m < 1 || p->k < 1 || p->n < 1 || p->m % KF_RB_PAD || p->k % KF_RB_PAD) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: %d x %d weight, %d rows", p->m, p->k, p->n);
    if (p->ldx < p->k || p->ldy < (p->epilogue == KF_RB_GATED ? p->m / 2 : p->m) || p->ldx % 8 || p->ldy % 4) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: row strides");
    if (!al16(p->w) || !al16(p->x) || !al16(p->y)) return abi_fail(KF_BLAS_UNALIGN, "kf_rb_linear: unaligned pointer");
    if (p->epilogue < KF_RB_STORE || p->epilogue > KF_RB_GATED || p->mode < KF_RB_ALL || p->mode > KF_RB_SUM) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: epilogue or mode");
    if (p->epilogue == KF_RB_RESIDUAL && (!p->res || !al16(p->res) || p->ldr < p->m || p->ldr % 4)) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: residual");
    if (p->act_lo < p->act_hi && (p->epilogue != KF_RB_STORE || p->mode != KF_RB_ALL || p->act_lo < 0 || p->act_hi > p->m)) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: activated columns");
    if (p->ssq && (!kf_rb_linear_norms(p->type, p->n, p->m) || p->epilogue != KF_RB_RESIDUAL)) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: sums of squares");
    if (p->norm_z && (!kf_rb_linear_norms(p->type, p->n, p->k) || p->mode != KF_RB_ALL || p->epilogue == KF_RB_RESIDUAL || !p->norm_w || !p->norm_x || !p->norm_ssq || p->norm_dim < 1 || p->norm_dim > p->k || p->ldx != p->k || !al16(p->norm_z) ||
                      !al16(p->norm_w) || !al16(p->norm_x)))
        return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: norm in front of the product");
    RbProduct q;
    q.p = *p;
    q.e = kf_rb_experts{};
    if (p->mode != KF_RB_ALL) {
        const kf_rb_experts* e = p->experts;
        if (!e || e->n_expert < 1 || e->top < 1 || e->tile < 1 || e->n_tile < 1 || !e->tile_expert || !e->list || !e->ids || !e->weight) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: experts");
        if (e->w_stride < (int64_t)p->m * p->k || e->w_stride % 8) return abi_fail(KF_INVALID_ARGS, "kf_rb_linear: expert stride");
        if ((p->mode == KF_RB_UP) != (p->epilogue == KF_RB_GATED) || (p->mode == KF_RB_DOWN && p->epilogue != KF_RB_STORE) || (p->mode == KF_RB_SUM && p->epilogue != KF_RB_RESIDUAL))
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
