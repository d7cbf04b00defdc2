// kf_rb_recur.h -- shared by the recurrent row-batch kernels: 32-bit elementary functions on the hardware's exp2 / log2 / rcp, barriers, a decode step's state in registers, and the
// decode step of the decayed sum (kf_rb_recur.hip launches it alone, kf_rb_attn.hip beside a layer's attention).
#pragma once
#include <math.h>

#include "kf_ctx.h"
#include "kf_rb_common.h"

namespace kf {

__device__ __forceinline__ float row16_sum(float v) { /* over the 16 lanes of a row, in all of them */
    v += dpp_f<0xB1>(v);
    v += dpp_f<0x4E>(v);
    v += dpp_f<0x141>(v);
    return v + dpp_f<0x140>(v);
}
__device__ __forceinline__ float rc_silu(float z) { return z * rb_sigmoid(z); }
__device__ __forceinline__ void rc_st_sc1(float* p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ float rc_ld_sc1(const float* p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
// a barrier for what passes through LDS only: loads and stores of global memory stay in flight over it
__device__ __forceinline__ void rc_lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
constexpr int RC_CNT_STRIDE = 16; /* words between arrival counters */
static __host__ __device__ inline int rc_up(int n, int m) { return (n + m - 1) / m * m; }

__device__ __forceinline__ float rc_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
constexpr float RC_LOG2E = 1.44269502162933349609375f;
__device__ __forceinline__ float rc_fast_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + rc_exp2(-RC_LOG2E * z)); }
// softplus in units of ln 2: log2(1 + e^z); the correction factor keeps the small ones exact to rounding
__device__ __forceinline__ float rc_softplus2(float z) {
    const float e = rc_exp2(-RC_LOG2E * fabsf(z)), u = 1.0f + e, d = u - 1.0f;
    const float l = d == 0.f ? e * RC_LOG2E : __builtin_amdgcn_logf(u) * (e * __builtin_amdgcn_rcpf(d));
    return fmaxf(z, 0.f) * RC_LOG2E + l;
}
__device__ __forceinline__ float rb_ld1(uint16_t v) { return bf2f(v); }
__device__ __forceinline__ float rb_ld1(float v) { return v; }

// A head's state matrix [dim][vs] in the registers of NT threads: groups of vs / 4 threads side by side, each group the rows rg, rg + RG, ..., four neighbouring columns per thread.
// RPT: rows of a thread at most (0: not kept, read where they are needed)
template <int NT, int RPT>
struct RcStep {
    int dim, vs, c4, RG, rg, col;
    bool on;
    f32x4 S[RPT ? RPT : 1];
    __device__ __forceinline__ RcStep(int dim_, int vdim, int tid) {
        dim = dim_, vs = rc_up(vdim, 4), c4 = vs / 4, RG = NT / c4, rg = tid / c4, col = 4 * (tid - rg * c4), on = rg < RG;
    }
    __device__ __forceinline__ void load(const float* S0, bool old) {
        if constexpr (RPT > 0) {
#pragma unroll
            for (int i = 0; i < RPT; i++) {
                S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (on && old && rg + i * RG < dim) S[i] = *reinterpret_cast<const f32x4*>(S0 + (size_t)(rg + i * RG) * vs + col);
            }
        }
    }
    template <class F>
    __device__ __forceinline__ void each(const float* S0, bool old, F f) const { /* f(row, its four columns) */
        if (!on) return;
        if constexpr (RPT > 0) {
#pragma unroll
            for (int i = 0; i < RPT; i++)
                if (rg + i * RG < dim) f(rg + i * RG, S[i]);
        } else {
            for (int r = rg; r < dim; r += RG) f(r, old ? *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col) : f32x4{0.f, 0.f, 0.f, 0.f});
        }
    }
    // the groups' sums over their rows -> red [parts()][vs]: groups that share a wave are added up first where a group is 16 or 32 lanes
    __device__ __forceinline__ int parts() const { return c4 == 32 ? RG / 2 : (c4 == 16 ? RG / 4 : RG); }
    __device__ __forceinline__ void partial(f32x4 v, float* red) const {
        if (c4 == 32 || c4 == 16) {
#pragma unroll
            for (int j = 0; j < 4; j++) {
                v[j] = xsum32(v[j]);
                if (c4 == 16) v[j] = xsum16(v[j]);
            }
            const int lane = threadIdx.x & 63;
            if (lane < c4) *reinterpret_cast<f32x4*>(red + (size_t)(threadIdx.x >> 6) * vs + col) = v;
        } else if (on) {
            *reinterpret_cast<f32x4*>(red + (size_t)rg * vs + col) = v;
        }
    }
};
// threads of a decode workgroup: 0: 1024 that read the state twice
static inline int rc_step_threads(int dim, int vdim) {
    const int c4 = rc_up(vdim, 4) / 4;
    for (int nt : {256, 512, 1024})
        if (c4 <= nt && (dim + nt / c4 - 1) / (nt / c4) <= (nt == 1024 ? 16 : 8)) return nt;
    return 0;
}
static inline size_t rc_decay_step_lds(int dim, int vdim, int nt) { return (2 * (size_t)rc_up(dim, 4) + rc_up(vdim, 4) + 4 * (size_t)nt + 40) * 4; }

int rc_check_decay(const kf_rb_decay* a, const int32_t* meta, int n, const char* who); // kf_rb_recur.hip
// head h of row rr (of n_rows): o = decay S^T q + (q . k) v, S' = decay S + k v^T; the row's last head norms and gates all of them
template <class T, int NT, int RPT>
__device__ __forceinline__ void rc_decay_step(const kf_rb_decay& a, const int32_t* __restrict__ meta, int h, int rr, int n_rows, float* smem) {
    constexpr int NW = NT / 64;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int pos = meta[KF_RB_META * rr], slot = meta[KF_RB_META * rr + 1];
    if (pos < 0) return; /* workgroup-uniform */
    const int dim = a.dim, vdim = a.vdim, vs = rc_up(vdim, 4);
    float *s_q = smem, *s_k = s_q + rc_up(dim, 4), *s_v = s_k + rc_up(dim, 4), *s_red = s_v + vs /* [parts][vs] */, *s_one = s_red + NT * 4;
    int* s_last = reinterpret_cast<int*>(s_one + 32);
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)rr * a.ldraw;
    const T *q = raw + a.col_q + (size_t)h * dim, *k = q + (size_t)a.n_head * dim, *v = raw + a.col_q + (size_t)2 * a.n_head * dim + (size_t)h * vdim;
    const float lam = a.decay[h];
    T first = T(); /* the first of this thread's inputs sets out in front of the state */
    const int n_in = 2 * dim + vdim;
    auto input = [&](int i) { return i < dim ? q[i] : (i < 2 * dim ? k[i - dim] : v[i - 2 * dim]); };
    if (tid < n_in) first = input(tid);
    RcStep<NT, RPT> st(dim, vdim, tid);
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + (pos & 1)) * side + h * head;
    st.load(S0, pos > 0);
    for (int i = tid; i < n_in; i += NT) (i < dim ? s_q[i] : (i < 2 * dim ? s_k[i - dim] : s_v[i - 2 * dim])) = rb_ld1(i == tid ? first : input(i));
    for (int i = vdim + tid; i < vs; i += NT) s_v[i] = 0.f;
    rc_lds_barrier();
    if (wid == NW - 1) {
        float d = 0.f;
        for (int i = lane; i < dim; i += 64) d = fmaf(s_q[i], s_k[i], d);
        d = wave_sum(d);
        if (lane == 0) s_one[0] = d;
    }
    f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
    const f32x4 u = *reinterpret_cast<const f32x4*>(s_v + st.col);
    st.each(S0, pos > 0, [&](int r, f32x4 s) {
        const float qq = s_q[r], kk = s_k[r];
        f32x4 n;
#pragma unroll
        for (int j = 0; j < 4; j++) o[j] = fmaf(qq, s[j], o[j]), n[j] = fmaf(kk, u[j], lam * s[j]);
        *reinterpret_cast<f32x4*>(S1 + (size_t)r * vs + st.col) = n;
    });
    st.partial(o, s_red);
    rc_lds_barrier();
    const int all = a.n_head * vdim, parts = st.parts();
    float* row = a.scratch + (size_t)RC_CNT_STRIDE * n_rows + (size_t)rr * all; /* behind the arrival counters: the row's heads */
    for (int i = tid; i < vdim; i += NT) {
        float so = 0.f;
        for (int g = 0; g < parts; g++) so += s_red[(size_t)g * vs + i];
        rc_st_sc1(row + h * vdim + i, fmaf(s_one[0], s_v[i], lam * so));
    }
    // the heads' outputs leave with write-through stores; every wave has their acknowledgements before one lane counts the workgroup in; the last one in norms and gates the row
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    int* counter = reinterpret_cast<int*>(a.scratch) + RC_CNT_STRIDE * (size_t)rr;
    if (tid == 0) *s_last = __hip_atomic_fetch_add(counter, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == a.n_head - 1;
    __syncthreads();
    if (!*s_last) return;
    if (tid == 0) __hip_atomic_store(counter, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    constexpr int KEEP = 8; /* of the row's outputs per thread in registers */
    float y[KEEP], ss = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; j++) {
        const int i = tid + j * NT;
        y[j] = i < all ? rc_ld_sc1(row + i) : 0.f;
    }
#pragma unroll
    for (int j = 0; j < KEEP; j++) ss = fmaf(y[j], y[j], ss);
    for (int i = tid + KEEP * NT; i < all; i += NT) {
        const float x = rc_ld_sc1(row + i);
        ss = fmaf(x, x, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) s_one[4 + wid] = ss;
    rc_lds_barrier();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < NW; w++) ss += s_one[4 + w];
    const float rs = a.out_scale / sqrtf(ss / (float)all + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)rr * a.ldout;
    auto finish = [&](int i, float x) { rb_st(out + i, x * rs * rb_ld(reinterpret_cast<const T*>(a.norm_w) + i) * rb_sigmoid(rb_ld(raw + a.col_g + i))); };
#pragma unroll
    for (int j = 0; j < KEEP; j++)
        if (tid + j * NT < all) finish(tid + j * NT, y[j]);
    for (int i = tid + KEEP * NT; i < all; i += NT) finish(i, rc_ld_sc1(row + i));
}

}  // namespace kf
