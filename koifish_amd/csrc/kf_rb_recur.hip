// kf_rb_recur.hip -- the recurrent layers of a row batch (kf_rb.h): the gated delta rule with a decay per key channel, and the sum with one constant decay per head.
//
// Decode: one workgroup per (head, row) holds the head's whole state matrix in registers -- a thread a few rows of four neighbouring columns -- and does the whole layer between the
// two products: convolution, SiLU, unit norms, the low-rank decay and gate, the state's step, the norm and the gate of the output.  S^T k and S^T q come from ONE walk over the old
// state: with k' = g k and q' = g q (row by row) S'^T q = S^T q' + (q . k) u, so the new state is only written, never read again.
// Prompts: a preparation pass per row and head, the walk over the tokens, the norm and gate per row.
#include <math.h>

#include <algorithm>

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
constexpr int RC_CNT_STRIDE = 16; /* words between arrival counters */
static __host__ __device__ inline int rc_up(int n, int m) { return (n + m - 1) / m * m; }

// row r of a product's weight (ld columns) times a[0 .. rank), a in LDS padded with zeros to a multiple of 8
__device__ __forceinline__ float rc_weight_dot(const uint16_t* __restrict__ w, int ld, int r, const float* a, int rank) {
    const uint16_t* tile = w + (size_t)(r / 16) * (ld / 32) * 512 + (r & 15) * 8;
    float s = 0.f;
    for (int o = 0; o < (rank + 7) / 8; o++) {
        const u32x4 v = *reinterpret_cast<const u32x4*>(tile + (o >> 2) * 512 + (o & 3) * 128);
        const float* x = a + 8 * o;
        s = fmaf(bf_lo(v.x), x[0], s), s = fmaf(bf_hi(v.x), x[1], s), s = fmaf(bf_lo(v.y), x[2], s), s = fmaf(bf_hi(v.y), x[3], s);
        s = fmaf(bf_lo(v.z), x[4], s), s = fmaf(bf_hi(v.z), x[5], s), s = fmaf(bf_lo(v.w), x[6], s), s = fmaf(bf_hi(v.w), x[7], s);
    }
    return s;
}
__device__ __forceinline__ float rc_weight_dot(const float* __restrict__ w, int ld, int r, const float* a, int rank) {
    float s = 0.f;
    for (int i = 0; i < rank; i++) s = fmaf(w[(size_t)r * ld + i], a[i], s);
    return s;
}
// channel c of the convolution at position pos, batch row r (the batch holds the sequence's positions from pos0 on), before the activation
template <class T>
__device__ __forceinline__ float rc_conv(const kf_rb_delta& a, const T* raw_r, const T* hist, int channels, int c, int pos, int pos0) {
    const T* w = reinterpret_cast<const T*>(a.conv) + (size_t)c * a.taps;
    float s = 0.f;
    for (int j = a.taps - 1; j >= 0; j--) {
        const int p = pos - j;
        if (p < 0) continue;
        const float x = p >= pos0 ? rb_ld(raw_r - (int64_t)j * a.ldraw + c) : rb_ld(hist + (size_t)(p % a.taps) * channels + c);
        s = fmaf(rb_ld(w + a.taps - 1 - j), x, s);
    }
    return s;
}

// ---- decode.  NT threads: groups of vs / 4 threads side by side, each group the rows rg, rg + RG, ...; RPT rows of a thread stay in registers (KEEP), otherwise they are read twice
constexpr int RC_RPT = 16;
template <class T, int NT, bool KEEP>
__global__ void __launch_bounds__(NT) rb_delta_step_kernel(const kf_rb_delta a, const int32_t* __restrict__ meta) {
    extern __shared__ float smem[];
    const int h = blockIdx.x, rr = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int pos = meta[KF_RB_META * rr], slot = meta[KF_RB_META * rr + 1];
    if (pos < 0) return; /* workgroup-uniform */
    const int dim = a.dim, vdim = a.vdim, vs = rc_up(vdim, 4), c4 = vs / 4, RG = NT / c4, rg = tid / c4, col = 4 * (tid - rg * c4);
    const int kvh = h / (a.n_head / a.n_kv), qd = a.n_kv * dim, channels = 2 * qd + a.n_head * vdim;
    const int ra8 = rc_up(a.rank_a, 8), rg8 = rc_up(a.rank_g, 8), d4 = rc_up(dim, 4);
    float *s_q = smem, *s_k = s_q + d4, *s_g = s_k + d4, *s_v = s_g + d4, *s_z = s_v + vs, *s_a = s_z + vs, *s_gl = s_a + ra8, *s_red = s_gl + rg8 /* [2][RG][vs] */, *s_one = s_red + 2 * NT * 4;
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + (pos & 1)) * side + h * head;
    const bool on = rg < RG, old = pos > 0;
    f32x4 S[KEEP ? RC_RPT : 1];
    if constexpr (KEEP) {
#pragma unroll
        for (int i = 0; i < RC_RPT; i++) {
            const int r = rg + i * RG;
            S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (on && old && r < dim) S[i] = *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col);
        }
    }
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)rr * a.ldraw;
    T* hist = reinterpret_cast<T*>(a.hist) + (size_t)slot * a.hist_slot;
    for (int i = tid; i < ra8 + rg8; i += NT) {
        const bool g = i >= ra8;
        const int j = g ? i - ra8 : i;
        s_a[i] = j < (g ? a.rank_g : a.rank_a) ? rb_ld(raw + (g ? a.col_g : a.col_a) + j) : 0.f;
    }
    for (int i = tid; i < 2 * dim + vdim; i += NT) { /* the head's channels: q, k, v */
        const int c = i < dim ? kvh * dim + i : (i < 2 * dim ? qd + kvh * dim + (i - dim) : 2 * qd + h * vdim + (i - 2 * dim));
        const float y = rc_silu(rc_conv(a, raw, hist, channels, c, pos, pos));
        (i < dim ? s_q[i] : (i < 2 * dim ? s_k[i - dim] : s_v[i - 2 * dim])) = y;
        if (i >= 2 * dim || h == kvh * (a.n_head / a.n_kv)) hist[(size_t)(pos % a.taps) * channels + c] = raw[c];
    }
    for (int i = vdim + tid; i < vs; i += NT) s_v[i] = 0.f;
    __syncthreads();
    for (int w = wid; w < 2; w += NT / 64) { /* 1 / length of q and of k, and q . k between them below */
        float ss = 0.f;
        const float* x = w ? s_k : s_q;
        for (int i = lane; i < dim; i += 64) ss = fmaf(x[i], x[i], ss);
        ss = wave_sum(ss);
        if (lane == 0) s_one[w] = 1.0f / sqrtf(ss + a.unit_eps);
    }
    const T *wa = reinterpret_cast<const T*>(a.w_a2), *wg = reinterpret_cast<const T*>(a.w_g2);
    const float rate = expf(rb_ld(reinterpret_cast<const T*>(a.a_log) + h));
    for (int i = tid; i < dim; i += NT) {
        const float z = rc_weight_dot(wa, a.ld_a, h * dim + i, s_a, a.rank_a) + rb_ld(reinterpret_cast<const T*>(a.dt_bias) + h * dim + i);
        s_g[i] = expf(-rate * rb_softplus(z));
    }
    for (int i = tid; i < vdim; i += NT) s_z[i] = rb_sigmoid(rc_weight_dot(wg, a.ld_g, h * vdim + i, s_gl, a.rank_g));
    __syncthreads();
    const float qn = s_one[0] * a.q_scale, kn = s_one[1];
    if (wid == 0) {
        float d = 0.f;
        for (int i = lane; i < dim; i += 64) d = fmaf(s_q[i], s_k[i], d);
        d = wave_sum(d);
        if (lane == 0) s_one[2] = d * qn * kn;
    }
    f32x4 p = f32x4{0.f, 0.f, 0.f, 0.f}, o = p;
    auto walk = [&](int r, f32x4 s) {
        const float g = s_g[r], kk = g * (s_k[r] * kn), qq = g * (s_q[r] * qn);
#pragma unroll
        for (int j = 0; j < 4; j++) p[j] = fmaf(kk, s[j], p[j]), o[j] = fmaf(qq, s[j], o[j]);
    };
    if (on && old) {
        if constexpr (KEEP) {
#pragma unroll
            for (int i = 0; i < RC_RPT; i++)
                if (rg + i * RG < dim) walk(rg + i * RG, S[i]);
        } else {
            for (int r = rg; r < dim; r += RG) walk(r, *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col));
        }
    }
    if (on) {
        *reinterpret_cast<f32x4*>(s_red + (size_t)rg * vs + col) = p;
        *reinterpret_cast<f32x4*>(s_red + (size_t)(RG + rg) * vs + col) = o;
    }
    __syncthreads();
    const float beta = rb_sigmoid(rb_ld(raw + a.col_b + h)), qk = s_one[2];
    float ss = 0.f;
    for (int i = tid; i < vs; i += NT) {
        float sp = 0.f, so = 0.f;
        for (int g = 0; g < RG; g++) sp += s_red[(size_t)g * vs + i], so += s_red[(size_t)(RG + g) * vs + i];
        const float u = beta * (s_v[i] - sp), y = fmaf(qk, u, so);
        s_v[i] = i < vdim ? u : 0.f;
        s_red[i] = y; /* this thread's column of the first group: nobody else's */
        if (i < vdim) ss = fmaf(y, y, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) s_one[4 + wid] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; w++) ss += s_one[4 + w];
    const float rs = 1.0f / sqrtf(ss / (float)vdim + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)rr * a.ldout + (size_t)h * vdim;
    for (int i = tid; i < vdim; i += NT) rb_st(out + i, s_red[i] * rs * rb_ld(reinterpret_cast<const T*>(a.norm_w) + i) * s_z[i]);
    if (on) {
        const f32x4 u = *reinterpret_cast<const f32x4*>(s_v + col);
        auto write = [&](int r, f32x4 s) {
            const float g = s_g[r], kk = s_k[r] * kn;
            f32x4 n;
#pragma unroll
            for (int j = 0; j < 4; j++) n[j] = fmaf(kk, u[j], g * s[j]);
            *reinterpret_cast<f32x4*>(S1 + (size_t)r * vs + col) = n;
        };
        if constexpr (KEEP) {
#pragma unroll
            for (int i = 0; i < RC_RPT; i++)
                if (rg + i * RG < dim) write(rg + i * RG, S[i]);
        } else {
            for (int r = rg; r < dim; r += RG) {
                f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
                if (old) s = *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col);
                write(r, s);
            }
        }
    }
}
template <class T, int NT, bool KEEP>
__global__ void __launch_bounds__(NT) rb_decay_step_kernel(const kf_rb_decay a, const int32_t* __restrict__ meta) {
    extern __shared__ float smem[];
    const int h = blockIdx.x, rr = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int pos = meta[KF_RB_META * rr], slot = meta[KF_RB_META * rr + 1];
    if (pos < 0) return; /* workgroup-uniform */
    const int dim = a.dim, vdim = a.vdim, vs = rc_up(vdim, 4), c4 = vs / 4, RG = NT / c4, rg = tid / c4, col = 4 * (tid - rg * c4);
    float *s_q = smem, *s_k = s_q + rc_up(dim, 4), *s_v = s_k + rc_up(dim, 4), *s_red = s_v + vs /* [RG][vs] */, *s_one = s_red + NT * 4;
    __shared__ int s_last;
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + (pos & 1)) * side + h * head;
    const bool on = rg < RG, old = pos > 0;
    const float lam = a.decay[h];
    f32x4 S[KEEP ? RC_RPT : 1];
    if constexpr (KEEP) {
#pragma unroll
        for (int i = 0; i < RC_RPT; i++) {
            const int r = rg + i * RG;
            S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (on && old && r < dim) S[i] = *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col);
        }
    }
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)rr * a.ldraw;
    const T* q = raw + a.col_q + (size_t)h * dim;
    const T* v = raw + a.col_q + (size_t)2 * a.n_head * dim + (size_t)h * vdim;
    for (int i = tid; i < dim; i += NT) s_q[i] = rb_ld(q + i), s_k[i] = rb_ld(q + (size_t)a.n_head * dim + i);
    for (int i = tid; i < vs; i += NT) s_v[i] = i < vdim ? rb_ld(v + i) : 0.f;
    __syncthreads();
    if (wid == 0) {
        float d = 0.f;
        for (int i = lane; i < dim; i += 64) d = fmaf(s_q[i], s_k[i], d);
        d = wave_sum(d);
        if (lane == 0) s_one[0] = d;
    }
    f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f}, u = o;
    if (on) u = *reinterpret_cast<const f32x4*>(s_v + col);
    auto step = [&](int r, f32x4 s) {
        const float qq = s_q[r], kk = s_k[r];
        f32x4 n;
#pragma unroll
        for (int j = 0; j < 4; j++) o[j] = fmaf(qq, s[j], o[j]), n[j] = fmaf(kk, u[j], lam * s[j]);
        *reinterpret_cast<f32x4*>(S1 + (size_t)r * vs + col) = n;
    };
    if (on) {
        if constexpr (KEEP) {
#pragma unroll
            for (int i = 0; i < RC_RPT; i++)
                if (rg + i * RG < dim) step(rg + i * RG, S[i]);
        } else {
            for (int r = rg; r < dim; r += RG) {
                f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
                if (old) s = *reinterpret_cast<const f32x4*>(S0 + (size_t)r * vs + col);
                step(r, s);
            }
        }
        *reinterpret_cast<f32x4*>(s_red + (size_t)rg * vs + col) = o;
    }
    __syncthreads();
    const int all = a.n_head * vdim;
    float* parts = a.scratch + (size_t)RC_CNT_STRIDE * gridDim.y + (size_t)rr * all; /* behind the arrival counters: the row's heads */
    for (int i = tid; i < vdim; i += NT) {
        float so = 0.f;
        for (int g = 0; g < RG; g++) so += s_red[(size_t)g * vs + i];
        rc_st_sc1(parts + h * vdim + i, fmaf(s_one[0], s_v[i], lam * so));
    }
    // the heads' outputs leave with write-through stores; every wave has their acknowledgements before one lane counts the workgroup in; the last one in norms and gates the row
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    int* counter = reinterpret_cast<int*>(a.scratch) + RC_CNT_STRIDE * (size_t)rr;
    if (tid == 0) s_last = __hip_atomic_fetch_add(counter, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (int)gridDim.x - 1;
    __syncthreads();
    if (!s_last) return;
    if (tid == 0) __hip_atomic_store(counter, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    float ss = 0.f;
    for (int i = tid; i < all; i += NT) {
        const float y = rc_ld_sc1(parts + i);
        ss = fmaf(y, y, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) s_one[4 + wid] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; w++) ss += s_one[4 + w];
    const float rs = a.out_scale / sqrtf(ss / (float)all + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)rr * a.ldout;
    for (int i = tid; i < all; i += NT) rb_st(out + i, rc_ld_sc1(parts + i) * rs * rb_ld(reinterpret_cast<const T*>(a.norm_w) + i) * rb_sigmoid(rb_ld(raw + a.col_g + i)));
}

// ---- prompts
// where a delta layer's prepared rows lie in its scratch (floats)
struct RcPrep {
    float *qk, *v, *g, *beta; /* [rows][2 n_kv dim] q then k, [rows][n_head vdim] (the outputs take its place), [rows][n_head dim], [rows][n_head] */
};
static RcPrep rc_prep_at(float* s, size_t rows, int n_head, int n_kv, int dim, int vdim) {
    RcPrep p;
    p.qk = s, p.v = p.qk + rows * 2 * n_kv * dim, p.g = p.v + rows * n_head * vdim, p.beta = p.g + rows * n_head * dim;
    return p;
}
// one wave per (row, unit): a q head, a k head, a v head, a head's decays and step size
template <class T>
__global__ void __launch_bounds__(256) rb_delta_prep_kernel(const kf_rb_delta a, const RcPrep out, const int32_t* __restrict__ meta) {
    const int r = blockIdx.x, lane = threadIdx.x & 63;
    int u = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int pos = meta[KF_RB_META * r], pos0 = meta[KF_RB_META * r + 2];
    if (u >= 2 * a.n_kv + 2 * a.n_head) return; /* no barrier below */
    const int dim = a.dim, vdim = a.vdim, qd = a.n_kv * dim, channels = 2 * qd + a.n_head * vdim;
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)r * a.ldraw;
    const T* hist = reinterpret_cast<const T*>(a.hist) + (size_t)meta[KF_RB_META * r + 1] * a.hist_slot;
    if (u < 2 * a.n_kv) {
        float x[8], ss = 0.f; /* dim <= 512 */
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const int c = lane + 64 * i;
            x[i] = 0.f;
            if (c < dim) x[i] = rc_silu(rc_conv(a, raw, hist, channels, u * dim + c, pos, pos0));
            ss = fmaf(x[i], x[i], ss);
        }
        const float f = (u < a.n_kv ? a.q_scale : 1.f) / sqrtf(wave_sum(ss) + a.unit_eps);
#pragma unroll
        for (int i = 0; i < 8; i++)
            if (lane + 64 * i < dim) out.qk[(size_t)r * 2 * qd + u * dim + lane + 64 * i] = x[i] * f;
        return;
    }
    u -= 2 * a.n_kv;
    if (u < a.n_head) {
        for (int c = lane; c < vdim; c += 64) out.v[(size_t)r * a.n_head * vdim + u * vdim + c] = rc_silu(rc_conv(a, raw, hist, channels, 2 * qd + u * vdim + c, pos, pos0));
        return;
    }
    u -= a.n_head;
    const float rate = expf(rb_ld(reinterpret_cast<const T*>(a.a_log) + u));
    for (int c = lane; c < dim; c += 64)
        out.g[((size_t)r * a.n_head + u) * dim + c] = expf(-rate * rb_softplus(a.a_z[(size_t)r * a.ld_az + u * dim + c] + rb_ld(reinterpret_cast<const T*>(a.dt_bias) + u * dim + c)));
    if (lane == 0) out.beta[(size_t)r * a.n_head + u] = rb_sigmoid(rb_ld(raw + a.col_b + u));
}
// the batch's last `taps` rows of every sequence into its slot's ring
template <class T>
__global__ void __launch_bounds__(256) rb_hist_kernel(const kf_rb_delta a, const int32_t* __restrict__ meta) {
    const int r = blockIdx.x, pos = meta[KF_RB_META * r], last = meta[KF_RB_META * r + 3];
    if (pos < 0 || pos <= last - a.taps) return;
    const int channels = 2 * a.n_kv * a.dim + a.n_head * a.vdim;
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)r * a.ldraw;
    T* hist = reinterpret_cast<T*>(a.hist) + (size_t)meta[KF_RB_META * r + 1] * a.hist_slot + (size_t)(pos % a.taps) * channels;
    for (int i = threadIdx.x; i < channels; i += 256) hist[i] = raw[i];
}

// token by token: a wave owns four columns of a head's state, its 16-lane rows share the key channels (rg, rg + 16, ...); the next token's rows are on their way while one is done
template <class T>
struct RcScan {
    const T *q, *k, *v; /* rows ldq / ldq / ldv apart; heads dim / dim / vdim apart */
    const float *g, *beta, *decay;
    float *o, *state;
    int64_t ldq, ldv, ldo;
    int n_head, per_k, dim, vdim; /* per_k: heads that share a k */
};
template <class T, int RPL, bool DELTA>
__global__ void __launch_bounds__(64) rb_scan_kernel(const RcScan<T> a, const int32_t* __restrict__ seqs) {
    const int h = blockIdx.x, lane = threadIdx.x, rg = lane & 15, col = blockIdx.y * 4 + (lane >> 4);
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3];
    const int dim = a.dim, vs = rc_up(a.vdim, 4);
    const bool on = col < a.vdim;
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos0 + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + ((pos0 + n - 1) & 1)) * side + h * head;
    const T *q = a.q + (size_t)row0 * a.ldq + (size_t)(h / a.per_k) * dim, *k = a.k + (size_t)row0 * a.ldq + (size_t)(h / a.per_k) * dim;
    const T* v = a.v + (size_t)row0 * a.ldv + (size_t)h * a.vdim + (on ? col : 0);
    const float* g = DELTA ? a.g + ((size_t)row0 * a.n_head + h) * dim : nullptr;
    const float* beta = DELTA ? a.beta + (size_t)row0 * a.n_head + h : nullptr;
    float* o = a.o + (size_t)row0 * a.ldo + (size_t)h * a.vdim + col;
    const float lam = DELTA ? 0.f : a.decay[h];
    float S[RPL], qn[RPL], kn[RPL], gn[RPL], vn, bn = 0.f;
#pragma unroll
    for (int i = 0; i < RPL; i++) {
        const int r = rg + 16 * i;
        S[i] = pos0 > 0 && r < dim ? S0[(size_t)r * vs + col] : 0.f; /* (columns past vdim, below vs: zeros) */
    }
    auto fetch = [&](int t) {
#pragma unroll
        for (int i = 0; i < RPL; i++) {
            const int r = rg + 16 * i;
            qn[i] = kn[i] = gn[i] = 0.f;
            if (r < dim) {
                qn[i] = rb_ld(q + (size_t)t * a.ldq + r), kn[i] = rb_ld(k + (size_t)t * a.ldq + r);
                if constexpr (DELTA) gn[i] = g[(size_t)t * a.n_head * dim + r];
            }
        }
        vn = on ? rb_ld(v + (size_t)t * a.ldv) : 0.f;
        if constexpr (DELTA) bn = beta[(size_t)t * a.n_head];
    };
    fetch(0);
    for (int t = 0; t < n; t++) {
        float qc[RPL], kc[RPL], gc[RPL];
#pragma unroll
        for (int i = 0; i < RPL; i++) qc[i] = qn[i], kc[i] = kn[i], gc[i] = gn[i];
        float u = vn;
        const float b = bn;
        if (t + 1 < n) fetch(t + 1);
        if constexpr (DELTA) {
            float p = 0.f;
#pragma unroll
            for (int i = 0; i < RPL; i++) S[i] *= gc[i], p = fmaf(kc[i], S[i], p);
            u = b * (u - row16_sum(p));
        } else {
#pragma unroll
            for (int i = 0; i < RPL; i++) S[i] *= lam;
        }
        float y = 0.f;
#pragma unroll
        for (int i = 0; i < RPL; i++) S[i] = fmaf(kc[i], u, S[i]), y = fmaf(qc[i], S[i], y);
        y = row16_sum(y);
        if (on && rg == 0) o[(size_t)t * a.ldo] = y;
    }
    if (col < vs)
#pragma unroll
        for (int i = 0; i < RPL; i++)
            if (rg + 16 * i < dim) S1[(size_t)(rg + 16 * i) * vs + col] = S[i];
}
template <class T, bool DELTA>
static int scan_go(hipStream_t st, const RcScan<T>& a, const int32_t* seqs, int n_seq) {
    const dim3 grid(a.n_head, (a.vdim + 3) / 4, n_seq);
    const int rpl = (a.dim + 15) / 16;
    if (rpl <= 2) hipLaunchKernelGGL((rb_scan_kernel<T, 2, DELTA>), grid, dim3(64), 0, st, a, seqs);
    else if (rpl <= 4) hipLaunchKernelGGL((rb_scan_kernel<T, 4, DELTA>), grid, dim3(64), 0, st, a, seqs);
    else if (rpl <= 8) hipLaunchKernelGGL((rb_scan_kernel<T, 8, DELTA>), grid, dim3(64), 0, st, a, seqs);
    else if (rpl <= 16) hipLaunchKernelGGL((rb_scan_kernel<T, 16, DELTA>), grid, dim3(64), 0, st, a, seqs);
    else if (rpl <= 32) hipLaunchKernelGGL((rb_scan_kernel<T, 32, DELTA>), grid, dim3(64), 0, st, a, seqs);
    else return 1;
    return KF_OK;
}

// out = scale * o / sqrt(mean(o^2) + eps) * w * sigmoid(gate), the mean over groups of `size` columns; w: of one group (shared) or of all
struct RcGate {
    const float* o;
    const void *w, *gate;
    void* out;
    int64_t ldo, ldg, ldout;
    int groups, size;
    float scale, eps;
};
template <class T>
__device__ __forceinline__ void rc_gate_store(const RcGate& a, const float* o, const T* gate, T* out, int c, int wc, float rs) {
    rb_st(out + c, o[c] * rs * rb_ld(reinterpret_cast<const T*>(a.w) + wc) * rb_sigmoid(rb_ld(gate + c)));
}
template <class T>
__global__ void __launch_bounds__(256) rb_gate_kernel(const RcGate a) {
    __shared__ float red[4];
    const int r = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const float* o = a.o + (size_t)r * a.ldo;
    const T* gate = reinterpret_cast<const T*>(a.gate) + (size_t)r * a.ldg;
    T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.ldout;
    if (a.groups == 1) {
        float ss = 0.f;
        for (int c = tid; c < a.size; c += 256) ss = fmaf(o[c], o[c], ss);
        ss = wave_sum(ss);
        if (lane == 0) red[wid] = ss;
        __syncthreads();
        const float rs = a.scale / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.size + a.eps);
        for (int c = tid; c < a.size; c += 256) rc_gate_store<T>(a, o, gate, out, c, c, rs);
        return;
    }
    for (int g = wid; g < a.groups; g += 4) {
        float ss = 0.f;
        for (int c = lane; c < a.size; c += 64) ss = fmaf(o[g * a.size + c], o[g * a.size + c], ss);
        const float rs = a.scale / sqrtf(wave_sum(ss) / (float)a.size + a.eps);
        for (int c = lane; c < a.size; c += 64) rc_gate_store<T>(a, o, gate, out, g * a.size + c, c, rs);
    }
}

template <class T>
static int delta_prefill_go(hipStream_t st, const kf_rb_delta& a, const int32_t* meta, int n, const int32_t* seqs, int n_seq) {
    const RcPrep p = rc_prep_at(a.scratch, n, a.n_head, a.n_kv, a.dim, a.vdim);
    hipLaunchKernelGGL(rb_delta_prep_kernel<T>, dim3(n, (2 * a.n_kv + 2 * a.n_head + 3) / 4), dim3(256), 0, st, a, p, meta);
    const int64_t ldq = 2 * (int64_t)a.n_kv * a.dim, ldv = (int64_t)a.n_head * a.vdim;
    const RcScan<float> s{p.qk, p.qk + (size_t)a.n_kv * a.dim, p.v, p.g, p.beta, nullptr, p.v, a.state, ldq, ldv, ldv, a.n_head, a.n_head / a.n_kv, a.dim, a.vdim};
    if (scan_go<float, true>(st, s, seqs, n_seq)) return 1;
    hipLaunchKernelGGL(rb_hist_kernel<T>, dim3(n), dim3(256), 0, st, a, meta);
    const RcGate g{p.v, a.norm_w, a.g_z, a.out, ldv, a.ld_gz, a.ldout, a.n_head, a.vdim, 1.f, a.eps};
    hipLaunchKernelGGL(rb_gate_kernel<T>, dim3(n), dim3(256), 0, st, g);
    return KF_OK;
}
template <class T>
static int decay_prefill_go(hipStream_t st, const kf_rb_decay& a, int n, const int32_t* seqs, int n_seq) {
    const int64_t ldo = (int64_t)a.n_head * a.vdim;
    float* o = a.scratch + (size_t)RC_CNT_STRIDE * n;
    const T* q = reinterpret_cast<const T*>(a.raw) + a.col_q;
    const RcScan<T> s{q, q + (size_t)a.n_head * a.dim, q + (size_t)2 * a.n_head * a.dim, nullptr, nullptr, a.decay, o, a.state, a.ldraw, a.ldraw, ldo, a.n_head, 1, a.dim, a.vdim};
    if (scan_go<T, false>(st, s, seqs, n_seq)) return 1;
    const RcGate g{o, a.norm_w, reinterpret_cast<const T*>(a.raw) + a.col_g, a.out, ldo, a.ldraw, a.ldout, 1, a.n_head * a.vdim, a.out_scale, a.eps};
    hipLaunchKernelGGL(rb_gate_kernel<T>, dim3(n), dim3(256), 0, st, g);
    return KF_OK;
}
// threads of a decode workgroup: at most RC_RPT rows of four columns each where the state allows it
static int step_threads(int dim, int vdim) {
    const int vs = rc_up(vdim, 4);
    for (int nt : {256, 512, 1024})
        if (vs / 4 <= nt && (dim + nt / (vs / 4) - 1) / (nt / (vs / 4)) <= RC_RPT) return nt;
    return 0; /* 1024 threads that read the state twice */
}
template <class T>
static void delta_step_go(hipStream_t st, const kf_rb_delta& a, const int32_t* meta, int n) {
    const int nt = step_threads(a.dim, a.vdim);
    const size_t smem = (3 * (size_t)rc_up(a.dim, 4) + 2 * rc_up(a.vdim, 4) + rc_up(a.rank_a, 8) + rc_up(a.rank_g, 8) + 8 * (size_t)(nt ? nt : 1024) + 32) * 4;
    const dim3 grid(a.n_head, n);
    if (nt == 256) hipLaunchKernelGGL((rb_delta_step_kernel<T, 256, true>), grid, dim3(256), smem, st, a, meta);
    else if (nt == 512) hipLaunchKernelGGL((rb_delta_step_kernel<T, 512, true>), grid, dim3(512), smem, st, a, meta);
    else if (nt == 1024) hipLaunchKernelGGL((rb_delta_step_kernel<T, 1024, true>), grid, dim3(1024), smem, st, a, meta);
    else hipLaunchKernelGGL((rb_delta_step_kernel<T, 1024, false>), grid, dim3(1024), smem, st, a, meta);
}
template <class T>
static void decay_step_go(hipStream_t st, const kf_rb_decay& a, const int32_t* meta, int n) {
    const int nt = step_threads(a.dim, a.vdim);
    const size_t smem = (2 * (size_t)rc_up(a.dim, 4) + rc_up(a.vdim, 4) + 4 * (size_t)(nt ? nt : 1024) + 32) * 4;
    const dim3 grid(a.n_head, n);
    if (nt == 256) hipLaunchKernelGGL((rb_decay_step_kernel<T, 256, true>), grid, dim3(256), smem, st, a, meta);
    else if (nt == 512) hipLaunchKernelGGL((rb_decay_step_kernel<T, 512, true>), grid, dim3(512), smem, st, a, meta);
    else if (nt == 1024) hipLaunchKernelGGL((rb_decay_step_kernel<T, 1024, true>), grid, dim3(1024), smem, st, a, meta);
    else hipLaunchKernelGGL((rb_decay_step_kernel<T, 1024, false>), grid, dim3(1024), smem, st, a, meta);
}

}  // namespace kf

using namespace kf;
constexpr int RC_MAX_DIM = 512;
static int check_delta(const kf_rb_delta* a, const int32_t* meta, int n, const char* who) {
    if (!a || !meta || n < 1 || !a->raw || !a->out || !a->conv || !a->a_log || !a->dt_bias || !a->norm_w || !a->state || !a->hist) return abi_fail(KF_INVALID_ARGS, "%s: null pointer", who);
    if (a->type != KF_BF16 && a->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: storage %d", who, a->type);
    if (a->n_head < 1 || a->n_kv < 1 || a->n_head % a->n_kv || a->dim < 1 || a->vdim < 1 || a->taps < 1) return abi_fail(KF_INVALID_ARGS, "%s: %d / %d heads of %d / %d, %d taps", who, a->n_head, a->n_kv, a->dim, a->vdim, a->taps);
    if (a->dim > RC_MAX_DIM || a->vdim > RC_MAX_DIM) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: head sizes %d / %d (served: up to %d)", who, a->dim, a->vdim, RC_MAX_DIM);
    const int64_t channels = 2 * (int64_t)a->n_kv * a->dim + (int64_t)a->n_head * a->vdim;
    if (a->hist_slot < channels * a->taps || a->ldout < (int64_t)a->n_head * a->vdim || a->col_b < channels || a->ldraw < a->col_b + a->n_head) return abi_fail(KF_INVALID_ARGS, "%s: strides", who);
    if (!al16(a->state) || !al16(a->raw) || !al16(a->out)) return abi_fail(KF_BLAS_UNALIGN, "%s: unaligned pointer", who);
    return KF_OK;
}
static int check_decay(const kf_rb_decay* a, const int32_t* meta, int n, const char* who) {
    if (!a || !meta || n < 1 || !a->raw || !a->out || !a->norm_w || !a->decay || !a->state || !a->scratch) return abi_fail(KF_INVALID_ARGS, "%s: null pointer", who);
    if (a->type != KF_BF16 && a->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: storage %d", who, a->type);
    if (a->n_head < 1 || a->dim < 1 || a->vdim < 1) return abi_fail(KF_INVALID_ARGS, "%s: %d heads of %d / %d", who, a->n_head, a->dim, a->vdim);
    if (a->dim > RC_MAX_DIM || a->vdim > RC_MAX_DIM) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: head sizes %d / %d (served: up to %d)", who, a->dim, a->vdim, RC_MAX_DIM);
    const int64_t qk = 2 * (int64_t)a->n_head * a->dim, all = (int64_t)a->n_head * a->vdim;
    if (a->col_q < 0 || a->col_g < 0 || a->ldraw < a->col_q + qk + all || a->ldraw < a->col_g + all || a->ldout < all) return abi_fail(KF_INVALID_ARGS, "%s: strides", who);
    if (!al16(a->state) || !al16(a->scratch)) return abi_fail(KF_BLAS_UNALIGN, "%s: unaligned pointer", who);
    return KF_OK;
}
static int launched(int rc, const char* who) {
    if (rc == 1) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: no kernel for these sizes", who);
    if (rc != KF_OK) return abi_fail(rc, "%s: launch failed", who);
    return hipGetLastError() == hipSuccess ? KF_OK : abi_fail(KF_HIP_CHECK, "%s: launch failed", who);
}
extern "C" {

size_t kf_rb_delta_scratch(int type, int n_rows, int n_seq, int n_head, int n_kv, int dim, int vdim) {
    if (n_rows < 1 || n_seq < 1) return 0;
    return ((size_t)n_rows * (2 * (size_t)n_kv * dim + (size_t)n_head * (dim + vdim + 1)) + 16) * 4;
}
size_t kf_rb_decay_scratch(int type, int n_rows, int n_seq, int n_head, int dim, int vdim) {
    if (n_rows < 1) return 0;
    return ((size_t)n_rows * (RC_CNT_STRIDE + (size_t)n_head * vdim) + 16) * 4;
}
int kf_rb_delta_prefill(kf_ctx* c, const kf_rb_delta* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n) {
    CHKCTX(c);
    const int rc = check_delta(a, meta, n_rows, "kf_rb_delta_prefill");
    if (rc) return rc;
    if (!seqs || n_seq < 1 || max_n < 1 || max_n > n_rows || !a->a_z || !a->g_z || !a->scratch || !al16(a->scratch) || a->ld_az < (int64_t)a->n_head * a->dim || a->ld_gz < (int64_t)a->n_head * a->vdim)
        return abi_fail(KF_INVALID_ARGS, "kf_rb_delta_prefill: bad arguments");
    return launched(a->type == KF_BF16 ? delta_prefill_go<uint16_t>(c->stream, *a, meta, n_rows, seqs, n_seq) : delta_prefill_go<float>(c->stream, *a, meta, n_rows, seqs, n_seq), "kf_rb_delta_prefill");
}
int kf_rb_delta_decode(kf_ctx* c, const kf_rb_delta* a, const int32_t* meta, int n_rows) {
    CHKCTX(c);
    const int rc = check_delta(a, meta, n_rows, "kf_rb_delta_decode");
    if (rc) return rc;
    if (!a->w_a2 || !a->w_g2 || a->rank_a < 1 || a->rank_g < 1 || a->rank_a > 2048 || a->rank_g > 2048 || a->ld_a < a->rank_a || a->ld_g < a->rank_g || a->ld_a % KF_RB_PAD || a->ld_g % KF_RB_PAD ||
        a->col_a < 0 || a->col_g < 0 || a->ldraw < a->col_a + a->rank_a || a->ldraw < a->col_g + a->rank_g || !al16(a->w_a2) || !al16(a->w_g2))
        return abi_fail(KF_INVALID_ARGS, "kf_rb_delta_decode: low-rank factors");
    if (a->type == KF_BF16) delta_step_go<uint16_t>(c->stream, *a, meta, n_rows);
    else delta_step_go<float>(c->stream, *a, meta, n_rows);
    return launched(KF_OK, "kf_rb_delta_decode");
}
int kf_rb_decay_prefill(kf_ctx* c, const kf_rb_decay* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n) {
    CHKCTX(c);
    const int rc = check_decay(a, meta, n_rows, "kf_rb_decay_prefill");
    if (rc) return rc;
    if (!seqs || n_seq < 1 || max_n < 1 || max_n > n_rows) return abi_fail(KF_INVALID_ARGS, "kf_rb_decay_prefill: bad arguments");
    return launched(a->type == KF_BF16 ? decay_prefill_go<uint16_t>(c->stream, *a, n_rows, seqs, n_seq) : decay_prefill_go<float>(c->stream, *a, n_rows, seqs, n_seq), "kf_rb_decay_prefill");
}
int kf_rb_decay_decode(kf_ctx* c, const kf_rb_decay* a, const int32_t* meta, int n_rows) {
    CHKCTX(c);
    const int rc = check_decay(a, meta, n_rows, "kf_rb_decay_decode");
    if (rc) return rc;
    if (a->type == KF_BF16) decay_step_go<uint16_t>(c->stream, *a, meta, n_rows);
    else decay_step_go<float>(c->stream, *a, meta, n_rows);
    return launched(KF_OK, "kf_rb_decay_decode");
}

}  // extern "C"
