// kf_rb_recur.hip -- the recurrent layers of a row batch (kf_rb.h): the gated delta rule with a decay per key channel, and the sum with one constant decay per head.
//
// Decode: one workgroup per (head, row) holds the head's whole state matrix in registers -- a thread a few rows of four neighbouring columns -- and does the whole layer between the
// two products: convolution, SiLU, unit norms, the low-rank decay and gate, the state's step, the norm and the gate of the output.  S^T k and S^T q come from ONE walk over the old
// state: with k' = g k and q' = g q (row by row) S'^T q = S^T q' + (q . k) u, so the new state is only written, never read again.
// Prompts: in chunks (below), or where the sizes are not served that way a preparation pass per row and head and a walk over the tokens; then the norm and gate per row.
#include <math.h>

#include <algorithm>

#include "kf_ctx.h"
#include "kf_rb_recur.h"

namespace kf {

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

// ---- decode
// eight consecutive columns of row r of a product's weight (ld columns), octet o, and their product with eight floats of LDS
__device__ __forceinline__ u32x4 rc_octet(const uint16_t* __restrict__ w, int ld, int r, int o) { return *reinterpret_cast<const u32x4*>(w + ((size_t)(r / 16) * (ld / 32) + (o >> 2)) * 512 + (r & 15) * 8 + (o & 3) * 128); }
__device__ __forceinline__ float rc_octet_dot(u32x4 v, const float* x, float s) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(x), b = *reinterpret_cast<const f32x4*>(x + 4);
    s = fmaf(bf_lo(v.x), a.x, s), s = fmaf(bf_hi(v.x), a.y, s), s = fmaf(bf_lo(v.y), a.z, s), s = fmaf(bf_hi(v.y), a.w, s);
    return fmaf(bf_hi(v.w), b.w, fmaf(bf_lo(v.w), b.z, fmaf(bf_hi(v.z), b.y, fmaf(bf_lo(v.z), b.x, s))));
}
struct RcOctet32 {
    f32x4 a, b;
};
__device__ __forceinline__ RcOctet32 rc_octet(const float* __restrict__ w, int ld, int r, int o) {
    const float* p = w + (size_t)r * ld + 8 * o;
    return RcOctet32{*reinterpret_cast<const f32x4*>(p), *reinterpret_cast<const f32x4*>(p + 4)};
}
__device__ __forceinline__ float rc_octet_dot(const RcOctet32& v, const float* x, float s) {
#pragma unroll
    for (int j = 0; j < 4; j++) s = fmaf(v.b[j], x[4 + j], fmaf(v.a[j], x[j], s));
    return s;
}
// One workgroup per (head, row).  What it reads sets out at once, in the order of its use: the channels' last inputs, the low-rank rows, the state (barriers wait for LDS only)
template <class T, int NT, int RPT>
__global__ void __launch_bounds__(NT, 4) rb_delta_step_kernel(const kf_rb_delta a, const int32_t* __restrict__ meta) {
    extern __shared__ float smem[];
    constexpr int NW = NT / 64, PF = NT > 512 || sizeof(T) == 4 ? 4 : 8; /* octets in flight per lane */
    const int h = blockIdx.x, rr = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int pos = meta[KF_RB_META * rr], slot = meta[KF_RB_META * rr + 1];
    if (pos < 0) return; /* workgroup-uniform */
    const int dim = a.dim, vdim = a.vdim, kvh = h / (a.n_head / a.n_kv), qd = a.n_kv * dim, channels = 2 * qd + a.n_head * vdim, n_ch = 2 * dim + vdim;
    const int ra8 = rc_up(a.rank_a, 8), rg8 = rc_up(a.rank_g, 8), d4 = rc_up(dim, 4), vs = rc_up(vdim, 4);
    float *s_a = smem, *s_gl = s_a + ra8, *s_q = s_gl + rg8, *s_k = s_q + d4, *s_g = s_k + d4, *s_v = s_g + d4, *s_z = s_v + vs, *s_red = s_z + vs /* [2][parts][vs] */, *s_one = s_red + 8 * NT;
    const T* raw = reinterpret_cast<const T*>(a.raw) + (size_t)rr * a.ldraw;
    T* hist = reinterpret_cast<T*>(a.hist) + (size_t)slot * a.hist_slot;
    auto channel = [&](int i) { return i < dim ? kvh * dim + i : (i < 2 * dim ? qd + kvh * dim + (i - dim) : 2 * qd + h * vdim + (i - 2 * dim)); };
    T x0[4], w0[4]; /* four taps: this thread's first channel */
    const bool four = a.taps == 4, ch_on = tid < n_ch;
    if (four && ch_on) {
        const int c = channel(tid);
#pragma unroll
        for (int j = 0; j < 4; j++) {
            x0[j] = j == 3 ? raw[c] : hist[(size_t)((pos + 1 + j) & 3) * channels + c]; /* row (pos - 3 + j) % 4 */
            w0[j] = reinterpret_cast<const T*>(a.conv)[(size_t)c * 4 + j];
        }
    }
    T lr0 = T();
    auto low_rank_input = [&](int i) { return i < ra8 ? (i < a.rank_a ? raw[a.col_a + i] : T()) : (i - ra8 < a.rank_g ? raw[a.col_g + i - ra8] : T()); };
    if (tid < ra8 + rg8) lr0 = low_rank_input(tid);
    // rows of the two factors: 32 of them per wave and turn, two lanes (16 apart) share a row's octets
    const T *wa = reinterpret_cast<const T*>(a.w_a2), *wg = reinterpret_cast<const T*>(a.w_g2);
    const int half = lane >> 4 & 1, n_row = dim + vdim;
    decltype(rc_octet(wa, 0, 0, 0)) pre[PF];
    {
        const int i = 32 * wid + (lane & 15) + 16 * (lane >> 5);
        const bool is_a = i < dim;
        const int no = (is_a ? ra8 : rg8) / 8;
#pragma unroll
        for (int j = 0; j < PF; j++) {
            pre[j] = decltype(rc_octet(wa, 0, 0, 0)){};
            if (i < n_row && half + 2 * j < no) pre[j] = is_a ? rc_octet(wa, a.ld_a, h * dim + i, half + 2 * j) : rc_octet(wg, a.ld_g, h * vdim + i - dim, half + 2 * j);
        }
    }
    RcStep<NT, RPT> st(dim, vdim, tid);
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + (pos & 1)) * side + h * head;
    st.load(S0, pos > 0);
    for (int i = tid; i < ra8 + rg8; i += NT) s_a[i] = rb_ld1(i == tid ? lr0 : low_rank_input(i));
    const bool first = h == kvh * (a.n_head / a.n_kv);
    for (int i = tid; i < n_ch; i += NT) { /* the head's channels: q, k, v */
        const int c = channel(i);
        float y;
        if (four && i == tid) {
            y = 0.f;
#pragma unroll
            for (int j = 0; j < 4; j++)
                if (pos - 3 + j >= 0) y = fmaf(rb_ld1(w0[j]), rb_ld1(x0[j]), y);
        } else {
            y = rc_conv(a, raw, hist, channels, c, pos, pos);
        }
        y *= rc_fast_sigmoid(y);
        (i < dim ? s_q[i] : (i < 2 * dim ? s_k[i - dim] : s_v[i - 2 * dim])) = y;
        if (i >= 2 * dim || first) hist[(size_t)(pos % a.taps) * channels + c] = raw[c];
    }
    for (int i = vdim + tid; i < vs; i += NT) s_v[i] = 0.f;
    const float rate = expf(rb_ld(reinterpret_cast<const T*>(a.a_log) + h)), beta = rb_sigmoid(rb_ld(raw + a.col_b + h));
    rc_lds_barrier();
    for (int g = wid; 32 * g < n_row; g += NW) {
        const int i = 32 * g + (lane & 15) + 16 * (lane >> 5);
        const bool is_a = i < dim, in = i < n_row;
        const int no = in ? (is_a ? ra8 : rg8) / 8 : 0, r = is_a ? h * dim + i : h * vdim + i - dim;
        const float* x = is_a ? s_a : s_gl;
        float z = 0.f;
#pragma unroll
        for (int j = 0; j < PF; j++) {
            const int o = half + 2 * j;
            if (o < no) z = rc_octet_dot(g == wid ? pre[j] : (is_a ? rc_octet(wa, a.ld_a, r, o) : rc_octet(wg, a.ld_g, r, o)), x + 8 * o, z);
        }
        for (int o = half + 2 * PF; o < no; o += 2) z = rc_octet_dot(is_a ? rc_octet(wa, a.ld_a, r, o) : rc_octet(wg, a.ld_g, r, o), x + 8 * o, z);
        z = xsum16(z);
        if (in && half == 0) {
            if (is_a) s_g[i] = rc_exp2(-rate * rc_softplus2(z + rb_ld(reinterpret_cast<const T*>(a.dt_bias) + r)));
            else s_z[i - dim] = rb_sigmoid(z);
        }
    }
    for (int w = NW - 1 - wid; w < 3; w += NW) { /* squares of q, of k, and q . k */
        const float *x = w == 1 ? s_k : s_q, *y = w ? s_k : s_q;
        float d = 0.f;
        for (int i = lane; i < dim; i += 64) d = fmaf(x[i], y[i], d);
        d = wave_sum(d);
        if (lane == 0) s_one[w] = d;
    }
    rc_lds_barrier();
    const float qn = a.q_scale / sqrtf(s_one[0] + a.unit_eps), kn = 1.0f / sqrtf(s_one[1] + a.unit_eps), qk = s_one[2] * qn * kn;
    f32x4 p = f32x4{0.f, 0.f, 0.f, 0.f}, o = p;
    st.each(S0, pos > 0, [&](int r, f32x4 s) {
        const float g = s_g[r], kk = g * (s_k[r] * kn), qq = g * (s_q[r] * qn);
#pragma unroll
        for (int j = 0; j < 4; j++) p[j] = fmaf(kk, s[j], p[j]), o[j] = fmaf(qq, s[j], o[j]);
    });
    const int parts = st.parts();
    st.partial(p, s_red), st.partial(o, s_red + (size_t)parts * vs);
    rc_lds_barrier();
    float ss = 0.f;
    for (int i = tid; i < vs; i += NT) {
        float sp = 0.f, so = 0.f;
        for (int g = 0; g < parts; g++) sp += s_red[(size_t)g * vs + i], so += s_red[(size_t)(parts + g) * vs + i];
        const float u = beta * (s_v[i] - sp), y = fmaf(qk, u, so);
        s_v[i] = i < vdim ? u : 0.f;
        s_red[i] = y; /* this thread's column of the first part: nobody else's */
        if (i < vdim) ss = fmaf(y, y, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) s_one[4 + wid] = ss;
    rc_lds_barrier();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < NW; w++) ss += s_one[4 + w];
    const float rs = 1.0f / sqrtf(ss / (float)vdim + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)rr * a.ldout + (size_t)h * vdim;
    for (int i = tid; i < vdim; i += NT) rb_st(out + i, s_red[i] * rs * rb_ld(reinterpret_cast<const T*>(a.norm_w) + i) * s_z[i]);
    const f32x4 u = *reinterpret_cast<const f32x4*>(s_v + st.col);
    st.each(S0, pos > 0, [&](int r, f32x4 s) {
        const float g = s_g[r], kk = s_k[r] * kn;
        f32x4 n;
#pragma unroll
        for (int j = 0; j < 4; j++) n[j] = fmaf(kk, u[j], g * s[j]);
        *reinterpret_cast<f32x4*>(S1 + (size_t)r * vs + st.col) = n;
    });
}
template <class T, int NT, int RPT>
__global__ void __launch_bounds__(NT) rb_decay_step_kernel(const kf_rb_decay a, const int32_t* __restrict__ meta) {
    extern __shared__ float smem[];
    rc_decay_step<T, NT, RPT>(a, meta, blockIdx.x, blockIdx.y, gridDim.y, smem);
}

// ---- prompts
// where a delta layer's prepared rows lie in its scratch (floats)
struct RcPrep {
    float *v, *qk, *g, *beta; /* [rows][n_head vdim] (the outputs take its place), [rows][2 n_kv dim] q then k, [rows][n_head dim], [rows][n_head] */
};
static RcPrep rc_prep_at(float* s, size_t rows, int n_head, int n_kv, int dim, int vdim) {
    RcPrep p;
    p.v = s, p.qk = p.v + rows * n_head * vdim, p.g = p.qk + rows * 2 * n_kv * dim, p.beta = p.g + rows * n_head * dim;
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
// the batch's last `taps` rows of every sequence into its slot's ring: grid (column blocks, taps, sequences)
template <class T>
__global__ void __launch_bounds__(256) rb_hist_kernel(const kf_rb_delta a, const int32_t* __restrict__ seqs) {
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3];
    const int channels = 2 * a.n_kv * a.dim + a.n_head * a.vdim, t = n - 1 - (int)blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (t < 0 || c >= channels) return;
    reinterpret_cast<T*>(a.hist)[(size_t)slot * a.hist_slot + (size_t)((pos0 + t) % a.taps) * channels + c] = reinterpret_cast<const T*>(a.raw)[(size_t)(row0 + t) * a.ldraw + c];
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

// ---- the delta rule in chunks of 64 tokens (prompts).  With G the logarithm of the decays' product from the chunk's start through a token, S0 the state in front of the chunk:
//   A_ij = sum over d of k_i k_j e^(G_i - G_j),  (I + diag(beta) A below the diagonal) [W U] = diag(beta) [k e^G, v],  u = U - W S0
//   o = (q e^G) S0 + (the same A with q_i, diagonal included) u,   S = e^(G_end) S0 + (k e^(G_end - G))^T u
// Everything but u is known without the state: one workgroup per (chunk, head) prepares it (rb_delta_chunk_kernel), then a workgroup per (head, 16 value columns) walks the chunks
// (rb_delta_walk_kernel).  All of it in 32 bits: v_mfma_f32_16x16x4_f32.  Its operands are read four k at a time (lane group g, register i holds k = 4 g + i): the register layout of a
// result is then the layout of a right operand, and a solved block feeds the next product without leaving its registers.
// No exponent is ever positive beyond what a float holds: logarithms are summed within blocks of 16 tokens and between blocks; a block row's left factors are taken from its own start
// (e^(G_i - start) <= 1), its right factors to that start (<= 1 in earlier blocks).  In the diagonal block the right factor is e^(start - G_j) >= 1: where a block's decays multiply to less
// than 2^-100 its entries are summed pair by pair instead.
constexpr int RC_C = 64;
__device__ __forceinline__ f32x4 rc_mfma(f32x4 a, f32x4 b, f32x4 c) { /* 16 x 16 x 16 */
#pragma unroll
    for (int i = 0; i < 4; i++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
    return c;
}
// what a chunk leaves for the walk, floats: W [64][DP], q e^G [64][DP], (k e^(G_end - G))^T [DP][64], q-k products [64][64], U [64][Vp], e^(G_end) [DP].  The matrices lie in 16 x 16
// tiles, row of tiles after row of tiles, 64 x 4 floats each in the order of a left operand (lane 16 g + r: row r, columns 4 g ..; U: of a result, rows 4 g .., column r): a wave reads a
// tile as one contiguous kilobyte
static __host__ __device__ inline size_t rc_chunk_floats(int DP, int Vp) { return (size_t)RC_C * (3 * DP + RC_C + Vp) + DP; }
// where element (row, col) of such a matrix lies
__device__ __forceinline__ int rc_tiled(int row, int col, int tiles) { return ((row / 16 * tiles + col / 16) * 64 + col % 16 / 4 * 16 + row % 16) * 4 + col % 4; }
static __host__ __device__ inline int rc_chunk_index(int row0, int seq) { return row0 / RC_C + seq; } /* of a sequence's first chunk: the sequences' chunks never meet */

template <class T>
__device__ __forceinline__ const T* rc_input_row(const kf_rb_delta& a, const T* raw0, const T* hist, int channels, int row, int pos0) {
    /* the projected channels of the sequence's row `row` (row < 0: before the batch), NULL: before the sequence */
    if (row >= 0) return raw0 + (int64_t)row * a.ldraw;
    const int p = pos0 + row;
    return p < 0 ? nullptr : hist + (size_t)(p % a.taps) * channels;
}
// two neighbouring channels of a row (the second may not exist), as they lie in memory: one load where they share one
__device__ __forceinline__ uint32_t rc_ld_pair(const uint16_t* p, bool paired, bool second) {
    if (paired) return *reinterpret_cast<const uint32_t*>(p);
    return p[0] | (second ? (uint32_t)p[1] << 16 : 0u);
}
__device__ __forceinline__ float2 rc_ld_pair(const float* p, bool paired, bool second) {
    if (paired) return *reinterpret_cast<const float2*>(p);
    return make_float2(p[0], second ? p[1] : 0.f);
}
__device__ __forceinline__ float2 rc_pair(uint32_t v) { return make_float2(bf_lo(v), bf_hi(v)); }
__device__ __forceinline__ float2 rc_pair(float2 v) { return v; }
template <class T>
struct RcPairOf {
    typedef uint32_t type;
};
template <>
struct RcPairOf<float> {
    typedef float2 type;
};
// the convolution and SiLU of channels c and c + 1 at 16 rows from `row` (a multiple of 16): the rows on their way (load), the results into dst [16][LD] (finish).  Rows at or past n_end give 0
template <class T>
struct RcConv {
    typename RcPairOf<T>::type x[19]; /* four taps; other numbers of taps load where they multiply */
    __device__ __forceinline__ void load(const kf_rb_delta& a, const T* raw0, const T* hist, int channels, int c, bool paired, bool second, int row, int n_end, int pos0) {
        if (a.taps != 4) return;
        const uint32_t ld = (uint32_t)a.ldraw;
#pragma unroll
        for (int t = 3; t < 19; t++) {
            const int r = row + t - 3;
            x[t] = rc_ld_pair(raw0 + ((uint32_t)(r < n_end ? r : n_end - 1) * ld + c), paired, second);
        }
        if (row >= 3) {
#pragma unroll
            for (int t = 0; t < 3; t++) x[t] = rc_ld_pair(raw0 + ((uint32_t)(row + t - 3 < n_end ? row + t - 3 : n_end - 1) * ld + c), paired, second);
        } else { /* the batch's first rows */
#pragma unroll
            for (int t = 0; t < 3; t++) {
                const T* p = rc_input_row(a, raw0, hist, channels, row + t - 3, pos0);
                x[t] = typename RcPairOf<T>::type{};
                if (p) x[t] = rc_ld_pair(p + c, paired, second);
            }
        }
    }
    template <int LD>
    __device__ __forceinline__ void finish(const kf_rb_delta& a, const T* raw0, const T* hist, int channels, int c, bool paired, bool second, int row, int n_end, int pos0, float* dst) const {
        const T* w = reinterpret_cast<const T*>(a.conv) + (size_t)c * a.taps;
        float2 y[16];
#pragma unroll
        for (int t = 0; t < 16; t++) y[t] = make_float2(0.f, 0.f);
        if (a.taps == 4) {
            float2 wt[4];
#pragma unroll
            for (int j = 0; j < 4; j++) wt[j] = make_float2(rb_ld(w + j), second ? rb_ld(w + 4 + j) : 0.f);
#pragma unroll
            for (int t = 0; t < 19; t++) {
                const float2 v = rc_pair(x[t]);
#pragma unroll
                for (int j = 0; j < 4; j++)
                    if (t - j >= 0 && t - j < 16) y[t - j].x = fmaf(wt[j].x, v.x, y[t - j].x), y[t - j].y = fmaf(wt[j].y, v.y, y[t - j].y);
            }
        } else {
            for (int j = 0; j < a.taps; j++) {
                const float w0 = rb_ld(w + a.taps - 1 - j), w1 = second ? rb_ld(w + 2 * a.taps - 1 - j) : 0.f;
#pragma unroll
                for (int t = 0; t < 16; t++) {
                    const T* p = row + t < n_end ? rc_input_row(a, raw0, hist, channels, row + t - j, pos0) : nullptr;
                    if (!p) continue;
                    const float2 v = rc_pair(rc_ld_pair(p + c, paired, second));
                    y[t].x = fmaf(w0, v.x, y[t].x), y[t].y = fmaf(w1, v.y, y[t].y);
                }
            }
        }
#pragma unroll
        for (int t = 0; t < 16; t++) {
            const bool on = row + t < n_end;
            *reinterpret_cast<float2*>(dst + t * LD) = make_float2(on ? y[t].x * rc_fast_sigmoid(y[t].x) : 0.f, on ? y[t].y * rc_fast_sigmoid(y[t].y) : 0.f);
        }
    }
};

// sB[J] + ... + sB[I - 1] of channels d .. d + 3
template <int DP>
__device__ __forceinline__ f32x4 rc_between(const float* sB, int J, int I, int d) {
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int m = J; m < I; m++) s += *reinterpret_cast<const f32x4*>(sB + m * DP + d);
    return s;
}
template <class T, int DP>
__global__ void __launch_bounds__(512) rb_delta_chunk_kernel(const kf_rb_delta a, float* __restrict__ chunks, const int32_t* __restrict__ seqs) {
    constexpr int LD = DP + 4, NB = RC_C / 16, LA = RC_C + 4, NE = NB * (NB + 1) / 2;
    extern __shared__ float smem[];
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3];
    const int h = blockIdx.x, c0 = blockIdx.y * RC_C;
    if (c0 >= n) return; /* workgroup-uniform */
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r16 = lane & 15, g4 = lane >> 4;
    // three arrays of rows: k, q, logs of the decays within the block; then k e^g, q e^g, k e^(block's end - g); the second becomes v
    float *sk = smem, *sq = sk + RC_C * LD, *sg = sq + RC_C * LD, *sB = sg + RC_C * LD /* [4][DP] logs of whole blocks */, *sE = sB + NB * DP /* [10][DP] factors of a block pair */,
          *sA = sE + NE * DP /* [64][LA] minus beta A */, *sT = sA + RC_C * LA /* [4][16][20] */, *s_kn = sT + NB * 16 * 20, *s_qn = s_kn + RC_C, *s_beta = s_qn + RC_C;
    const int dim = a.dim, vdim = a.vdim, Vp = rc_up(vdim, 16), qd = a.n_kv * dim, channels = 2 * qd + a.n_head * vdim, kvh = h / (a.n_head / a.n_kv);
    const T* raw0 = reinterpret_cast<const T*>(a.raw) + (size_t)row0 * a.ldraw;
    const T* hist = reinterpret_cast<const T*>(a.hist) + (size_t)slot * a.hist_slot;
    float* out = chunks + ((size_t)(rc_chunk_index(row0, blockIdx.z) + blockIdx.y) * a.n_head + h) * rc_chunk_floats(DP, Vp);
    float *oW = out, *oQ = oW + RC_C * DP, *oK = oQ + RC_C * DP, *oP = oK + RC_C * DP, *oU = oP + RC_C * RC_C, *oG = oU + RC_C * Vp;
    const bool paired = dim % 2 == 0 && vdim % 2 == 0 && a.ldraw % 2 == 0 && a.hist_slot % 2 == 0;
    auto zero16 = [&](float* dst) {
#pragma unroll
        for (int t = 0; t < 16; t++) *reinterpret_cast<float2*>(dst + t * LD) = make_float2(0.f, 0.f);
    };
    // everything this thread reads of the rows sets out together: a pair of q's or k's channels, the logs' inputs of a channel, a pair of v's
    constexpr int QK = DP * NB; /* work items of q and k (half of them each), of the decays; v: half as many.  At most one of each kind per thread */
    static_assert(QK <= 512, "an item per thread");
    const int qc = 2 * (tid % (DP / 2)), qw = tid / (DP / 2) & 1, qb = tid / DP, dc = tid % DP, db = tid / DP, vb = tid / (DP / 2);
    const bool q_on = tid < QK && qc < dim, d_on = tid < QK && dc < dim, v_on = tid < QK / 2 && qc < vdim;
    RcConv<T> cq, cv;
    if (q_on) cq.load(a, raw0, hist, channels, qw * qd + kvh * dim + qc, paired, qc + 1 < dim, c0 + 16 * qb, n, pos0);
    float z[16];
    if (d_on) {
        const float* zp = a.a_z + (size_t)(row0 + c0) * a.ld_az + h * dim + dc;
#pragma unroll
        for (int t = 0; t < 16; t++) z[t] = zp[(uint32_t)(c0 + 16 * db + t < n ? 16 * db + t : n - 1 - c0) * (uint32_t)a.ld_az];
    }
    if (v_on) cv.load(a, raw0, hist, channels, 2 * qd + h * vdim + qc, paired, qc + 1 < vdim, c0 + 16 * vb, n, pos0);
    if (tid < QK) {
        float* dst = (qw ? sk : sq) + 16 * qb * LD + qc;
        if (q_on) cq.template finish<LD>(a, raw0, hist, channels, qw * qd + kvh * dim + qc, paired, qc + 1 < dim, c0 + 16 * qb, n, pos0, dst);
        else zero16(dst);
        // decays: a thread a block of a channel
        const float rate = expf(rb_ld(reinterpret_cast<const T*>(a.a_log) + h)), bias = d_on ? rb_ld(reinterpret_cast<const T*>(a.dt_bias) + h * dim + dc) : 0.f;
        float l = 0.f;
#pragma unroll
        for (int t = 0; t < 16; t++) {
            if (d_on && c0 + 16 * db + t < n) l -= rate * rc_softplus2(z[t] + bias);
            sg[(16 * db + t) * LD + dc] = l;
        }
        sB[db * DP + dc] = l;
    }
    if (tid < RC_C) s_beta[tid] = c0 + tid < n ? rb_sigmoid(rb_ld(raw0 + (size_t)(c0 + tid) * a.ldraw + a.col_b + h)) : 0.f;
    rc_lds_barrier();
    { /* 1 / length: a wave eight tokens of q and of k, four lanes each */
        const int t = 8 * wid + (lane & 7);
        const float* x = ((lane & 8) ? sk : sq) + t * LD + g4 * (DP / 4);
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < DP / 4; i += 4) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(x + i);
#pragma unroll
            for (int j = 0; j < 4; j++) ss = fmaf(v[j], v[j], ss);
        }
        ss = xsum32(xsum16(ss));
        if (g4 == 0) {
            if (lane & 8) s_kn[t] = 1.0f / sqrtf(ss + a.unit_eps);
            else s_qn[t] = a.q_scale / sqrtf(ss + a.unit_eps);
        }
    }
    // the 16 x 16 blocks of A on and below the diagonal, with k and with q on the left: block (I, J) is number I (I + 1) / 2 + J
    auto finish = [&](int I, int J, f32x4 kk, f32x4 qk) {
        const int tj = 16 * J + r16;
        const float knj = s_kn[tj];
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = 16 * I + 4 * g4 + e;
            sA[t * LA + tj] = t > tj ? -s_beta[t] * s_kn[t] * knj * kk[e] : 0.f;
            oP[rc_tiled(t, tj, NB)] = t >= tj ? s_qn[t] * knj * qk[e] : 0.f;
        }
    };
    // a diagonal block whose decays multiply to next to nothing: pair by pair, while q, k and the logs are there.  Waves I and I + 4 see to block I: one tells, one sums
    bool by_pairs;
    {
        float least = 0.f;
        for (int d = lane; d < DP; d += 64) least = fminf(least, sB[(wid & 3) * DP + d]);
        by_pairs = wave_max(-least) >= 100.f;
    }
    rc_lds_barrier(); /* (the lengths) */
    if (by_pairs && wid < NB) { /* the layout of a result: rows 4 g4 + e, column r16 */
        f32x4 kk = f32x4{0.f, 0.f, 0.f, 0.f}, qk = kk;
        const int tj = 16 * wid + r16;
        for (int d = 0; d < DP; d++) {
            const float kj = sk[tj * LD + d], gj = sg[tj * LD + d];
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int t = 16 * wid + 4 * g4 + e;
                const float x = kj * rc_exp2(fminf(sg[t * LD + d] - gj, 0.f));
                kk[e] = fmaf(sk[t * LD + d], x, kk[e]), qk[e] = fmaf(sq[t * LD + d], x, qk[e]);
            }
        }
        finish(wid, wid, kk, qk);
    }
    rc_lds_barrier();
    for (int i = tid; i < RC_C * DP / 4; i += 512) {
        const int at = i / (DP / 4) * LD + 4 * (i % (DP / 4));
        f32x4 k = *reinterpret_cast<const f32x4*>(sk + at), q = *reinterpret_cast<const f32x4*>(sq + at), g = *reinterpret_cast<const f32x4*>(sg + at);
        const f32x4 B = *reinterpret_cast<const f32x4*>(sB + i / (DP / 4) / 16 * DP + 4 * (i % (DP / 4)));
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const float f = rc_exp2(g[e]);
            g[e] = k[e] * rc_exp2(B[e] - g[e]), k[e] *= f, q[e] *= f;
        }
        *reinterpret_cast<f32x4*>(sk + at) = k, *reinterpret_cast<f32x4*>(sq + at) = q, *reinterpret_cast<f32x4*>(sg + at) = g;
    }
    for (int i = tid; i < NE * DP / 4; i += 512) { /* from the end of block J to the start of block I; J = I: from its end back to its start */
        const int b = i / (DP / 4), d = 4 * (i % (DP / 4)), I = b < 1 ? 0 : (b < 3 ? 1 : (b < 6 ? 2 : 3)), J = b - I * (I + 1) / 2;
        f32x4 x = J < I ? rc_between<DP>(sB, J + 1, I, d) : -*reinterpret_cast<const f32x4*>(sB + I * DP + d);
#pragma unroll
        for (int e = 0; e < 4; e++) x[e] = rc_exp2(fminf(x[e], 100.f));
        *reinterpret_cast<f32x4*>(sE + b * DP + d) = x;
    }
    rc_lds_barrier();
    for (int b = wid; b < NE; b += 8) {
        const int I = b < 1 ? 0 : (b < 3 ? 1 : (b < 6 ? 2 : 3)), J = b - I * (I + 1) / 2;
        if (I == J) { /* (block I is this wave's or its partner's: 0, 2, 5 and 9 go to waves 0, 2, 5 and 1) */
            float least = 0.f;
            for (int d = lane; d < DP; d += 64) least = fminf(least, sB[I * DP + d]);
            if (wave_max(-least) >= 100.f) continue;
        }
        const float *pk = sk + (16 * I + r16) * LD + 4 * g4, *pq = sq + (16 * I + r16) * LD + 4 * g4, *pj = sg + (16 * J + r16) * LD + 4 * g4, *pe = sE + b * DP + 4 * g4;
        f32x4 kk[2], qk[2]; /* two chains each */
#pragma unroll
        for (int j = 0; j < 2; j++) kk[j] = qk[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int kb = 0; kb < DP / 16; kb++) {
            const f32x4 B = *reinterpret_cast<const f32x4*>(pj + 16 * kb) * *reinterpret_cast<const f32x4*>(pe + 16 * kb);
            const f32x4 k = *reinterpret_cast<const f32x4*>(pk + 16 * kb), q = *reinterpret_cast<const f32x4*>(pq + 16 * kb);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                kk[kb & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[e], B[e], kk[kb & 1], 0, 0, 0);
                qk[kb & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e], B[e], qk[kb & 1], 0, 0, 0);
            }
        }
        finish(I, J, kk[0] + kk[1], qk[0] + qk[1]);
    }
    // q e^G and (k e^(G_end - G))^T for the walk, in tiles
    for (int i = tid; i < RC_C * DP / 4; i += 512) {
        const int tile = i / 64, t = tile / (DP / 16) * 16 + r16, d = tile % (DP / 16) * 16 + 4 * g4;
        f32x4 q = *reinterpret_cast<const f32x4*>(sq + t * LD + d);
        const f32x4 x = rc_between<DP>(sB, 0, t / 16, d);
        const float f = s_qn[t];
#pragma unroll
        for (int e = 0; e < 4; e++) q[e] *= f * rc_exp2(x[e]);
        *reinterpret_cast<f32x4*>(oQ + 4 * i) = q;
    }
    for (int i = tid; i < RC_C * DP / 4; i += 512) {
        const int tile = i / 64, d = tile / NB * 16 + r16, t = tile % NB * 16 + 4 * g4;
        float x = 0.f;
        for (int m = t / 16 + 1; m < NB; m++) x += sB[m * DP + d];
        x = rc_exp2(x);
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = sg[(t + e) * LD + d] * s_kn[t + e] * x;
        *reinterpret_cast<f32x4*>(oK + 4 * i) = o;
    }
    for (int d = tid; d < DP; d += 512) oG[d] = rc_exp2(sB[d] + sB[DP + d] + sB[2 * DP + d] + sB[3 * DP + d]);
    rc_lds_barrier();
    if (wid == 7) { /* the diagonal blocks' inverses: a lane column r16 of block g4 */
        const float* Lb = sA + (16 * g4) * LA + 16 * g4;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; i++) {
            float s = i == r16 ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; j++) s = fmaf(Lb[i * LA + j], x[j], s); /* (the stored sign is minus) */
            x[i] = s;
            sT[(g4 * 16 + i) * 20 + r16] = s;
        }
    }
    // W, and U as many columns at a time as one array of rows holds
    for (int v0 = 0; v0 < Vp; v0 += DP) {
        if (tid < QK / 2) {
            const int c = v0 + qc;
            float* dst = sq + 16 * vb * LD + qc;
            if (v0 && c < vdim) cv.load(a, raw0, hist, channels, 2 * qd + h * vdim + c, paired, c + 1 < vdim, c0 + 16 * vb, n, pos0);
            if (c < vdim) cv.template finish<LD>(a, raw0, hist, channels, 2 * qd + h * vdim + c, paired, c + 1 < vdim, c0 + 16 * vb, n, pos0, dst);
            else zero16(dst);
        }
        rc_lds_barrier();
        const int first = v0 ? DP / 16 : 0, cols = Vp - v0 < DP ? Vp - v0 : DP;
        for (int ct = first + wid; ct < (DP + cols) / 16; ct += 8) { /* 16 columns: of W, of U */
            const bool is_w = ct < DP / 16;
            const int col = is_w ? 16 * ct + r16 : 16 * ct - DP + r16;
            f32x4 X[NB];
            float ahead = 0.f; /* the logs of the blocks in front, of this lane's channel */
#pragma unroll
            for (int I = 0; I < NB; I++) {
                const int t = 16 * I + 4 * g4;
                f32x4 acc;
                const float f = is_w ? rc_exp2(ahead) : 1.f;
                const float* src = (is_w ? sk : sq) + t * LD + col;
#pragma unroll
                for (int e = 0; e < 4; e++) acc[e] = s_beta[t + e] * (is_w ? s_kn[t + e] * f : 1.f) * src[e * LD];
                if (is_w) ahead += sB[I * DP + col];
#pragma unroll
                for (int J = 0; J < I; J++) acc = rc_mfma(*reinterpret_cast<const f32x4*>(sA + (16 * I + r16) * LA + 16 * J + 4 * g4), X[J], acc);
                X[I] = rc_mfma(*reinterpret_cast<const f32x4*>(sT + (16 * I + r16) * 20 + 4 * g4), acc, f32x4{0.f, 0.f, 0.f, 0.f});
                if (is_w) {
#pragma unroll
                    for (int e = 0; e < 4; e++) oW[rc_tiled(t + e, col, DP / 16)] = X[I][e];
                } else {
                    *reinterpret_cast<f32x4*>(oU + ((I * (Vp / 16) + (v0 + col) / 16) * 64 + lane) * 4) = X[I];
                }
            }
        }
        rc_lds_barrier();
    }
}

// the walk: four waves, wave w the chunk's tokens 16 w .. and the state's rows w DP / 4 ..; S^T and u^T pass between them through LDS
template <int DP>
__global__ void __launch_bounds__(256, 1) rb_delta_walk_kernel(const kf_rb_delta a, const float* __restrict__ chunks, float* __restrict__ o, const int32_t* __restrict__ seqs) {
    constexpr int LS = DP + 4, LU = RC_C + 4, NT = DP / 64 /* 16-row tiles of the state per wave */;
    __shared__ __attribute__((aligned(16))) float sS[16 * LS], sU[16 * LU];
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3];
    const int h = blockIdx.x, v0 = 16 * blockIdx.y, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r16 = lane & 15, g4 = lane >> 4;
    const int dim = a.dim, vdim = a.vdim, Vp = rc_up(vdim, 16), vs = rc_up(vdim, 4), col = v0 + r16;
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head, step = (size_t)a.n_head * rc_chunk_floats(DP, Vp);
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos0 + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + ((pos0 + n - 1) & 1)) * side + h * head;
    f32x4 S[NT]; /* rows d0 + 16 t + 4 g4 + e, column r16 */
    const int d0 = wid * 16 * NT;
#pragma unroll
    for (int t = 0; t < NT; t++) {
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int d = d0 + 16 * t + 4 * g4 + e;
            S[t][e] = pos0 > 0 && d < dim && col < vdim ? S0[(size_t)d * vs + col] : 0.f;
        }
        *reinterpret_cast<f32x4*>(sS + r16 * LS + d0 + 16 * t + 4 * g4) = S[t];
    }
    const float* c = chunks + ((size_t)rc_chunk_index(row0, blockIdx.z) * a.n_head + h) * rc_chunk_floats(DP, Vp);
    const int nc = (n + RC_C - 1) / RC_C;
    // what a wave reads of a chunk.  A register is loaded for the next chunk as soon as this one has used it, a load or two between the products: a CU takes in 64 bytes a cycle, and a
    // wave that issued a chunk's loads in one go would wait for that instead of multiplying
    f32x4 w[DP / 16], q[DP / 16], p[RC_C / 16], kt[NT][RC_C / 16], u, gt[NT];
    auto ld_w = [&](const float* c, int k) { w[k] = *reinterpret_cast<const f32x4*>(c + ((wid * (DP / 16) + k) * 64 + lane) * 4); };
    auto ld_q = [&](const float* c, int k) { q[k] = *reinterpret_cast<const f32x4*>(c + RC_C * DP + ((wid * (DP / 16) + k) * 64 + lane) * 4); };
    auto ld_k = [&](const float* c, int t, int b) { kt[t][b] = *reinterpret_cast<const f32x4*>(c + 2 * RC_C * DP + (((wid * NT + t) * (RC_C / 16) + b) * 64 + lane) * 4); };
    auto ld_p = [&](const float* c, int b) { p[b] = *reinterpret_cast<const f32x4*>(c + 3 * RC_C * DP + ((wid * (RC_C / 16) + b) * 64 + lane) * 4); }; /* (above the diagonal: tiles nobody wrote, not used) */
    auto ld_u = [&](const float* c) { u = *reinterpret_cast<const f32x4*>(c + RC_C * (3 * DP + RC_C) + ((wid * (Vp / 16) + v0 / 16) * 64 + lane) * 4); };
    auto ld_g = [&](const float* c, int t) { gt[t] = *reinterpret_cast<const f32x4*>(c + RC_C * (3 * DP + RC_C + Vp) + d0 + 16 * t + 4 * g4); };
#pragma unroll
    for (int k = 0; k < DP / 16; k++) ld_w(c, k), ld_q(c, k);
    ld_u(c);
#pragma unroll
    for (int t = 0; t < NT; t++) {
        ld_g(c, t);
#pragma unroll
        for (int b = 0; b < RC_C / 16; b++) ld_k(c, t, b);
    }
#pragma unroll
    for (int b = 0; b < RC_C / 16; b++) ld_p(c, b);
    f32x4 done = f32x4{0.f, 0.f, 0.f, 0.f}; /* the last chunk's outputs: stored while this one multiplies, a chunk's time before the next wait for memory */
    auto store = [&](int i) {
        if (col < vdim) {
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int row = RC_C * i + 16 * wid + 4 * g4 + e;
                if (row < n) o[(size_t)(row0 + row) * a.n_head * vdim + (size_t)h * vdim + col] = done[e];
            }
        }
    };
    for (int i = 0; i < nc; i++) {
        const float* next = i + 1 < nc ? c + step : c; /* (the last chunk again: not used) */
        rc_lds_barrier(); /* the state of the last chunk is in LDS */
        f32x4 ws[2], y[2]; /* two chains each */
#pragma unroll
        for (int j = 0; j < 2; j++) ws[j] = y[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        f32x4 s = *reinterpret_cast<const f32x4*>(sS + r16 * LS + 4 * g4);
#pragma unroll
        for (int k = 0; k < DP / 16; k++) {
            f32x4 s1 = s;
            if (k + 1 < DP / 16) s1 = *reinterpret_cast<const f32x4*>(sS + r16 * LS + 16 * (k + 1) + 4 * g4);
            ws[k & 1] = rc_mfma(w[k], s, ws[k & 1]);
            if (k > 0) ld_q(next, k - 1);
            __builtin_amdgcn_sched_barrier(0);
            y[k & 1] = rc_mfma(q[k], s, y[k & 1]);
            ld_w(next, k);
            s = s1;
            __builtin_amdgcn_sched_barrier(0);
            if (k == 0 && i > 0) store(i - 1);
        }
        *reinterpret_cast<f32x4*>(sU + r16 * LU + 16 * wid + 4 * g4) = u - (ws[0] + ws[1]);
        ld_q(next, DP / 16 - 1), ld_u(next);
        rc_lds_barrier();
        f32x4 ub = *reinterpret_cast<const f32x4*>(sU + r16 * LU + 4 * g4);
#pragma unroll
        for (int t = 0; t < NT; t++) {
            S[t] *= gt[t];
            ld_g(next, t);
        }
#pragma unroll
        for (int b = 0; b < RC_C / 16; b++) {
            f32x4 u1 = ub;
            if (b + 1 < RC_C / 16) u1 = *reinterpret_cast<const f32x4*>(sU + r16 * LU + 16 * (b + 1) + 4 * g4);
#pragma unroll
            for (int t = 0; t < NT; t++) {
                S[t] = rc_mfma(kt[t][b], ub, S[t]);
                ld_k(next, t, b);
                __builtin_amdgcn_sched_barrier(0);
            }
            if (b <= wid) y[b & 1] = rc_mfma(p[b], ub, y[b & 1]); /* wave-uniform */
            ld_p(next, b);
            ub = u1;
            __builtin_amdgcn_sched_barrier(0);
        }
#pragma unroll
        for (int t = 0; t < NT; t++) *reinterpret_cast<f32x4*>(sS + r16 * LS + d0 + 16 * t + 4 * g4) = S[t];
        done = y[0] + y[1];
        c = next;
    }
    store(nc - 1);
    if (col < vs) {
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int d = d0 + 16 * t + 4 * g4 + e;
                if (d < dim) S1[(size_t)d * vs + col] = S[t][e];
            }
    }
}
static int rc_delta_padded(int dim, int vdim) { return vdim > 256 ? 0 : (dim <= 64 ? 64 : (dim <= 128 ? 128 : 0)); } /* 0: not served in chunks */
template <class T, int DP>
static int delta_chunks_go(hipStream_t st, const kf_rb_delta& a, float* chunks, float* o, const int32_t* seqs, int n_seq, int max_n) {
    constexpr size_t smem = (3 * RC_C * (DP + 4) + 14 * DP + RC_C * (RC_C + 4) + 4 * 16 * 20 + 3 * RC_C) * sizeof(float);
    static_assert(smem <= 160 * 1024, "LDS");
    static int done = 0;
    if (!done) {
        if (hipFuncSetAttribute((const void*)rb_delta_chunk_kernel<T, DP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess) return KF_HIP_CHECK;
        done = 1;
    }
    hipLaunchKernelGGL((rb_delta_chunk_kernel<T, DP>), dim3(a.n_head, (max_n + RC_C - 1) / RC_C, n_seq), dim3(512), smem, st, a, chunks, seqs);
    hipLaunchKernelGGL((rb_delta_walk_kernel<DP>), dim3(a.n_head, (a.vdim + 15) / 16, n_seq), dim3(256), 0, st, a, chunks, o, seqs);
    return KF_OK;
}

// ---- the decayed sum in chunks (prompts, bf16 rows): S_c, the state in front of a chunk of 256 tokens, from one product per chunk and a walk over the chunks; then blocks of 128 queries
//   o_i = decay^(i - c + 1) S_c^T q_i + sum over the chunk's j <= i of decay^(i - j) (q_i . k_j) v_j
// on v_mfma_f32_32x32x16_bf16: q, k, v are exact, what has been multiplied by a decay enters as two (weights, S_c where it is read) or three (values on their way into the state) bf16 terms.
typedef __bf16 rc_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 rc_bf4 __attribute__((ext_vector_type(4)));
typedef float rc_f16 __attribute__((ext_vector_type(16)));
constexpr int RC_SPAN = 256, RC_QB = 128;
__device__ __forceinline__ rc_f16 rc_mfma32(u32x4 a, u32x4 b, rc_f16 c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rc_bf8, a), __builtin_bit_cast(rc_bf8, b), c, 0, 0, 0); }
// decay^n, n >= 0
struct RcPower {
    float l2;
    bool neg;
    __device__ __forceinline__ explicit RcPower(float decay) : l2(log2f(fabsf(decay))), neg(decay < 0.f) {}
    __device__ __forceinline__ float operator()(int n) const {
        const float p = n == 0 ? 1.f : __builtin_amdgcn_exp2f((float)n * l2); /* decay 0: e^-inf */
        return neg && (n & 1) ? -p : p;
    }
};
// keys (values) r0 .. of 32 rows staged [32][LDR]: a lane's operand of the 16 keys 16 s .. for column 32 b + lane % 32.  Element e is key 16 s + 4 (lane / 32) + e % 4 + 8 (e / 4)
template <int LDR>
__device__ __forceinline__ u32x4 rc_transposed(const uint16_t* rows, int s, int b, int lane) {
    const uint16_t* p = rows + (16 * s + 4 * (lane >> 5) + ((lane & 15) >> 2)) * LDR + b * 32 + (lane & 16) + 4 * (lane & 3);
    const rc_bf4 x = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) rc_bf4*)(p));
    const rc_bf4 y = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) rc_bf4*)(p + 8 * LDR));
    return __builtin_bit_cast(u32x4, rc_bf8{x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]});
}
__device__ __forceinline__ int rc_tile_key(int h, int i) { return 4 * h + (i & 3) + 8 * (i >> 2); } /* row of register i of a 32 x 32 result */

// the scratch behind the counters and outputs: per (span, head) the span's own sum [HD v][HD d] fp32, and the state in front of it as two bf16 planes of the same layout
static __host__ __device__ inline int rc_span_index(int row0, int seq) { return row0 / RC_SPAN + seq; }

template <int HD>
struct RcStage { /* 32 rows of k and of v: global -> registers -> LDS, 256 threads */
    static constexpr int KS = HD + 8, VS = HD + 32, CH = HD / 8, CPT = 32 * CH / 256, BYTES = 32 * (KS + VS) * 2;
    u32x4 kr[CPT], vr[CPT];
    __device__ __forceinline__ void load(const uint16_t* k, const uint16_t* v, int64_t ld, int dim, int vdim, int r0, int r_end, int tid) {
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int c = tid + 256 * i, r = r0 + c / CH, d = c % CH * 8;
            kr[i] = vr[i] = u32x4{0, 0, 0, 0};
            if (r < r_end) {
                if (d < dim) kr[i] = *reinterpret_cast<const u32x4*>(k + (int64_t)r * ld + d);
                if (d < vdim) vr[i] = *reinterpret_cast<const u32x4*>(v + (int64_t)r * ld + d);
            }
        }
    }
    __device__ __forceinline__ void store(uint16_t* ks, uint16_t* vs, int tid) const {
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int c = tid + 256 * i, r = c / CH, d = c % CH * 8;
            *reinterpret_cast<u32x4*>(ks + r * KS + d) = kr[i];
            *reinterpret_cast<u32x4*>(vs + r * VS + d) = vr[i];
        }
    }
};

template <int HD>
__global__ void __launch_bounds__(256) rb_decay_part_kernel(const kf_rb_decay a, float* __restrict__ sums, const int32_t* __restrict__ seqs) {
    using Stage = RcStage<HD>;
    constexpr int DB = HD == 128 ? 4 : 1; /* 32 x 32 tiles of a wave: HD 128: v block w, all d blocks; HD 64: one tile */
    static_assert(HD == 64 || HD == 128, "tiles dealt to four waves");
    __shared__ __attribute__((aligned(16))) uint16_t lds[2][32 * (Stage::KS + Stage::VS)];
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], t0 = blockIdx.y * RC_SPAN, h = blockIdx.x;
    if (t0 >= n) return; /* workgroup-uniform */
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r = lane & 31, hh = lane >> 5;
    const int vb = HD == 128 ? wid : wid >> 1, db0 = HD == 128 ? 0 : wid & 1;
    const uint16_t* k = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)row0 * a.ldraw + a.col_q + (size_t)a.n_head * a.dim + (size_t)h * a.dim;
    const uint16_t* v = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)row0 * a.ldraw + a.col_q + (size_t)2 * a.n_head * a.dim + (size_t)h * a.vdim;
    const int t1 = t0 + RC_SPAN < n ? t0 + RC_SPAN : n, nt = (t1 - t0 + 31) / 32;
    const RcPower pw(a.decay[h]);
    rc_f16 acc[DB];
#pragma unroll
    for (int d = 0; d < DB; d++)
#pragma unroll
        for (int i = 0; i < 16; i++) acc[d][i] = 0.f;
    Stage st;
    st.load(k, v, a.ldraw, a.dim, a.vdim, t0, t1, tid);
    st.store(lds[0], lds[0] + 32 * Stage::KS, tid);
    rc_lds_barrier();
    for (int t = 0; t < nt; t++) {
        const int k0 = t0 + 32 * t, m = t1 - k0 < 32 ? t1 - k0 : 32; /* the tile's keys */
        if (t + 1 < nt) st.load(k, v, a.ldraw, a.dim, a.vdim, k0 + 32, t1, tid);
        const uint16_t *ks = lds[t & 1], *vs = ks + 32 * Stage::KS;
        const float f = pw(m);
#pragma unroll
        for (int d = 0; d < DB; d++)
#pragma unroll
            for (int i = 0; i < 16; i++) acc[d][i] *= f;
#pragma unroll
        for (int s = 0; s < 2; s++) {
            const u32x4 raw = rc_transposed<Stage::VS>(vs, s, vb, lane);
            u32x4 p0, p1, p2; /* decay^(m - 1 - key) v as three bf16 terms */
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const int e = 2 * j, key = 16 * s + 4 * hh + (e & 3) + 8 * (e >> 2);
                const float x = key < m ? bf_lo(raw[j]) * pw(m - 1 - key) : 0.f, y = key + 1 < m ? bf_hi(raw[j]) * pw(m - 2 - key) : 0.f;
                p0[j] = pack_bf16x2(x, y);
                const float x1 = x - bf_lo(p0[j]), y1 = y - bf_hi(p0[j]);
                p1[j] = pack_bf16x2(x1, y1);
                p2[j] = pack_bf16x2(x1 - bf_lo(p1[j]), y1 - bf_hi(p1[j]));
            }
#pragma unroll
            for (int d = 0; d < DB; d++) {
                const u32x4 B = rc_transposed<Stage::KS>(ks, s, db0 + d, lane);
                acc[d] = rc_mfma32(p0, B, acc[d]), acc[d] = rc_mfma32(p1, B, acc[d]), acc[d] = rc_mfma32(p2, B, acc[d]);
            }
        }
        if (t + 1 < nt) st.store(lds[(t + 1) & 1], lds[(t + 1) & 1] + 32 * Stage::KS, tid);
        rc_lds_barrier();
    }
    float* out = sums + ((size_t)(rc_span_index(row0, blockIdx.z) + blockIdx.y) * a.n_head + h) * HD * HD;
#pragma unroll
    for (int d = 0; d < DB; d++)
#pragma unroll
        for (int i = 0; i < 16; i++) out[(32 * vb + rc_tile_key(hh, i)) * HD + 32 * (db0 + d) + r] = acc[d][i];
}
// a thread four neighbouring d of a v row: the state in front of every span, and the state after the batch
template <int HD>
__global__ void __launch_bounds__(256) rb_decay_states_kernel(const kf_rb_decay a, const float* __restrict__ sums, uint16_t* __restrict__ planes, const int32_t* __restrict__ seqs) {
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3], h = blockIdx.x;
    const int at = 4 * (blockIdx.y * 256 + threadIdx.x), v = at / HD, d = at % HD;
    const int dim = a.dim, vs = rc_up(a.vdim, 4), ns = (n + RC_SPAN - 1) / RC_SPAN;
    const size_t head = (size_t)dim * vs, side = (size_t)a.n_head * head;
    const float* S0 = a.state + ((size_t)slot * 2 + ((pos0 + 1) & 1)) * side + h * head;
    float* S1 = a.state + ((size_t)slot * 2 + ((pos0 + n - 1) & 1)) * side + h * head;
    const RcPower pw(a.decay[h]);
    f32x4 S = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (pos0 > 0 && v < a.vdim && d + j < dim) S[j] = S0[(size_t)(d + j) * vs + v];
    const size_t step = (size_t)a.n_head * HD * HD, first = ((size_t)rc_span_index(row0, blockIdx.z) * a.n_head + h) * HD * HD + at;
    const float* x = sums + first;
    f32x4 next = *reinterpret_cast<const f32x4*>(x);
    for (int c = 0; c < ns; c++) {
        const f32x4 add = next;
        if (c + 1 < ns) next = *reinterpret_cast<const f32x4*>(x + (c + 1) * step);
        uint16_t* hi = planes + 2 * ((size_t)(rc_span_index(row0, blockIdx.z) + c) * a.n_head + h) * HD * HD + at;
        const u32x2 p = u32x2{pack_bf16x2(S.x, S.y), pack_bf16x2(S.z, S.w)};
        *reinterpret_cast<u32x2*>(hi) = p;
        *reinterpret_cast<u32x2*>(hi + HD * HD) = u32x2{pack_bf16x2(S.x - bf_lo(p.x), S.y - bf_hi(p.x)), pack_bf16x2(S.z - bf_lo(p.y), S.w - bf_hi(p.y))};
        const float f = pw(n - c * RC_SPAN < RC_SPAN ? n - c * RC_SPAN : RC_SPAN);
#pragma unroll
        for (int j = 0; j < 4; j++) S[j] = fmaf(f, S[j], add[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (v < vs && d + j < dim) S1[(size_t)(d + j) * vs + v] = S[j];
}
// 128 queries of a head: a wave 32 of them, one per lane pair
template <int HD>
__global__ void __launch_bounds__(256) rb_decay_out_kernel(const kf_rb_decay a, const uint16_t* __restrict__ planes, float* __restrict__ o, const int32_t* __restrict__ seqs) {
    using Stage = RcStage<HD>;
    constexpr int NS = HD / 16, NB = HD / 32;
    __shared__ __attribute__((aligned(16))) uint16_t lds[2][32 * (Stage::KS + Stage::VS)];
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], h = blockIdx.x, q0 = blockIdx.y * RC_QB;
    if (q0 >= n) return; /* workgroup-uniform */
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r = lane & 31, hh = lane >> 5;
    const uint16_t* q = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)row0 * a.ldraw + a.col_q + (size_t)h * a.dim;
    const uint16_t* k = q + (size_t)a.n_head * a.dim;
    const uint16_t* v = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)row0 * a.ldraw + a.col_q + (size_t)2 * a.n_head * a.dim + (size_t)h * a.vdim;
    const int tok = q0 + 32 * wid + r, row = tok < n ? tok : n - 1, c0 = q0 / RC_SPAN * RC_SPAN; /* queries past the end repeat the last one and are not stored */
    const int last = q0 + RC_QB < n ? q0 + RC_QB : n, nt = (last - c0 + 31) / 32;
    Stage st;
    st.load(k, v, a.ldraw, a.dim, a.vdim, c0, last, tid);
    u32x4 qf[NS];
#pragma unroll
    for (int s = 0; s < NS; s++) {
        qf[s] = u32x4{0, 0, 0, 0};
        if (16 * s + 8 * hh < a.dim) qf[s] = *reinterpret_cast<const u32x4*>(q + (int64_t)row * a.ldraw + 16 * s + 8 * hh);
    }
    const RcPower pw(a.decay[h]);
    rc_f16 acc[NB];
    const uint16_t* S = planes + 2 * ((size_t)(rc_span_index(row0, blockIdx.z) + c0 / RC_SPAN) * a.n_head + h) * HD * HD;
    st.store(lds[0], lds[0] + 32 * Stage::KS, tid);
    const float f0 = pw(row - c0 + 1);
#pragma unroll
    for (int b = 0; b < NB; b++) {
#pragma unroll
        for (int i = 0; i < 16; i++) acc[b][i] = 0.f;
#pragma unroll
        for (int s = 0; s < NS; s++) {
            const uint16_t* p = S + (32 * b + r) * HD + 16 * s + 8 * hh;
            acc[b] = rc_mfma32(*reinterpret_cast<const u32x4*>(p), qf[s], acc[b]);
            acc[b] = rc_mfma32(*reinterpret_cast<const u32x4*>(p + HD * HD), qf[s], acc[b]);
        }
#pragma unroll
        for (int i = 0; i < 16; i++) acc[b][i] *= f0;
    }
    float tail[16]; /* decay^(31 - key) of a tile's keys */
#pragma unroll
    for (int i = 0; i < 16; i++) tail[i] = pw(31 - rc_tile_key(hh, i));
    rc_lds_barrier();
    for (int t = 0; t < nt; t++) {
        const int k0 = c0 + 32 * t;
        if (t + 1 < nt) st.load(k, v, a.ldraw, a.dim, a.vdim, k0 + 32, last, tid);
        const uint16_t *ks = lds[t & 1], *vs = ks + 32 * Stage::KS;
        if (k0 <= q0 + 32 * wid + 31) { /* wave-uniform */
            rc_f16 s;
#pragma unroll
            for (int i = 0; i < 16; i++) s[i] = 0.f;
#pragma unroll
            for (int j = 0; j < NS; j++) s = rc_mfma32(*reinterpret_cast<const u32x4*>(ks + r * Stage::KS + 16 * j + 8 * hh), qf[j], s);
            if (k0 + 31 <= q0 + 32 * wid) {
                const float f = pw((row > k0 + 31 ? row : k0 + 31) - k0 - 31);
#pragma unroll
                for (int i = 0; i < 16; i++) s[i] *= f * tail[i];
            } else {
#pragma unroll
                for (int i = 0; i < 16; i++) {
                    const int age = row - k0 - rc_tile_key(hh, i);
                    s[i] = age >= 0 ? s[i] * pw(age) : 0.f;
                }
            }
            uint32_t ph[8], pl[8];
#pragma unroll
            for (int i = 0; i < 8; i++) {
                ph[i] = pack_bf16x2(s[2 * i], s[2 * i + 1]);
                pl[i] = pack_bf16x2(s[2 * i] - bf_lo(ph[i]), s[2 * i + 1] - bf_hi(ph[i]));
            }
#pragma unroll
            for (int s2 = 0; s2 < 2; s2++) {
                const u32x4 B = u32x4{ph[4 * s2], ph[4 * s2 + 1], ph[4 * s2 + 2], ph[4 * s2 + 3]}, B2 = u32x4{pl[4 * s2], pl[4 * s2 + 1], pl[4 * s2 + 2], pl[4 * s2 + 3]};
#pragma unroll
                for (int b = 0; b < NB; b++) {
                    const u32x4 A = rc_transposed<Stage::VS>(vs, s2, b, lane);
                    acc[b] = rc_mfma32(A, B, acc[b]), acc[b] = rc_mfma32(A, B2, acc[b]);
                }
            }
        }
        if (t + 1 < nt) st.store(lds[(t + 1) & 1], lds[(t + 1) & 1] + 32 * Stage::KS, tid);
        rc_lds_barrier();
    }
    if (tok >= n) return;
    float* out = o + (size_t)(row0 + tok) * a.n_head * a.vdim + (size_t)h * a.vdim;
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int g = 0; g < 4; g++) {
            const int c = 32 * b + 8 * g + 4 * hh;
            if (c < a.vdim) rb_st4(out + c, f32x4{acc[b][4 * g], acc[b][4 * g + 1], acc[b][4 * g + 2], acc[b][4 * g + 3]});
        }
}
static int rc_decay_padded(int type, int dim, int vdim) { /* 0: not served in chunks */
    const int m = std::max(dim, vdim);
    return type != KF_BF16 || dim % 8 || vdim % 8 || m > 128 ? 0 : (m <= 64 ? 64 : 128);
}
template <int HD>
static void decay_chunks_go(hipStream_t st, const kf_rb_decay& a, float* sums, uint16_t* planes, float* o, const int32_t* seqs, int n_seq, int max_n) {
    hipLaunchKernelGGL(rb_decay_part_kernel<HD>, dim3(a.n_head, (max_n + RC_SPAN - 1) / RC_SPAN, n_seq), dim3(256), 0, st, a, sums, seqs);
    hipLaunchKernelGGL(rb_decay_states_kernel<HD>, dim3(a.n_head, HD * HD / 1024, n_seq), dim3(256), 0, st, a, sums, planes, seqs);
    hipLaunchKernelGGL(rb_decay_out_kernel<HD>, dim3(a.n_head, (max_n + RC_QB - 1) / RC_QB, n_seq), dim3(256), 0, st, a, planes, o, seqs);
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

// the same, four columns of a thread in registers; a group is a power-of-two run of at most 64 threads, or the row (GROUPED: false)
template <class T, int VPT, bool GROUPED>
__global__ void __launch_bounds__(256) rb_gate_vec_kernel(const RcGate a) {
    __shared__ float red[4];
    const int r = blockIdx.x, tid = threadIdx.x, cols = a.groups * a.size;
    const float* o = a.o + (size_t)r * a.ldo;
    const T* gate = reinterpret_cast<const T*>(a.gate) + (size_t)r * a.ldg;
    T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.ldout;
    f32x4 v[VPT];
    float ss[VPT], all = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * (tid + 256 * i);
        v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (c < cols) v[i] = rb_ld4(o + c);
        ss[i] = 0.f;
#pragma unroll
        for (int j = 0; j < 4; j++) ss[i] = fmaf(v[i][j], v[i][j], ss[i]);
        if (GROUPED)
            for (int w = 1; w < a.size / 4; w <<= 1) ss[i] += __shfl_xor(ss[i], w, 64);
        else all += ss[i];
    }
    if (!GROUPED) {
        all = wave_sum(all);
        if ((tid & 63) == 0) red[tid >> 6] = all;
        __syncthreads();
        all = red[0] + red[1] + red[2] + red[3];
    }
#pragma unroll
    for (int i = 0; i < VPT; i++) {
        const int c = 4 * (tid + 256 * i);
        if (c >= cols) continue;
        const float rs = a.scale / sqrtf((GROUPED ? ss[i] : all) / (float)a.size + a.eps);
        const f32x4 w = rb_ld4(reinterpret_cast<const T*>(a.w) + (GROUPED ? c % a.size : c)), g = rb_ld4(gate + c);
        f32x4 y;
#pragma unroll
        for (int j = 0; j < 4; j++) y[j] = v[i][j] * rs * w[j] * rb_sigmoid(g[j]);
        rb_st4(out + c, y);
    }
}
template <class T, int VPT>
static void gate_vec(hipStream_t st, const RcGate& a, int n) {
    if (a.groups > 1) hipLaunchKernelGGL((rb_gate_vec_kernel<T, VPT, true>), dim3(n), dim3(256), 0, st, a);
    else hipLaunchKernelGGL((rb_gate_vec_kernel<T, VPT, false>), dim3(n), dim3(256), 0, st, a);
}
template <class T>
static void gate_go(hipStream_t st, const RcGate& a, int n) {
    const int cols = a.groups * a.size, quads = a.size / 4, vpt = (cols + 1023) / 1024;
    const bool aligned = a.size % 4 == 0 && a.ldo % 4 == 0 && a.ldg % 4 == 0 && a.ldout % 4 == 0 && (uintptr_t)a.gate % 16 == 0 && (uintptr_t)a.out % 16 == 0 && (uintptr_t)a.w % 16 == 0 && (uintptr_t)a.o % 16 == 0;
    const bool grouped = a.groups > 1;
    if (!aligned || vpt > 8 || (grouped && (quads > 64 || (quads & (quads - 1))))) {
        hipLaunchKernelGGL(rb_gate_kernel<T>, dim3(n), dim3(256), 0, st, a);
        return;
    }
    if (vpt <= 1) gate_vec<T, 1>(st, a, n);
    else if (vpt <= 2) gate_vec<T, 2>(st, a, n);
    else if (vpt <= 4) gate_vec<T, 4>(st, a, n);
    else gate_vec<T, 8>(st, a, n);
}
constexpr int RC_MIN_CHUNKED = 16; /* rows of the longest sequence from which the chunked forms are taken */
template <class T>
static int delta_prefill_go(hipStream_t st, const kf_rb_delta& a, const int32_t* meta, int n, const int32_t* seqs, int n_seq, int max_n) {
    const int64_t ldv = (int64_t)a.n_head * a.vdim;
    float* o = a.scratch; /* [n][n_head vdim] */
    const bool offsets = (int64_t)n * std::max(a.ldraw, a.ld_az) < ((int64_t)1 << 30); /* of a row inside the batch: 32 bits */
    const int DP = max_n >= RC_MIN_CHUNKED && offsets ? rc_delta_padded(a.dim, a.vdim) : 0;
    if (DP) {
        float* chunks = o + ((size_t)n * ldv + 3) / 4 * 4;
        const int rc = DP == 64 ? delta_chunks_go<T, 64>(st, a, chunks, o, seqs, n_seq, max_n) : delta_chunks_go<T, 128>(st, a, chunks, o, seqs, n_seq, max_n);
        if (rc) return rc;
    } else {
        const RcPrep p = rc_prep_at(a.scratch, n, a.n_head, a.n_kv, a.dim, a.vdim);
        hipLaunchKernelGGL(rb_delta_prep_kernel<T>, dim3(n, (2 * a.n_kv + 2 * a.n_head + 3) / 4), dim3(256), 0, st, a, p, meta);
        const int64_t ldq = 2 * (int64_t)a.n_kv * a.dim;
        const RcScan<float> s{p.qk, p.qk + (size_t)a.n_kv * a.dim, p.v, p.g, p.beta, nullptr, p.v, a.state, ldq, ldv, ldv, a.n_head, a.n_head / a.n_kv, a.dim, a.vdim};
        if (scan_go<float, true>(st, s, seqs, n_seq)) return 1;
    }
    hipLaunchKernelGGL(rb_hist_kernel<T>, dim3((2 * a.n_kv * a.dim + a.n_head * a.vdim + 255) / 256, a.taps, n_seq), dim3(256), 0, st, a, seqs);
    gate_go<T>(st, RcGate{o, a.norm_w, a.g_z, a.out, ldv, a.ld_gz, a.ldout, a.n_head, a.vdim, 1.f, a.eps}, n);
    return KF_OK;
}
template <class T>
static int decay_prefill_go(hipStream_t st, const kf_rb_decay& a, int n, const int32_t* seqs, int n_seq, int max_n) {
    const int64_t ldo = (int64_t)a.n_head * a.vdim;
    float* o = a.scratch + (size_t)RC_CNT_STRIDE * n;
    const int HD = max_n >= RC_MIN_CHUNKED && a.col_q % 8 == 0 && a.ldraw % 8 == 0 ? rc_decay_padded(a.type, a.dim, a.vdim) : 0;
    if (HD) {
        float* sums = o + ((size_t)n * ldo + 3) / 4 * 4;
        uint16_t* planes = reinterpret_cast<uint16_t*>(sums + (size_t)(n / RC_SPAN + n_seq) * a.n_head * HD * HD);
        HD == 64 ? decay_chunks_go<64>(st, a, sums, planes, o, seqs, n_seq, max_n) : decay_chunks_go<128>(st, a, sums, planes, o, seqs, n_seq, max_n);
    } else {
        const T* q = reinterpret_cast<const T*>(a.raw) + a.col_q;
        const RcScan<T> s{q, q + (size_t)a.n_head * a.dim, q + (size_t)2 * a.n_head * a.dim, nullptr, nullptr, a.decay, o, a.state, a.ldraw, a.ldraw, ldo, a.n_head, 1, a.dim, a.vdim};
        if (scan_go<T, false>(st, s, seqs, n_seq)) return 1;
    }
    gate_go<T>(st, RcGate{o, a.norm_w, reinterpret_cast<const T*>(a.raw) + a.col_g, a.out, ldo, a.ldraw, a.ldout, 1, a.n_head * a.vdim, a.out_scale, a.eps}, n);
    return KF_OK;
}
template <class T>
static void delta_step_go(hipStream_t st, const kf_rb_delta& a, const int32_t* meta, int n) {
    const int nt = rc_step_threads(a.dim, a.vdim);
    const size_t smem = (3 * (size_t)rc_up(a.dim, 4) + 2 * rc_up(a.vdim, 4) + rc_up(a.rank_a, 8) + rc_up(a.rank_g, 8) + 8 * (size_t)(nt ? nt : 1024) + 32) * 4;
    const dim3 grid(a.n_head, n);
    if (nt == 256) hipLaunchKernelGGL((rb_delta_step_kernel<T, 256, 8>), grid, dim3(256), smem, st, a, meta);
    else if (nt == 512) hipLaunchKernelGGL((rb_delta_step_kernel<T, 512, 8>), grid, dim3(512), smem, st, a, meta);
    else if (nt == 1024) hipLaunchKernelGGL((rb_delta_step_kernel<T, 1024, 16>), grid, dim3(1024), smem, st, a, meta);
    else hipLaunchKernelGGL((rb_delta_step_kernel<T, 1024, 0>), grid, dim3(1024), smem, st, a, meta);
}
template <class T>
static void decay_step_go(hipStream_t st, const kf_rb_decay& a, const int32_t* meta, int n) {
    const int nt = rc_step_threads(a.dim, a.vdim);
    const size_t smem = rc_decay_step_lds(a.dim, a.vdim, nt ? nt : 1024);
    const dim3 grid(a.n_head, n);
    if (nt == 256) hipLaunchKernelGGL((rb_decay_step_kernel<T, 256, 8>), grid, dim3(256), smem, st, a, meta);
    else if (nt == 512) hipLaunchKernelGGL((rb_decay_step_kernel<T, 512, 8>), grid, dim3(512), smem, st, a, meta);
    else if (nt == 1024) hipLaunchKernelGGL((rb_decay_step_kernel<T, 1024, 16>), grid, dim3(1024), smem, st, a, meta);
    else hipLaunchKernelGGL((rb_decay_step_kernel<T, 1024, 0>), grid, dim3(1024), smem, st, a, meta);
}

constexpr int RC_MAX_DIM = 512;
int rc_check_decay(const kf_rb_decay* a, const int32_t* meta, int n, const char* who) {
    if (!a || !meta || n < 1 || !a->raw || !a->out || !a->norm_w || !a->decay || !a->state || !a->scratch) return abi_fail(KF_INVALID_ARGS, "%s: null pointer", who);
    if (a->type != KF_BF16 && a->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: storage %d", who, a->type);
    if (a->n_head < 1 || a->dim < 1 || a->vdim < 1) return abi_fail(KF_INVALID_ARGS, "%s: %d heads of %d / %d", who, a->n_head, a->dim, a->vdim);
    if (a->dim > RC_MAX_DIM || a->vdim > RC_MAX_DIM) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: head sizes %d / %d (served: up to %d)", who, a->dim, a->vdim, RC_MAX_DIM);
    const int64_t qk = 2 * (int64_t)a->n_head * a->dim, all = (int64_t)a->n_head * a->vdim;
    if (a->col_q < 0 || a->col_g < 0 || a->ldraw < a->col_q + qk + all || a->ldraw < a->col_g + all || a->ldout < all) return abi_fail(KF_INVALID_ARGS, "%s: strides", who);
    if (!al16(a->state) || !al16(a->scratch) || !al16(a->raw)) return abi_fail(KF_BLAS_UNALIGN, "%s: unaligned pointer", who);
    return KF_OK;
}

}  // namespace kf

using namespace kf;
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
static int launched(int rc, const char* who) {
    if (rc == 1) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: no kernel for these sizes", who);
    if (rc != KF_OK) return abi_fail(rc, "%s: launch failed", who);
    return hipGetLastError() == hipSuccess ? KF_OK : abi_fail(KF_HIP_CHECK, "%s: launch failed", who);
}
extern "C" {

size_t kf_rb_delta_scratch(int type, int n_rows, int n_seq, int n_head, int n_kv, int dim, int vdim) {
    if (n_rows < 1 || n_seq < 1 || n_head < 1 || n_kv < 1 || dim < 1 || vdim < 1) return 0;
    const size_t o = (size_t)n_rows * n_head * vdim + 4, rows = (size_t)n_rows * (2 * (size_t)n_kv * dim + (size_t)n_head * (dim + 1));
    const int DP = rc_delta_padded(dim, vdim);
    const size_t chunks = DP ? (size_t)(n_rows / RC_C + n_seq) * n_head * rc_chunk_floats(DP, rc_up(vdim, 16)) : 0;
    return (o + std::max(rows, chunks) + 16) * 4;
}
size_t kf_rb_decay_scratch(int type, int n_rows, int n_seq, int n_head, int dim, int vdim) {
    if (n_rows < 1 || n_seq < 1 || n_head < 1 || dim < 1 || vdim < 1) return 0;
    const int HD = rc_decay_padded(type, dim, vdim);
    const size_t spans = HD ? (size_t)(n_rows / RC_SPAN + n_seq) * n_head * HD * HD * 2 : 0; /* a sum and two half-width planes */
    return ((size_t)n_rows * (RC_CNT_STRIDE + (size_t)n_head * vdim) + 4 + spans + 16) * 4;
}
int kf_rb_delta_prefill(kf_ctx* c, const kf_rb_delta* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n) {
    CHKCTX(c);
    const int rc = check_delta(a, meta, n_rows, "kf_rb_delta_prefill");
    if (rc) return rc;
    if (!seqs || n_seq < 1 || max_n < 1 || max_n > n_rows || !a->a_z || !a->g_z || !a->scratch || !al16(a->scratch) || a->ld_az < (int64_t)a->n_head * a->dim || a->ld_gz < (int64_t)a->n_head * a->vdim)
        return abi_fail(KF_INVALID_ARGS, "kf_rb_delta_prefill: bad arguments");
    return launched(a->type == KF_BF16 ? delta_prefill_go<uint16_t>(c->stream, *a, meta, n_rows, seqs, n_seq, max_n) : delta_prefill_go<float>(c->stream, *a, meta, n_rows, seqs, n_seq, max_n), "kf_rb_delta_prefill");
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
    const int rc = rc_check_decay(a, meta, n_rows, "kf_rb_decay_prefill");
    if (rc) return rc;
    if (!seqs || n_seq < 1 || max_n < 1 || max_n > n_rows) return abi_fail(KF_INVALID_ARGS, "kf_rb_decay_prefill: bad arguments");
    return launched(a->type == KF_BF16 ? decay_prefill_go<uint16_t>(c->stream, *a, n_rows, seqs, n_seq, max_n) : decay_prefill_go<float>(c->stream, *a, n_rows, seqs, n_seq, max_n), "kf_rb_decay_prefill");
}
int kf_rb_decay_decode(kf_ctx* c, const kf_rb_decay* a, const int32_t* meta, int n_rows) {
    CHKCTX(c);
    const int rc = rc_check_decay(a, meta, n_rows, "kf_rb_decay_decode");
    if (rc) return rc;
    if (a->type == KF_BF16) decay_step_go<uint16_t>(c->stream, *a, meta, n_rows);
    else decay_step_go<float>(c->stream, *a, meta, n_rows);
    return launched(KF_OK, "kf_rb_decay_decode");
}

}  // extern "C"
