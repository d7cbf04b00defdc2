// kf_rb_attn.hip -- attention of a row batch (kf_rb.h): per-head RMS norm and partial rotation of q and k, unrotated k as the value, chunks, free scale, output gate, a ring
// of cache rows per slot.
//
// bf16, dim a multiple of 8 up to 256: MFMA flash form, the register / LDS scheme of kf_attn_prefill.hip (S^T = K Q^T by v_mfma_f32_32x32x16_bf16, a column = one (token,
// query head) pair per lane pair, P split into a bf16 pair for the P.V product, V^T fragments by ds_read_b64_tr_b16), with
//   * columns flattened over (token, head): any number of query heads per kv-head;
//   * keys and values of the batch's own tokens read from the batch, older ones from the slot's ring: a prompt is attended to before its rows overwrite the ring;
//   * only the tiles between a wave's first chunk start and its last position.
// A decode row is one workgroup per (kv-head, key range): q and the new key are prepared in LDS, each of its four waves walks its own 32-key tiles (staged into LDS of its
// own, no barrier in the walk) and the four partial softmaxes meet at the end.
// fp32 storage (and other head sizes): a plain form, one wave per (row, head), 32-bit throughout.
#include <algorithm>

#include "kf_ctx.h"
#include "kf_rb_recur.h"

namespace kf {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));

constexpr float RB_LOG2E = 1.44269502162933349609375f;
__device__ __forceinline__ float rb_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ void rb_st_sc1(float* p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ float rb_ld_sc1(const float* p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
constexpr int RB_CNT_STRIDE = 16; /* words between arrival counters: one cache line each */
__device__ __forceinline__ int rb_first_key(int pos, const kf_rb_attention& a) {
    if (a.window > 0) return pos >= a.window ? pos - a.window + 1 : 0;
    return a.chunk > 0 ? pos - pos % a.chunk : 0;
}
// the launchers fill in what the caller left zero (whole_form): vdim, v_col, gate_col and out_scale hold real values in the kernels

// one head (dim elements at src) normed and rotated by one wave into dst; buf: dim floats of LDS of this wave
template <class T>
__device__ __forceinline__ void rb_prep_head(const T* __restrict__ src, T* dst, const T* __restrict__ w, bool unit, const float* __restrict__ rope, int rot, int dim, int pos, float eps,
                                             float* buf, int lane) {
    float ss = 0.f;
    for (int i = lane; i < dim; i += 64) {
        const float v = rb_ld(src + i);
        buf[i] = v;
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    const float rs = w || unit ? 1.0f / sqrtf(ss / (float)dim + eps) : 1.0f;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    const int half = rot >> 1;
    for (int i = lane; i < half; i += 64) {
        const float u = buf[i] * rs * (w ? rb_ld(w + i) : 1.f), v = buf[i + half] * rs * (w ? rb_ld(w + i + half) : 1.f);
        const float2 cs = *reinterpret_cast<const float2*>(rope + ((size_t)pos * half + i) * 2);
        rb_st(dst + i, u * cs.x - v * cs.y);
        rb_st(dst + i + half, v * cs.x + u * cs.y);
    }
    for (int i = rot + lane; i < dim; i += 64) rb_st(dst + i, buf[i] * rs * (w ? rb_ld(w + i) : 1.f));
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// ---- q in place, k -> k_new (prefill) or, STORE: k and v into the slot's ring (decode)
template <class T, bool STORE>
__global__ void __launch_bounds__(256) rb_prep_kernel(const kf_rb_attention a, const int32_t* __restrict__ meta) {
    extern __shared__ float s_buf[];
    const int r = blockIdx.x, wid = threadIdx.x >> 6, lane = threadIdx.x & 63, u = blockIdx.y * 4 + wid;
    const int pos = meta[KF_RB_META * r];
    if (pos < 0 || u >= a.n_head + a.n_kv) return; /* no barrier below */
    T* raw = reinterpret_cast<T*>(a.raw) + (size_t)r * a.ldraw;
    float* buf = s_buf + wid * a.dim;
    if (u < a.n_head) {
        T* q = raw + (size_t)u * a.dim;
        rb_prep_head(q, q, reinterpret_cast<const T*>(a.q_norm), a.unit, a.rope, a.rot_dims, a.dim, pos, a.eps, buf, lane);
        return;
    }
    const int g = u - a.n_head, kvd = a.n_kv * a.dim;
    const T* k = raw + (size_t)u * a.dim;
    T* dst;
    if constexpr (STORE) {
        const size_t head = (size_t)meta[KF_RB_META * r + 1] * a.slot_stride + (size_t)g * a.head_stride, row = pos % a.cache_rows;
        dst = reinterpret_cast<T*>(a.k_cache) + head + row * a.dim;
        const T* vn = raw + a.v_col + (size_t)g * a.vdim;
        T* v = reinterpret_cast<T*>(a.v_cache) + head + row * a.vdim;
        for (int i = lane; i < a.vdim; i += 64) v[i] = vn[i];
    } else {
        dst = reinterpret_cast<T*>(a.k_new) + (size_t)r * kvd + (size_t)g * a.dim;
    }
    rb_prep_head(k, dst, reinterpret_cast<const T*>(a.k_norm), a.unit, a.rope, a.rot_dims, a.dim, pos, a.eps, buf, lane);
}
// the prompt form, bf16, L lanes per head: lane j < rot / 8 holds the rotation pairs 4 j .. 4 j + 3 (a quad of each half), the next lanes a quad of the dimensions behind
template <int L>
__global__ void __launch_bounds__(256) rb_prep_vec_kernel(const kf_rb_attention a, const int32_t* __restrict__ meta) {
    const int r = blockIdx.x, u = blockIdx.y * (256 / L) + (int)threadIdx.x / L, j = threadIdx.x % L;
    const int pos = meta[KF_RB_META * r];
    const bool head_on = pos >= 0 && u < a.n_head + a.n_kv;
    uint16_t* src = reinterpret_cast<uint16_t*>(a.raw) + (size_t)r * a.ldraw + (size_t)(head_on ? u : 0) * a.dim;
    const bool key = u >= a.n_head;
    uint16_t* dst = key ? reinterpret_cast<uint16_t*>(a.k_new) + ((size_t)r * a.n_kv + (u - a.n_head)) * a.dim : src;
    const uint16_t* w = reinterpret_cast<const uint16_t*>(key ? a.k_norm : a.q_norm);
    const int half = a.rot_dims / 2, np = a.rot_dims / 8, i0 = j < np ? 4 * j : a.rot_dims + 4 * (j - np);
    const bool on = head_on && i0 < a.dim, pair = on && j < np;
    f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f}, y = x;
    if (on) x = rb_ld4(src + i0);
    if (pair) y = rb_ld4(src + i0 + half);
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 4; e++) ss = fmaf(x[e], x[e], fmaf(y[e], y[e], ss));
#pragma unroll
    for (int o = 1; o < L; o <<= 1) ss += __shfl_xor(ss, o, 64);
    if (!on) return;
    const float rs = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
    const f32x4 one = f32x4{1.f, 1.f, 1.f, 1.f}, wx = w ? rb_ld4(w + i0) : one;
#pragma unroll
    for (int e = 0; e < 4; e++) x[e] *= rs * wx[e];
    if (pair) {
        const f32x4 wy = w ? rb_ld4(w + i0 + half) : one;
        const f32x4* cs = reinterpret_cast<const f32x4*>(a.rope + ((size_t)pos * half + i0) * 2);
        const f32x4 c01 = cs[0], c23 = cs[1];
        const float co[4] = {c01.x, c01.z, c23.x, c23.z}, si[4] = {c01.y, c01.w, c23.y, c23.w};
        f32x4 p, q;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const float yy = y[e] * rs * wy[e];
            p[e] = x[e] * co[e] - yy * si[e], q[e] = yy * co[e] + x[e] * si[e];
        }
        rb_st4(dst + i0, p), rb_st4(dst + i0 + half, q);
    } else {
        rb_st4(dst + i0, x);
    }
}
// ---- the batch's last cache_rows keys / values of every sequence into its slot's ring
template <class T>
__global__ void __launch_bounds__(256) rb_store_kernel(const kf_rb_attention a, const int32_t* __restrict__ meta) {
    const int r = blockIdx.x, pos = meta[KF_RB_META * r], last = meta[KF_RB_META * r + 3];
    if (pos < 0 || pos <= last - a.cache_rows) return;
    const int kvd = a.n_kv * a.dim, vvd = a.n_kv * a.vdim;
    const size_t slot = (size_t)meta[KF_RB_META * r + 1] * a.slot_stride, row = pos % a.cache_rows, head = a.head_stride;
    const T* k = reinterpret_cast<const T*>(a.k_new) + (size_t)r * kvd;
    const T* v = reinterpret_cast<const T*>(a.raw) + (size_t)r * a.ldraw + a.v_col;
    T *kc = reinterpret_cast<T*>(a.k_cache) + slot + row * a.dim, *vc = reinterpret_cast<T*>(a.v_cache) + slot + row * a.vdim;
    for (int i = threadIdx.x; i < kvd; i += blockDim.x) {
        const int g = i / a.dim;
        kc[g * head + (i - g * a.dim)] = k[i];
    }
    for (int i = threadIdx.x; i < vvd; i += blockDim.x) {
        const int g = i / a.vdim;
        vc[g * head + (i - g * a.vdim)] = v[i];
    }
}

// ---- the plain form: one wave per (row, head); scores of 64 keys at a time, one key per lane, then the values with one dimension per lane.
// ring_only: every key up to the row's own is in the ring already (decode)
template <class T>
__global__ void __launch_bounds__(64) rb_attn_plain_kernel(const kf_rb_attention a, const int32_t* __restrict__ meta, int ring_only) {
    extern __shared__ float s_q[]; /* [dim] */
    __shared__ float s_p[64];
    __shared__ const T* s_v[64];
    const int r = blockIdx.x, n = blockIdx.y, lane = threadIdx.x;
    const int pos = meta[KF_RB_META * r], slot = meta[KF_RB_META * r + 1], pos0 = ring_only ? pos + 1 : meta[KF_RB_META * r + 2];
    if (pos < 0) return;
    const int g = n / (a.n_head / a.n_kv), kvd = a.n_kv * a.dim;
    const T* raw = reinterpret_cast<const T*>(a.raw);
    for (int i = lane; i < a.dim; i += 64) s_q[i] = rb_ld(raw + (size_t)r * a.ldraw + (size_t)n * a.dim + i);
    __syncthreads();
    constexpr int ND = 8; /* dims per lane: vdim <= 512 */
    float o[ND];
#pragma unroll
    for (int j = 0; j < ND; j++) o[j] = 0.f;
    float M = -__builtin_inff(), l = 0.f;
    for (int k0 = rb_first_key(pos, a); k0 <= pos; k0 += 64) {
        const int key = k0 + lane;
        float s = -__builtin_inff();
        const T* v = nullptr;
        if (key <= pos) {
            const T* k;
            if (key >= pos0) {
                const size_t row = (size_t)r - (pos - key);
                k = reinterpret_cast<const T*>(a.k_new) + row * kvd + (size_t)g * a.dim;
                v = raw + row * a.ldraw + a.v_col + (size_t)g * a.vdim;
            } else {
                const size_t head = (size_t)slot * a.slot_stride + (size_t)g * a.head_stride, row = key % a.cache_rows;
                k = reinterpret_cast<const T*>(a.k_cache) + head + row * a.dim, v = reinterpret_cast<const T*>(a.v_cache) + head + row * a.vdim;
            }
            float d = 0.f;
            for (int i = 0; i < a.dim; i++) d = fmaf(s_q[i], rb_ld(k + i), d);
            s = d * a.scale;
        }
        const float mt = wave_max(s), Mn = fmaxf(M, mt);
        const float alpha = expf(M - Mn), p = expf(s - Mn); /* masked: 0 */
        l = l * alpha + wave_sum(p);
        M = Mn;
        __syncthreads();
        s_p[lane] = p, s_v[lane] = v;
        __syncthreads();
        const int nk = pos - k0 + 1 < 64 ? pos - k0 + 1 : 64;
#pragma unroll
        for (int j = 0; j < ND; j++) o[j] *= alpha;
        for (int i = 0; i < nk; i++) {
            const float pi = s_p[i];
            const T* vi = s_v[i];
#pragma unroll
            for (int j = 0; j < ND; j++) {
                const int d = lane + 64 * j;
                if (d < a.vdim) o[j] = fmaf(pi, rb_ld(vi + d), o[j]);
            }
        }
    }
    float f = a.out_scale;
    if (a.sink) {
        const float Ms = fmaxf(M, 0.f), fs = expf(M - Ms);
        l = l * fs + expf(-Ms), f *= fs;
    }
    const T* gate = raw + (size_t)r * a.ldraw + a.gate_col + (size_t)n * a.vdim;
    T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.ldout + (size_t)n * a.vdim;
#pragma unroll
    for (int j = 0; j < ND; j++) {
        const int d = lane + 64 * j;
        if (d < a.vdim) rb_st(out + d, o[j] * f / l * (a.gated ? rb_sigmoid(rb_ld(gate + d)) : 1.f));
    }
}

// what a column's sum of values is multiplied by, from its maximum M (in powers of two) and its sum l: 1 / l, or with the sink's score of 0 in the denominator
__device__ __forceinline__ float rb_softmax_factor(float M, float l, int sink) {
    if (!sink) return 1.0f / l;
    const float Ms = fmaxf(M, 0.f), f = rb_exp2(M - Ms);
    return f / (l * f + rb_exp2(-Ms));
}

// ---- MFMA form: one 32-key tile against a wave's 32 columns
constexpr int RB_VPAD = 32; /* V row padding, elements: the 4 rows of a transposing read land on distinct bank groups */
template <int HD>
struct RbTile {
    static constexpr int NS = HD / 16, NDB = HD / 32, KS = HD + 8, VS = HD + RB_VPAD;
    f32x16_t o[NDB];
    float M, l;
    __device__ __forceinline__ void init() {
#pragma unroll
        for (int db = 0; db < NDB; db++)
#pragma unroll
            for (int i = 0; i < 16; i++) o[db][i] = 0.f;
        M = -__builtin_inff(), l = 0.f;
    }
    // keys k0 .. k0 + 31 staged at kb [32][KS], vb [32][VS]; the column sees keys lo .. hi (every: the whole tile is visible to every column of the wave)
    __device__ __forceinline__ void step(const uint16_t* kb, const uint16_t* vb, const u32x4 (&qf)[NS], float sc2, int k0, int lo, int hi, bool every, int lane) {
        const int r = lane & 31, h = lane >> 5;
        f32x16_t st;
#pragma unroll
        for (int i = 0; i < 16; i++) st[i] = 0.f;
#pragma unroll
        for (int s = 0; s < NS; s++) {
            const u32x4 A = *reinterpret_cast<const u32x4*>(kb + r * KS + 16 * s + 8 * h);
            st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, A), __builtin_bit_cast(bf16x8_t, qf[s]), st, 0, 0, 0);
        }
        float mt = -__builtin_inff();
        if (every) {
#pragma unroll
            for (int i = 0; i < 16; i++) st[i] *= sc2, mt = fmaxf(mt, st[i]);
        } else {
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const int key = k0 + 4 * h + (i & 3) + 8 * (i >> 2);
                st[i] = key >= lo && key <= hi ? st[i] * sc2 : -__builtin_inff();
                mt = fmaxf(mt, st[i]);
            }
        }
        mt = xmax32(mt);
        if (mt > M) {
            const float alpha = rb_exp2(M - mt);
            l *= alpha;
#pragma unroll
            for (int db = 0; db < NDB; db++)
#pragma unroll
                for (int i = 0; i < 16; i++) o[db][i] *= alpha;
            M = mt;
        }
        const float Mref = M == -__builtin_inff() ? 0.f : M; /* a column that has seen nothing: p = 0 */
        uint32_t ph[8], pl[8];
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const float p0 = rb_exp2(st[2 * i] - Mref), p1 = rb_exp2(st[2 * i + 1] - Mref);
            l += p0;
            l += p1;
            ph[i] = pack_bf16x2(p0, p1);
            pl[i] = pack_bf16x2(p0 - bf_lo(ph[i]), p1 - bf_hi(ph[i]));
        }
#pragma unroll
        for (int s2 = 0; s2 < 2; s2++) {
            const u32x4 B = u32x4{ph[4 * s2], ph[4 * s2 + 1], ph[4 * s2 + 2], ph[4 * s2 + 3]}, B2 = u32x4{pl[4 * s2], pl[4 * s2 + 1], pl[4 * s2 + 2], pl[4 * s2 + 3]};
#pragma unroll
            for (int db = 0; db < NDB; db++) {
                const uint16_t* vp = vb + (16 * s2 + 4 * h + ((lane & 15) >> 2)) * VS + db * 32 + (lane & 16) + 4 * (lane & 3);
                const bf16x4_t x = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(vp));
                const bf16x4_t y = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(vp + 8 * VS));
                const bf16x8_t A = bf16x8_t{x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
                o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(A, __builtin_bit_cast(bf16x8_t, B), o[db], 0, 0, 0);
                o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(A, __builtin_bit_cast(bf16x8_t, B2), o[db], 0, 0, 0);
            }
        }
    }
};

// q, k_new prepared.  grid (column blocks of the longest sequence, n_kv, sequences), 128 columns per workgroup, 32 per wave.  KH = 2: waves 0 - 3 walk the even key tiles,
// waves 4 - 7 the odd ones, the two partial softmaxes of a column meet in LDS at the end (launches of about one workgroup per CU last as long as their longest walk).
// Key `key` lies in the batch from the sequence's first position on, in the slot's ring before it.
template <int HD, int KH>
__global__ void __launch_bounds__(256 * KH, HD <= 128 ? 2 : 1) rb_attn_prefill_kernel(const kf_rb_attention a, const int32_t* __restrict__ seqs) {
    using Tile = RbTile<HD>;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    constexpr int KS = Tile::KS, VS = Tile::VS, CH = HD / 8, CPT = (32 * CH + 255) / 256, NREG = Tile::NDB * 16;
    const int tid = threadIdx.x & 255, lane = tid & 63, wid = tid >> 6, kh = KH == 2 ? (int)threadIdx.x >> 8 : 0, r = lane & 31, h = lane >> 5, kvd = a.n_kv * a.dim;
    uint16_t* ks = reinterpret_cast<uint16_t*>(smem_raw) + (size_t)kh * 2 * 32 * (KS + VS); /* 2 x [32][KS] */
    uint16_t* vs = ks + 2 * 32 * KS;                                                         /* 2 x [32][VS] */
    const int row0 = seqs[4 * blockIdx.z], n = seqs[4 * blockIdx.z + 1], pos0 = seqs[4 * blockIdx.z + 2], slot = seqs[4 * blockIdx.z + 3];
    // consecutive workgroups go to consecutive XCDs: the workgroups of a kv-head stay on the same ones, its keys and values in their L2
    const int wg = (int)blockIdx.x + (int)gridDim.x * (int)blockIdx.y, g = wg % a.n_kv, bx = (int)gridDim.x - 1 - wg / a.n_kv;
    const int GQ = a.n_head / a.n_kv, ncol = n * GQ;
    if (bx * 128 >= ncol) return; /* workgroup-uniform */
    const uint16_t* raw = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)row0 * a.ldraw;
    const uint16_t *k_new = reinterpret_cast<const uint16_t*>(a.k_new) + (size_t)row0 * kvd + (size_t)g * a.dim, *v_new = raw + a.v_col + (size_t)g * a.vdim;
    const uint16_t* k_ring = reinterpret_cast<const uint16_t*>(a.k_cache) + (size_t)slot * a.slot_stride + (size_t)g * a.head_stride;
    const uint16_t* v_ring = reinterpret_cast<const uint16_t*>(a.v_cache) + (size_t)slot * a.slot_stride + (size_t)g * a.head_stride;
    // this lane pair's column; columns past the end repeat the last one and are not stored
    int c = bx * 128 + wid * 32 + r;
    const bool col_ok = c < ncol;
    c = col_ok ? c : ncol - 1;
    const int tok = c / GQ, head = g * GQ + (c - tok * GQ), pos = pos0 + tok, lo = rb_first_key(pos, a);
    // the wave's and the workgroup's key ranges
    auto tok_of = [&](int cc) { return (cc < ncol ? cc : ncol - 1) / GQ; };
    const int w0 = pos0 + tok_of(bx * 128 + wid * 32), w1 = pos0 + tok_of(bx * 128 + wid * 32 + 31);
    const int wlo = rb_first_key(w0, a), wlo1 = rb_first_key(w1, a);
    const int klo = rb_first_key(pos0 + tok_of(bx * 128), a), khi = pos0 + tok_of(bx * 128 + 127);
    u32x4 qf[Tile::NS];
    {
        const uint16_t* q = raw + (size_t)tok * a.ldraw + (size_t)head * a.dim;
#pragma unroll
        for (int s = 0; s < Tile::NS; s++) {
            qf[s] = u32x4{0, 0, 0, 0};
            if (16 * s + 8 * h < a.dim) qf[s] = *reinterpret_cast<const u32x4*>(q + 16 * s + 8 * h);
        }
    }
    u32x4 kr[CPT], vr[CPT];
    const uint32_t ldk = (uint32_t)kvd, ldv = (uint32_t)a.ldraw, ring = (uint32_t)a.cache_rows; /* offsets inside a batch or a ring fit 32 bits (checked by the launcher) */
    auto tload = [&](int k0) {
        const int where = k0 >= pos0 ? 0 : (k0 + 31 < pos0 && k0 + 31 <= khi ? 1 : 2); /* all new, all old, a mixture (workgroup-uniform) */
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int ch = tid + 256 * i, key = ch / CH, d = (ch - key * CH) * 8;
            kr[i] = vr[i] = u32x4{0, 0, 0, 0};
            if (32 * CH % 256 == 0 || key < 32) {
                const int kk = k0 + key < khi ? k0 + key : khi; /* past the last key: masked, never read past it */
                const uint16_t *kb = k_new, *vb = v_new;
                uint32_t ok, ov;
                if (where == 0 || (where == 2 && kk >= pos0)) {
                    ok = (uint32_t)(kk - pos0) * ldk, ov = (uint32_t)(kk - pos0) * ldv;
                } else {
                    kb = k_ring, vb = v_ring;
                    const uint32_t row = (uint32_t)kk % ring;
                    ok = row * (uint32_t)a.dim, ov = row * (uint32_t)a.vdim;
                }
                if (d < a.dim) kr[i] = *reinterpret_cast<const u32x4*>(kb + (ok + d));
                if (d < a.vdim) vr[i] = *reinterpret_cast<const u32x4*>(vb + (ov + d));
            }
        }
    };
    auto tstore = [&](int b) {
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int ch = tid + 256 * i, key = ch / CH, d = (ch - key * CH) * 8;
            if (32 * CH % 256 == 0 || key < 32) {
                *reinterpret_cast<u32x4*>(ks + (b * 32 + key) * KS + d) = kr[i];
                *reinterpret_cast<u32x4*>(vs + (b * 32 + key) * VS + d) = vr[i];
            }
        }
    };
    Tile T;
    T.init();
    const float sc2 = a.scale * RB_LOG2E;
    const int ntile = (khi - klo) / 32 + 1, nstep = (ntile + KH - 1) / KH; /* both key halves make the same steps and barriers; the odd half's last may be empty */
    tload(klo + 32 * (kh < ntile ? kh : ntile - 1));
    tstore(0);
    __syncthreads();
    for (int j = 0; j < nstep; j++) {
        const int t = kh + KH * j, k0 = klo + 32 * t, b = j & 1;
        const bool more = t + KH < ntile;
        if (more) tload(k0 + 32 * KH);
        if (t < ntile && k0 + 31 >= wlo && k0 <= w1) /* wave-uniform */
            T.step(ks + b * 32 * KS, vs + b * 32 * VS, qf, sc2, k0, lo, pos, k0 >= wlo1 && k0 + 31 <= w0, lane);
        if (more) tstore(b ^ 1);
        __syncthreads();
    }
    if constexpr (KH == 2) { /* the odd half hands its part over, the even half merges */
        float* ex = reinterpret_cast<float*>(smem_raw); /* [NREG + 2][256] */
        if (kh == 1) {
#pragma unroll
            for (int db = 0; db < Tile::NDB; db++)
#pragma unroll
                for (int i = 0; i < 16; i++) ex[(db * 16 + i) * 256 + tid] = T.o[db][i];
            ex[NREG * 256 + tid] = T.M, ex[(NREG + 1) * 256 + tid] = T.l;
        }
        __syncthreads();
        if (kh == 1) return;
        const float M1 = ex[NREG * 256 + tid], Mm = fmaxf(T.M, M1); /* one of the halves has seen a key of the column */
        const float f0 = rb_exp2(T.M - Mm), f1 = rb_exp2(M1 - Mm);
        T.l = T.l * f0 + ex[(NREG + 1) * 256 + tid] * f1, T.M = Mm;
#pragma unroll
        for (int db = 0; db < Tile::NDB; db++)
#pragma unroll
            for (int i = 0; i < 16; i++) T.o[db][i] = T.o[db][i] * f0 + ex[(db * 16 + i) * 256 + tid] * f1;
    }
    const float l = xsum32(T.l);
    if (!col_ok) return;
    const float inv = a.out_scale * rb_softmax_factor(T.M, l, a.sink);
    const uint16_t* gate = raw + (size_t)tok * a.ldraw + a.gate_col + (size_t)head * a.vdim;
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out) + (size_t)(row0 + tok) * a.ldout + (size_t)head * a.vdim;
#pragma unroll
    for (int db = 0; db < Tile::NDB; db++)
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const int d = 32 * db + 8 * q + 4 * h;
            if (d >= a.vdim) continue;
            f32x4 v = f32x4{T.o[db][4 * q] * inv, T.o[db][4 * q + 1] * inv, T.o[db][4 * q + 2] * inv, T.o[db][4 * q + 3] * inv};
            if (a.gated) {
                const f32x4 gv = rb_ld4(gate + d);
#pragma unroll
                for (int j = 0; j < 4; j++) v[j] *= rb_sigmoid(gv[j]);
            }
            rb_st4(out + d, v);
        }
}

// decode: grid (n_kv * column blocks of 32 query heads, key ranges of `span` keys, rows).  raw is not prepared: q and the new key are normed and rotated here while the first
// tiles are on their way; the workgroup whose range holds the row's position patches the new key and value into its tile and puts them into the ring.
template <int HD>
__device__ __forceinline__ void rb_attn_decode(const kf_rb_attention& a, const int32_t* __restrict__ meta, int span, int n_range, int block, int range, int rr, int n_rows, unsigned char* smem_raw) {
    using Tile = RbTile<HD>;
    constexpr int KS = Tile::KS, VS = Tile::VS, CH = HD / 8, WAVE_EL = 32 * (KS + VS), NREG = Tile::NDB * 16;
    const int pos = meta[KF_RB_META * rr], slot = meta[KF_RB_META * rr + 1];
    if (pos < 0) return; /* workgroup-uniform, like the next */
    const int first = rb_first_key(pos, a), k_lo = first + range * span, k_hi = k_lo + span - 1 < pos ? k_lo + span - 1 : pos;
    if (k_lo > pos) return;
    const int GQ = a.n_head / a.n_kv, ncb = (GQ + 31) / 32, g = block / ncb, cb = block % ncb, col0 = cb * 32, ncol = GQ - col0 < 32 ? GQ - col0 : 32;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, r = lane & 31, h = lane >> 5;
    uint16_t* s_new = reinterpret_cast<uint16_t*>(smem_raw);             /* the new key, the new value: [2][HD] */
    uint16_t* s_kv = s_new + 2 * HD;                                     /* [4 waves] [32][KS] + [32][VS]; before the walk: */
    uint16_t* s_q = s_kv;                                                /* [32][KS] */
    float* s_buf = reinterpret_cast<float*>(s_q + 32 * KS);              /* [4][HD] */
    __shared__ int s_last;
    const uint16_t* raw = reinterpret_cast<const uint16_t*>(a.raw) + (size_t)rr * a.ldraw;
    const size_t base = (size_t)slot * a.slot_stride + (size_t)g * a.head_stride;
    uint16_t *kc = reinterpret_cast<uint16_t*>(a.k_cache) + base, *vc = reinterpret_cast<uint16_t*>(a.v_cache) + base;
    constexpr int CPT = CH / 2; /* chunks per lane of a 32-row tile */
    u32x4 kr[CPT], vr[CPT];
    auto tload = [&](int k0) { /* (the row's own position still holds an older key: patched below) */
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int ch = lane + 64 * i, key = ch / CH, d = (ch - key * CH) * 8;
            kr[i] = vr[i] = u32x4{0, 0, 0, 0};
            const int kk = k0 + key < k_hi ? k0 + key : k_hi;
            const uint32_t row = (uint32_t)kk % (uint32_t)a.cache_rows;
            if (d < a.dim) kr[i] = *reinterpret_cast<const u32x4*>(kc + (row * (uint32_t)a.dim + d));
            if (d < a.vdim) vr[i] = *reinterpret_cast<const u32x4*>(vc + (row * (uint32_t)a.vdim + d));
        }
    };
    int k0 = k_lo + wid * 32;
    if (k0 <= k_hi) tload(k0);
    for (int i = tid; i < 32 * KS / 8; i += 256) reinterpret_cast<u32x4*>(s_q)[i] = u32x4{0, 0, 0, 0};
    __syncthreads();
    for (int u = wid; u <= ncol; u += 4) {
        if (u < ncol) {
            rb_prep_head(raw + (size_t)(g * GQ + col0 + u) * a.dim, s_q + u * KS, reinterpret_cast<const uint16_t*>(a.q_norm), a.unit, a.rope, a.rot_dims, a.dim, pos, a.eps, s_buf + wid * HD, lane);
        } else if (k_hi == pos) {
            const uint16_t* k = raw + (size_t)(a.n_head + g) * a.dim;
            rb_prep_head(k, s_new, reinterpret_cast<const uint16_t*>(a.k_norm), a.unit, a.rope, a.rot_dims, a.dim, pos, a.eps, s_buf + wid * HD, lane);
            const uint16_t* vn = raw + a.v_col + (size_t)g * a.vdim;
            const size_t row = pos % a.cache_rows;
            for (int i = lane; i < HD; i += 64) {
                const uint16_t v = i < a.vdim ? vn[i] : (uint16_t)0;
                s_new[HD + i] = v;
                if (i >= a.dim) s_new[i] = 0;
                if (i < a.dim && cb == 0) kc[row * a.dim + i] = s_new[i];
                if (i < a.vdim && cb == 0) vc[row * a.vdim + i] = v;
            }
        }
    }
    __syncthreads();
    u32x4 qf[Tile::NS];
#pragma unroll
    for (int s = 0; s < Tile::NS; s++) qf[s] = *reinterpret_cast<const u32x4*>(s_q + r * KS + 16 * s + 8 * h);
    __syncthreads(); /* the queries are in registers: their place is a tile's from here on */
    uint16_t *ks = s_kv + (size_t)wid * WAVE_EL, *vs = ks + 32 * KS;
    Tile T;
    T.init();
    const float sc2 = a.scale * RB_LOG2E;
    for (; k0 <= k_hi; k0 += 128) {
        __builtin_amdgcn_wave_barrier(); /* the tile is this wave's own: its LDS accesses are in order, only the compiler has to be told */
#pragma unroll
        for (int i = 0; i < CPT; i++) {
            const int ch = lane + 64 * i, key = ch / CH, d = (ch - key * CH) * 8;
            const bool own = k_hi == pos && k0 + key >= pos; /* (and the rows behind it: masked, but finite) */
            *reinterpret_cast<u32x4*>(ks + key * KS + d) = own ? *reinterpret_cast<const u32x4*>(s_new + d) : kr[i];
            *reinterpret_cast<u32x4*>(vs + key * VS + d) = own ? *reinterpret_cast<const u32x4*>(s_new + HD + d) : vr[i];
        }
        if (k0 + 128 <= k_hi) tload(k0 + 128);
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        T.step(ks, vs, qf, sc2, k0, k_lo, k_hi, k0 + 31 <= k_hi, lane);
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
    }
    // the four waves' partial softmaxes: registers lane-major per wave, every wave finishes a quarter of them
    __syncthreads();
    float* ex = reinterpret_cast<float*>(s_kv); /* [4][NREG + 2][64] */
#pragma unroll
    for (int db = 0; db < Tile::NDB; db++)
#pragma unroll
        for (int i = 0; i < 16; i++) ex[((size_t)wid * (NREG + 2) + db * 16 + i) * 64 + lane] = T.o[db][i];
    ex[((size_t)wid * (NREG + 2) + NREG) * 64 + lane] = T.M;
    ex[((size_t)wid * (NREG + 2) + NREG + 1) * 64 + lane] = xsum32(T.l);
    __syncthreads();
    float f[4], M = -__builtin_inff(), L = 0.f;
#pragma unroll
    for (int w = 0; w < 4; w++) M = fmaxf(M, ex[((size_t)w * (NREG + 2) + NREG) * 64 + lane]); /* wave 0 has seen a key: finite */
#pragma unroll
    for (int w = 0; w < 4; w++) {
        f[w] = rb_exp2(ex[((size_t)w * (NREG + 2) + NREG) * 64 + lane] - M);
        L += f[w] * ex[((size_t)w * (NREG + 2) + NREG + 1) * 64 + lane];
    }
    const int n_used = (pos - first) / span + 1; /* key ranges this row has */
    const int head = g * GQ + col0 + (r < ncol ? r : 0);
    const uint16_t* gate = raw + a.gate_col + (size_t)head * a.vdim;
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out) + (size_t)rr * a.ldout + (size_t)head * a.vdim;
    float* parts = reinterpret_cast<float*>(a.scratch) + RB_CNT_STRIDE * (size_t)n_rows * a.n_head; /* behind the arrival counters: [row][head][range][vdim + 2] */
    float* part = parts + (((size_t)rr * a.n_head + head) * n_range + range) * (a.vdim + 2);
    const float inv = a.out_scale * rb_softmax_factor(M, L, a.sink);
    for (int q = wid; q < Tile::NDB * 4 && r < ncol; q += 4) { /* a quad of registers = four consecutive d */
        const int d = 8 * q + 4 * h;
        if (d >= a.vdim) continue;
        f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 4; w++)
#pragma unroll
            for (int j = 0; j < 4; j++) v[j] = fmaf(f[w], ex[((size_t)w * (NREG + 2) + 4 * q + j) * 64 + lane], v[j]);
        if (n_used > 1) {
#pragma unroll
            for (int j = 0; j < 4; j++) rb_st_sc1(part + 2 + d + j, v[j]);
        } else {
            const f32x4 gv = a.gated ? rb_ld4(gate + d) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < 4; j++) v[j] *= a.gated ? inv * rb_sigmoid(gv[j]) : inv;
            rb_st4(out + d, v);
        }
    }
    if (n_used == 1) return;
    // the ranges' parts leave with write-through stores; every wave has their acknowledgements before one lane counts the workgroup in; the last one in merges and puts the
    // counter back to zero (kf_attn.hip's scheme)
    if (wid == 0 && h == 0 && r < ncol) rb_st_sc1(part, M), rb_st_sc1(part + 1, L);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    int* counter = reinterpret_cast<int*>(a.scratch) + RB_CNT_STRIDE * ((size_t)rr * a.n_head + block);
    if (tid == 0) s_last = __hip_atomic_fetch_add(counter, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == n_used - 1;
    __syncthreads();
    if (!s_last) return;
    if (tid == 0) __hip_atomic_store(counter, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    for (int c = wid; c < ncol; c += 4) {
        const int hd = g * GQ + col0 + c;
        const float* p = parts + ((size_t)rr * a.n_head + hd) * n_range * (a.vdim + 2);
        const bool mine = lane < n_used;
        const float ms = mine ? rb_ld_sc1(p + (size_t)lane * (a.vdim + 2)) : -__builtin_inff(), ls = mine ? rb_ld_sc1(p + (size_t)lane * (a.vdim + 2) + 1) : 0.f;
        const float mw = wave_max(ms), mx = a.sink ? fmaxf(mw, 0.f) : mw, fs = rb_exp2(ms - mx), tot = a.out_scale / (wave_sum(fs * ls) + (a.sink ? rb_exp2(-mx) : 0.f));
        constexpr int DPL = (HD + 63) / 64;
        float v[DPL];
#pragma unroll
        for (int e = 0; e < DPL; e++) v[e] = 0.f;
        for (int s0 = 0; s0 < n_used; s0 += 8) {
            float w[DPL][8];
#pragma unroll
            for (int e = 0; e < DPL; e++)
#pragma unroll
                for (int s = 0; s < 8; s++) w[e][s] = s0 + s < n_used && lane + 64 * e < a.vdim ? rb_ld_sc1(p + (size_t)(s0 + s) * (a.vdim + 2) + 2 + lane + 64 * e) : 0.f;
#pragma unroll
            for (int s = 0; s < 8; s++) {
                const float f1 = __shfl(fs, (s0 + s) & 63, 64); /* past n_used: exp2(-inf) = 0 */
#pragma unroll
                for (int e = 0; e < DPL; e++) v[e] = fmaf(f1, w[e][s], v[e]);
            }
        }
#pragma unroll
        for (int e = 0; e < DPL; e++) {
            const int d = lane + 64 * e;
            if (d < a.vdim)
                reinterpret_cast<uint16_t*>(a.out)[(size_t)rr * a.ldout + (size_t)hd * a.vdim + d] =
                    f2bf(v[e] * tot * (a.gated ? rb_sigmoid(bf2f(raw[a.gate_col + (size_t)hd * a.vdim + d])) : 1.f));
        }
    }
}
template <int HD>
__global__ void __launch_bounds__(256) rb_attn_decode_kernel(const kf_rb_attention a, const int32_t* __restrict__ meta, int span, int n_range) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    rb_attn_decode<HD>(a, meta, span, n_range, blockIdx.x, blockIdx.y, blockIdx.z, gridDim.z, smem_raw);
}
// a layer's decayed sum (its heads first) and its attention in one launch: neither waits for the other
template <int HD>
__global__ void __launch_bounds__(256) rb_attn_decay_decode_kernel(const kf_rb_attention a, const kf_rb_decay d, const int32_t* __restrict__ meta, int span, int n_range) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    const int block = (int)blockIdx.x - d.n_head, blocks = ((int)gridDim.x - d.n_head) / n_range;
    if (block < 0) rc_decay_step<uint16_t, 256, 16>(d, meta, blockIdx.x, blockIdx.y, gridDim.y, reinterpret_cast<float*>(smem_raw));
    else rb_attn_decode<HD>(a, meta, span, n_range, block % blocks, block / blocks, blockIdx.y, gridDim.y, smem_raw);
}
constexpr int RB_MAX_RANGES = 32;
static void decode_ranges(int n_rows, int n_kv, int keys, int& span, int& n_range) {
    n_range = (keys + 255) / 256; /* a range is at least two tiles per wave */
    const int want = (512 + n_rows * n_kv - 1) / (n_rows * n_kv); /* two workgroups per CU: one round */
    n_range = std::max(1, std::min(n_range, std::min(want, RB_MAX_RANGES)));
    span = ((keys + n_range - 1) / n_range + 127) / 128 * 128;
    n_range = (keys + span - 1) / span;
}
template <class K>
static int big_lds(K kernel, size_t smem, int& done) {
    if (done || smem <= 64 * 1024) return KF_OK;
    if (hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess) return KF_HIP_CHECK;
    done = 1;
    return KF_OK;
}
template <int HD, int KH>
static int prefill_kh(hipStream_t st, const kf_rb_attention& a, const int32_t* seqs, dim3 grid) {
    constexpr size_t tiles = KH * 2 * 2 * 32 * (size_t)(RbTile<HD>::KS + RbTile<HD>::VS), merge = KH == 2 ? 256 * 4 * (size_t)(RbTile<HD>::NDB * 16 + 2) : 0;
    constexpr size_t smem = tiles > merge ? tiles : merge;
    static_assert(smem <= 160 * 1024, "LDS");
    static int done = 0;
    if (big_lds(rb_attn_prefill_kernel<HD, KH>, smem, done)) return KF_HIP_CHECK;
    hipLaunchKernelGGL((rb_attn_prefill_kernel<HD, KH>), grid, dim3(256 * KH), smem, st, a, seqs);
    return KF_OK;
}
template <int HD>
static int prefill_go(hipStream_t st, const kf_rb_attention& a, const int32_t* seqs, int n_seq, int max_n) {
    const dim3 grid((unsigned)(((long long)max_n * (a.n_head / a.n_kv) + 127) / 128), a.n_kv, n_seq);
    if constexpr (HD <= 128) {
        if ((long)grid.x * grid.y * grid.z <= 512 && max_n >= 256) return prefill_kh<HD, 2>(st, a, seqs, grid);
    }
    return prefill_kh<HD, 1>(st, a, seqs, grid);
}
template <int HD>
static int decode_go(hipStream_t st, const kf_rb_attention& a, const kf_rb_decay* d, const int32_t* meta, int n_rows, int span, int n_range) {
    constexpr size_t tiles = 4 * 2 * 32 * (size_t)(RbTile<HD>::KS + RbTile<HD>::VS), merge = 4 * (size_t)(RbTile<HD>::NDB * 16 + 2) * 256;
    constexpr size_t smem = 4 * HD + (tiles > merge ? tiles : merge);
    static_assert(32 * RbTile<HD>::KS * 2 + 16 * HD <= tiles, "queries in the tiles' place");
    static_assert(smem <= 160 * 1024, "LDS");
    const int blocks = a.n_kv * ((a.n_head / a.n_kv + 31) / 32);
    if (d) {
        static int done = 0;
        const size_t both = std::max(smem, rc_decay_step_lds(d->dim, d->vdim, 256));
        if (both > 150 * 1024) return 1;
        if (!done && hipFuncSetAttribute((const void*)rb_attn_decay_decode_kernel<HD>, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024) != hipSuccess) return KF_HIP_CHECK;
        done = 1;
        hipLaunchKernelGGL(rb_attn_decay_decode_kernel<HD>, dim3(d->n_head + blocks * n_range, n_rows), dim3(256), both, st, a, *d, meta, span, n_range);
        return KF_OK;
    }
    static int done = 0;
    if (big_lds(rb_attn_decode_kernel<HD>, smem, done)) return KF_HIP_CHECK;
    hipLaunchKernelGGL(rb_attn_decode_kernel<HD>, dim3(blocks, n_range, n_rows), dim3(256), smem, st, a, meta, span, n_range);
    return KF_OK;
}
static bool mfma_served(const kf_rb_attention& a, int n_rows) {
    return a.type == KF_BF16 && (int64_t)n_rows * a.ldraw < ((int64_t)1 << 30) && (int64_t)a.cache_rows * a.n_kv * std::max(a.dim, a.vdim) < ((int64_t)1 << 30) && a.dim % 8 == 0 && a.dim <= 256 && a.vdim % 8 == 0 && a.vdim <= 256 && a.v_col % 8 == 0 && a.gate_col % 4 == 0 && a.ldraw % 8 == 0 && a.ldout % 4 == 0 && a.slot_stride % 8 == 0 && a.head_stride % 8 == 0;
}
#define RB_BY_DIM(call)                                 \
    (std::max(a.dim, a.vdim) <= 32    ? call(32)        \
     : std::max(a.dim, a.vdim) <= 64  ? call(64)        \
     : std::max(a.dim, a.vdim) <= 96  ? call(96)        \
     : std::max(a.dim, a.vdim) <= 128 ? call(128)       \
     : std::max(a.dim, a.vdim) <= 192 ? call(192)       \
                                      : call(256))

/* vector form of the prep of a prompt batch: a head's lanes fit 16 or 32, quads of both halves */
static int prep_vec_lanes(const kf_rb_attention& a) {
    if (a.type != KF_BF16 || a.dim % 4 || a.rot_dims % 8 || a.ldraw % 4 || (!a.unit && (!a.q_norm || !a.k_norm))) return 0;
    const int need = a.rot_dims / 8 + (a.dim - a.rot_dims) / 4;
    return need <= 16 ? 16 : (need <= 32 ? 32 : 0);
}
template <class T>
static void prep_go(hipStream_t st, const kf_rb_attention& a, const int32_t* meta, int n, bool store) {
    const dim3 grid(n, (a.n_head + a.n_kv + 3) / 4);
    const size_t smem = 4 * (size_t)a.dim * sizeof(float);
    if (const int L = store ? 0 : prep_vec_lanes(a)) {
        const dim3 vgrid(n, (a.n_head + a.n_kv + 256 / L - 1) / (256 / L));
        if (L == 16) hipLaunchKernelGGL(rb_prep_vec_kernel<16>, vgrid, dim3(256), 0, st, a, meta);
        else hipLaunchKernelGGL(rb_prep_vec_kernel<32>, vgrid, dim3(256), 0, st, a, meta);
        return;
    }
    if (store) hipLaunchKernelGGL((rb_prep_kernel<T, true>), grid, dim3(256), smem, st, a, meta);
    else hipLaunchKernelGGL((rb_prep_kernel<T, false>), grid, dim3(256), smem, st, a, meta);
}
template <class T>
static void plain_go(hipStream_t st, const kf_rb_attention& a, const int32_t* meta, int n, int ring_only) {
    hipLaunchKernelGGL(rb_attn_plain_kernel<T>, dim3(n, a.n_head), dim3(64), (size_t)a.dim * sizeof(float), st, a, meta, ring_only);
}
template <class T>
static void store_go(hipStream_t st, const kf_rb_attention& a, const int32_t* meta, int n) {
    const int kvd = a.n_kv * a.dim;
    hipLaunchKernelGGL(rb_store_kernel<T>, dim3(n), dim3(kvd >= 256 ? 256 : 64), 0, st, a, meta);
}

}  // namespace kf

using namespace kf;
static kf_rb_attention whole_form(const kf_rb_attention& in) {
    kf_rb_attention a = in;
    if (!a.vdim) a.vdim = a.dim;
    if (!a.v_col) a.v_col = a.n_head * a.dim;                       /* the keys as they were projected */
    if (!a.gate_col) a.gate_col = (a.n_head + a.n_kv) * a.dim;
    if (!a.scaled) a.out_scale = 1.f;
    return a;
}
static int check_attention(const kf_rb_attention* a, const int32_t* meta, int n, const char* who) {
    if (!a || !meta || n < 1 || !a->raw || !a->out || !a->k_cache || !a->v_cache || (a->rot_dims && !a->rope)) return abi_fail(KF_INVALID_ARGS, "%s: null pointer", who);
    if (a->type != KF_BF16 && a->type != KF_F32) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: storage %d", who, a->type);
    if (a->n_head < 1 || a->n_kv < 1 || a->n_head % a->n_kv || a->dim < 1 || a->rot_dims < 0 || a->rot_dims > a->dim || (a->rot_dims & 1) || a->chunk < 0 || a->cache_rows < 1)
        return abi_fail(KF_INVALID_ARGS, "%s: %d / %d heads of %d, %d rotated, chunk %d, %d cache rows", who, a->n_head, a->n_kv, a->dim, a->rot_dims, a->chunk, a->cache_rows);
    if (a->dim > 512 || a->vdim > 512) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: head sizes %d / %d (served: up to 512)", who, a->dim, a->vdim);
    if (a->vdim < 1 || a->window < 0 || (a->window && a->chunk) || (a->unit && (a->q_norm || a->k_norm)) || a->v_col < a->n_head * a->dim) return abi_fail(KF_INVALID_ARGS, "%s: values or mask", who);
    const int64_t cols = std::max((int64_t)a->v_col + (int64_t)a->n_kv * a->vdim, a->gated ? (int64_t)a->gate_col + (int64_t)a->n_head * a->vdim : 0);
    if (a->ldraw < cols || a->ldout < (int64_t)a->n_head * a->vdim || a->head_stride < (int64_t)a->cache_rows * std::max(a->dim, a->vdim) || a->slot_stride < a->head_stride * a->n_kv) return abi_fail(KF_INVALID_ARGS, "%s: strides", who);
    if (!al16(a->raw) || !al16(a->out) || !al16(a->k_cache) || !al16(a->v_cache)) return abi_fail(KF_BLAS_UNALIGN, "%s: unaligned pointer", who);
    return KF_OK;
}
constexpr int RB_BESIDE_ROWS = 16; /* rows up to which a decayed sum goes into the attention's launch */
static int attention_decode(kf_ctx* c, const kf_rb_attention* ap, const kf_rb_decay* d, const int32_t* meta, int n_rows, int max_pos, const char* who) {
    CHKCTX(c);
    if (!ap) return abi_fail(KF_INVALID_ARGS, "%s: null pointer", who);
    const kf_rb_attention a = whole_form(*ap);
    const int rc = check_attention(&a, meta, n_rows, who);
    if (rc) return rc;
    if (max_pos < 0) return abi_fail(KF_INVALID_ARGS, "%s: max_pos %d", who, max_pos);
    hipStream_t st = c->stream;
    int r = KF_OK;
    if (mfma_served(a, n_rows)) {
        int keys = max_pos + 1, span, n_range;
        const int seen = a.window > 0 ? a.window : a.chunk;
        if (seen > 0 && keys > seen) keys = seen;
        decode_ranges(n_rows, a.n_kv * ((a.n_head / a.n_kv + 31) / 32), keys, span, n_range);
        if (n_range > 1 && !a.scratch) return abi_fail(KF_INVALID_ARGS, "%s: null scratch", who);
#define RB_CALL(HD) decode_go<HD>(st, a, d, meta, n_rows, span, n_range)
        r = RB_BY_DIM(RB_CALL);
#undef RB_CALL
    } else if (a.type == KF_BF16) {
        prep_go<uint16_t>(st, a, meta, n_rows, true);
        plain_go<uint16_t>(st, a, meta, n_rows, 1);
    } else {
        prep_go<float>(st, a, meta, n_rows, true);
        plain_go<float>(st, a, meta, n_rows, 1);
    }
    if (r == 1) return abi_fail(KF_UNSUPPORTED_DATATYPE, "%s: these sizes do not share a launch", who);
    if (r != KF_OK || hipGetLastError() != hipSuccess) return abi_fail(KF_HIP_CHECK, "%s: launch failed", who);
    return KF_OK;
}
extern "C" {

size_t kf_rb_attention_scratch(int n_rows, int n_head, int dim) { return n_rows < 1 || n_head < 1 || dim < 1 ? 0 : (size_t)n_rows * n_head * (RB_CNT_STRIDE + (size_t)RB_MAX_RANGES * (dim + 2)) * sizeof(float); }

int kf_rb_attention_prefill(kf_ctx* c, const kf_rb_attention* ap, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n) {
    CHKCTX(c);
    if (!ap) return abi_fail(KF_INVALID_ARGS, "kf_rb_attention_prefill: null pointer");
    const kf_rb_attention a = whole_form(*ap);
    const int rc = check_attention(&a, meta, n_rows, "kf_rb_attention_prefill");
    if (rc) return rc;
    if (!seqs || n_seq < 1 || max_n < 1 || max_n > n_rows || !a.k_new || !al16(a.k_new)) return abi_fail(KF_INVALID_ARGS, "kf_rb_attention_prefill: bad arguments");
    hipStream_t st = c->stream;
    int r = KF_OK;
    if (a.type == KF_BF16) {
        prep_go<uint16_t>(st, a, meta, n_rows, false);
        if (mfma_served(a, n_rows)) {
#define RB_CALL(HD) prefill_go<HD>(st, a, seqs, n_seq, max_n)
            r = RB_BY_DIM(RB_CALL);
#undef RB_CALL
        } else {
            plain_go<uint16_t>(st, a, meta, n_rows, 0);
        }
        store_go<uint16_t>(st, a, meta, n_rows);
    } else {
        prep_go<float>(st, a, meta, n_rows, false);
        plain_go<float>(st, a, meta, n_rows, 0);
        store_go<float>(st, a, meta, n_rows);
    }
    if (r != KF_OK || hipGetLastError() != hipSuccess) return abi_fail(KF_HIP_CHECK, "kf_rb_attention_prefill: launch failed");
    return KF_OK;
}
int kf_rb_attention_decode(kf_ctx* c, const kf_rb_attention* ap, const int32_t* meta, int n_rows, int max_pos) { return attention_decode(c, ap, nullptr, meta, n_rows, max_pos, "kf_rb_attention_decode"); }
int kf_rb_attention_decay_decode(kf_ctx* c, const kf_rb_attention* ap, const kf_rb_decay* d, const int32_t* meta, int n_rows, int max_pos) {
    CHKCTX(c);
    int rc = rc_check_decay(d, meta, n_rows, "kf_rb_attention_decay_decode");
    if (rc) return rc;
    // one launch where a head's state fits the registers of an attention workgroup and the rows are few (more of them fill the chip either way)
    const int c4 = (d->vdim + 3) / 4;
    const bool fits = d->type == KF_BF16 && c4 <= 256 && (d->dim + 256 / c4 - 1) / (256 / c4) <= 16 && n_rows <= RB_BESIDE_ROWS;
    if (fits && ap && mfma_served(whole_form(*ap), n_rows)) return attention_decode(c, ap, d, meta, n_rows, max_pos, "kf_rb_attention_decay_decode");
    rc = kf_rb_attention_decode(c, ap, meta, n_rows, max_pos);
    return rc ? rc : kf_rb_decay_decode(c, d, meta, n_rows);
}

}  // extern "C"
