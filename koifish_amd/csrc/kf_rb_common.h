// kf_rb_common.h -- shared by the row-batch kernels (kf_rb_*.hip): the two storages, activations, launch interfaces.
#pragma once
#include "../../include/kf_rb.h"
#include "kf_device.h"

namespace kf {

// storage of weights and activations: bf16 bits or fp32; arithmetic is fp32 in both
__device__ __forceinline__ float rb_ld(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float rb_ld(const float* p) { return *p; }
__device__ __forceinline__ void rb_st(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void rb_st(float* p, float v) { *p = v; }
__device__ __forceinline__ f32x4 rb_ld4(const uint16_t* p) {
    const u32x2 v = *reinterpret_cast<const u32x2*>(p);
    return f32x4{bf_lo(v.x), bf_hi(v.x), bf_lo(v.y), bf_hi(v.y)};
}
__device__ __forceinline__ f32x4 rb_ld4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ void rb_st4(uint16_t* p, f32x4 v) { *reinterpret_cast<u32x2*>(p) = u32x2{pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w)}; }
__device__ __forceinline__ void rb_st4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }

__device__ __forceinline__ float rb_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float rb_softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float rb_activate(int act, float z) {
    if (act == KF_RB_RELU) return fmaxf(z, 0.0f);
    if (act == KF_RB_SILU) return z * rb_sigmoid(z);
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * fmaf(0.044715f * z * z, z, z)));
}

// what the product kernels get: kf_rb_product and its experts by value
struct RbProduct {
    kf_rb_product p;
    kf_rb_experts e;
};
// kf_rb_gemm.hip: bf16 tile kernels (any number of rows); kf_rb_linear.hip: streaming form (<= KF_RB_DECODE_MAX rows) and the fp32 product
int rb_gemm_launch(hipStream_t st, const RbProduct& a);
int rb_stream_launch(hipStream_t st, const RbProduct& a);
int rb_f32_launch(hipStream_t st, const RbProduct& a);

}  // namespace kf
