// Element access for kernels templated on the activation type: bf16 (as uint16_t) or f32.
#pragma once
#include "common.h"
#include "../../include/skyrl_layers.h"

namespace skyrl {

__device__ __forceinline__ float ld(const uint16_t* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ float ld(const float* p) { return *p; }
__device__ __forceinline__ void st(uint16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void st(float* p, float v) { *p = v; }

__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 ld4(const uint16_t* p) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                       __uint_as_float(v.y & 0xffff0000u));
}
__device__ __forceinline__ void st4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void st4(uint16_t* p, float4 v) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
}

// VEC consecutive elements (1 or 8, 8 aligned to 16 bytes) as floats.
template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T* p, float (&o)[VEC]) {
    if constexpr (VEC == 1) {
        o[0] = ld(p);
    } else {
        static_assert(VEC == 8);
        const float4 a = ld4(p), b = ld4(p + 4);
        o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
        o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
    }
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
    st4(p, make_float4(v[0], v[1], v[2], v[3]));
    st4(p + 4, make_float4(v[4], v[5], v[6], v[7]));
}
__device__ __forceinline__ void st8(uint16_t* p, const float (&v)[8]) {
    *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                                              pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
}
__device__ __forceinline__ void unpack8(uint4 x, float (&o)[8]) {
    const uint32_t w[4] = {x.x, x.y, x.z, x.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        o[2 * i] = __uint_as_float(w[i] << 16);
        o[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}
__device__ __forceinline__ void stv(float* p, const float (&v)[1]) { *p = v[0]; }
__device__ __forceinline__ void stv(uint16_t* p, const float (&v)[1]) { st(p, v[0]); }
template <typename T>
__device__ __forceinline__ void stv(T* p, const float (&v)[8]) {
    st8(p, v);
}

constexpr float kLog2e = 1.4426950408889634f;

// exp(x): the bare base-2 instruction for a model in bf16 (its error is a few f32 roundings of x), expf for f32.
template <typename T>
__device__ __forceinline__ float exp_(float x) {
    if constexpr (sizeof(T) == 2) return fast_exp2(x * kLog2e);
    return expf(x);
}
template <typename T>
__device__ __forceinline__ float inv_(float x) {
    if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(x);
    return 1.f / x;
}
template <typename T>
__device__ __forceinline__ float sigmoid_(float x) {
    return inv_<T>(1.f + exp_<T>(-x));
}
template <typename T>
__device__ __forceinline__ float gelu_tanh_(float z) {  // 0.5 z (1 + tanh(a)) = z sigmoid(2 a)
    return z * sigmoid_<T>(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

__device__ __forceinline__ float sigmoidf_(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float siluf_(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplusf_(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// Sum over a block of NT threads, in every thread; lds holds NT / 64 floats and is free again on return.
template <int NT>
__device__ __forceinline__ float block_total(float v, float* lds) {
    v = wave_sum(v);
    if ((threadIdx.x & (kWave - 1)) == 0) lds[threadIdx.x / kWave] = v;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < NT / kWave; ++j) s += lds[j];
    __syncthreads();
    return s;
}

inline bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace skyrl

// Host: run BODY with T bound to the element type of a SKYRL_* dtype code.
#define SKYRL_DISPATCH_T(dtype, ...)             \
    if ((dtype) == SKYRL_BF16) {                 \
        using T = uint16_t;                      \
        __VA_ARGS__                              \
    } else {                                     \
        using T = float;                         \
        __VA_ARGS__                              \
    }
#define SKYRL_REQUIRE_T(dtype, name) \
    SKYRL_REQUIRE((dtype) == SKYRL_BF16 || (dtype) == SKYRL_F32, name ": dtype must be bf16 or f32")
