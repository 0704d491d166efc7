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
