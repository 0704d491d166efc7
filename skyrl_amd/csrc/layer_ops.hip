// Norms, gated activations and the logit cap of the hybrid decoders (include/skyrl_layers.h). The
// residual stream stays f32 in HBM: the add, the norm and the optional per-pass step vector of a
// looped layer stack are one pass over a row.
#include "elem.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;

// One block per row, the row in registers: kMaxV groups of VEC elements per thread.
template <typename T, int VEC, int kMaxV>
__global__ __launch_bounds__(kNT) void add_norm_kernel(const T* __restrict__ delta, float* __restrict__ h,
                                                       const T* __restrict__ step, const T* __restrict__ w, int H,
                                                       float eps, int kind, T* __restrict__ out) {
    __shared__ float s_red[kNT / kWave];
    const int64_t base = (int64_t)blockIdx.x * H;
    const int nv = H / VEC;
    float x[kMaxV][VEC];
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * kNT;
        if (v < nv) {
            if constexpr (VEC == 4) {
                float4 a = ld4(h + base + 4 * v);
                if (delta) {
                    const float4 d = ld4(delta + base + 4 * v);
                    a.x += d.x; a.y += d.y; a.z += d.z; a.w += d.w;
                }
                if (step) {
                    const float4 d = ld4(step + 4 * v);
                    a.x += d.x; a.y += d.y; a.z += d.z; a.w += d.w;
                }
                if (delta || step) st4(h + base + 4 * v, a);
                x[k][0] = a.x; x[k][1] = a.y; x[k][2] = a.z; x[k][3] = a.w;
            } else {
                float a = h[base + v];
                if (delta) a += ld(delta + base + v);
                if (step) a += ld(step + v);
                if (delta || step) h[base + v] = a;
                x[k][0] = a;
            }
#pragma unroll
            for (int j = 0; j < VEC; ++j) sum += x[k][j];
        }
    }
    const float mean = kind == SKYRL_NORM_LAYER ? block_total<kNT>(sum, s_red) / (float)H : 0.f;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        if (threadIdx.x + k * kNT < nv) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                x[k][j] -= mean;
                ss += x[k][j] * x[k][j];
            }
        }
    }
    const float r = 1.f / sqrtf(block_total<kNT>(ss, s_red) / (float)H + eps);
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * kNT;
        if (v < nv) {
            if constexpr (VEC == 4) {
                const float4 a = ld4(w + 4 * v);
                st4(out + base + 4 * v,
                    make_float4(x[k][0] * r * a.x, x[k][1] * r * a.y, x[k][2] * r * a.z, x[k][3] * r * a.w));
            } else {
                st(out + base + v, x[k][0] * r * ld(w + v));
            }
        }
    }
}

__device__ __forceinline__ float activate(float x, int act) {
    if (act == SKYRL_ACT_SILU) return siluf_(x);
    return 0.5f * x * (1.f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
}

template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void gate_mul_kernel(const T* __restrict__ gu, int64_t n, int I, int act,
                                                       T* __restrict__ out) {
    const int iv = I / VEC;
    const int64_t total = n * iv;
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < total; e += (int64_t)gridDim.x * kNT) {
        const int64_t row = e / iv;
        const int c = (int)(e - row * iv) * VEC;
        const T* g = gu + row * 2 * I + c;
        if constexpr (VEC == 4) {
            const float4 a = ld4(g), b = ld4(g + I);
            st4(out + row * I + c, make_float4(activate(a.x, act) * b.x, activate(a.y, act) * b.y,
                                               activate(a.z, act) * b.z, activate(a.w, act) * b.w));
        } else {
            st(out + row * I + c, activate(ld(g), act) * ld(g + I));
        }
    }
}

template <typename T>
__global__ __launch_bounds__(kNT) void softcap_kernel(const T* __restrict__ x, float* __restrict__ out, int64_t n,
                                                      float cap) {
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < n; e += (int64_t)gridDim.x * kNT) {
        const float v = ld(x + e);
        out[e] = cap > 0.f ? cap * tanhf(v / cap) : v;
    }
}

unsigned grid_for(int64_t items) {
    const int64_t b = (items + kNT - 1) / kNT;
    return (unsigned)(b > 8192 ? 8192 : b);
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_NORM(V, K) \
    hipLaunchKernelGGL((add_norm_kernel<T, V, K>), dim3(n), dim3(kNT), 0, s, d, hidden, st_, w, H, eps, kind, o)

extern "C" int skyrl_add_norm(const void* delta, float* hidden, const void* step, const void* weight, int32_t n,
                              int32_t H, float eps, int32_t kind, void* out, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "add_norm");
    SKYRL_REQUIRE(n >= 0 && H > 0 && H <= 8192, "add_norm: H must be in [1, 8192]");
    SKYRL_REQUIRE(kind == SKYRL_NORM_LAYER || kind == SKYRL_NORM_RMS, "add_norm: unknown norm kind");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(hidden && weight && out, "add_norm: null pointer");
    hipStream_t s = as_stream(stream);
    SKYRL_DISPATCH_T(dtype, {
        const T* d = reinterpret_cast<const T*>(delta);
        const T* st_ = reinterpret_cast<const T*>(step);
        const T* w = reinterpret_cast<const T*>(weight);
        T* o = reinterpret_cast<T*>(out);
        if (H % 4 == 0) {
            if (H <= 4 * kNT) LAUNCH_NORM(4, 1);
            else if (H <= 8 * kNT) LAUNCH_NORM(4, 2);
            else if (H <= 16 * kNT) LAUNCH_NORM(4, 4);
            else LAUNCH_NORM(4, 8);
        } else {
            if (H <= 4 * kNT) LAUNCH_NORM(1, 4);
            else LAUNCH_NORM(1, 32);
        }
    })
    return check_launch("add_norm_kernel");
}

extern "C" int skyrl_gate_mul(const void* gate_up, int64_t n, int32_t I, int32_t act, void* out, int32_t dtype,
                              void* stream) {
    SKYRL_REQUIRE_T(dtype, "gate_mul");
    SKYRL_REQUIRE(n >= 0 && I > 0, "gate_mul: bad sizes");
    SKYRL_REQUIRE(act == SKYRL_ACT_SILU || act == SKYRL_ACT_GELU_TANH, "gate_mul: unknown activation");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(gate_up && out, "gate_mul: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const T* g = reinterpret_cast<const T*>(gate_up);
        T* o = reinterpret_cast<T*>(out);
        if (I % 4 == 0)
            hipLaunchKernelGGL((gate_mul_kernel<T, 4>), dim3(grid_for(n * (I / 4))), dim3(kNT), 0, as_stream(stream),
                               g, n, I, act, o);
        else
            hipLaunchKernelGGL((gate_mul_kernel<T, 1>), dim3(grid_for(n * I)), dim3(kNT), 0, as_stream(stream), g, n,
                               I, act, o);
    })
    return check_launch("gate_mul_kernel");
}

extern "C" int skyrl_softcap(const void* x, float* out, int64_t count, float cap, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "softcap");
    SKYRL_REQUIRE(count >= 0, "softcap: bad count");
    if (count == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && out, "softcap: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((softcap_kernel<T>), dim3(grid_for(count)), dim3(kNT), 0, as_stream(stream),
                           reinterpret_cast<const T*>(x), out, count, cap);
    })
    return check_launch("softcap_kernel");
}
