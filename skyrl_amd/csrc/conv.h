// Short causal convolutions over time (one filter per channel, the last tap on the current token) for
// kernels templated on the activation type. A sequence's last `taps` inputs are kept in a ring
// T [taps, channels] of its state row, the input of position p at p % taps: the slot that a one-token
// step writes is none that it reads.
#pragma once
#include "elem.h"

namespace skyrl {

constexpr int kConvWindow = 8;  // taps whose loads are all in flight at once

// Convolution of channel ch at token t (position pos, r = pos % taps) of a sequence whose first token in
// this step is t0; inputs before t0 come from the ring, before position 0 they are zero. w T [channels, taps].
template <typename T>
__device__ __forceinline__ float short_conv(const T* __restrict__ proj, int64_t stride, const T* __restrict__ w,
                                            const T* __restrict__ ring, int channels, int taps, int ch, int t, int t0,
                                            int pos, int r) {
    float y = 0.f;
    auto input = [&](int back) -> float {
        if (t - back >= t0) return ld(proj + (int64_t)(t - back) * stride + ch);
        const int slot = r - back < 0 ? r - back + taps : r - back;
        return ld(ring + (int64_t)slot * channels + ch);
    };
    if (taps <= kConvWindow) {
        float x[kConvWindow], f[kConvWindow];
#pragma unroll
        for (int back = 0; back < kConvWindow; ++back) {
            const bool on = back < taps && back <= pos;
            x[back] = on ? input(back) : 0.f;
            f[back] = on ? ld(w + (int64_t)ch * taps + taps - 1 - back) : 0.f;
        }
#pragma unroll
        for (int back = 0; back < kConvWindow; ++back) y += x[back] * f[back];
    } else {
        for (int back = 0; back < taps && back <= pos; ++back)
            y += input(back) * ld(w + (int64_t)ch * taps + taps - 1 - back);
    }
    return y;
}

// The same of VEC channels with the filters transposed, conv_t f32 [taps, channels]; x0: the token's own inputs.
template <typename T, int VEC>
__device__ __forceinline__ void conv_at(const T* __restrict__ proj, int64_t stride, const float* __restrict__ conv_t,
                                        const T* __restrict__ ring, int channels, int taps, int ch, int t, int t0,
                                        int pos, float (&y)[VEC], float (&x0)[VEC]) {
    constexpr int W = 4;
    const int r = pos % taps;
    auto input = [&](int back, float (&x)[VEC]) {
        if (t - back >= t0) {
            ldv<T, VEC>(proj + (int64_t)(t - back) * stride + ch, x);
        } else {
            const int slot = r - back < 0 ? r - back + taps : r - back;
            ldv<T, VEC>(ring + (int64_t)slot * channels + ch, x);
        }
    };
#pragma unroll
    for (int i = 0; i < VEC; ++i) y[i] = 0.f;
    if (taps <= W) {
        float x[W][VEC], f[W][VEC];
#pragma unroll
        for (int back = 0; back < W; ++back) {
            if (back < taps && back <= pos) {
                input(back, x[back]);
                ldv<float, VEC>(conv_t + (int64_t)(taps - 1 - back) * channels + ch, f[back]);
            } else {
#pragma unroll
                for (int i = 0; i < VEC; ++i) x[back][i] = f[back][i] = 0.f;
            }
        }
#pragma unroll
        for (int back = 0; back < W; ++back)
#pragma unroll
            for (int i = 0; i < VEC; ++i) y[i] += x[back][i] * f[back][i];
#pragma unroll
        for (int i = 0; i < VEC; ++i) x0[i] = x[0][i];
    } else {
        input(0, x0);
        for (int back = 0; back < taps && back <= pos; ++back) {
            float x[VEC], f[VEC];
            input(back, x);
            ldv<float, VEC>(conv_t + (int64_t)(taps - 1 - back) * channels + ch, f);
#pragma unroll
            for (int i = 0; i < VEC; ++i) y[i] += x[i] * f[i];
        }
    }
}

}  // namespace skyrl
