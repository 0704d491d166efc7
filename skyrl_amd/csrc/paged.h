// Pieces of the attention kernels over paged keys and values (blocks of 16 tokens).
#pragma once
#include "elem.h"

namespace skyrl {

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kBS = 16;  // tokens per cache block

// Four consecutive outputs of a head from column e on.
__device__ __forceinline__ void store4(uint16_t* orow, int e, int V, bool vec, const float (&v)[4]) {
    if (vec && e + 4 <= V) {
        *reinterpret_cast<uint2*>(orow + e) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (e + i < V) orow[e + i] = f32_to_bf16(v[i]);
    }
}
__device__ __forceinline__ bool out_vec(const uint16_t* out, int64_t out_stride, int V) {
    return V % 4 == 0 && out_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & 7) == 0;
}

// A context of ctx tokens over at most nparts waves, each share a multiple of 16 and at least part_min tokens.
__device__ __forceinline__ void ctx_split(int ctx, int part_min, int nparts, int& part, int& np) {
    const int p = ((ctx + nparts - 1) / nparts + kBS - 1) / kBS * kBS;
    part = max(p, part_min);
    np = (ctx + part - 1) / part;
}

}  // namespace skyrl
