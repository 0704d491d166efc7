// Short causal convolutions of a prompt's tokens (include/skyrl_layers.h): bias and activation in the same
// pass, the results as rows of padded units, as transposed tiles of a chunk's tokens, or both.
//
// A thread takes VEC channels of eight consecutive tokens of a chunk, a wave eight such runs of eight pieces:
// inputs are read in 128-byte rows, and a channel's 64 tokens leave as one 128-byte line of the transposed tile.
#include "conv.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kC = 64;    // tokens per chunk
constexpr int kRun = 8;   // tokens per thread
constexpr int kMaxSections = 3;

template <typename T>
struct Section {
    int first, units, size, padded;  // channels [first, first + units size)
    T* rows;                         // [tokens, units, padded]
    T* cols;                         // [chunks, units, padded, 64]
};

template <typename T>
struct ConvArgs {
    const T* x;
    int64_t stride;
    int channels, taps, act, nsec;
    const float *conv_t, *bias;
    const int32_t *chunk, *cu, *rows;
    const int64_t* positions;
    const T* ring;
    Section<T> sec[kMaxSections];
};

// TW >= taps: the inputs of a run and the tokens before it stay in registers; TW 0: any number of taps.
template <typename T, int VEC, int TW>
__global__ __launch_bounds__(kNT) void conv_chunk_kernel(ConvArgs<T> p) {
    const int32_t* ck = p.chunk + 4 * blockIdx.y;
    const int t0 = ck[0], n = ck[1], seq = ck[2];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int ch = ((blockIdx.x * (kNT / kWave) + wave) * 8 + (lane >> 3)) * VEC, r0 = (lane & 7) * kRun;
    if (ch >= p.channels) return;
    const int sfirst = p.cu[seq];
    const int pos0 = (int)p.positions[sfirst] + (t0 - sfirst);  // of the chunk's first token
    const T* ring = p.ring + (int64_t)p.rows[seq] * p.taps * p.channels + ch;
    // input at chunk token i: from the step, from the stored inputs, or zero before the sequence's start
    auto input = [&](int i, float (&o)[VEC]) {
        if (pos0 + i < 0 || i >= n) {
#pragma unroll
            for (int v = 0; v < VEC; ++v) o[v] = 0.f;
        } else if (t0 + i >= sfirst) {
            ldv<T, VEC>(p.x + (int64_t)(t0 + i) * p.stride + ch, o);
        } else {
            ldv<T, VEC>(ring + (int64_t)((pos0 + i) % p.taps) * p.channels, o);
        }
    };
    // all inputs are the step's own: no case to tell apart
    const bool inner = n == kC && t0 - (p.taps - 1) >= sfirst;
    float y[kRun][VEC];
    float b[VEC];
#pragma unroll
    for (int v = 0; v < VEC; ++v) b[v] = 0.f;
    if (r0 >= n) {
#pragma unroll
        for (int j = 0; j < kRun; ++j)
#pragma unroll
            for (int v = 0; v < VEC; ++v) y[j][v] = 0.f;
    }
    if (p.bias) ldv<float, VEC>(p.bias + ch, b);
    if (r0 < n) {
        if constexpr (TW > 0) {
            float x[TW - 1 + kRun][VEC];
            if (inner) {
                const T* src = p.x + (int64_t)(t0 + r0 - (TW - 1)) * p.stride + ch;
#pragma unroll
                for (int k = 0; k < TW - 1 + kRun; ++k)
                    ldv<T, VEC>(src + max(k, TW - p.taps) * p.stride, x[k]);  // rows before the filter are not used
            } else {
#pragma unroll
                for (int k = 0; k < TW - 1 + kRun; ++k) {
                    if (k >= TW - p.taps) {
                        input(r0 + k - (TW - 1), x[k]);
                    } else {
#pragma unroll
                        for (int v = 0; v < VEC; ++v) x[k][v] = 0.f;
                    }
                }
            }
#pragma unroll
            for (int j = 0; j < kRun; ++j)
#pragma unroll
                for (int v = 0; v < VEC; ++v) y[j][v] = b[v];
#pragma unroll
            for (int k = 0; k < TW; ++k) {
                if (k < TW - p.taps) continue;
                float f[VEC];
                ldv<float, VEC>(p.conv_t + (int64_t)(k - (TW - p.taps)) * p.channels + ch, f);
#pragma unroll
                for (int j = 0; j < kRun; ++j)
#pragma unroll
                    for (int v = 0; v < VEC; ++v) y[j][v] += x[j + k][v] * f[v];
            }
        } else {
#pragma unroll
            for (int j = 0; j < kRun; ++j)
#pragma unroll
                for (int v = 0; v < VEC; ++v) y[j][v] = b[v];
            for (int k = 0; k < p.taps; ++k) {
                float f[VEC], x[VEC];
                ldv<float, VEC>(p.conv_t + (int64_t)k * p.channels + ch, f);
#pragma unroll
                for (int j = 0; j < kRun; ++j) {
                    input(r0 + j + k - (p.taps - 1), x);
#pragma unroll
                    for (int v = 0; v < VEC; ++v) y[j][v] += x[v] * f[v];
                }
            }
        }
    }
#pragma unroll
    for (int j = 0; j < kRun; ++j)
#pragma unroll
        for (int v = 0; v < VEC; ++v) {
            if (p.act == SKYRL_CONV_SILU) y[j][v] = y[j][v] * sigmoid_<T>(y[j][v]);
            if (r0 + j >= n) y[j][v] = 0.f;
        }
    int k = 0;
    while (k + 1 < p.nsec && ch >= p.sec[k + 1].first) ++k;
    const Section<T> s = p.sec[k];
    const int unit = (ch - s.first) / s.size, e = ch - s.first - unit * s.size, wide = s.units * s.padded;
    const int col = unit * s.padded + e;
    if (s.rows) {
#pragma unroll
        for (int j = 0; j < kRun; ++j)
            if (r0 + j < n) stv(s.rows + (int64_t)(t0 + r0 + j) * wide + col, y[j]);
    }
    if (s.cols) {
        T* dst = s.cols + ((int64_t)blockIdx.y * wide + col) * kC + r0;
#pragma unroll
        for (int v = 0; v < VEC; ++v) {
            float z[kRun];
#pragma unroll
            for (int j = 0; j < kRun; ++j) z[j] = y[j][v];
            st8(dst + v * kC, z);
        }
    }
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_CONV(VEC, TW)                                                                                      \
    hipLaunchKernelGGL((conv_chunk_kernel<T, VEC, TW>), dim3((channels + 32 * VEC - 1) / (32 * VEC), nchunks), \
                       dim3(kNT), 0, as_stream(stream), p)

extern "C" int skyrl_conv_chunk(const void* x, int64_t stride, int32_t channels, int32_t taps, const float* conv_t,
                                const float* bias, int32_t act, const int32_t* chunk, int32_t nchunks,
                                const int32_t* cu, const int32_t* rows, const int64_t* positions, const void* ring,
                                const skyrl_conv_section* sections, int32_t nsections, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "conv_chunk");
    SKYRL_REQUIRE(channels > 0 && taps > 0 && stride >= channels && nchunks >= 0 && nchunks <= 65535,
                  "conv_chunk: bad sizes");
    SKYRL_REQUIRE(act == SKYRL_CONV_NONE || act == SKYRL_CONV_SILU, "conv_chunk: unknown activation");
    SKYRL_REQUIRE(sections && nsections >= 1 && nsections <= kMaxSections, "conv_chunk: 1 to 3 sections");
    if (nchunks == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && conv_t && chunk && cu && rows && positions && ring, "conv_chunk: null pointer");
    SKYRL_REQUIRE(aligned16(conv_t) && aligned16(bias) && aligned16(ring), "conv_chunk: 16-byte alignment");
    SKYRL_DISPATCH_T(dtype, {
        ConvArgs<T> p{reinterpret_cast<const T*>(x), stride, channels, taps, act, nsections, conv_t, bias, chunk, cu,
                      rows, positions, reinterpret_cast<const T*>(ring), {}};
        bool wide = channels % 8 == 0 && stride % 8 == 0 && aligned16(x);
        int first = 0;
        for (int i = 0; i < nsections; ++i) {
            const skyrl_conv_section& s = sections[i];
            SKYRL_REQUIRE(s.units > 0 && s.size > 0 && s.padded >= s.size, "conv_chunk: bad section");
            SKYRL_REQUIRE(aligned16(s.rows) && aligned16(s.cols), "conv_chunk: 16-byte alignment");
            p.sec[i] = Section<T>{first, s.units, s.size, s.padded, reinterpret_cast<T*>(s.rows),
                                  reinterpret_cast<T*>(s.cols)};
            first += s.units * s.size;
            wide = wide && s.size % 8 == 0 && s.padded % 8 == 0;
        }
        SKYRL_REQUIRE(first == channels, "conv_chunk: the sections must cover the channels");
        if (wide) {
            if (taps <= 4) LAUNCH_CONV(8, 4);
            else if (taps <= 8) LAUNCH_CONV(8, 8);
            else LAUNCH_CONV(8, 0);
        } else {
            if (taps <= 4) LAUNCH_CONV(1, 4);
            else if (taps <= 8) LAUNCH_CONV(1, 8);
            else LAUNCH_CONV(1, 0);
        }
    })
    return check_launch("conv_chunk_kernel");
}
