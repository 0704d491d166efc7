// Gated linear recurrence over channels (include/skyrl_layers.h has the equations and the tensor layouts).
//
// The two gates are block-diagonal products of the convolved input, so a workgroup takes one block's input
// tile, forms 16 columns of both gates per wave on the matrix instructions and finishes its channels in the
// accumulators: lane (c, g) holds channel c of rows 4 g .. 4 g + 3.
//
// Decode (rglru_step): the rows are 16 sequences' tokens. Convolution, gates, state update and output gate in
// one launch.
//
// Prompts (rglru_gates, rglru_chain, rglru_out): the rows are consecutive tokens of a chunk of 64, a workgroup
// walks a run of chunks. A state from the run's own tokens and the product of the decays up to each token give
// S_t = h_t + A_t S_in, so runs are independent but for one multiply-add per run and channel (rglru_chain).
// Within a chunk the pairs (A, h) compose along the accumulators: four tokens in a lane, four lane groups by
// shuffles, four tiles in order.
#include "conv.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kC = 64;     // tokens per chunk
constexpr int kSlab = 128; // input channels of a block in LDS at a time (prompts)
constexpr int kHeld = 4;   // 32-wide steps of the gate matrices held in registers

typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

struct Dims {
    int W, nb, bs, taps;
    __host__ __device__ int np() const { return (bs + 15) / 16 * 16; }  // padded outputs of a block
    __host__ __device__ int kp() const { return (bs + 31) / 32 * 32; }  // padded inputs
    __host__ __device__ int splits() const { return (np() + 63) / 64; } // workgroups of 64 columns per block
};

template <typename T>
struct Gates {
    const T* w;         // [nb, 2, np, kp]
    const float* bias;  // [2, W]
    const float* rate;  // [W]: log a = rate r
};

// A lane's part of 16 rows of a 32-wide operand, and acc += A B^T over it.
template <typename T>
struct Frag;
template <>
struct Frag<uint16_t> {
    s16x8 x;
    __device__ __forceinline__ void load(const uint16_t* row, int g) { x = *reinterpret_cast<const s16x8*>(row + 8 * g); }
};
template <>
struct Frag<float> {
    float4 x[2];
    __device__ __forceinline__ void load(const float* row, int g) {
        x[0] = ld4(row + 4 * g);
        x[1] = ld4(row + 16 + 4 * g);
    }
};
__device__ __forceinline__ f32x4 product32(const Frag<uint16_t>& a, const Frag<uint16_t>& b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.x, b.x, acc, 0, 0, 0);
}
__device__ __forceinline__ f32x4 product32(const Frag<float>& a, const Frag<float>& b, f32x4 acc) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x[s].x, b.x[s].x, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x[s].y, b.x[s].y, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x[s].z, b.x[s].z, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x[s].w, b.x[s].w, acc, 0, 0, 0);
    }
    return acc;
}

// VEC consecutive elements on their way to LDS.
template <typename T, int VEC>
struct Piece {
    static constexpr int kWords = VEC * sizeof(T) / 16;
    uint4 w[kWords];
    __device__ __forceinline__ void clear() {
#pragma unroll
        for (int i = 0; i < kWords; ++i) w[i] = make_uint4(0, 0, 0, 0);
    }
    __device__ __forceinline__ void load(const T* p) {
#pragma unroll
        for (int i = 0; i < kWords; ++i) w[i] = reinterpret_cast<const uint4*>(p)[i];
    }
    __device__ __forceinline__ void store(T* p) const {
#pragma unroll
        for (int i = 0; i < kWords; ++i) reinterpret_cast<uint4*>(p)[i] = w[i];
    }
};
template <typename T>
struct Piece<T, 1> {
    T w;
    __device__ __forceinline__ void clear() { w = 0; }
    __device__ __forceinline__ void load(const T* p) { w = *p; }
    __device__ __forceinline__ void store(T* p) const { *p = w; }
};

// Decay a and input b of S <- a S + b from the gates' sums: b = sqrt(1 - a^2) i u.
template <typename T>
__device__ __forceinline__ void recurrence_of(float zr, float zi, float u, float rate, float& a, float& b) {
    const float la = rate * sigmoid_<T>(zr), x = 2.f * la;
    a = exp_<T>(la);
    float one_minus;  // 1 - a^2, without cancellation where a is near 1
    if constexpr (sizeof(T) == 2) {
        const float series = -x * (1.f + x * (0.5f + x * (1.f / 6 + x * (1.f / 24 + x * (1.f / 120)))));
        one_minus = x > -0.2f ? series : fmaf(-a, a, 1.f);
        b = __builtin_amdgcn_sqrtf(one_minus) * sigmoid_<T>(zi) * u;
    } else {
        one_minus = -expm1f(x);
        b = sqrtf(one_minus) * sigmoid_<T>(zi) * u;
    }
}

// ---- decode: one token per sequence; grid (nb splits, ceil(n / 16)) ---------------------------------
template <typename T, int VEC>
__global__ __launch_bounds__(kNT) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 4 : 2))) void rglru_step_kernel(Dims d, const T* __restrict__ proj, int64_t stride,
                                                         const float* __restrict__ conv_t,
                                                         const float* __restrict__ conv_b, Gates<T> gt,
                                                         const int32_t* __restrict__ rows,
                                                         const int64_t* __restrict__ positions, int n,
                                                         float* __restrict__ state, T* __restrict__ ring_base,
                                                         T* __restrict__ out, int64_t out_stride) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* s_u = reinterpret_cast<T*>(smem);
    const int LD = d.kp() + 16 / (int)sizeof(T), ns = d.splits();
    const int blk = blockIdx.x / ns, split = blockIdx.x - blk * ns, q0 = 16 * blockIdx.y;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int o0 = 64 * split + 16 * wave, ks = d.kp() / 32;
    const bool on = o0 < d.np();
    const T* wr = gt.w + ((int64_t)blk * 2 * d.np() + (on ? o0 : 0) + c) * d.kp();
    const T* wi = wr + (int64_t)d.np() * d.kp();
    // what does not wait for the convolution: matrices, states, output gates
    Frag<T> fr[kHeld], fi[kHeld];
#pragma unroll
    for (int k = 0; k < kHeld; ++k) {
        if (k < ks) {
            fr[k].load(wr + 32 * k, g);
            fi[k].load(wi + 32 * k, g);
        }
    }
    const int ch_own = blk * d.bs + min(o0 + c, d.bs - 1);
    float old[4], yg[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int s = min(q0 + 4 * g + i, n - 1), row = rows[s];
        old[i] = row >= 0 && positions[s] > 0 ? state[(int64_t)row * d.W + ch_own] : 0.f;
        yg[i] = ld(proj + (int64_t)s * stride + ch_own);
    }
    const int pieces = d.kp() / VEC;
    for (int e = tid; e < 16 * pieces; e += kNT) {
        const int i = e / pieces, k = (e - i * pieces) * VEC, s = q0 + i;
        float y[VEC], x0[VEC];
#pragma unroll
        for (int v = 0; v < VEC; ++v) y[v] = 0.f;
        if (s < n && k < d.bs && rows[s] >= 0) {
            const int ch = blk * d.bs + k, pos = (int)positions[s];
            T* ring = ring_base + (int64_t)rows[s] * d.taps * d.W;
            conv_at<T, VEC>(proj + d.W, stride, conv_t, ring, d.W, d.taps, ch, s, s, pos, y, x0);
            float b[VEC];
            ldv<float, VEC>(conv_b + ch, b);
#pragma unroll
            for (int v = 0; v < VEC; ++v) y[v] += b[v];
            if (k / 64 == split) stv(ring + (int64_t)(pos % d.taps) * d.W + ch, x0);  // no convolution reads this slot now
        }
        stv(s_u + i * LD + k, y);
    }
    __syncthreads();
    if (!on) return;
    f32x4 ar = {0.f, 0.f, 0.f, 0.f}, ai = ar;
    Frag<T> fu;
#pragma unroll
    for (int k = 0; k < kHeld; ++k) {
        if (k < ks) {
            fu.load(s_u + c * LD + 32 * k, g);
            ar = product32(fu, fr[k], ar);
            ai = product32(fu, fi[k], ai);
        }
    }
    for (int k = kHeld; k < ks; ++k) {
        fu.load(s_u + c * LD + 32 * k, g);
        fr[0].load(wr + 32 * k, g);
        fi[0].load(wi + 32 * k, g);
        ar = product32(fu, fr[0], ar);
        ai = product32(fu, fi[0], ai);
    }
    if (o0 + c >= d.bs) return;
    const int ch = ch_own;
    const float br = gt.bias[ch], bi = gt.bias[d.W + ch], rate = gt.rate[ch];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int s = q0 + 4 * g + i;
        if (s >= n) break;
        const int row = rows[s];
        if (row < 0) continue;
        float a, b;
        recurrence_of<T>(ar[i] + br, ai[i] + bi, ld(s_u + (4 * g + i) * LD + o0 + c), rate, a, b);
        const float S = fmaf(a, old[i], b);
        state[(int64_t)row * d.W + ch] = S;
        st(out + (int64_t)s * out_stride + ch, S * gelu_tanh_<T>(yg[i]));
    }
}

// ---- prompts, step 1: gates and each run's own states; grid (nb splits, nruns) ----------------------
// FIT: a block's inputs are one slab, so that its matrices stay in registers and the next chunk's inputs are
// on their way while a chunk is finished.
template <typename T, int VEC, bool FIT>
__global__ __launch_bounds__(kNT) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 4 : 2))) void rglru_gates_kernel(Dims d, const T* __restrict__ u, Gates<T> gt,
                                                          const int32_t* __restrict__ chunk,
                                                          const int32_t* __restrict__ runs, float* __restrict__ hbuf,
                                                          float* __restrict__ abuf) {
    constexpr int LD = kSlab + 16 / (int)sizeof(T);
    constexpr int kPieces = FIT && VEC > 1 ? kC * kSlab / VEC / kNT : 1;  // of a thread, per chunk
    __shared__ __attribute__((aligned(16))) T s_u[kC * LD];
    const int ns = d.splits(), kp = d.kp();
    const int blk = blockIdx.x / ns, split = blockIdx.x - blk * ns;
    const int c0 = runs[4 * blockIdx.y], c1 = c0 + runs[4 * blockIdx.y + 1];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int o0 = 64 * split + 16 * wave;
    const bool on = o0 < d.np(), real = on && o0 + c < d.bs;
    const T* wr = gt.w + ((int64_t)blk * 2 * d.np() + (on ? o0 : 0) + c) * kp;
    const T* wi = wr + (int64_t)d.np() * kp;
    const T* ub = u + blk * d.bs;
    Frag<T> fr[kHeld], fi[kHeld];
    if constexpr (FIT) {
#pragma unroll
        for (int k = 0; k < kHeld; ++k) {
            if (32 * k < kp) {
                fr[k].load(wr + 32 * k, g);
                fi[k].load(wi + 32 * k, g);
            }
        }
    }
    const int och = real ? o0 + c : 0, ch = blk * d.bs + och;
    const float br = gt.bias[ch], bi = gt.bias[d.W + ch], rate = gt.rate[ch];
    float CA = 1.f, CB = 0.f;  // decay and state over the run so far

    // token e / pieces of a chunk, inputs k0 + VEC (e % pieces) .. of the block, zero past their ends
    auto fetch = [&](int t0, int n, int k0, int e, int pieces, Piece<T, VEC>& y) {
        const int i = e / pieces, k = (e - i * pieces) * VEC;
        y.clear();
        if (i < n && k0 + k < d.bs) y.load(ub + (int64_t)(t0 + i) * d.W + k0 + k);
    };
    auto place = [&](int e, int pieces, const Piece<T, VEC>& y) {
        const int i = e / pieces, k = (e - i * pieces) * VEC;
        y.store(s_u + i * LD + k);
    };
    Piece<T, VEC> held[kPieces];
    const int fitp = kp / VEC;
    if constexpr (kPieces > 1) {
#pragma unroll
        for (int j = 0; j < kPieces; ++j)
            if (tid + j * kNT < kC * fitp) fetch(chunk[4 * c0], chunk[4 * c0 + 1], 0, tid + j * kNT, fitp, held[j]);
    }
    for (int ci = c0; ci < c1; ++ci) {
        const int t0 = chunk[4 * ci], n = chunk[4 * ci + 1];
        f32x4 ar[4], ai[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) ar[t] = ai[t] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int k0 = 0; k0 < kp; k0 += kSlab) {
            const int w = min(kSlab, kp - k0), pieces = w / VEC;
            __syncthreads();
            if constexpr (kPieces > 1) {
#pragma unroll
                for (int j = 0; j < kPieces; ++j)
                    if (tid + j * kNT < kC * fitp) place(tid + j * kNT, fitp, held[j]);
            } else {
                for (int e = tid; e < kC * pieces; e += kNT) {
                    Piece<T, VEC> y;
                    fetch(t0, n, k0, e, pieces, y);
                    place(e, pieces, y);
                }
            }
            __syncthreads();
            if constexpr (kPieces > 1) {
                if (ci + 1 < c1) {
#pragma unroll
                    for (int j = 0; j < kPieces; ++j)
                        if (tid + j * kNT < kC * fitp)
                            fetch(chunk[4 * ci + 4], chunk[4 * ci + 5], 0, tid + j * kNT, fitp, held[j]);
                }
            }
            if (!on) continue;
#pragma unroll
            for (int k = 0; k < kSlab / 32; ++k) {
                if (32 * k >= w) break;
                if constexpr (!FIT) {
                    fr[0].load(wr + k0 + 32 * k, g);
                    fi[0].load(wi + k0 + 32 * k, g);
                }
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    Frag<T> fu;
                    fu.load(s_u + (16 * t + c) * LD + 32 * k, g);
                    ar[t] = product32(fu, fr[FIT ? k : 0], ar[t]);
                    ai[t] = product32(fu, fi[FIT ? k : 0], ai[t]);
                }
            }
        }
        if (!on) continue;
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if (16 * t >= n) break;
            float A[4], B[4];  // prefixes of this lane's four tokens
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int j = 16 * t + 4 * g + i;
                float x, a, b;
                if constexpr (FIT) x = ld(s_u + j * LD + och);
                else x = ld(ub + (int64_t)(t0 + min(j, n - 1)) * d.W + och);
                recurrence_of<T>(ar[t][i] + br, ai[t][i] + bi, x, rate, a, b);
                if (j >= n) {
                    a = 1.f;
                    b = 0.f;
                }
                A[i] = i ? a * A[i - 1] : a;
                B[i] = i ? fmaf(a, B[i - 1], b) : b;
            }
            float TA = A[3], TB = B[3];
#pragma unroll
            for (int o = 16; o <= 32; o <<= 1) {
                const float pa = __shfl_up(TA, o, kWave), pb = __shfl_up(TB, o, kWave);
                if (lane >= o) {
                    TB = fmaf(TA, pb, TB);
                    TA *= pa;
                }
            }
            float ea = __shfl_up(TA, 16, kWave), eb = __shfl_up(TB, 16, kWave);
            if (g == 0) {
                ea = 1.f;
                eb = 0.f;
            }
            const float PA = ea * CA, PB = fmaf(ea, CB, eb);
            const int64_t e = (int64_t)(t0 + 16 * t + 4 * g) * d.W + ch;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (16 * t + 4 * g + i < n && real) {
                    hbuf[e + i * d.W] = fmaf(A[i], PB, B[i]);
                    abuf[e + i * d.W] = A[i] * PA;
                }
            }
            const float la = __shfl(TA, 48 + c, kWave), lb = __shfl(TB, 48 + c, kWave);
            CB = fmaf(la, CB, lb);
            CA *= la;
        }
    }
}

// ---- step 2: the state before every run, and the sequence's last; grid (ceil(W / 64), nseq) ---------
__global__ __launch_bounds__(kWave) void rglru_chain_kernel(int W, const int32_t* __restrict__ chunk,
                                                            const int32_t* __restrict__ runs,
                                                            const int32_t* __restrict__ seq_runs,
                                                            const int32_t* __restrict__ cu,
                                                            const int32_t* __restrict__ rows,
                                                            const int64_t* __restrict__ positions, int seq0,
                                                            const float* __restrict__ hbuf,
                                                            const float* __restrict__ abuf, float* __restrict__ state,
                                                            float* __restrict__ s_in) {
    constexpr int kAhead = 32;
    const int lane = threadIdx.x, ch = blockIdx.x * kWave + lane, si = blockIdx.y, seq = seq0 + si, row = rows[seq];
    const int r0 = seq_runs[si], r1 = seq_runs[si + 1];
    if (row < 0 || r0 >= r1) return;
    const bool on = ch < W;
    const int col = on ? ch : 0;
    float* st_ = state + (int64_t)row * W + col;
    float S = positions[cu[seq]] > 0 ? *st_ : 0.f;
    for (int b0 = r0; b0 < r1; b0 += kAhead) {
        int last = 0;  // the last token of run b0 + lane
        if (lane < kAhead && b0 + lane < r1) {
            const int ci = runs[4 * (b0 + lane)] + runs[4 * (b0 + lane) + 1] - 1;
            last = chunk[4 * ci] + chunk[4 * ci + 1] - 1;
        }
        float a[kAhead], h[kAhead];
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            const int64_t e = (int64_t)__builtin_amdgcn_readlane(last, i) * W + col;
            a[i] = abuf[e];
            h[i] = hbuf[e];
        }
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            if (b0 + i < r1) {
                if (on) s_in[(int64_t)(b0 + i) * W + col] = S;
                S = fmaf(a[i], S, h[i]);
            }
        }
    }
    if (on) *st_ = S;
}

// ---- step 3: out = (h + A S_in) gelu(y); grid (ceil(W / (256 VEC)), nchunks, 4): 16 tokens each -----
template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void rglru_out_kernel(int W, const int32_t* __restrict__ chunk,
                                                        const float* __restrict__ hbuf,
                                                        const float* __restrict__ abuf,
                                                        const float* __restrict__ s_in, const T* __restrict__ proj,
                                                        int64_t stride, T* __restrict__ out, int64_t out_stride) {
    const int ch = (blockIdx.x * kNT + threadIdx.x) * VEC;
    const int t0 = chunk[4 * blockIdx.y], n = chunk[4 * blockIdx.y + 1], run = chunk[4 * blockIdx.y + 3];
    if (ch >= W) return;
    float S[VEC];
    ldv<float, VEC>(s_in + (int64_t)run * W + ch, S);
    const int j1 = min(n, 16 * (int)blockIdx.z + 16);
#pragma unroll 2
    for (int j = 16 * blockIdx.z; j < j1; ++j) {
        const int64_t t = t0 + j;
        float h[VEC], a[VEC], y[VEC];
        ldv<float, VEC>(hbuf + t * W + ch, h);
        ldv<float, VEC>(abuf + t * W + ch, a);
        ldv<T, VEC>(proj + t * stride + ch, y);
#pragma unroll
        for (int v = 0; v < VEC; ++v) h[v] = fmaf(a[v], S[v], h[v]) * gelu_tanh_<T>(y[v]);
        stv(out + t * out_stride + ch, h);
    }
}

const char* bad_dims(const Dims& d) {
    if (d.W <= 0 || d.nb <= 0 || d.bs * d.nb != d.W) return "rglru: width must be a multiple of blocks";
    if (d.taps <= 0 || d.taps > 64) return "rglru: taps must be in [1, 64]";
    return nullptr;
}
template <typename T>
size_t tile_bytes(int rows, int k) {
    return (size_t)rows * (k * sizeof(T) + 16);
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_STEP(VEC)                                                                                           \
    hipLaunchKernelGGL((rglru_step_kernel<T, VEC>), dim3(d.nb * d.splits(), (n + 15) / 16), dim3(kNT), lds,      \
                       as_stream(stream), d, reinterpret_cast<const T*>(proj), proj_stride, conv_t, conv_b, gt, rows, \
                       positions, n, state, reinterpret_cast<T*>(ring), reinterpret_cast<T*>(out), out_stride)

extern "C" int skyrl_rglru_step(const void* proj, int64_t proj_stride, int32_t width, int32_t blocks, int32_t taps,
                                const float* conv_t, const float* conv_b, const void* gate_w, const float* gate_b,
                                const float* rate, const int32_t* rows, const int64_t* positions, int32_t n,
                                float* state, void* ring, void* out, int64_t out_stride, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "rglru_step");
    const Dims d{width, blocks, blocks > 0 ? width / blocks : 0, taps};
    const char* bad = bad_dims(d);
    SKYRL_REQUIRE(!bad, bad);
    SKYRL_REQUIRE(n >= 0 && n <= 16 * 65535 && proj_stride >= 2 * (int64_t)width && out_stride >= width,
                  "rglru_step: bad sizes");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_t && conv_b && gate_w && gate_b && rate && rows && positions && state && ring && out,
                  "rglru_step: null pointer");
    SKYRL_REQUIRE(aligned16(conv_t) && aligned16(conv_b) && aligned16(gate_w) && aligned16(ring),
                  "rglru_step: 16-byte alignment");
    SKYRL_DISPATCH_T(dtype, {
        const Gates<T> gt{reinterpret_cast<const T*>(gate_w), gate_b, rate};
        const size_t lds = tile_bytes<T>(16, d.kp());
        SKYRL_REQUIRE(lds <= 65536, "rglru_step: a block's inputs do not fit (width / blocks too large)");
        if (d.bs % 8 == 0 && d.W % 8 == 0 && proj_stride % 8 == 0 && aligned16(proj)) LAUNCH_STEP(8);
        else LAUNCH_STEP(1);
    })
    return check_launch("rglru_step_kernel");
}

#define LAUNCH_GATES(VEC, FIT)                                                                                    \
    hipLaunchKernelGGL((rglru_gates_kernel<T, VEC, FIT>), grid, dim3(kNT), 0, s, d, u_, gt, chunk, runs, hbuf, abuf)

extern "C" int skyrl_rglru_prompt(const void* proj, int64_t proj_stride, int32_t width, int32_t blocks,
                                  const void* u, const void* gate_w, const float* gate_b, const float* rate,
                                  const int32_t* chunk, int32_t nchunks, const int32_t* runs, int32_t nruns,
                                  const int32_t* seq_runs, int32_t seq0, int32_t nseq, const int32_t* cu, const int32_t* rows, const int64_t* positions,
                                  float* state, float* hbuf, float* abuf, float* s_in, void* out, int64_t out_stride,
                                  int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "rglru_prompt");
    const Dims d{width, blocks, blocks > 0 ? width / blocks : 0, 1};
    const char* bad = bad_dims(d);
    SKYRL_REQUIRE(!bad, bad);
    SKYRL_REQUIRE(nchunks >= 0 && nchunks <= 65535 && nruns >= 0 && nruns <= nchunks && nseq >= 0 && nseq <= 65535 && seq0 >= 0 &&
                      proj_stride >= width && out_stride >= width,
                  "rglru_prompt: bad sizes");
    if (nchunks == 0 || nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && u && gate_w && gate_b && rate && chunk && runs && seq_runs && cu && rows && positions && state &&
                      hbuf && abuf && s_in && out,
                  "rglru_prompt: null pointer");
    SKYRL_REQUIRE(aligned16(u) && aligned16(gate_w) && aligned16(hbuf) && aligned16(abuf) && aligned16(s_in),
                  "rglru_prompt: 16-byte alignment");
    hipStream_t s = as_stream(stream);
    SKYRL_DISPATCH_T(dtype, {
        const Gates<T> gt{reinterpret_cast<const T*>(gate_w), gate_b, rate};
        const T* u_ = reinterpret_cast<const T*>(u);
        const T* p_ = reinterpret_cast<const T*>(proj);
        T* o_ = reinterpret_cast<T*>(out);
        const dim3 grid(d.nb * d.splits(), nruns);
        const bool fit = d.kp() <= kSlab;
        if (d.bs % 8 == 0 && fit) LAUNCH_GATES(8, true);
        else if (d.bs % 8 == 0) LAUNCH_GATES(8, false);
        else if (fit) LAUNCH_GATES(1, true);
        else LAUNCH_GATES(1, false);
        hipLaunchKernelGGL(rglru_chain_kernel, dim3((d.W + kWave - 1) / kWave, nseq), dim3(kWave), 0, s, d.W, chunk,
                           runs, seq_runs, cu, rows, positions, seq0, hbuf, abuf, state, s_in);
        if (d.W % 8 == 0 && proj_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(p_) && aligned16(o_))
            hipLaunchKernelGGL((rglru_out_kernel<T, 8>), dim3((d.W + 8 * kNT - 1) / (8 * kNT), nchunks, 4), dim3(kNT),
                               0, s, d.W, chunk, hbuf, abuf, s_in, p_, proj_stride, o_, out_stride);
        else
            hipLaunchKernelGGL((rglru_out_kernel<T, 1>), dim3((d.W + kNT - 1) / kNT, nchunks, 4), dim3(kNT), 0, s, d.W,
                               chunk, hbuf, abuf, s_in, p_, proj_stride, o_, out_stride);
    })
    return check_launch("rglru_prompt kernels");
}
