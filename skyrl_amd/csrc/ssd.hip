// State space mixer with a scalar decay per head and token (include/skyrl_layers.h has the equations and the
// tensor layouts).
//
// Token form (ssd_scan): one workgroup per (sequence, head), the state in registers over the sequence's tokens:
// convolution, step size, decay, update and read-out in one launch. A decode step reads and writes the state once.
//
// Prompt form: the convolutions run once for all heads (skyrl_conv_chunk: x and B also transposed), so do the
// products C B^T of every chunk and group (ssd_scores). ssd_walk takes one (run of chunks, head, 64 value columns) per workgroup and walks the chunks of 64 tokens with
// the state in registers:
//   Y = (L o C B^T) X + diag(e^G) C S,   S <- e^{G_n} S + B^T diag(e^{G_n - G} dt) X,
// G the summed log decays, L_ij = e^{G_i - G_j} dt_j (j <= i), the skip D on L's diagonal. Long sequences are cut
// into several runs of chunks: a first walk forms each run's own last state, ssd_chain carries them from run to
// run, and the second walk starts every run from the state before it.
//
// x, B and C are bf16; state, decays and L are f32. A product of an f32 matrix with a bf16 one runs on the bf16
// matrix instructions, the f32 operand split exactly into three bf16 terms (8 + 8 + 8 bits of its significand),
// about a fifth of the time of the f32 instructions. Accumulators hold rows 4 g + i of a 16 x 16 tile, which is the
// operand layout of the next product over those rows, so neither L nor S needs a transposition.
#include "conv.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kC = 64;  // tokens per chunk

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

struct Dims {
    int H, P, N, G, taps;
    __host__ __device__ int inner() const { return H * P; }
    __host__ __device__ int channels() const { return H * P + 2 * G * N; }
    __host__ __device__ int ppad() const { return (P + 3) / 4 * 4; }
    __host__ __device__ int vp() const { return (P + 15) / 16 * 16; }
    __host__ __device__ int np() const { return (N + 31) / 32 * 32; }
    __host__ __device__ int group(int h) const { return h / (H / G); }
};

// ---- token form: thread (cg, rg) holds columns 4 cg .. 4 cg + 3 of state rows rg, rg + RG, ... -------
template <typename T, int NT, int RPT>
__global__ __launch_bounds__(NT) __attribute__((amdgpu_waves_per_eu(4))) void ssd_scan_kernel(
    Dims d, const T* __restrict__ proj, int64_t stride, const float* __restrict__ conv_t,
    const float* __restrict__ conv_b, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    const float* __restrict__ skip, const int32_t* __restrict__ cu, const int32_t* __restrict__ rows,
    const int64_t* __restrict__ positions, float* __restrict__ state, T* __restrict__ ring_base, int save_conv,
    T* __restrict__ y, int64_t y_stride) {
    extern __shared__ float smem[];
    const int h = blockIdx.x, s = blockIdx.y, row = rows[s];
    if (row < 0) return;
    const int t0 = cu[s], t1 = cu[s + 1];
    if (t0 >= t1) return;
    const int N = d.N, P = d.P, VP = d.ppad(), NC = VP / 4, RG = NT / NC, n_all = d.channels();
    float* s_b = smem;         // N
    float* s_c = s_b + N;      // N
    float* s_x = s_c + N;      // VP (N may be odd: not read as vectors)
    float* s_red = smem + (2 * N + VP + 3) / 4 * 4;  // RG * VP
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cg = tid % NC, rg = tid / NC;
    const bool act = rg < RG;
    const bool fold = NC <= kWave && (NC & (NC - 1)) == 0;  // a wave holds whole row groups
    const int nrec = fold ? NT / kWave : RG;
    const int64_t pos0 = positions[t0];
    T* ring = ring_base + (int64_t)row * d.taps * n_all;
    float* st_ = state + ((int64_t)row * d.H + h) * N * VP;
    float S[RPT][4];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (act && r < N && pos0 > 0) v = ld4(st_ + (int64_t)r * VP + 4 * cg);
        S[i][0] = v.x; S[i][1] = v.y; S[i][2] = v.z; S[i][3] = v.w;
    }
    const float rate = -expf(a_log[h]), dtb = dt_bias[h], D = skip[h];
    const int boff = d.inner() + d.group(h) * N, coff = boff + d.G * N;
    const T* xbc = proj + d.inner();  // z comes first
    for (int t = t0; t < t1; ++t) {
        const int pos = (int)pos0 + (t - t0);
        const float raw = ld(xbc + (int64_t)t * stride + n_all + h);
        for (int e = tid; e < 2 * N + VP; e += NT) {
            float v = 0.f;
            if (e < 2 * N + P) {
                const int ch = e < N ? boff + e : e < 2 * N ? coff + e - N : h * P + e - 2 * N;
                float c[1], x0[1];
                conv_at<T, 1>(xbc, stride, conv_t, ring, n_all, d.taps, ch, t, t0, pos, c, x0);
                v = siluf_(c[0] + conv_b[ch]);
                // one token: no convolution reads the slot written here
                if (save_conv && (e >= 2 * N || h % (d.H / d.G) == 0))
                    st(ring + (int64_t)(pos % d.taps) * n_all + ch, x0[0]);
            }
            smem[e] = v;
        }
        __syncthreads();
        const float dt = softplusf_(raw + dtb), decay = expf(rate * dt);
        const float x[4] = {s_x[4 * cg], s_x[4 * cg + 1], s_x[4 * cg + 2], s_x[4 * cg + 3]};
        float o[4] = {0.f, 0.f, 0.f, 0.f};
        if (act) {
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const int r = rg + i * RG;
                if (r < N) {
                    const float b = dt * s_b[r], c = s_c[r];
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        S[i][j] = decay * S[i][j] + b * x[j];
                        o[j] += S[i][j] * c;
                    }
                }
            }
            if (fold)
                for (int k = NC; k < kWave; k <<= 1)
#pragma unroll
                    for (int j = 0; j < 4; ++j) o[j] += __shfl_xor(o[j], k, kWave);
            if (!fold || lane < NC)
                st4(s_red + (fold ? wave : rg) * VP + 4 * cg, make_float4(o[0], o[1], o[2], o[3]));
        }
        __syncthreads();
        if (tid < VP && tid < P) {
            float v = D * s_x[tid];
            for (int r = 0; r < nrec; ++r) v += s_red[r * VP + tid];
            st(y + (int64_t)t * y_stride + h * P + tid, v);
        }
        for (int e = tid + NT; e < P; e += NT) {
            float v = D * s_x[e];
            for (int r = 0; r < nrec; ++r) v += s_red[r * VP + e];
            st(y + (int64_t)t * y_stride + h * P + e, v);
        }
        if (t + 1 < t1) __syncthreads();  // s_x is rewritten
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        if (act && r < N) st4(st_ + (int64_t)r * VP + 4 * cg, make_float4(S[i][0], S[i][1], S[i][2], S[i][3]));
    }
}

// ---- prompt form ----------------------------------------------------------------------------------
struct SeqRef {
    const int32_t* chunk;  // [nchunks, 4]: first token, tokens, sequence, 0
    const int32_t* super;  // [nsuper, 4]: first chunk, chunks, sequence, kind (kMany, kLast)
    const int32_t* cu;
    const int32_t* rows;
    const int64_t* positions;
};
constexpr int kMany = 1;  // the sequence has several runs of chunks: the state before this one is in the buffer
constexpr int kLast = 2;  // its last: leaves the sequence's state

struct Split {
    s16x8 hi, mid, lo;
};
// Eight f32 values as the sums of three bf16 values each (truncated, so that the remainders are exact).
__device__ __forceinline__ Split split3(const float (&x)[8]) {
    uint32_t h[4], m[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        uint32_t a[2], b[2], c[2];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const float v = x[2 * i + k];
            a[k] = __float_as_uint(v) & 0xffff0000u;
            const float r = v - __uint_as_float(a[k]);
            b[k] = __float_as_uint(r) & 0xffff0000u;
            c[k] = __float_as_uint(r - __uint_as_float(b[k]));
        }
        h[i] = __builtin_amdgcn_perm(a[1], a[0], 0x07060302u);  // the upper halves of both
        m[i] = __builtin_amdgcn_perm(b[1], b[0], 0x07060302u);
        l[i] = __builtin_amdgcn_perm(c[1], c[0], 0x07060302u);
    }
    return Split{__builtin_bit_cast(s16x8, make_uint4(h[0], h[1], h[2], h[3])),
                 __builtin_bit_cast(s16x8, make_uint4(m[0], m[1], m[2], m[3])),
                 __builtin_bit_cast(s16x8, make_uint4(l[0], l[1], l[2], l[3]))};
}
__device__ __forceinline__ f32x4 mma(const s16x8& a, const s16x8& b, const f32x4& acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma3(const Split& a, const s16x8& b, f32x4 acc) {
    return mma(a.hi, b, mma(a.mid, b, mma(a.lo, b, acc)));
}
__device__ __forceinline__ f32x4 mma3(const s16x8& a, const Split& b, f32x4 acc) {
    return mma(a, b.hi, mma(a, b.mid, mma(a, b.lo, acc)));
}
__device__ __forceinline__ void put16(uint16_t* p, uint4 v) {  // 16 bytes to an address on 8
    *reinterpret_cast<uint2*>(p) = make_uint2(v.x, v.y);
    *reinterpret_cast<uint2*>(p + 4) = make_uint2(v.z, v.w);
}
// Elements 4 g .. 4 g + 3 of both 16-wide halves of a 32-wide step: the accumulators' order of rows.
__device__ __forceinline__ s16x8 halves(const uint16_t* p) {
    const s16x4 a = *reinterpret_cast<const s16x4*>(p), b = *reinterpret_cast<const s16x4*>(p + 16);
    return s16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// C B^T of a chunk and group, transposed (keys in the rows): 16 x 16 tiles at and below the diagonal as the walk's
// accumulators, query tile w's first at w (w + 1) / 2. grid nchunks G.
constexpr int kTiles = 10;
constexpr int kLTerm = 6 * kWave * 8;  // L^T in LDS: 32-key steps 0 .. qt / 2 of each query tile qt
__device__ __forceinline__ int l_step(int qt, int kk) { return (qt < 2 ? qt : 2 * qt - 2 + kk) * kWave * 8; }
__global__ __launch_bounds__(kNT) void ssd_scores_kernel(int G, int np, const int32_t* __restrict__ chunk,
                                                         const uint16_t* __restrict__ brow,
                                                         const uint16_t* __restrict__ crow, float* __restrict__ scores) {
    const int ci = blockIdx.x / G, gi = blockIdx.x - ci * G;
    const int t0 = chunk[4 * ci], n = chunk[4 * ci + 1];
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int64_t bw = (int64_t)G * np;
    const uint16_t* cr = crow + (t0 + min(16 * wave + c, n - 1)) * bw + gi * np + 8 * g;
    f32x4 acc[4];
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) acc[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < np; k += 32) {
        const s16x8 q = *reinterpret_cast<const s16x8*>(cr + k);
#pragma unroll
        for (int tt = 0; tt < 4; ++tt)
            if (tt <= wave)
                acc[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    *reinterpret_cast<const s16x8*>(brow + (t0 + min(16 * tt + c, n - 1)) * bw + gi * np + 8 * g + k), q,
                    acc[tt], 0, 0, 0);
    }
    float* dst = scores + ((int64_t)blockIdx.x * kTiles + wave * (wave + 1) / 2) * 256 + 4 * lane;
#pragma unroll
    for (int tt = 0; tt < 4; ++tt)
        if (tt <= wave) *reinterpret_cast<f32x4*>(dst + tt * 256) = acc[tt];
}

// NS: 32-wide steps of the padded state dimension at least. OUT: the second walk; otherwise the first, over the
// runs that `pick` lists.
template <int NS, bool OUT>
__global__ __launch_bounds__(kNT) __attribute__((amdgpu_waves_per_eu(NS <= 4 ? 3 : 1))) void ssd_walk_kernel(
    Dims d, SeqRef sq, const int32_t* __restrict__ pick, int slices, const uint16_t* __restrict__ xt,
    const uint16_t* __restrict__ bt, const float* __restrict__ scores, const uint16_t* __restrict__ crow,
    const uint16_t* __restrict__ dt_raw, int64_t dt_stride, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const float* __restrict__ skip, float* __restrict__ state,
    float* __restrict__ runs, float* __restrict__ gtot, uint16_t* __restrict__ y, int64_t y_stride) {
    constexpr int LDC = NS * 32 + 4, LDB = kC + 4;  // rows on 8 bytes
    __shared__ __attribute__((aligned(16))) uint16_t s_c[OUT ? kC * LDC : 8];
    __shared__ __attribute__((aligned(16))) uint16_t s_bt[NS * 32 * LDB];
    __shared__ __attribute__((aligned(16))) uint16_t s_l[OUT ? 3 * kLTerm : 8];  // L^T: term, (query tile, step)
    __shared__ __attribute__((aligned(16))) float s_g[kC], s_d[kC], s_w[kC];
    const int slice = blockIdx.x % slices, hs = blockIdx.x / slices, h = hs % d.H;
    const int ri = OUT ? hs / d.H : pick[hs / d.H];
    const int32_t* sp = sq.super + 4 * ri;
    const int c0 = sp[0], nchunk = sp[1], seq = sp[2], kind = sp[3];
    const int row = sq.rows[seq];
    if (row < 0) return;
    const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int np = d.np(), vp = d.vp(), VP = d.ppad(), ns = np / 32, gi = d.group(h), bw = d.G * np;
    const int pt = slice * 4 + wave;  // this wave's 16 value columns
    const bool on = 16 * pt < vp;
    const int pcol = 16 * pt + c;
    float* st_ = state + ((int64_t)row * d.H + h) * d.N * VP;
    float* rbuf = runs + ((int64_t)ri * d.H + h) * np * vp;

    f32x4 S[NS][2];  // rows 32 s + 16 k + 4 g + i, column pcol
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = 32 * s + 16 * k + 4 * g + i;
                float v = 0.f;
                if (OUT && on && s < ns) {
                    if (kind & kMany) v = rbuf[(int64_t)n * vp + pcol];
                    else if (n < d.N && pcol < VP && sq.positions[sq.cu[seq]] > 0) v = st_[(int64_t)n * VP + pcol];
                }
                S[s][k][i] = v;
            }
    const float rate = -expf(a_log[h]), dtb = dt_bias[h], D = OUT ? skip[h] : 0.f;
    float gsum = 0.f;
    for (int k = 0; k < nchunk; ++k) {
        const int ci = c0 + k, t0 = sq.chunk[4 * ci], n = sq.chunk[4 * ci + 1];
        __syncthreads();  // the previous chunk's tiles are consumed
        if constexpr (OUT) {
            const int pieces = np / 8;
            for (int e = tid; e < kC * pieces; e += kNT) {
                const int i = e / pieces, x = (e - i * pieces) * 8;
                put16(&s_c[i * LDC + x],
                      *reinterpret_cast<const uint4*>(crow + (int64_t)(t0 + min(i, n - 1)) * bw + gi * np + x));
            }
        }
        for (int e = tid; e < np * 8; e += kNT)
            put16(&s_bt[(e >> 3) * LDB + (e & 7) * 8],
                  *reinterpret_cast<const uint4*>(bt + ((int64_t)ci * bw + gi * np) * kC + e * 8));
        f32x4 sc[4];
        if constexpr (OUT) {
            const float* src = scores + (((int64_t)ci * d.G + gi) * kTiles + wave * (wave + 1) / 2) * 256 + 4 * lane;
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)
                if (tt <= wave) sc[tt] = *reinterpret_cast<const f32x4*>(src + tt * 256);
        }
        s16x8 xf[2];
#pragma unroll
        for (int kk = 0; kk < 2; ++kk)
            xf[kk] = on ? halves(xt + ((int64_t)ci * d.H * vp + h * vp + pcol) * kC + 32 * kk + 4 * g)
                        : s16x8{0, 0, 0, 0, 0, 0, 0, 0};
        // a lane per token, in every wave: step size, summed log decays; no decay and no input past the end
        const float raw = ld(dt_raw + (int64_t)(t0 + min(lane, n - 1)) * dt_stride + h);
        const float dt = lane < n ? softplusf_(raw + dtb) : 0.f;
        float G = rate * dt;
#pragma unroll
        for (int o = 1; o < kWave; o <<= 1) {
            const float v = __shfl_up(G, o, kWave);
            if (lane >= o) G += v;
        }
        const float gl = __shfl(G, kWave - 1, kWave);
        if (wave == 0) {
            s_g[lane] = G;
            s_d[lane] = dt;
            s_w[lane] = expf(gl - G) * dt;
        }
        __syncthreads();
        f32x4 o[4];
        if constexpr (OUT) {
            // L^T of this wave's 16 queries: keys in the rows
            const int q = 16 * wave + c;
            const float gq = s_g[q];
            float w[2][8];
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) {
                float* dst = &w[tt >> 1][4 * (tt & 1)];
                if (tt <= wave) {
                    const int j0 = 16 * tt + 4 * g;
                    const float4 gk = ld4(&s_g[j0]), dk = ld4(&s_d[j0]);
                    const float gv[4] = {gk.x, gk.y, gk.z, gk.w}, dv[4] = {dk.x, dk.y, dk.z, dk.w};
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const float l = j0 + i <= q ? sc[tt][i] * fast_exp2((gq - gv[i]) * kLog2e) * dv[i] : 0.f;
                        dst[i] = j0 + i == q ? l + D : l;
                    }
                } else {
#pragma unroll
                    for (int i = 0; i < 4; ++i) dst[i] = 0.f;
                }
            }
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                if (kk > wave / 2) break;
                const Split f = split3(w[kk]);
                uint16_t* p = &s_l[l_step(wave, kk) + lane * 8];
                *reinterpret_cast<s16x8*>(p) = f.hi;
                *reinterpret_cast<s16x8*>(p + kLTerm) = f.mid;
                *reinterpret_cast<s16x8*>(p + 2 * kLTerm) = f.lo;
            }
            // what the state before the chunk gives: (C S)^T
#pragma unroll
            for (int qt = 0; qt < 4; ++qt) o[qt] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (on) {
#pragma unroll
                for (int s = 0; s < NS; ++s) {
                    if (s < ns) {
                        float v[8];
#pragma unroll
                        for (int i = 0; i < 8; ++i) v[i] = S[s][i >> 2][i & 3];
                        const Split f = split3(v);
#pragma unroll
                        for (int qt = 0; qt < 4; ++qt) o[qt] = mma3(f, halves(&s_c[(16 * qt + c) * LDC + 32 * s + 4 * g]), o[qt]);
                    }
                }
#pragma unroll
                for (int qt = 0; qt < 4; ++qt) o[qt] = o[qt] * fast_exp2(s_g[16 * qt + c] * kLog2e);
            }
            __syncthreads();  // L^T of all queries is there
            if (on) {
#pragma unroll
                for (int qt = 0; qt < 4; ++qt) {
#pragma unroll
                    for (int kk = 0; kk <= qt / 2; ++kk) {
                        const uint16_t* p = &s_l[l_step(qt, kk) + lane * 8];
                        const Split f{*reinterpret_cast<const s16x8*>(p), *reinterpret_cast<const s16x8*>(p + kLTerm),
                                      *reinterpret_cast<const s16x8*>(p + 2 * kLTerm)};
                        o[qt] = mma3(xf[kk], f, o[qt]);
                    }
                    const int tq = 16 * qt + c, p0 = 16 * pt + 4 * g;
                    if (tq < n) {
                        uint16_t* dst = y + (int64_t)(t0 + tq) * y_stride + h * d.P + p0;
                        if (d.P % 4 == 0) {
                            if (p0 < d.P) st4(dst, make_float4(o[qt][0], o[qt][1], o[qt][2], o[qt][3]));
                        } else {
#pragma unroll
                            for (int i = 0; i < 4; ++i)
                                if (p0 + i < d.P) st(dst + i, o[qt][i]);
                        }
                    }
                }
            }
        }
        gsum += gl;
        if (!on) continue;
        const float decay = fast_exp2(gl * kLog2e);
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            S[s][0] = S[s][0] * decay;
            S[s][1] = S[s][1] * decay;
        }
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            if (32 * kk >= n) break;
            const float4 w0 = ld4(&s_w[32 * kk + 4 * g]), w1 = ld4(&s_w[32 * kk + 16 + 4 * g]);
            const float wv[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
            float v[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = bf16_to_f32((uint16_t)xf[kk][i]) * wv[i];
            const Split f = split3(v);
#pragma unroll
            for (int s = 0; s < NS; ++s) {
                if (s < ns) {
#pragma unroll
                    for (int e = 0; e < 2; ++e)
                        S[s][e] = mma3(halves(&s_bt[(32 * s + 16 * e + c) * LDB + 32 * kk + 4 * g]), f, S[s][e]);
                }
            }
        }
    }
    if (!OUT && slice == 0 && tid == 0) gtot[(int64_t)ri * d.H + h] = gsum;
    if (!on || (OUT && !(kind & kLast))) return;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
        if (s < ns) {
#pragma unroll
            for (int k = 0; k < 2; ++k)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int n = 32 * s + 16 * k + 4 * g + i;
                    if constexpr (OUT) {
                        if (n < d.N && pcol < VP) st_[(int64_t)n * VP + pcol] = S[s][k][i];
                    } else {
                        rbuf[(int64_t)n * vp + pcol] = S[s][k][i];
                    }
                }
        }
    }
}

// The state before every run of chunks of sequences that have several: chain i32 [n, 2] (first run, runs).
// grid (ceil(H np vp / 256), n).
__global__ __launch_bounds__(kNT) void ssd_chain_kernel(Dims d, SeqRef sq, const int32_t* __restrict__ chain,
                                                        const float* __restrict__ state,
                                                        const float* __restrict__ gtot, float* __restrict__ runs) {
    constexpr int kAhead = 4;
    const int np = d.np(), vp = d.vp(), VP = d.ppad();
    const int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x, size = (int64_t)d.H * np * vp;
    if (e >= size) return;
    const int h = (int)(e / (np * vp)), n = (int)(e / vp) % np, p = (int)(e % vp);
    const int r0 = chain[2 * blockIdx.y], cnt = chain[2 * blockIdx.y + 1];
    const int seq = sq.super[4 * r0 + 2], row = sq.rows[seq];
    float S = 0.f;
    if (row >= 0 && n < d.N && p < VP && sq.positions[sq.cu[seq]] > 0)
        S = state[(((int64_t)row * d.H + h) * d.N + n) * VP + p];
    for (int b = 0; b < cnt; b += kAhead) {
        float own[kAhead], gt[kAhead];
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            const int r = r0 + min(b + i, cnt - 1);
            own[i] = b + i + 1 < cnt ? runs[r * size + e] : 0.f;  // the last run's own state is not formed
            gt[i] = b + i + 1 < cnt ? gtot[(int64_t)r * d.H + h] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            if (b + i < cnt) {
                runs[(r0 + b + i) * size + e] = S;
                S = fmaf(expf(gt[i]), S, own[i]);
            }
        }
    }
}

const char* bad_shape(const skyrl_ssd_shape* sh) {
    if (!sh) return "ssd: null shape";
    if (sh->heads <= 0 || sh->groups <= 0 || sh->heads % sh->groups) return "ssd: heads must be a multiple of groups";
    if (sh->vdim <= 0 || sh->state <= 0 || sh->vdim > 1024 || sh->state > 1024) return "ssd: vdim and state must be in [1, 1024]";
    if (sh->taps <= 0 || sh->taps > 64) return "ssd: taps must be in [1, 64]";
    return nullptr;
}
Dims dims_of(const skyrl_ssd_shape* s) { return Dims{s->heads, s->vdim, s->state, s->groups, s->taps}; }
int rows_per_thread(const Dims& d, int nt) {
    const int RG = nt / (d.ppad() / 4);
    return (d.N + RG - 1) / RG;
}
int64_t proj_width(const Dims& d) { return d.inner() + d.channels() + (int64_t)d.H; }

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_SCAN(NT, R)                                                                                          \
    hipLaunchKernelGGL((ssd_scan_kernel<T, NT, R>), dim3(d.H, nseq), dim3(NT), lds, as_stream(stream), d,         \
                       reinterpret_cast<const T*>(proj), proj_stride, conv_t, conv_b, a_log, dt_bias, skip, cu, rows, \
                       positions, state, reinterpret_cast<T*>(ring), save_conv, reinterpret_cast<T*>(y), y_stride)

extern "C" int skyrl_ssd_scan(const skyrl_ssd_shape* shape, const void* proj, int64_t proj_stride, const float* conv_t,
                              const float* conv_b, const float* a_log, const float* dt_bias, const float* skip,
                              const int32_t* cu, const int32_t* rows, const int64_t* positions, int32_t nseq,
                              float* state, void* ring, int32_t save_conv, void* y, int64_t y_stride, int32_t dtype,
                              void* stream) {
    SKYRL_REQUIRE_T(dtype, "ssd_scan");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nseq >= 0 && nseq <= 65535 && proj_stride >= proj_width(d) && y_stride >= d.inner(),
                  "ssd_scan: bad sizes");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_t && conv_b && a_log && dt_bias && skip && cu && rows && positions && state && ring && y,
                  "ssd_scan: null pointer");
    SKYRL_REQUIRE(aligned16(state), "ssd_scan: 16-byte alignment");
    const int nt = rows_per_thread(d, 256) <= 8 ? 256 : rows_per_thread(d, 512) <= 8 ? 512 : 1024;
    const int rpt = rows_per_thread(d, nt), RG = nt / (d.ppad() / 4);
    SKYRL_REQUIRE(rpt <= 16, "ssd_scan: state * vdim too large for one workgroup's registers (at most 65536)");
    const size_t lds = ((size_t)(2 * d.N + d.ppad() + 3) / 4 * 4 + (size_t)RG * d.ppad()) * sizeof(float);
    SKYRL_DISPATCH_T(dtype, {
        if (nt == 256 && rpt <= 4) LAUNCH_SCAN(256, 4);
        else if (nt == 256) LAUNCH_SCAN(256, 8);
        else if (nt == 512) LAUNCH_SCAN(512, 8);
        else if (rpt <= 8) LAUNCH_SCAN(1024, 8);
        else LAUNCH_SCAN(1024, 16);
    })
    return check_launch("ssd_scan_kernel");
}

#define LAUNCH_WALK(NS, OUT, grid, pick)                                                                             \
    hipLaunchKernelGGL((ssd_walk_kernel<NS, OUT>), dim3(grid), dim3(kNT), 0, s, d, sq, pick, slices, u16(xt), u16(bt), \
                       scores, u16(crow), u16(dt_raw), dt_stride, a_log, dt_bias, skip, state, runs, gtot,        \
                       reinterpret_cast<uint16_t*>(y), y_stride)
#define LAUNCH_WALKS(OUT, grid, pick)                      \
    if (d.np() <= 64) LAUNCH_WALK(2, OUT, grid, pick);       \
    else if (d.np() <= 128) LAUNCH_WALK(4, OUT, grid, pick); \
    else LAUNCH_WALK(8, OUT, grid, pick)

extern "C" int skyrl_ssd_prompt(const skyrl_ssd_shape* shape, const void* xt, const void* bt, const void* brow,
                                const void* crow, const void* dt_raw, int64_t dt_stride, const float* a_log,
                                const float* dt_bias, const float* skip, const int32_t* chunk, int32_t nchunks,
                                const int32_t* super, int32_t nsuper, const int32_t* pick, int32_t npick, const int32_t* chain,
                                int32_t nchain, const int32_t* cu, const int32_t* rows, const int64_t* positions,
                                float* state, float* scores, float* runs, float* gtot, void* y,
                                int64_t y_stride, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    const int slices = (d.vp() + 63) / 64;
    SKYRL_REQUIRE(d.N <= 256, "ssd_prompt: state must be at most 256");
    SKYRL_REQUIRE(nchunks >= nsuper && nsuper >= 0 && npick >= 0 && nchain >= 0 && nchain <= 65535 && dt_stride >= d.H &&
                      (int64_t)nsuper * d.H * slices < (1 << 30) && (int64_t)npick * d.H * slices < (1 << 30) &&
                      y_stride >= d.inner(),
                  "ssd_prompt: bad sizes");
    if (nsuper == 0) return SKYRL_OK;
    SKYRL_REQUIRE(xt && bt && brow && crow && dt_raw && a_log && dt_bias && skip && chunk && super && cu && rows &&
                      positions && state && scores && runs && gtot && y && (pick || !npick) && (chain || !nchain),
                  "ssd_prompt: null pointer");
    SKYRL_REQUIRE(aligned16(xt) && aligned16(bt) && aligned16(brow) && aligned16(crow) && aligned16(scores),
                  "ssd_prompt: 16-byte alignment");
    SKYRL_REQUIRE(d.P % 4 || (y_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(y) & 7) == 0),
                  "ssd_prompt: y must be aligned to four elements");
    hipStream_t s = as_stream(stream);
    const SeqRef sq{chunk, super, cu, rows, positions};
    auto u16 = [](const void* p) { return reinterpret_cast<const uint16_t*>(p); };
    hipLaunchKernelGGL(ssd_scores_kernel, dim3((unsigned)nchunks * d.G), dim3(kNT), 0, s, d.G, d.np(), chunk, u16(brow),
                       u16(crow), scores);
    if (npick) {
        LAUNCH_WALKS(false, (unsigned)(npick * d.H * slices), pick);
        const int64_t size = (int64_t)d.H * d.np() * d.vp();
        hipLaunchKernelGGL(ssd_chain_kernel, dim3((unsigned)((size + kNT - 1) / kNT), nchain), dim3(kNT), 0, s, d, sq,
                           chain, state, gtot, runs);
    }
    LAUNCH_WALKS(true, (unsigned)(nsuper * d.H * slices), nullptr);
    return check_launch("ssd_prompt kernels");
}
