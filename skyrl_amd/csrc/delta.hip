// Gated delta rule: a recurrent layer with a [dim x vdim] matrix state per head
// (include/skyrl_layers.h has the equations and the tensor layouts).
//
// Token form (delta_scan): one workgroup per (sequence, head). The state is read once into registers,
// carried over the sequence's tokens and written once, so a decode step costs one read and one write
// of the state. Convolution, unit norms, gates, recurrence, output norm and output gate are one pass.
// Both products with the state are taken before the update, S^T k and S^T q, in one sweep:
// o = (g S + k u^T)^T q = g S^T q + (k . q) u.
//
// Prompt form (conv, chunk, chain, out): chunks of 64 tokens. Unrolling the recurrence over a chunk
// with G_i the summed log decays up to token i gives
//   u_i = beta_i (v_i - e^{G_i} S0^T k_i - sum_{j<i} e^{G_i - G_j} (k_i . k_j) u_j),
// i.e. (I + A) U = diag(beta) V - diag(beta e^G) K S0 with A_ij = beta_i e^{G_i - G_j} k_i . k_j below
// the diagonal. delta_chunk solves it for both right-hand sides, all chunks at once: U0 = (I + A)^-1
// diag(beta) V and W = (I + A)^-1 diag(beta e^G) K, and forms P_ij = e^{G_i - G_j} q_i . k_j (j <= i).
// delta_chain then walks a sequence's chunks with a 16-column slice of S per workgroup:
//   U = U0 - W S,   O = diag(e^G) Q S + P U,   S <- e^{G_n} S + K^T diag(e^{G_n - G}) U.
// Everything is f32, the products on the f32 matrix instructions (v_mfma_f32_16x16x4_f32): a lane's
// four consecutive k values of a 16-step feed four instructions, the same permutation of k on both sides.
#include "conv.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kMaxTaps = 64;
constexpr int kC = 64;       // tokens per chunk

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct Dims {
    int H, K, D, V, taps;
    float eps;
    __host__ __device__ int vpad() const { return (V + 3) / 4 * 4; }
    __host__ __device__ int d16() const { return (D + 15) / 16 * 16; }
    __host__ __device__ int v16() const { return (V + 15) / 16 * 16; }
    __host__ __device__ int channels() const { return 2 * K * D + H * V; }
};

template <typename T>
__device__ __forceinline__ float conv_silu(const T* __restrict__ proj, int64_t stride, const T* __restrict__ w,
                                           const T* __restrict__ ring, int channels, int taps, int ch, int t, int t0,
                                           int pos, int r) {
    return siluf_(short_conv(proj, stride, w, ring, channels, taps, ch, t, t0, pos, r));
}

// NT threads, RPT state rows per thread: thread (cg, rg) holds columns 4 cg .. 4 cg + 3 of rows rg, rg + RG, ...
template <typename T, int NT, int RPT>
__global__ __launch_bounds__(NT) __attribute__((amdgpu_waves_per_eu(4))) void delta_scan_kernel(Dims d, const T* __restrict__ proj, int64_t stride,
                                                         const T* __restrict__ conv_w, const float* __restrict__ a_log,
                                                         const float* __restrict__ dt_bias,
                                                         const T* __restrict__ norm_w, const int32_t* __restrict__ cu,
                                                         const int32_t* __restrict__ rows,
                                                         const int64_t* __restrict__ positions,
                                                         float* __restrict__ state, T* __restrict__ conv_state,
                                                         int save_conv, T* __restrict__ out, int64_t out_stride) {
    extern __shared__ float smem[];
    const int h = blockIdx.x, s = blockIdx.y;
    const int row = rows[s];
    if (row < 0) return;
    const int t0 = cu[s], t1 = cu[s + 1];
    if (t0 >= t1) return;
    const int D = d.D, V = d.V, VP = d.vpad(), NC = VP / 4, RG = NT / NC;
    const int ch_all = d.channels();
    const int kh = h / (d.H / d.K);
    float* s_q = smem;             // D
    float* s_k = s_q + D;          // D
    float* s_v = s_k + D;          // VP
    float* s_o = s_v + VP;         // VP
    float* s_red = s_o + VP;       // RG * VP * 2
    float* s_n = s_red + RG * VP * 2;  // 4 scalars
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cg = tid % NC, rg = tid / NC;
    const bool act = rg < RG;
    const bool fold = NC <= kWave && (NC & (NC - 1)) == 0;  // a wave holds whole row groups
    const int nrec = fold ? NT / kWave : RG;
    const int64_t pos0 = positions[t0];
    T* ring = conv_state + (int64_t)row * d.taps * ch_all;
    float* st_ = state + ((int64_t)row * d.H + h) * D * VP;
    float S[RPT][4];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (act && r < D && pos0 > 0) v = ld4(st_ + (int64_t)r * VP + 4 * cg);
        S[i][0] = v.x; S[i][1] = v.y; S[i][2] = v.z; S[i][3] = v.w;
    }
    const float neg_rate = -expf(a_log[h]), dt = dt_bias[h];
    const float qscale = 1.f / sqrtf((float)D);
    const int qoff = kh * D, koff = (d.K + kh) * D, voff = 2 * d.K * D + h * V;
    const int goff = ch_all + h * V, boff = ch_all + d.H * V + h, aoff = boff + d.H;
    for (int t = t0; t < t1; ++t) {
        const int pos = (int)pos0 + (t - t0);
        const T* p = proj + (int64_t)t * stride;
        const int slot = pos % d.taps;
        const float b_raw = ld(p + boff), a_raw = ld(p + aoff);
        const float gate = tid < V ? ld(p + goff + tid) : 0.f, nw = tid < V ? ld(norm_w + tid) : 0.f;
        for (int e = tid; e < 2 * D + VP; e += NT) {
            float y = 0.f;
            if (e < 2 * D + V) {
                const int ch = e < D ? qoff + e : e < 2 * D ? koff + e - D : voff + e - 2 * D;
                y = conv_silu(proj, stride, conv_w, ring, ch_all, d.taps, ch, t, t0, pos, slot);
            }
            smem[e] = y;  // s_q | s_k | s_v are contiguous
        }
        __syncthreads();
        if (wave < 3) {  // |q|^2, |k|^2, q . k of the raw vectors
            const float* a = wave == 1 ? s_k : s_q;
            const float* b = wave == 0 ? s_q : s_k;
            float x = 0.f;
            for (int i = lane; i < D; i += kWave) x += a[i] * b[i];
            x = wave_sum(x);
            if (lane == 0) s_n[wave] = x;
        }
        __syncthreads();
        const float rq = qscale / sqrtf(s_n[0] + 1e-6f), rk = 1.f / sqrtf(s_n[1] + 1e-6f);
        const float kq = s_n[2] * rq * rk;
        const float beta = sigmoidf_(b_raw);
        const float g = expf(neg_rate * softplusf_(a_raw + dt));
        float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
        if (act) {
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const int r = rg + i * RG;
                if (r < D) {
                    const float kr = s_k[r] * rk, qr = s_q[r] * rq;
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        a[j] += S[i][j] * kr;
                        b[j] += S[i][j] * qr;
                    }
                }
            }
            if (fold)  // the wave's own row groups first
                for (int o = NC; o < kWave; o <<= 1) {
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        a[j] += __shfl_xor(a[j], o, kWave);
                        b[j] += __shfl_xor(b[j], o, kWave);
                    }
                }
            if (!fold || lane < NC) {
                const int rec = fold ? wave : rg;
                st4(s_red + (rec * 2) * VP + 4 * cg, make_float4(a[0], a[1], a[2], a[3]));
                st4(s_red + (rec * 2 + 1) * VP + 4 * cg, make_float4(b[0], b[1], b[2], b[3]));
            }
        }
        __syncthreads();
        if (act) {
            float4 A = make_float4(0.f, 0.f, 0.f, 0.f), B = A;
            for (int r = 0; r < nrec; ++r) {
                const float4 x = ld4(s_red + (r * 2) * VP + 4 * cg), y = ld4(s_red + (r * 2 + 1) * VP + 4 * cg);
                A.x += x.x; A.y += x.y; A.z += x.z; A.w += x.w;
                B.x += y.x; B.y += y.y; B.z += y.z; B.w += y.w;
            }
            const float4 v = ld4(s_v + 4 * cg);
            const float u[4] = {beta * (v.x - g * A.x), beta * (v.y - g * A.y), beta * (v.z - g * A.z),
                                beta * (v.w - g * A.w)};
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const int r = rg + i * RG;
                if (r < D) {
                    const float kr = s_k[r] * rk;
#pragma unroll
                    for (int j = 0; j < 4; ++j) S[i][j] = g * S[i][j] + kr * u[j];
                }
            }
            if (rg == 0)
                st4(s_o + 4 * cg,
                    make_float4(g * B.x + kq * u[0], g * B.y + kq * u[1], g * B.z + kq * u[2], g * B.w + kq * u[3]));
        }
        __syncthreads();
        if (wave * kWave < V) {
            float x = 0.f;
            for (int i = lane; i < V; i += kWave) x += s_o[i] * s_o[i];
            x = wave_sum(x);
            const float r = 1.f / sqrtf(x / (float)V + d.eps);
            T* dst = out + (int64_t)t * out_stride + h * V;
            if (tid < V) st(dst + tid, s_o[tid] * r * nw * siluf_(gate));
            for (int i = tid + NT; i < V; i += NT) st(dst + i, s_o[i] * r * ld(norm_w + i) * siluf_(ld(p + goff + i)));
        }
        // s_q/s_k/s_v are rewritten only after every thread passed the barrier above; s_o not before the next two
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        if (act && r < D) st4(st_ + (int64_t)r * VP + 4 * cg, make_float4(S[i][0], S[i][1], S[i][2], S[i][3]));
    }
    if (save_conv) {  // one token: its slot is not among those the convolutions read
        const T* p = proj + (int64_t)t0 * stride;
        T* dst = ring + (int64_t)(pos0 % d.taps) * ch_all;
        for (int e = tid; e < V; e += NT) dst[voff + e] = p[voff + e];
        if (h % (d.H / d.K) == 0)
            for (int e = tid; e < D; e += NT) {
                dst[qoff + e] = p[qoff + e];
                dst[koff + e] = p[koff + e];
            }
    }
}

// ---- prompt form ------------------------------------------------------------------------------
struct SeqRef {
    const int32_t* chunk;  // [nchunks, 4]: first token, tokens, sequence, 0
    const int32_t* cu;
    const int32_t* rows;
    const int64_t* positions;
};

// Convolution, silu, unit norms and gates. grid (nchunks, K + ceil(H V / 256)): the first K groups are the
// key heads (q and k), the others 256 value channels each; gates with group 0.
template <typename T>
__global__ __launch_bounds__(kNT) void delta_conv_kernel(Dims d, SeqRef sq, const T* __restrict__ proj, int64_t stride,
                                                         const T* __restrict__ conv_w, const float* __restrict__ a_log,
                                                         const float* __restrict__ dt_bias,
                                                         const T* __restrict__ conv_state, float* __restrict__ qk,
                                                         float* __restrict__ kt, float* __restrict__ vout, float* __restrict__ lg,
                                                         float* __restrict__ beta) {
    extern __shared__ float smem[];  // [16][2 D] of the key heads
    const int32_t* ck = sq.chunk + 4 * blockIdx.x;
    const int t0 = ck[0], n = ck[1], seq = ck[2];
    const int sfirst = sq.cu[seq];
    const int pos0 = (int)sq.positions[sfirst] + (t0 - sfirst);
    const int ch_all = d.channels(), D = d.D, D16 = d.d16();
    const T* ring = conv_state + (int64_t)sq.rows[seq] * d.taps * ch_all;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const bool keys = (int)blockIdx.y < d.K;
    const int kh = blockIdx.y;
    if (blockIdx.y == 0) {
        for (int e = tid; e < n * d.H; e += kNT) {
            const int i = e / d.H, h = e - i * d.H;
            const T* p = proj + (int64_t)(t0 + i) * stride + ch_all + d.H * d.V;
            beta[(int64_t)(t0 + i) * d.H + h] = sigmoidf_(ld(p + h));
            lg[(int64_t)(t0 + i) * d.H + h] = -expf(a_log[h]) * softplusf_(ld(p + d.H + h) + dt_bias[h]);
        }
    }
    // input of channel ch at local token i (negative: before the chunk, from the portion or the stored inputs)
    auto input = [&](int ch, int i) -> float {
        if (pos0 + i < 0) return 0.f;
        if (t0 + i >= sfirst) return ld(proj + (int64_t)(t0 + i) * stride + ch);
        return ld(ring + (int64_t)((pos0 + i) % d.taps) * ch_all + ch);
    };
    const int nch = keys ? 2 * D : min(kNT, d.H * d.V - ((int)blockIdx.y - d.K) * kNT);
    const bool held = d.taps <= kConvWindow, carry = nch <= kNT;  // carry: one channel per thread, inputs stay in registers
    constexpr int kSub = 16, kBack = kConvWindow - 1;
    float x[kBack + kSub];
    for (int i0 = 0; i0 < n; i0 += kSub) {
        const int m = min(kSub, n - i0);
        for (int e = tid; e < nch; e += kNT) {
            const int ch = !keys ? 2 * d.K * D + ((int)blockIdx.y - d.K) * kNT + e
                                 : e < D ? kh * D + e : (d.K + kh) * D + (e - D);
            float w[kConvWindow];
            if (held) {
                if (carry && i0 > 0) {
#pragma unroll
                    for (int j = 0; j < kBack; ++j) x[j] = x[j + kSub];
                } else {
#pragma unroll
                    for (int j = 0; j < kBack; ++j) x[j] = j >= kConvWindow - d.taps ? input(ch, i0 - kBack + j) : 0.f;
                }
#pragma unroll
                for (int j = 0; j < kSub; ++j)
                    x[kBack + j] = ld(proj + (int64_t)(t0 + min(i0 + j, n - 1)) * stride + ch);
#pragma unroll
                for (int j = 0; j < kConvWindow; ++j)
                    w[j] = j >= kConvWindow - d.taps ? ld(conv_w + (int64_t)ch * d.taps + j - (kConvWindow - d.taps)) : 0.f;
            }
#pragma unroll
            for (int i = 0; i < kSub; ++i) {
                float y = 0.f;
                if (held) {
#pragma unroll
                    for (int j = 0; j < kConvWindow; ++j) y += x[i + j] * w[j];
                } else if (i < m) {
                    for (int j = 0; j < d.taps; ++j)
                        y += input(ch, i0 + i - (d.taps - 1) + j) * ld(conv_w + (int64_t)ch * d.taps + j);
                }
                y = siluf_(y);
                if (keys) smem[i * 2 * D + e] = y;
                else if (i < m) vout[(int64_t)(t0 + i0 + i) * d.H * d.V + ((int)blockIdx.y - d.K) * kNT + e] = y;
            }
        }
        if (!keys) continue;
        __syncthreads();
        for (int e = wave; e < 2 * m; e += kNT / kWave) {
            const int i = e >> 1, which = e & 1;
            float* src = smem + i * 2 * D + which * D;
            float ss = 0.f;
            for (int k = lane; k < D; k += kWave) ss += src[k] * src[k];
            float r = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
            if (which == 0) r *= 1.f / sqrtf((float)D);
            float* dst = qk + (((int64_t)(t0 + i0 + i) * 2 + which) * d.K + kh) * D16;
            for (int k = lane; k < D16; k += kWave) {
                const float y = k < D ? src[k] * r : 0.f;
                dst[k] = y;
                if (which && k < D) src[k] = y;
            }
        }
        __syncthreads();
        float* tr = kt + (((int64_t)blockIdx.x * d.K + kh) * D16) * kC + i0;  // K^T, zero past the chunk's end
        for (int e = tid; e < D16 * 4; e += kNT) {
            const int k = e >> 2, i = (e & 3) * 4;
            float y[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) y[j] = (k < D && i + j < m) ? smem[(i + j) * 2 * D + D + k] : 0.f;
            st4(tr + (int64_t)k * kC + i, make_float4(y[0], y[1], y[2], y[3]));
        }
        __syncthreads();
    }
    if (keys)
        for (int i0 = (n + kSub - 1) / kSub * kSub; i0 < kC; i0 += kSub)
            for (int e = tid; e < D16 * 4; e += kNT)
                st4(kt + (((int64_t)blockIdx.x * d.K + kh) * D16 + (e >> 2)) * kC + i0 + (e & 3) * 4,
                    make_float4(0.f, 0.f, 0.f, 0.f));
}

__device__ __forceinline__ f32x4 mma4(const float4& a, const float4& b, f32x4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}
__device__ __forceinline__ float4 as_float4(const f32x4& v) { return make_float4(v[0], v[1], v[2], v[3]); }

// One workgroup per (chunk, head). The 64 x 64 system is solved in 16 x 16 blocks: each wave inverts one
// diagonal block by substitution, the blocks below follow diagonal by diagonal from
// T_rb = -T_rr sum_k A_rk T_kb, and T then multiplies both right-hand sides. A 16 x 16 result's registers
// (rows 4 g + i, column c) are the next product's right operand as they are.
__global__ __launch_bounds__(kNT) void delta_chunk_kernel(Dims d, const int32_t* __restrict__ chunk,
                                                          const float* __restrict__ qk, const float* __restrict__ v,
                                                          const float* __restrict__ lg, const float* __restrict__ beta,
                                                          float* __restrict__ W, float* __restrict__ U,
                                                          float* __restrict__ P, float* __restrict__ G) {
    constexpr int LD = kC + 4;
    __shared__ __attribute__((aligned(16))) float s_k[kC * LD];  // a 64-wide slab of K; then A
    __shared__ __attribute__((aligned(16))) float s_q[kC * LD];  // a slab of Q; then T = (I + A)^-1
    __shared__ __attribute__((aligned(16))) float s_g[kC], s_b[kC], s_w[kC];
    const int h = blockIdx.x % d.H, ci = blockIdx.x / d.H;
    const int32_t* ck = chunk + 4 * ci;
    const int t0 = ck[0], n = ck[1];
    const int kh = h / (d.H / d.K), D16 = d.d16(), V16 = d.v16();
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int64_t ch = (int64_t)ci * d.H + h;
    if (wave == 0) {  // inclusive sums of the log decays; tokens past the chunk's end have beta 0 and decay 1
        float x = lane < n ? lg[(int64_t)(t0 + lane) * d.H + h] : 0.f;
#pragma unroll
        for (int o = 1; o < kWave; o <<= 1) {
            const float y = __shfl_up(x, o, kWave);
            if (lane >= o) x += y;
        }
        const float be = lane < n ? beta[(int64_t)(t0 + lane) * d.H + h] : 0.f;
        s_g[lane] = x;
        s_b[lane] = be;
        s_w[lane] = be * expf(x);
        G[ch * kC + lane] = x;
    }
    // K K^T and Q K^T on the ten blocks at and below the diagonal: 20 block products, five per wave
    f32x4 acc[5];
    int br[5], bc[5];
#pragma unroll
    for (int k = 0; k < 5; ++k) {
        acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int item = (wave + 4 * k) % 10;  // (0,0) (1,0) (1,1) (2,0) ...
        br[k] = item >= 6 ? 3 : item >= 3 ? 2 : item >= 1 ? 1 : 0;
        bc[k] = item - br[k] * (br[k] + 1) / 2;
    }
    for (int d0 = 0; d0 < D16; d0 += kC) {
        const int w4 = min(kC, D16 - d0) / 4;
        __syncthreads();
        for (int e = tid; e < kC * w4; e += kNT) {
            const int i = e / w4, x = (e - i * w4) * 4;
            const float* src = qk + ((int64_t)(t0 + min(i, n - 1)) * 2 * d.K + kh) * D16 + d0 + x;
            float4 qv = ld4(src), kv = ld4(src + (int64_t)d.K * D16);
            st4(&s_k[i * LD + x], kv);
            st4(&s_q[i * LD + x], qv);
        }
        __syncthreads();
        for (int s = 0; s < w4 / 4; ++s) {
#pragma unroll
            for (int k = 0; k < 5; ++k) {
                const float* left = wave + 4 * k < 10 ? s_k : s_q;
                acc[k] = mma4(ld4(&left[(16 * br[k] + c) * LD + 16 * s + 4 * g]),
                              ld4(&s_k[(16 * bc[k] + c) * LD + 16 * s + 4 * g]), acc[k]);
            }
        }
    }
    __syncthreads();
    float *s_a = s_k, *s_t = s_q;
#pragma unroll
    for (int k = 0; k < 5; ++k) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = 16 * br[k] + 4 * g + i, cc = 16 * bc[k] + c;
            const float dec = cc <= r ? expf(s_g[r] - s_g[cc]) : 0.f;
            if (wave + 4 * k < 10) s_a[r * LD + cc] = cc < r ? s_b[r] * dec * acc[k][i] : 0.f;
            else P[(ch * kC + r) * kC + cc] = dec * acc[k][i];
        }
    }
    __syncthreads();
    {  // diagonal block `wave`: column c of its inverse
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float r = i == c ? 1.f : 0.f;
#pragma unroll
            for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
                const float4 a = ld4(&s_a[(16 * wave + i) * LD + 16 * wave + 4 * j4]);
                r -= a.x * x[4 * j4];
                if (4 * j4 + 1 < i) r -= a.y * x[4 * j4 + 1];
                if (4 * j4 + 2 < i) r -= a.z * x[4 * j4 + 2];
                if (4 * j4 + 3 < i) r -= a.w * x[4 * j4 + 3];
            }
            x[i] = r;
        }
        if (g == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) s_t[(16 * wave + i) * LD + 16 * wave + c] = x[i];
        }
    }
#pragma unroll
    for (int lev = 1; lev < 4; ++lev) {
        __syncthreads();
        if (wave + lev < 4) {
            const int b = wave, r = wave + lev;
            f32x4 m = {0.f, 0.f, 0.f, 0.f}, tt = m;
            for (int k = b; k < r; ++k) {
                const float* tk = &s_t[(16 * k + 4 * g) * LD + 16 * b + c];
                m = mma4(ld4(&s_a[(16 * r + c) * LD + 16 * k + 4 * g]),
                         make_float4(tk[0], tk[LD], tk[2 * LD], tk[3 * LD]), m);
            }
            tt = mma4(ld4(&s_t[(16 * r + c) * LD + 16 * r + 4 * g]), as_float4(m), tt);
#pragma unroll
            for (int i = 0; i < 4; ++i) s_t[(16 * r + 4 * g + i) * LD + 16 * b + c] = -tt[i];
        }
    }
    __syncthreads();
    // T times [diag(beta e^G) K | diag(beta) V], 16 columns at a time
    const int nw = D16 / 16, ntile = nw + V16 / 16;
    for (int tile = wave; tile < ntile; tile += 4) {
        const bool isw = tile < nw;
        const int cc = 16 * (isw ? tile : tile - nw) + c;
        const float* src = isw ? qk + ((int64_t)t0 * 2 + 1) * d.K * D16 + (int64_t)kh * D16 + cc
                               : v + ((int64_t)t0 * d.H + h) * d.V + min(cc, d.V - 1);
        const int64_t step = isw ? (int64_t)2 * d.K * D16 : (int64_t)d.H * d.V;
        float x[16];
#pragma unroll
        for (int j = 0; j < 16; ++j) x[j] = src[min(16 * (j >> 2) + 4 * g + (j & 3), n - 1) * step];
        f32x4 o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            const float4 sc = ld4((isw ? s_w : s_b) + 16 * s + 4 * g);
            const float4 bv = make_float4(x[4 * s] * sc.x, x[4 * s + 1] * sc.y, x[4 * s + 2] * sc.z, x[4 * s + 3] * sc.w);
#pragma unroll
            for (int r = s; r < 4; ++r) o[r] = mma4(ld4(&s_t[(16 * r + c) * LD + 16 * s + 4 * g]), bv, o[r]);
        }
        if (isw) {
            float* dst = W + ch * kC * D16 + cc;
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
                for (int i = 0; i < 4; ++i) dst[(16 * r + 4 * g + i) * D16] = o[r][i];
        } else {  // U^T
            float* dst = U + (ch * V16 + cc) * kC + 4 * g;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                st4(dst + 16 * r, cc < d.V ? as_float4(o[r]) : make_float4(0.f, 0.f, 0.f, 0.f));
        }
    }
}

// One workgroup per (sequence, head, 16 columns of S). NS: 16-wide steps of dim (EXACT: dim = 16 NS); DT
// 16-row tiles of S per wave. What a phase has consumed is loaded for the next chunk at once, into the
// same registers: W and Q during the second phase, K^T and P during the next chunk's first.
template <int NS, bool EXACT>
__global__ __launch_bounds__(kNT) __attribute__((amdgpu_waves_per_eu(NS <= 8 ? 2 : 1))) void delta_chain_kernel(
    Dims d, SeqRef sq, const int32_t* __restrict__ seq_chunks, int seq0, int nseq, const float* __restrict__ qk,
    const float* __restrict__ kt, const float* __restrict__ W, const float* __restrict__ U, const float* __restrict__ P,
    const float* __restrict__ G, float* __restrict__ state, float* __restrict__ o) {
    constexpr int LS = NS * 16 + 4, LU = kC + 4, DT = (NS + 3) / 4;
    __shared__ __attribute__((aligned(16))) float s_s[16 * LS];      // S^T slice
    __shared__ __attribute__((aligned(16))) float s_u[2][16 * LU];   // U^T and its decayed copy
    const int V16 = d.v16(), D16 = EXACT ? NS * 16 : d.d16(), VP = d.vpad(), nt = V16 / 16;
    // the slices of one (sequence, head) read the same W, Q, K and P: consecutive on one XCD
    const int xcd = blockIdx.x % 8, slot = blockIdx.x / 8, grp = slot / nt * 8 + xcd;
    if (grp >= nseq * d.H) return;
    const int vt = slot % nt, h = grp % d.H, si = grp / d.H;
    const int seq = seq0 + si, row = sq.rows[seq];
    if (row < 0) return;
    const int64_t pos0 = sq.positions[sq.cu[seq]];
    const int kh = h / (d.H / d.K);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int ns = EXACT ? NS : D16 / 16;
    float* st_ = state + ((int64_t)row * d.H + h) * d.D * VP;
    const int vcol = 16 * vt + c;

    // this wave's rows of S: tiles wave, wave + 4, ...; element i: dim 16 tile + 4 g + i, column c
    f32x4 S[DT];
#pragma unroll
    for (int k = 0; k < DT; ++k) {
        const int tile = wave + 4 * k;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int dd = 16 * tile + 4 * g + i;
            S[k][i] = (pos0 > 0 && dd < d.D && vcol < VP) ? st_[(int64_t)dd * VP + vcol] : 0.f;
        }
        if (EXACT || tile < ns) *reinterpret_cast<f32x4*>(&s_s[c * LS + 16 * tile + 4 * g]) = S[k];
    }
    const int c0 = seq_chunks[si], c1 = seq_chunks[si + 1];
    const int woff = (16 * wave + c) * D16 + 4 * g, poff = (16 * wave + c) * kC + 4 * g;
    const int koff = (16 * wave + c) * kC + 4 * g, goff = 16 * wave + 4 * g, uoff = vcol * kC + goff;
    const int qstep = 2 * d.K * D16, ostep = d.H * d.V;
    float4 w[NS], q[NS], p[4], kk[DT][4], u0, gr;
    float gl;
    auto load_first = [&](int ci, int t0, int n) {
        const float* wp = W + ((int64_t)ci * d.H + h) * kC * D16;
        const float* qp = qk + ((int64_t)t0 * 2 * d.K + kh) * D16;
        const int qoff = min(16 * wave + c, n - 1) * qstep + 4 * g;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            if (EXACT || s < ns) {
                w[s] = ld4(wp + woff + 16 * s);
                q[s] = ld4(qp + qoff + 16 * s);
            }
        }
        const float* gp = G + ((int64_t)ci * d.H + h) * kC;
        u0 = ld4(U + ((int64_t)ci * d.H + h) * V16 * kC + uoff);
        gr = ld4(gp + goff);
        gl = gp[kC - 1];
    };
    auto load_second = [&](int ci) {
        const float* pp = P + ((int64_t)ci * d.H + h) * kC * kC;
        const float* kp = kt + ((int64_t)ci * d.K + kh) * D16 * kC;
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            if (s <= wave) p[s] = ld4(pp + poff + 16 * s);  // P is lower triangular
#pragma unroll
            for (int k = 0; k < DT; ++k)
                if (EXACT || wave + 4 * k < ns) kk[k][s] = ld4(kp + koff + 64 * k * kC + 16 * s);
        }
    };
    int t0 = 0, n = 0;
    if (c0 < c1) {
        t0 = sq.chunk[4 * c0];
        n = sq.chunk[4 * c0 + 1];
        load_first(c0, t0, n);
    }
    for (int ci = c0; ci < c1; ++ci) {
        load_second(ci);
        __syncthreads();  // S^T of the previous chunk is in LDS
        f32x4 aw = {0.f, 0.f, 0.f, 0.f}, ao = aw;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            if (EXACT || s < ns) {
                const float4 b = ld4(&s_s[c * LS + 16 * s + 4 * g]);
                aw = mma4(w[s], b, aw);
                ao = mma4(q[s], b, ao);
            }
        }
        const float4 u = make_float4(u0.x - aw[0], u0.y - aw[1], u0.z - aw[2], u0.w - aw[3]);
        const float4 ud = make_float4(u.x * expf(gl - gr.x), u.y * expf(gl - gr.y), u.z * expf(gl - gr.z),
                                      u.w * expf(gl - gr.w));
        ao[0] *= expf(gr.x);
        ao[1] *= expf(gr.y);
        ao[2] *= expf(gr.z);
        ao[3] *= expf(gr.w);
        const float decay = expf(gl);
        st4(&s_u[0][c * LU + goff], u);
        st4(&s_u[1][c * LU + goff], ud);
        __syncthreads();
        const int tc = t0, nc = n;
        if (ci + 1 < c1) {
            t0 = sq.chunk[4 * ci + 4];
            n = sq.chunk[4 * ci + 5];
            load_first(ci + 1, t0, n);
        }
#pragma unroll
        for (int k = 0; k < DT; ++k) S[k] = S[k] * decay;
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            const float4 b = ld4(&s_u[1][c * LU + 16 * s + 4 * g]);
            if (s <= wave) ao = mma4(p[s], ld4(&s_u[0][c * LU + 16 * s + 4 * g]), ao);
#pragma unroll
            for (int k = 0; k < DT; ++k)
                if (EXACT || wave + 4 * k < ns) S[k] = mma4(kk[k][s], b, S[k]);
        }
#pragma unroll
        for (int k = 0; k < DT; ++k)
            if (EXACT || wave + 4 * k < ns) *reinterpret_cast<f32x4*>(&s_s[c * LS + 16 * (wave + 4 * k) + 4 * g]) = S[k];
        float* op = o + ((int64_t)tc * d.H + h) * d.V;
        if (vcol < d.V) {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (goff + i < nc) op[(goff + i) * ostep + vcol] = ao[i];
        }
    }
#pragma unroll
    for (int k = 0; k < DT; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int dd = 16 * (wave + 4 * k) + 4 * g + i;
            if (dd < d.D && vcol < VP) st_[(int64_t)dd * VP + vcol] = S[k][i];
        }
}

// Output norm and gate of tokens [first, T). LG lanes share a (token, head), four values a lane (VEC: vdim
// a multiple of 4, at most 4 LG); otherwise a wave takes one and strides over vdim.
template <typename T, bool VEC>
__global__ __launch_bounds__(kNT) void delta_out_kernel(Dims d, const float* __restrict__ o, const T* __restrict__ proj,
                                                        int64_t stride, const T* __restrict__ norm_w, int first, int LG,
                                                        int64_t items, T* __restrict__ out, int64_t out_stride) {
    const int lane = threadIdx.x & 63;
    if constexpr (VEC) {
        const int per = kNT / LG, sub = threadIdx.x % LG, i = 4 * sub;
        constexpr int kIt = 4;
        const int64_t e0 = (int64_t)blockIdx.x * per * kIt + threadIdx.x / LG;
        float4 x[kIt], gt[kIt];
#pragma unroll
        for (int k = 0; k < kIt; ++k) {
            const int64_t e = min(e0 + (int64_t)k * per, items - 1), t = first + e / d.H;
            const int h = (int)(e % d.H), ii = min(i, d.V - 4);
            x[k] = ld4(o + (t * d.H + h) * d.V + ii);
            const T* gp = proj + t * stride + d.channels() + h * d.V + ii;
            gt[k] = make_float4(ld(gp), ld(gp + 1), ld(gp + 2), ld(gp + 3));
        }
        const int ii = min(i, d.V - 4);
        const float4 w = make_float4(ld(norm_w + ii), ld(norm_w + ii + 1), ld(norm_w + ii + 2), ld(norm_w + ii + 3));
#pragma unroll
        for (int k = 0; k < kIt; ++k) {
            float ss = i < d.V ? x[k].x * x[k].x + x[k].y * x[k].y + x[k].z * x[k].z + x[k].w * x[k].w : 0.f;
            for (int q = 1; q < LG; q <<= 1) ss += __shfl_xor(ss, q, kWave);
            const float r = 1.f / sqrtf(ss / (float)d.V + d.eps);
            const int64_t e = e0 + (int64_t)k * per;
            if (e < items && i < d.V) {
                T* dst = out + (first + e / d.H) * out_stride + (e % d.H) * d.V + i;
                st(dst, x[k].x * r * w.x * siluf_(gt[k].x));
                st(dst + 1, x[k].y * r * w.y * siluf_(gt[k].y));
                st(dst + 2, x[k].z * r * w.z * siluf_(gt[k].z));
                st(dst + 3, x[k].w * r * w.w * siluf_(gt[k].w));
            }
        }
        return;
    }
    const int64_t e = (int64_t)blockIdx.x * (kNT / kWave) + (threadIdx.x >> 6);
    if (e >= items) return;
    const int64_t t = first + e / d.H;
    const int h = (int)(e % d.H);
    const float* src = o + (t * d.H + h) * d.V;
    const T* gate = proj + t * stride + d.channels() + h * d.V;
    float ss = 0.f;
    for (int i = lane; i < d.V; i += kWave) ss += src[i] * src[i];
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)d.V + d.eps);
    for (int i = lane; i < d.V; i += kWave)
        st(out + t * out_stride + h * d.V + i, src[i] * r * ld(norm_w + i) * siluf_(ld(gate + i)));
}

int scan_rows_per_thread(const Dims& d, int nt) {
    const int RG = nt / (d.vpad() / 4);
    return (d.D + RG - 1) / RG;
}

const char* bad_shape(const skyrl_delta_shape* sh) {
    if (!sh) return "delta: null shape";
    if (sh->heads <= 0 || sh->kv_heads <= 0 || sh->heads % sh->kv_heads) return "delta: heads must be a multiple of kv_heads";
    if (sh->dim <= 0 || sh->vdim <= 0 || sh->dim > 1024 || sh->vdim > 1024) return "delta: dim and vdim must be in [1, 1024]";
    if (sh->taps <= 0 || sh->taps > kMaxTaps) return "delta: taps must be in [1, 64]";
    return nullptr;
}
Dims dims_of(const skyrl_delta_shape* sh) {
    return Dims{sh->heads, sh->kv_heads, sh->dim, sh->vdim, sh->taps, sh->eps};
}
int64_t proj_width(const Dims& d) { return d.channels() + (int64_t)d.H * d.V + 2 * d.H; }

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_SCAN(NT, R)                                                                                         \
    hipLaunchKernelGGL((delta_scan_kernel<T, NT, R>), dim3(d.H, nseq), dim3(NT), lds, as_stream(stream), d,        \
                       reinterpret_cast<const T*>(proj), proj_stride, reinterpret_cast<const T*>(conv_w), a_log,   \
                       dt_bias, reinterpret_cast<const T*>(norm_w), cu, rows, positions, state,                    \
                       reinterpret_cast<T*>(conv_state), save_conv, reinterpret_cast<T*>(out), out_stride)

extern "C" int skyrl_delta_scan(const skyrl_delta_shape* shape, const void* proj, int64_t proj_stride,
                                const void* conv_w, const float* a_log, const float* dt_bias, const void* norm_w,
                                const int32_t* cu, const int32_t* rows, const int64_t* positions, int32_t nseq,
                                float* state, void* conv_state, int32_t save_conv, void* out, int64_t out_stride,
                                int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "delta_scan");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nseq >= 0 && nseq <= 65535, "delta_scan: nseq must be in [0, 65535]");
    SKYRL_REQUIRE(proj_stride >= proj_width(d), "delta_scan: proj_stride");
    SKYRL_REQUIRE(out_stride >= (int64_t)d.H * d.V, "delta_scan: out_stride");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_w && a_log && dt_bias && norm_w && cu && rows && positions && state && conv_state && out,
                  "delta_scan: null pointer");
    const int nt = scan_rows_per_thread(d, 256) <= 8 ? 256 : scan_rows_per_thread(d, 512) <= 8 ? 512 : 1024;
    const int rpt = scan_rows_per_thread(d, nt), RG = nt / (d.vpad() / 4);
    SKYRL_REQUIRE(rpt <= 16, "delta_scan: dim * vdim too large for one workgroup's registers (at most 65536)");
    const size_t lds = (size_t)(2 * d.D + 2 * d.vpad() + 2 * RG * d.vpad() + 4) * sizeof(float);
    SKYRL_DISPATCH_T(dtype, {
        if (nt == 256 && rpt <= 4) LAUNCH_SCAN(256, 4);
        else if (nt == 256) LAUNCH_SCAN(256, 8);
        else if (nt == 512) LAUNCH_SCAN(512, 8);
        else if (rpt <= 8) LAUNCH_SCAN(1024, 8);
        else LAUNCH_SCAN(1024, 16);
    })
    return check_launch("delta_scan_kernel");
}

extern "C" int skyrl_delta_conv(const skyrl_delta_shape* shape, const void* proj, int64_t proj_stride,
                                const void* conv_w, const float* a_log, const float* dt_bias, const int32_t* chunk,
                                int32_t nchunks, const int32_t* cu, const int32_t* rows, const int64_t* positions,
                                const void* conv_state, float* qk, float* kt, float* v, float* lg, float* beta,
                                int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "delta_conv");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nchunks >= 0 && proj_stride >= proj_width(d), "delta_conv: bad sizes");
    if (nchunks == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_w && a_log && dt_bias && chunk && cu && rows && positions && conv_state && qk && kt && v &&
                      lg && beta,
                  "delta_conv: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((delta_conv_kernel<T>), dim3(nchunks, d.K + (d.H * d.V + kNT - 1) / kNT), dim3(kNT),
                           16 * 2 * d.D * sizeof(float), as_stream(stream), d, SeqRef{chunk, cu, rows, positions},
                           reinterpret_cast<const T*>(proj), proj_stride, reinterpret_cast<const T*>(conv_w), a_log,
                           dt_bias, reinterpret_cast<const T*>(conv_state), qk, kt, v, lg, beta);
    })
    return check_launch("delta_conv_kernel");
}

extern "C" int skyrl_delta_chunk(const skyrl_delta_shape* shape, const int32_t* chunk, int32_t nchunks,
                                 const float* qk, const float* v, const float* lg, const float* beta, float* W,
                                 float* U, float* P, float* G, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nchunks >= 0 && (int64_t)nchunks * d.H < (1 << 30), "delta_chunk: bad sizes");
    if (nchunks == 0) return SKYRL_OK;
    SKYRL_REQUIRE(chunk && qk && v && lg && beta && W && U && P && G, "delta_chunk: null pointer");
    hipLaunchKernelGGL(delta_chunk_kernel, dim3(nchunks * d.H), dim3(kNT), 0, as_stream(stream), d, chunk, qk, v, lg,
                       beta, W, U, P, G);
    return check_launch("delta_chunk_kernel");
}

#define LAUNCH_CHAIN(NS, EXACT)                                                                                 \
    hipLaunchKernelGGL((delta_chain_kernel<NS, EXACT>),                                                           \
                       dim3((unsigned)(nseq * d.H + 7) / 8 * 8 * (d.v16() / 16)), dim3(kNT), 0, as_stream(stream), \
                       d, SeqRef{chunk, cu, rows, positions}, seq_chunks, seq0, nseq, qk, kt, W, U, P, G, state, o)

extern "C" int skyrl_delta_chain(const skyrl_delta_shape* shape, const int32_t* chunk, const int32_t* seq_chunks,
                                 int32_t seq0, int32_t nseq, const int32_t* cu, const int32_t* rows,
                                 const int64_t* positions, const float* qk, const float* kt, const float* W,
                                 const float* U, const float* P, const float* G, float* state, float* o, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(d.D <= 256, "delta_chain: dim must be at most 256");
    SKYRL_REQUIRE(nseq >= 0 && seq0 >= 0 && (int64_t)nseq * d.H * (d.v16() / 16) < (1 << 30), "delta_chain: bad sizes");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(chunk && seq_chunks && cu && rows && positions && qk && kt && W && U && P && G && state && o,
                  "delta_chain: null pointer");
    if (d.D == 64) LAUNCH_CHAIN(4, true);
    else if (d.D < 64) LAUNCH_CHAIN(4, false);
    else if (d.D == 128) LAUNCH_CHAIN(8, true);
    else if (d.D < 128) LAUNCH_CHAIN(8, false);
    else LAUNCH_CHAIN(16, false);
    return check_launch("delta_chain_kernel");
}

extern "C" int skyrl_delta_out(const skyrl_delta_shape* shape, const float* o, const void* proj, int64_t proj_stride,
                               const void* norm_w, int32_t first, int32_t T_, void* out, int64_t out_stride,
                               int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "delta_out");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(first >= 0 && T_ >= first && proj_stride >= proj_width(d) && out_stride >= (int64_t)d.H * d.V,
                  "delta_out: bad sizes");
    const int64_t items = (int64_t)(T_ - first) * d.H;
    if (items == 0) return SKYRL_OK;
    SKYRL_REQUIRE(o && proj && norm_w && out, "delta_out: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        int LG = 1;
        while (4 * LG < d.V) LG <<= 1;
        const T* p = reinterpret_cast<const T*>(proj);
        const T* w = reinterpret_cast<const T*>(norm_w);
        T* dst = reinterpret_cast<T*>(out);
        if (d.V % 4 == 0 && LG <= kWave) {
            const int64_t per = (int64_t)kNT / LG * 4;
            hipLaunchKernelGGL((delta_out_kernel<T, true>), dim3((unsigned)((items + per - 1) / per)), dim3(kNT), 0,
                               as_stream(stream), d, o, p, proj_stride, w, first, LG, items, dst, out_stride);
        } else {
            hipLaunchKernelGGL((delta_out_kernel<T, false>), dim3((unsigned)((items + 3) / 4)), dim3(kNT), 0,
                               as_stream(stream), d, o, p, proj_stride, w, first, LG, items, dst, out_stride);
        }
    })
    return check_launch("delta_out_kernel");
}
