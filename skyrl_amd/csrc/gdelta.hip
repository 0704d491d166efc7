// Generalized delta rule: a recurrent layer with a [dim x dim] matrix state per head, a decay per key channel and a
// removal along the unit key (include/skyrl_layers.h has the equations and the tensor layouts):
//   S_t = diag(w_t) S - (a_t u_t) (u_t^T S) + k_t v_t^T,  o_t = S_t^T r_t,  S the state before t.
//
// Token form (gdelta_scan): one workgroup per (sequence, head), the state in registers over the sequence's tokens. Both
// products with the state read the old one, z = S^T u and y = S^T (w r), in one sweep:
//   o = y - (r . a u) z + (r . k) v.
//
// Prompt form (chunk, chain, out): chunks of 64 tokens. With G_t the summed log decays up to token t, per channel, and
//   al_t = e^{G_(t-1)} u_t,  be_t = e^{-G_t} a_t u_t,  ka_t = e^{-G_t} k_t,  rh_t = e^{G_t} r_t
// (a log decay is above -0.61, so 64 of them stay far inside the range of f32), z_t = u_t^T S_(t-1) solves
//   (I + A) Z = al S0 + B V,   A = al be^T, B = al ka^T below the diagonal,
// and with T = (I + A)^-1, W = T al, U = T B V, P = rh be^T and Q = rh ka^T up to the diagonal:
//   O = R S0 + O0,    R = rh - P W,                       O0 = Q V - P U,
//   S <- M S0 + N,    M = diag(e^{G_n}) (I - be^T W),     N = diag(e^{G_n}) (ka^T V - be^T U).
// gdelta_chunk forms M, N, R and O0 of all chunks at once, gdelta_chain walks a sequence's chunks (one product each)
// with a 16-column slice of S per workgroup and leaves every chunk's first state, gdelta_out forms O with the head
// norms and the output gate. Everything is f32, the products on v_mfma_f32_16x16x4_f32: a lane's four consecutive k
// values of a 16-step feed four instructions, the same permutation of k on both sides.
#include "elem.h"

namespace skyrl {
namespace {

constexpr int kC = 64;   // tokens per chunk
constexpr int LD = kC + 4;
constexpr float kRate = 0.6065306597126334f;  // e^(-1/2)
constexpr float kUnitEps = 1e-6f;

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct Dims {
    int H, D;
    float eps;
    __host__ __device__ int vpad() const { return (D + 3) / 4 * 4; }
    __host__ __device__ int d16() const { return (D + 15) / 16 * 16; }
    __host__ __device__ int width() const { return H * D; }
};

// Columns of a projection row: r | k | v | output gate | removal rate, each heads x dim; wl: the decay logits, a row each.
template <typename T>
struct In {
    const T* proj;
    int64_t stride;
    const T* wl;
    int64_t wl_stride;
    const float* w0;
    const float* ab;
};

__device__ __forceinline__ float log_decay(float z) { return -kRate * sigmoidf_(z); }

// ---- token form ---------------------------------------------------------------------------------
// NT threads, RPT state rows per thread: thread (cg, rg) holds columns 4 cg .. 4 cg + 3 of rows rg, rg + RG, ...
// dim <= NT: a thread loads one channel.
template <typename T, int NT, int RPT>
__global__ __launch_bounds__(NT) void gdelta_scan_kernel(Dims d, In<T> in, const T* __restrict__ norm_w,
                                                         const int32_t* __restrict__ cu,
                                                         const int32_t* __restrict__ rows,
                                                         const int64_t* __restrict__ positions,
                                                         float* __restrict__ state, T* __restrict__ out,
                                                         int64_t out_stride) {
    extern __shared__ float smem[];
    constexpr int NW = NT / kWave;
    const int h = blockIdx.x, s = blockIdx.y;
    const int row = rows[s];
    if (row < 0) return;
    const int t0 = cu[s], t1 = cu[s + 1];
    if (t0 >= t1) return;
    const int D = d.D, VP = d.vpad(), NC = VP / 4, RG = NT / NC, HD = d.width();
    float* s_k = smem;         // VP each: key, decayed query, decay, removal times key, value, output
    float* s_q = s_k + VP;
    float* s_w = s_q + VP;
    float* s_a = s_w + VP;
    float* s_v = s_a + VP;
    float* s_n = s_v + VP;     // 4 NW
    float* s_red = s_n + 4 * NW;  // 2 VP per record
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cg = tid % NC, rg = tid / NC;
    const bool act = rg < RG;
    const bool fold = NC <= kWave && (NC & (NC - 1)) == 0;  // a wave holds whole row groups
    const int nrec = fold ? NW : RG;
    float* st_ = state + ((int64_t)row * d.H + h) * D * VP;
    const bool fresh = positions[t0] == 0;
    float S[RPT][4];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (act && r < D && !fresh) v = ld4(st_ + (int64_t)r * VP + 4 * cg);
        S[i][0] = v.x; S[i][1] = v.y; S[i][2] = v.z; S[i][3] = v.w;
    }
    const bool ch = tid < D;
    const int c0 = h * D + (ch ? tid : 0);
    const float w0 = in.w0[c0], ab = in.ab[c0], nw = ld(norm_w + c0);
    float r_, k_, v_, g_, a_, l_;
    auto load = [&](int t) {
        const T* p = in.proj + (int64_t)t * in.stride + c0;
        r_ = ld(p);
        k_ = ld(p + HD);
        v_ = ld(p + 2 * HD);
        g_ = ld(p + 3 * HD);
        a_ = ld(p + 4 * HD);
        l_ = ld(in.wl + (int64_t)t * in.wl_stride + c0);
    };
    load(t0);
    for (int t = t0; t < t1; ++t) {
        const float k = ch ? k_ : 0.f, r = ch ? r_ : 0.f, a = sigmoidf_(a_ + ab), gate = g_;
        const float w = expf(log_decay(l_ + w0));
        if (tid < VP) {
            s_k[tid] = k;
            s_q[tid] = r * w;
            s_w[tid] = w;
            s_a[tid] = a * k;
            s_v[tid] = ch ? v_ : 0.f;
        }
        const float kk = wave_sum(k * k), ra = wave_sum(r * a * k), rk = wave_sum(r * k);
        if (lane == 0) {
            s_n[4 * wave] = kk;
            s_n[4 * wave + 1] = ra;
            s_n[4 * wave + 2] = rk;
        }
        if (t + 1 < t1) load(t + 1);
        __syncthreads();
        float n2 = 0.f, dra = 0.f, drk = 0.f;
#pragma unroll
        for (int j = 0; j < NW; ++j) {
            n2 += s_n[4 * j];
            dra += s_n[4 * j + 1];
            drk += s_n[4 * j + 2];
        }
        const float un = 1.f / sqrtf(n2 + kUnitEps);
        float z[4] = {0.f, 0.f, 0.f, 0.f}, y[4] = {0.f, 0.f, 0.f, 0.f};
        if (act) {
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const int rr = rg + i * RG;
                if (rr < D) {
                    const float kr = s_k[rr], qr = s_q[rr];
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        z[j] += S[i][j] * kr;
                        y[j] += S[i][j] * qr;
                    }
                }
            }
            if (fold)  // the wave's own row groups first
                for (int o = NC; o < kWave; o <<= 1) {
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        z[j] += __shfl_xor(z[j], o, kWave);
                        y[j] += __shfl_xor(y[j], o, kWave);
                    }
                }
            if (!fold || lane < NC) {
                const int rec = fold ? wave : rg;
                st4(s_red + (rec * 2) * VP + 4 * cg, make_float4(z[0], z[1], z[2], z[3]));
                st4(s_red + (rec * 2 + 1) * VP + 4 * cg, make_float4(y[0], y[1], y[2], y[3]));
            }
        }
        __syncthreads();
        if (act) {
            float4 Z = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int q = 0; q < nrec; ++q) {
                const float4 x = ld4(s_red + (q * 2) * VP + 4 * cg);
                Z.x += x.x; Z.y += x.y; Z.z += x.z; Z.w += x.w;
            }
            const float4 v = ld4(s_v + 4 * cg);
            const float zz[4] = {Z.x * un * un, Z.y * un * un, Z.z * un * un, Z.w * un * un}, vv[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const int rr = rg + i * RG;
                if (rr < D) {
                    const float wr = s_w[rr], ar = s_a[rr], kr = s_k[rr];
#pragma unroll
                    for (int j = 0; j < 4; ++j) S[i][j] = wr * S[i][j] - ar * zz[j] + kr * vv[j];
                }
            }
        }
        float o = 0.f;
        if (ch) {  // thread = column
            float Z = 0.f, Y = 0.f;
            for (int q = 0; q < nrec; ++q) {
                Z += s_red[(q * 2) * VP + tid];
                Y += s_red[(q * 2 + 1) * VP + tid];
            }
            o = Y - dra * un * un * Z + drk * s_v[tid];
        }
        const float ss = wave_sum(o * o);
        if (lane == 0) s_n[4 * wave + 3] = ss;
        __syncthreads();
        float tot = 0.f;
#pragma unroll
        for (int j = 0; j < NW; ++j) tot += s_n[4 * j + 3];
        if (ch)
            st(out + (int64_t)t * out_stride + c0, o * (1.f / sqrtf(tot / (float)D + d.eps)) * nw * sigmoidf_(gate));
        // the next token's writes of s_n[..3] come after two barriers, those of the rest after this one
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + i * RG;
        if (act && r < D) st4(st_ + (int64_t)r * VP + 4 * cg, make_float4(S[i][0], S[i][1], S[i][2], S[i][3]));
    }
}

// ---- prompt form ----------------------------------------------------------------------------------
__device__ __forceinline__ f32x4 mma4(const float4& a, const float4& b, f32x4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}
__device__ __forceinline__ float4 as_float4(const f32x4& v) { return make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ f32x4 zero4() { return f32x4{0.f, 0.f, 0.f, 0.f}; }
// exp of a summed log decay: the bare base-2 instruction (its argument is rounded once more than expf's)
__device__ __forceinline__ float exp_sum(float x) { return fast_exp2(x * kLog2e); }

// What gdelta_chunk leaves, all f32: M [chunk][head][d16][d16], N transposed [..][value][key], R and O0 [..][64][d16].
struct ChunkOut {
    float *M, *N, *R, *O;
};

constexpr int kNW = 8;  // waves

// One workgroup per (chunk, head). Channels come in slabs of 64: al, be, ka and rh of a slab are formed in LDS (token by
// channel), and the four 64 x 64 products sum over slabs. The triangular system is solved in 16 x 16 blocks: a wave
// inverts a diagonal block by substitution, the blocks of T = (I + A)^-1 below follow diagonal by diagonal and are kept
// in the unused blocks above A's diagonal (block (r, b) at (b, r)). Then every wave takes 16 columns of W or of V: a
// 16 x 16 result's registers (rows 4 g + i, column c) are the next product's right operand as they are. With more than
// one slab (dim > 64) the slabs are formed again where they are read. TPW: column tiles of each kind per wave.
template <typename T, int TPW>
__global__ __launch_bounds__(kNW * kWave) void gdelta_chunk_kernel(Dims d, In<T> in, const int32_t* __restrict__ chunk,
                                                                   ChunkOut co) {
    __shared__ __attribute__((aligned(16))) float s_al[kC * LD], s_be[kC * LD], s_ka[kC * LD], s_rh[kC * LD];
    __shared__ __attribute__((aligned(16))) float s_A[kC * LD], s_B[kC * LD], s_P[kC * LD], s_Q[kC * LD];
    __shared__ float s_seg[kNW * kC], s_un[kC], s_eg[kC];
    const int h = blockIdx.x % d.H, ci = blockIdx.x / d.H;
    const int32_t* ck = chunk + 4 * ci;
    const int t0 = ck[0], n = ck[1];
    const int D = d.D, D16 = d.d16(), HD = d.width(), nt = D16 / 16;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int64_t rec = (int64_t)ci * d.H + h;

    // 1 / |k| of every token
#pragma unroll
    for (int i = 0; i < kC / kNW; ++i) {
        const int t = wave * (kC / kNW) + i;
        float ss = 0.f;
        if (t < n)
            for (int e = lane; e < D; e += kWave) {
                const float k = ld(in.proj + (int64_t)(t0 + t) * in.stride + HD + h * D + e);
                ss += k * k;
            }
        ss = wave_sum(ss);
        if (lane == 0) s_un[t] = 1.f / sqrtf(ss + kUnitEps);
    }

    // channel d0 + lane, tokens 8 wave ..: two barriers, the first after everything that read the slab before
    auto load_slab = [&](int d0) {
        constexpr int kT = kC / kNW;
        const int e = d0 + lane;
        const bool on = e < D;
        const int col = h * D + (on ? e : 0);
        const float w0 = in.w0[col], ab = in.ab[col];
        float r[kT], k[kT], a[kT], G[kT];
#pragma unroll
        for (int i = 0; i < kT; ++i) {
            const int t = wave * kT + i;
            const T* p = in.proj + (int64_t)(t0 + min(t, n - 1)) * in.stride + col;
            r[i] = ld(p);
            k[i] = ld(p + HD);
            a[i] = ld(p + 4 * HD);
            G[i] = ld(in.wl + (int64_t)(t0 + min(t, n - 1)) * in.wl_stride + col);
        }
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < kT; ++i) {
            const bool use = on && wave * kT + i < n;
            const float lw = use ? log_decay(G[i] + w0) : 0.f;
            a[i] = sigmoidf_(a[i] + ab);
            if (!use) r[i] = k[i] = 0.f;
            sum += lw;
            G[i] = lw;
        }
        s_seg[wave * kC + lane] = sum;
        __syncthreads();
        float base = 0.f, all = 0.f;
#pragma unroll
        for (int j = 0; j < kNW; ++j) {
            const float x = s_seg[j * kC + lane];
            if (j < wave) base += x;
            all += x;
        }
        if (wave == 0) s_eg[lane] = exp_sum(all);
        float ep = exp_sum(base);
#pragma unroll
        for (int i = 0; i < kT; ++i) {
            const int t = wave * kT + i;
            base += G[i];
            const float ec = exp_sum(base), en = exp_sum(-base), u = k[i] * s_un[t];
            s_al[t * LD + lane] = ep * u;
            s_be[t * LD + lane] = en * a[i] * u;
            s_ka[t * LD + lane] = en * k[i];
            s_rh[t * LD + lane] = ec * r[i];
            ep = ec;
        }
        __syncthreads();
    };

    // the ten blocks at and below the diagonal of A, B, P and Q: five block products per wave
    {
        f32x4 acc[5];
        int mat[5], br[5], bc[5];
#pragma unroll
        for (int k = 0; k < 5; ++k) {
            acc[k] = zero4();
            const int item = wave * 5 + k, blk = item % 10;
            mat[k] = item / 10;
            br[k] = blk >= 6 ? 3 : blk >= 3 ? 2 : blk >= 1 ? 1 : 0;
            bc[k] = blk - br[k] * (br[k] + 1) / 2;
        }
        for (int d0 = 0; d0 < D16; d0 += kC) {
            load_slab(d0);
            const int steps = min(kC, D16 - d0) / 16;
            for (int s = 0; s < steps; ++s) {
#pragma unroll
                for (int k = 0; k < 5; ++k) {
                    const float* left = mat[k] < 2 ? s_al : s_rh;
                    const float* right = mat[k] & 1 ? s_ka : s_be;
                    acc[k] = mma4(ld4(&left[(16 * br[k] + c) * LD + 16 * s + 4 * g]),
                                  ld4(&right[(16 * bc[k] + c) * LD + 16 * s + 4 * g]), acc[k]);
                }
            }
        }
#pragma unroll
        for (int k = 0; k < 5; ++k) {
            float* dst = mat[k] == 0 ? s_A : mat[k] == 1 ? s_B : mat[k] == 2 ? s_P : s_Q;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * br[k] + 4 * g + i, cc = 16 * bc[k] + c;
                dst[r * LD + cc] = (cc < r || (mat[k] >= 2 && cc == r)) ? acc[k][i] : 0.f;
            }
        }
    }
    __syncthreads();
    auto t_at = [&](int r, int b) { return r == b ? 16 * r * LD + 16 * r : 16 * b * LD + 16 * r; };  // block (r, b) of T
    if (wave < 4) {  // diagonal block `wave`: column c of its inverse
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float r = i == c ? 1.f : 0.f;
#pragma unroll
            for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
                const float4 a = ld4(&s_A[(16 * wave + i) * LD + 16 * wave + 4 * j4]);
                r -= a.x * x[4 * j4];
                if (4 * j4 + 1 < i) r -= a.y * x[4 * j4 + 1];
                if (4 * j4 + 2 < i) r -= a.z * x[4 * j4 + 2];
                if (4 * j4 + 3 < i) r -= a.w * x[4 * j4 + 3];
            }
            x[i] = r;
        }
        if (g == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) s_A[(16 * wave + i) * LD + 16 * wave + c] = x[i];
        }
    }
#pragma unroll
    for (int lev = 1; lev < 4; ++lev) {
        __syncthreads();
        if (wave + lev < 4) {
            const int b = wave, r = wave + lev;
            f32x4 m = zero4(), tt = m;
            for (int k = b; k < r; ++k) {
                const float* tk = &s_A[t_at(k, b) + 4 * g * LD + c];
                m = mma4(ld4(&s_A[(16 * r + c) * LD + 16 * k + 4 * g]),
                         make_float4(tk[0], tk[LD], tk[2 * LD], tk[3 * LD]), m);
            }
            tt = mma4(ld4(&s_A[t_at(r, r) + c * LD + 4 * g]), as_float4(m), tt);
#pragma unroll
            for (int i = 0; i < 4; ++i) s_A[t_at(r, b) + (4 * g + i) * LD + c] = -tt[i];
        }
    }
    __syncthreads();

    // result block row r += lower block row r of a matrix times the right operand x
    auto lower = [&](const float* mtx, int r, const f32x4 (&x)[4], f32x4 acc) {
#pragma unroll
        for (int s = 0; s < 4; ++s)
            if (s <= r) acc = mma4(ld4(&mtx[(16 * r + c) * LD + 16 * s + 4 * g]), as_float4(x[s]), acc);
        return acc;
    };
    auto times_t = [&](const f32x4 (&x)[4], f32x4 (&y)[4]) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            y[r] = zero4();
#pragma unroll
            for (int s = 0; s < 4; ++s)
                if (s <= r) y[r] = mma4(ld4(&s_A[t_at(r, s) + c * LD + 4 * g]), as_float4(x[s]), y[r]);
        }
    };
    f32x4 W[TPW][4], U[TPW][4], V[TPW][4];
    int wt[TPW], vt[TPW];  // column tiles of this wave, >= nt: none
#pragma unroll
    for (int q = 0; q < TPW; ++q) {
        wt[q] = wave + kNW * q;
        vt[q] = (wave + kNW - nt % kNW) % kNW + kNW * q;
        if (vt[q] < nt) {
            const int cc = 16 * vt[q] + c;
            const T* src = in.proj + (int64_t)t0 * in.stride + 2 * HD + h * D + min(cc, D - 1);
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int t = 16 * s + 4 * g + j;
                    const float x = ld(src + (int64_t)min(t, n - 1) * in.stride);
                    V[q][s][j] = t < n && cc < D ? x : 0.f;
                }
            f32x4 bv[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) bv[r] = lower(s_B, r, V[q], zero4());
            times_t(bv, U[q]);
            float* dst = co.O + rec * kC * D16 + cc;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const f32x4 a = lower(s_Q, r, V[q], zero4()), b = lower(s_P, r, U[q], zero4());
#pragma unroll
                for (int i = 0; i < 4; ++i) dst[(int64_t)(16 * r + 4 * g + i) * D16] = a[i] - b[i];
            }
        }
    }
    const bool again = D16 > kC;
    for (int d0 = 0; d0 < D16; d0 += kC) {
        if (again) {
            __syncthreads();
            load_slab(d0);
        }
#pragma unroll
        for (int q = 0; q < TPW; ++q) {
            if (wt[q] >= nt || 16 * wt[q] < d0 || 16 * wt[q] >= d0 + kC) continue;
            const int col = 16 * wt[q] - d0 + c;
            f32x4 x[4];
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int j = 0; j < 4; ++j) x[s][j] = s_al[(16 * s + 4 * g + j) * LD + col];
            times_t(x, W[q]);
            float* dst = co.R + rec * kC * D16 + d0 + col;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const f32x4 pw = lower(s_P, r, W[q], zero4());
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = 16 * r + 4 * g + i;
                    dst[(int64_t)t * D16] = s_rh[t * LD + col] - pw[i];
                }
            }
        }
    }
    for (int d0 = 0; d0 < D16; d0 += kC) {
        if (again) {
            __syncthreads();
            load_slab(d0);
        }
        const int nb = min(kC, D16 - d0) / 16;
        for (int rb = 0; rb < nb; ++rb) {  // rows d0 + 16 rb .. of M and N
            // transposed left operands: channel 16 rb + c of tokens 16 s + 4 g ..
            float4 bt[4], kt[4];
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                const int at = (16 * s + 4 * g) * LD + 16 * rb + c;
                bt[s] = make_float4(s_be[at], s_be[at + LD], s_be[at + 2 * LD], s_be[at + 3 * LD]);
                kt[s] = make_float4(s_ka[at], s_ka[at + LD], s_ka[at + 2 * LD], s_ka[at + 3 * LD]);
            }
            const float4 eg = make_float4(s_eg[16 * rb + 4 * g], s_eg[16 * rb + 4 * g + 1], s_eg[16 * rb + 4 * g + 2],
                                          s_eg[16 * rb + 4 * g + 3]);
            const int dr = d0 + 16 * rb + 4 * g;
#pragma unroll
            for (int q = 0; q < TPW; ++q) {
                if (wt[q] < nt) {
                    f32x4 m = zero4();
#pragma unroll
                    for (int s = 0; s < 4; ++s) m = mma4(bt[s], as_float4(W[q][s]), m);
                    const int cc = 16 * wt[q] + c;
                    float* dst = co.M + (rec * D16 + dr) * D16 + cc;
                    dst[0] = eg.x * ((cc == dr ? 1.f : 0.f) - m[0]);
                    dst[D16] = eg.y * ((cc == dr + 1 ? 1.f : 0.f) - m[1]);
                    dst[2 * D16] = eg.z * ((cc == dr + 2 ? 1.f : 0.f) - m[2]);
                    dst[3 * D16] = eg.w * ((cc == dr + 3 ? 1.f : 0.f) - m[3]);
                }
                if (vt[q] < nt) {
                    f32x4 a = zero4(), b = a;
#pragma unroll
                    for (int s = 0; s < 4; ++s) {
                        a = mma4(kt[s], as_float4(V[q][s]), a);
                        b = mma4(bt[s], as_float4(U[q][s]), b);
                    }
                    st4(co.N + (rec * D16 + 16 * vt[q] + c) * D16 + dr,
                        make_float4(eg.x * (a[0] - b[0]), eg.y * (a[1] - b[1]), eg.z * (a[2] - b[2]), eg.w * (a[3] - b[3])));
                }
            }
        }
    }
}

struct SeqRef {
    const int32_t* chunk;  // [nchunks, 4]: first token, tokens, sequence, 0
    const int32_t* cu;
    const int32_t* rows;
    const int64_t* positions;
};

// One workgroup per (sequence, head, 16 columns of S), four waves. NS: 16-wide steps of dim at most; DT 16-row tiles of
// S per wave; PF chunks of M and N in flight. `first` holds every chunk's first state, transposed [value][key].
template <int NS, int PF>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void gdelta_chain_kernel(
    Dims d, SeqRef sq, const int32_t* __restrict__ seq_chunks, int seq0, int nseq, const float* __restrict__ M,
    const float* __restrict__ N, float* __restrict__ state, float* __restrict__ first) {
    constexpr int LS = NS * 16 + 4, DT = (NS + 3) / 4;
    __shared__ __attribute__((aligned(16))) float s_s[2][16 * LS];  // S^T slice
    const int D16 = d.d16(), VP = d.vpad(), nt = D16 / 16, ns = nt;
    // the slices of one (sequence, head) read the same M: consecutive on one XCD
    const int xcd = blockIdx.x % 8, slot = blockIdx.x / 8, grp = slot / nt * 8 + xcd;
    if (grp >= nseq * d.H) return;
    const int vt = slot % nt, h = grp % d.H, si = grp / d.H;
    const int seq = seq0 + si, row = sq.rows[seq];
    if (row < 0) return;
    const bool fresh = sq.positions[sq.cu[seq]] == 0;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4, vcol = 16 * vt + c;
    float* st_ = state + ((int64_t)row * d.H + h) * d.D * VP;
    f32x4 S[DT];  // rows 16 (wave + 4 k) + 4 g + i, column c
#pragma unroll
    for (int k = 0; k < DT; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int dd = 16 * (wave + 4 * k) + 4 * g + i;
            S[k][i] = (!fresh && dd < d.D && vcol < VP) ? st_[(int64_t)dd * VP + vcol] : 0.f;
        }
    const int c0 = seq_chunks[si], c1 = seq_chunks[si + 1];
    float4 m[PF][DT][NS], nn[PF][DT];
    auto fetch = [&](int ci, float4 (&mm)[DT][NS], float4 (&nv)[DT]) {
        const int64_t at = ((int64_t)min(ci, c1 - 1) * d.H + h) * D16 * D16;
#pragma unroll
        for (int k = 0; k < DT; ++k) {
            const int tile = min(wave + 4 * k, ns - 1);
            nv[k] = ld4(N + at + (int64_t)vcol * D16 + 16 * tile + 4 * g);
#pragma unroll
            for (int s = 0; s < NS; ++s) mm[k][s] = ld4(M + at + (int64_t)(16 * tile + c) * D16 + 16 * min(s, ns - 1) + 4 * g);
        }
    };
    if (c0 < c1)
#pragma unroll
        for (int p = 0; p < PF; ++p) fetch(c0 + p, m[p], nn[p]);
    for (int cb = c0; cb < c1; cb += PF) {
#pragma unroll
        for (int p = 0; p < PF; ++p) {
            const int ci = cb + p;
            if (ci >= c1) continue;
            float* buf = s_s[(ci - c0) & 1];
            float* fp = first + (((int64_t)ci * d.H + h) * D16 + vcol) * D16;
#pragma unroll
            for (int k = 0; k < DT; ++k) {
                const int tile = wave + 4 * k;
                if (tile < ns) {
                    *reinterpret_cast<f32x4*>(&buf[c * LS + 16 * tile + 4 * g]) = S[k];
                    *reinterpret_cast<f32x4*>(fp + 16 * tile + 4 * g) = S[k];
                }
            }
            __syncthreads();  // the other half is still read by waves that lag: it is written after the next barrier
            float4 b[NS];
#pragma unroll
            for (int s = 0; s < NS; ++s)
                if (s < ns) b[s] = ld4(&buf[c * LS + 16 * s + 4 * g]);
#pragma unroll
            for (int k = 0; k < DT; ++k) {
                f32x4 lo = {nn[p][k].x, nn[p][k].y, nn[p][k].z, nn[p][k].w}, hi = zero4();
#pragma unroll
                for (int s = 0; s < NS; ++s)
                    if (s < ns) {
                        if (s & 1) hi = mma4(m[p][k][s], b[s], hi);
                        else lo = mma4(m[p][k][s], b[s], lo);
                    }
                S[k] = lo + hi;
            }
            fetch(ci + PF, m[p], nn[p]);
        }
    }
#pragma unroll
    for (int k = 0; k < DT; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int dd = 16 * (wave + 4 * k) + 4 * g + i;
            if (dd < d.D && vcol < VP) st_[(int64_t)dd * VP + vcol] = vcol < d.D ? S[k][i] : 0.f;
        }
}

// O = R S + O0 of one (chunk, head), head norm, weight and output gate; a wave takes 16 tokens. NS: 16-wide steps of
// dim at most.
template <typename T, int NS>
__global__ __launch_bounds__(256) void gdelta_out_kernel(Dims d, const int32_t* __restrict__ chunk,
                                                         const float* __restrict__ R, const float* __restrict__ O0,
                                                         const float* __restrict__ first, const T* __restrict__ gate,
                                                         int64_t gate_stride, const T* __restrict__ norm_w,
                                                         T* __restrict__ out, int64_t out_stride) {
    const int h = blockIdx.x % d.H, ci = blockIdx.x / d.H;
    const int t0 = chunk[4 * ci], n = chunk[4 * ci + 1];
    const int D = d.D, D16 = d.d16(), ns = D16 / 16;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (16 * wave >= n) return;
    const int c = lane & 15, g = lane >> 4;
    const int64_t rec = (int64_t)ci * d.H + h;
    f32x4 o[NS];
#pragma unroll
    for (int v = 0; v < NS; ++v) {
        o[v] = zero4();
        if (v < ns)
#pragma unroll
            for (int i = 0; i < 4; ++i) o[v][i] = O0[(rec * kC + 16 * wave + 4 * g + i) * D16 + 16 * v + c];
    }
    const float* rp = R + (rec * kC + 16 * wave + c) * D16 + 4 * g;
    const float* sp = first + (rec * D16 + c) * D16 + 4 * g;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
        if (s >= ns) continue;
        const float4 r = ld4(rp + 16 * s);
#pragma unroll
        for (int v = 0; v < NS; ++v)
            if (v < ns) o[v] = mma4(r, ld4(sp + (int64_t)16 * v * D16 + 16 * s), o[v]);
    }
    float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < NS; ++v)
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (v < ns && 16 * v + c < D) ss[i] += o[v][i] * o[v][i];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int q = 1; q < 16; q <<= 1) ss[i] += __shfl_xor(ss[i], q, kWave);
        ss[i] = 1.f / sqrtf(ss[i] / (float)D + d.eps);
    }
#pragma unroll
    for (int v = 0; v < NS; ++v) {
        const int col = 16 * v + c;
        if (v >= ns || col >= D) continue;
        const float w = ld(norm_w + h * D + col);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * g + i;
            if (t < n) {
                const float gt = ld(gate + (int64_t)(t0 + t) * gate_stride + h * D + col);
                st(out + (int64_t)(t0 + t) * out_stride + h * D + col, o[v][i] * ss[i] * w * sigmoid_<T>(gt));
            }
        }
    }
}

const char* bad_shape(const skyrl_gdelta_shape* sh) {
    if (!sh) return "gdelta: null shape";
    if (sh->heads <= 0 || sh->heads > 65535) return "gdelta: heads must be in [1, 65535]";
    if (sh->dim <= 0 || sh->dim > 256) return "gdelta: dim must be in [1, 256]";
    return nullptr;
}
Dims dims_of(const skyrl_gdelta_shape* sh) { return Dims{sh->heads, sh->dim, sh->eps}; }

}  // namespace
}  // namespace skyrl

using namespace skyrl;

#define LAUNCH_SCAN(NT, R)                                                                                         \
    hipLaunchKernelGGL((gdelta_scan_kernel<T, NT, R>), dim3(d.H, nseq), dim3(NT), lds(NT), as_stream(stream), d,   \
                       (In<T>{reinterpret_cast<const T*>(proj), proj_stride, reinterpret_cast<const T*>(wl),       \
                              wl_stride, w0, a_bias}),                                                             \
                       reinterpret_cast<const T*>(norm_w), cu, rows, positions, state, reinterpret_cast<T*>(out), out_stride)

extern "C" int skyrl_gdelta_scan(const skyrl_gdelta_shape* shape, const void* proj, int64_t proj_stride, const void* wl,
                                 int64_t wl_stride, const float* w0, const float* a_bias, const void* norm_w,
                                 const int32_t* cu, const int32_t* rows, const int64_t* positions, int32_t nseq,
                                 float* state, void* out, int64_t out_stride, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gdelta_scan");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nseq >= 0 && nseq <= 65535, "gdelta_scan: nseq must be in [0, 65535]");
    SKYRL_REQUIRE(proj_stride >= 5 * (int64_t)d.width() && wl_stride >= d.width() && out_stride >= d.width(),
                  "gdelta_scan: strides");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && wl && w0 && a_bias && norm_w && cu && rows && positions && state && out,
                  "gdelta_scan: null pointer");
    auto lds = [&](int nt) {  // records: a wave's, or a row group's where columns do not fold in a wave
        const int VP = d.vpad(), NC = VP / 4, nw = nt / kWave;
        const bool fold = NC <= kWave && (NC & (NC - 1)) == 0;
        return (size_t)(5 * VP + 4 * nw + 2 * VP * (fold ? nw : nt / NC)) * sizeof(float);
    };
    SKYRL_DISPATCH_T(dtype, {
        if (d.D <= 32) LAUNCH_SCAN(64, 8);         // 8 column groups or fewer: 8 row groups or more, 4 rows each or fewer
        else if (d.D <= 64) LAUNCH_SCAN(64, 16);   // 16: 4, 16 rows
        else if (d.D <= 128) LAUNCH_SCAN(512, 8);  // 32: 16, 8 rows
        else LAUNCH_SCAN(1024, 16);                // 64: 16, 16 rows
    })
    return check_launch("gdelta_scan_kernel");
}

extern "C" int skyrl_gdelta_chunk(const skyrl_gdelta_shape* shape, const void* proj, int64_t proj_stride, const void* wl,
                                  int64_t wl_stride, const float* w0, const float* a_bias, const int32_t* chunk,
                                  int32_t nchunks, float* M, float* N, float* R, float* O, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gdelta_chunk");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nchunks >= 0 && (int64_t)nchunks * d.H < (1 << 30), "gdelta_chunk: bad sizes");
    SKYRL_REQUIRE(proj_stride >= 5 * (int64_t)d.width() && wl_stride >= d.width(), "gdelta_chunk: strides");
    if (nchunks == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && wl && w0 && a_bias && chunk && M && N && R && O, "gdelta_chunk: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const In<T> in{reinterpret_cast<const T*>(proj), proj_stride, reinterpret_cast<const T*>(wl), wl_stride, w0, a_bias};
        const ChunkOut co{M, N, R, O};
        if (d.D <= 128)
            hipLaunchKernelGGL((gdelta_chunk_kernel<T, 1>), dim3(nchunks * d.H), dim3(kNW * kWave), 0, as_stream(stream), d,
                               in, chunk, co);
        else
            hipLaunchKernelGGL((gdelta_chunk_kernel<T, 2>), dim3(nchunks * d.H), dim3(kNW * kWave), 0, as_stream(stream), d,
                               in, chunk, co);
    })
    return check_launch("gdelta_chunk_kernel");
}

#define LAUNCH_CHAIN(NS, PF)                                                                                      \
    hipLaunchKernelGGL((gdelta_chain_kernel<NS, PF>), dim3((unsigned)(nseq * d.H + 7) / 8 * 8 * (d.d16() / 16)),  \
                       dim3(256), 0, as_stream(stream), d, SeqRef{chunk, cu, rows, positions}, seq_chunks, seq0,  \
                       nseq, M, N, state, first)

extern "C" int skyrl_gdelta_chain(const skyrl_gdelta_shape* shape, const int32_t* chunk, const int32_t* seq_chunks,
                                  int32_t seq0, int32_t nseq, const int32_t* cu, const int32_t* rows,
                                  const int64_t* positions, const float* M, const float* N, float* state, float* first,
                                  void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nseq >= 0 && seq0 >= 0 && (int64_t)nseq * d.H * (d.d16() / 16) < (1 << 30), "gdelta_chain: bad sizes");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(chunk && seq_chunks && cu && rows && positions && M && N && state && first, "gdelta_chain: null pointer");
    if (d.D <= 64) LAUNCH_CHAIN(4, 4);
    else if (d.D <= 128) LAUNCH_CHAIN(8, 2);
    else LAUNCH_CHAIN(16, 1);
    return check_launch("gdelta_chain_kernel");
}

extern "C" int skyrl_gdelta_out(const skyrl_gdelta_shape* shape, const int32_t* chunk, int32_t nchunks, const float* R,
                                const float* O, const float* first, const void* gate, int64_t gate_stride,
                                const void* norm_w, void* out, int64_t out_stride, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gdelta_out");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nchunks >= 0 && (int64_t)nchunks * d.H < (1 << 30) && gate_stride >= d.width() && out_stride >= d.width(),
                  "gdelta_out: bad sizes");
    if (nchunks == 0) return SKYRL_OK;
    SKYRL_REQUIRE(chunk && R && O && first && gate && norm_w && out, "gdelta_out: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const T* gt = reinterpret_cast<const T*>(gate);
        const T* w = reinterpret_cast<const T*>(norm_w);
        T* o = reinterpret_cast<T*>(out);
        const dim3 grid(nchunks * d.H), block(256);
        if (d.D <= 64)
            hipLaunchKernelGGL((gdelta_out_kernel<T, 4>), grid, block, 0, as_stream(stream), d, chunk, R, O, first, gt,
                               gate_stride, w, o, out_stride);
        else if (d.D <= 128)
            hipLaunchKernelGGL((gdelta_out_kernel<T, 8>), grid, block, 0, as_stream(stream), d, chunk, R, O, first, gt,
                               gate_stride, w, o, out_stride);
        else
            hipLaunchKernelGGL((gdelta_out_kernel<T, 16>), grid, block, 0, as_stream(stream), d, chunk, R, O, first, gt,
                               gate_stride, w, o, out_stride);
    })
    return check_launch("gdelta_out_kernel");
}
