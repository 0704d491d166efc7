// Gated delta rule: a recurrent layer with a [dim x vdim] matrix state per head
// (include/skyrl_layers.h has the equations and the tensor layouts).
//
// Token form (delta_scan): one workgroup per (sequence, head). The state is read once into registers,
// carried over the sequence's tokens and written once, so a decode step costs one read and one write
// of the state. Convolution, unit norms, gates, recurrence, output norm and output gate are one pass.
// Both products with the state are taken before the update, S^T k and S^T q, in one sweep:
// o = (g S + k u^T)^T q = g S^T q + (k . q) u.
#include "elem.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kMaxTaps = 64;

struct Dims {
    int H, K, D, V, taps;
    float eps;
    __host__ __device__ int vpad() const { return (V + 3) / 4 * 4; }
    __host__ __device__ int channels() const { return 2 * K * D + H * V; }
};

// silu(causal convolution) of channel ch at token t of a sequence whose first token is t0 at position p0;
// inputs before t0 come from the stored ones (the input of position p at p % taps).
template <typename T>
__device__ __forceinline__ float conv_silu(const T* __restrict__ proj, int64_t stride, const T* __restrict__ w,
                                           const T* __restrict__ ring, int channels, int taps, int ch, int t, int t0,
                                           int pos) {
    float y = 0.f;
    for (int j = 0; j < taps; ++j) {
        const int back = taps - 1 - j;
        const int p = pos - back;
        if (p < 0) continue;
        const int tt = t - back;
        const float x = tt >= t0 ? ld(proj + (int64_t)tt * stride + ch) : ld(ring + (int64_t)(p % taps) * channels + ch);
        y += x * ld(w + (int64_t)ch * taps + j);
    }
    return siluf_(y);
}

// RPT: state rows per thread. Thread (cg, rg) holds columns 4 cg .. 4 cg + 3 of rows rg, rg + RG, ...
template <typename T, int RPT>
__global__ __launch_bounds__(kNT) void delta_scan_kernel(Dims d, const T* __restrict__ proj, int64_t stride,
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
    const int D = d.D, V = d.V, VP = d.vpad(), NC = VP / 4, RG = kNT / NC;
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
    const float neg_rate = -expf(a_log[h]);
    const float qscale = 1.f / sqrtf((float)D);
    const int qoff = kh * D, koff = (d.K + kh) * D, voff = 2 * d.K * D + h * V;
    const int goff = ch_all + h * V, boff = ch_all + d.H * V + h, aoff = boff + d.H;
    for (int t = t0; t < t1; ++t) {
        const int pos = (int)pos0 + (t - t0);
        const T* p = proj + (int64_t)t * stride;
        for (int e = tid; e < 2 * D + VP; e += kNT) {
            float y = 0.f;
            if (e < 2 * D + V) {
                const int ch = e < D ? qoff + e : e < 2 * D ? koff + e - D : voff + e - 2 * D;
                y = conv_silu(proj, stride, conv_w, ring, ch_all, d.taps, ch, t, t0, pos);
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
        const float beta = sigmoidf_(ld(p + boff));
        const float g = expf(neg_rate * softplusf_(ld(p + aoff) + dt_bias[h]));
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
            st4(s_red + (rg * 2) * VP + 4 * cg, make_float4(a[0], a[1], a[2], a[3]));
            st4(s_red + (rg * 2 + 1) * VP + 4 * cg, make_float4(b[0], b[1], b[2], b[3]));
        }
        __syncthreads();
        if (act) {
            float4 A = make_float4(0.f, 0.f, 0.f, 0.f), B = A;
            for (int r = 0; r < RG; ++r) {
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
        if (wave == 0) {
            float x = 0.f;
            for (int i = lane; i < V; i += kWave) x += s_o[i] * s_o[i];
            x = wave_sum(x);
            const float r = 1.f / sqrtf(x / (float)V + d.eps);
            for (int i = lane; i < V; i += kWave)
                st(out + (int64_t)t * out_stride + h * V + i, s_o[i] * r * ld(norm_w + i) * siluf_(ld(p + goff + i)));
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
        for (int e = tid; e < V; e += kNT) dst[voff + e] = p[voff + e];
        if (h % (d.H / d.K) == 0)
            for (int e = tid; e < D; e += kNT) {
                dst[qoff + e] = p[qoff + e];
                dst[koff + e] = p[koff + e];
            }
    }
}

template <typename T>
__global__ __launch_bounds__(kNT) void delta_save_kernel(Dims d, const T* __restrict__ proj, int64_t stride,
                                                         const int32_t* __restrict__ cu,
                                                         const int32_t* __restrict__ rows,
                                                         const int64_t* __restrict__ positions,
                                                         T* __restrict__ conv_state) {
    const int s = blockIdx.y, row = rows[s];
    if (row < 0) return;
    const int t0 = cu[s], t1 = cu[s + 1];
    const int ch = blockIdx.x * kNT + threadIdx.x, n = d.channels();
    if (ch >= n || t0 >= t1) return;
    const int64_t pos0 = positions[t0];
    for (int t = max(t0, t1 - d.taps); t < t1; ++t)
        conv_state[((int64_t)row * d.taps + (pos0 + t - t0) % d.taps) * n + ch] = proj[(int64_t)t * stride + ch];
}

int scan_rows_per_thread(const Dims& d) {
    const int RG = kNT / (d.vpad() / 4);
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

#define LAUNCH_SCAN(R)                                                                                             \
    hipLaunchKernelGGL((delta_scan_kernel<T, R>), dim3(d.H, nseq), dim3(kNT), lds, as_stream(stream), d,           \
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
    const int RG = kNT / (d.vpad() / 4), rpt = scan_rows_per_thread(d);
    SKYRL_REQUIRE(rpt <= 64, "delta_scan: dim * vdim too large for one workgroup's registers (at most 65536)");
    const size_t lds = (size_t)(2 * d.D + 2 * d.vpad() + 2 * RG * d.vpad() + 4) * sizeof(float);
    SKYRL_DISPATCH_T(dtype, {
        if (rpt <= 4) LAUNCH_SCAN(4);
        else if (rpt <= 8) LAUNCH_SCAN(8);
        else if (rpt <= 16) LAUNCH_SCAN(16);
        else if (rpt <= 32) LAUNCH_SCAN(32);
        else LAUNCH_SCAN(64);
    })
    return check_launch("delta_scan_kernel");
}

extern "C" int skyrl_delta_save(const skyrl_delta_shape* shape, const void* proj, int64_t proj_stride,
                                const int32_t* cu, const int32_t* rows, const int64_t* positions, int32_t nseq,
                                void* conv_state, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "delta_save");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nseq >= 0 && nseq <= 65535 && proj_stride >= proj_width(d), "delta_save: bad sizes");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && cu && rows && positions && conv_state, "delta_save: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((delta_save_kernel<T>), dim3((d.channels() + kNT - 1) / kNT, nseq), dim3(kNT), 0,
                           as_stream(stream), d, reinterpret_cast<const T*>(proj), proj_stride, cu, rows, positions,
                           reinterpret_cast<T*>(conv_state));
    })
    return check_launch("delta_save_kernel");
}
