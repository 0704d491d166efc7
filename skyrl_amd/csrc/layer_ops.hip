// Embedding, norms, activations, convolution state and the logit cap of the hybrid decoders
// (include/skyrl_layers.h). The residual stream stays f32 in HBM: the add, the norm and the optional
// per-pass step vector of a looped layer stack are one pass over a row.
#include "conv.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;

// One block per row, the row in registers: kMaxV groups of VEC elements per thread.
template <typename T, int VEC, int kMaxV>
__global__ __launch_bounds__(kNT) void add_norm_kernel(const T* __restrict__ delta, float* __restrict__ h,
                                                       const T* __restrict__ step, const T* __restrict__ w,
                                                       float w_base, int H, float eps, int kind,
                                                       T* __restrict__ out) {
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
                st4(out + base + 4 * v, make_float4(x[k][0] * r * (w_base + a.x), x[k][1] * r * (w_base + a.y),
                                                    x[k][2] * r * (w_base + a.z), x[k][3] * r * (w_base + a.w)));
            } else {
                st(out + base + v, x[k][0] * r * (w_base + ld(w + v)));
            }
        }
    }
}

// Norms of sublayer outputs added to the residual. Up to two outputs per row; the row in registers: kMaxV
// groups of VEC elements per thread.
template <typename T>
struct NormAdd {
    const T *a, *wa, *b, *wb;  // b, wa, wb: only with two outputs
    float share;
    float* h;
    const T* g;
    int gs;  // 0: g is one number, 1: a vector
    const T* gf;
    int fs;
    T* out;
    int H;
    float eps;
};

template <typename T, int VEC>
__device__ __forceinline__ void ldw(const T* p, float (&o)[VEC]) {
    if constexpr (VEC == 4) {
        const float4 v = ld4(p);
        o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
    } else {
        o[0] = ld(p);
    }
}
template <typename T, int VEC>
__device__ __forceinline__ void stw(T* p, const float (&v)[VEC]) {
    if constexpr (VEC == 4) st4(p, make_float4(v[0], v[1], v[2], v[3]));
    else st(p, v[0]);
}
// A weight's VEC values at element e: a vector's, or one number.
template <typename T, int VEC>
__device__ __forceinline__ void weights_at(const T* w, int step, int e, float (&o)[VEC]) {
    if (step) {
        ldw<T, VEC>(w + e, o);
    } else {
        const float x = ld(w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] = x;
    }
}

template <typename T, int VEC, int kMaxV, bool PAIR>
__global__ __launch_bounds__(kNT) void norm_add_kernel(NormAdd<T> p) {
    __shared__ float s_red[kNT / kWave];
    const int64_t base = (int64_t)blockIdx.x * p.H;
    const int nv = p.H / VEC;
    float a[kMaxV][VEC], b[PAIR ? kMaxV : 1][VEC], h[kMaxV][VEC];
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * kNT;
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            a[k][j] = h[k][j] = 0.f;
            if constexpr (PAIR) b[k][j] = 0.f;
        }
        if (v < nv) {
            ldw<T, VEC>(p.a + base + VEC * v, a[k]);
            if constexpr (PAIR) ldw<T, VEC>(p.b + base + VEC * v, b[k]);
            ldw<float, VEC>(p.h + base + VEC * v, h[k]);
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            sa += a[k][j] * a[k][j];
            if constexpr (PAIR) sb += b[k][j] * b[k][j];
        }
    }
    float r = 1.f / sqrtf(block_total<kNT>(sa, s_red) / (float)p.H + p.eps);
    if constexpr (PAIR) {
        const float rb = 1.f / sqrtf(block_total<kNT>(sb, s_red) / (float)p.H + p.eps);
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < kMaxV; ++k) {
            const int v = threadIdx.x + k * kNT;
            if (v < nv) {
                float wa[VEC], wb[VEC];
                ldw<T, VEC>(p.wa + VEC * v, wa);
                ldw<T, VEC>(p.wb + VEC * v, wb);
#pragma unroll
                for (int j = 0; j < VEC; ++j) {
                    a[k][j] = p.share * (a[k][j] * r * wa[j] + b[k][j] * rb * wb[j]);
                    ss += a[k][j] * a[k][j];
                }
            }
        }
        r = 1.f / sqrtf(block_total<kNT>(ss, s_red) / (float)p.H + p.eps);
    }
    float sh = 0.f;
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * kNT;
        if (v < nv) {
            float g[VEC];
            weights_at<T, VEC>(p.g, p.gs, VEC * v, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                h[k][j] += a[k][j] * r * g[j];
                sh += h[k][j] * h[k][j];
            }
            stw<float, VEC>(p.h + base + VEC * v, h[k]);
        }
    }
    float rf = 1.f;
    if (p.gf) rf = 1.f / sqrtf(block_total<kNT>(sh, s_red) / (float)p.H + p.eps);
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * kNT;
        if (v < nv) {
            if (p.gf) {
                float g[VEC];
                weights_at<T, VEC>(p.gf, p.fs, VEC * v, g);
#pragma unroll
                for (int j = 0; j < VEC; ++j) h[k][j] *= rf * g[j];
            }
            stw<T, VEC>(p.out + base + VEC * v, h[k]);
        }
    }
}

struct Gate {
    int act;
    float alpha, limit;  // of the clamped form
};

// The gated product of one pair.
__device__ __forceinline__ float gated(float g, float u, const Gate& f) {
    if (f.act == SKYRL_ACT_SILU) return siluf_(g) * u;
    if (f.act == SKYRL_ACT_CLAMPED) {
        g = fminf(g, f.limit);
        u = fminf(fmaxf(u, -f.limit), f.limit);
        return g / (1.f + expf(-f.alpha * g)) * (u + 1.f);
    }
    return 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
}

template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void gate_mul_kernel(const T* __restrict__ gu, int64_t gu_stride, int64_t n, int I,
                                                       Gate f, T* __restrict__ out, int64_t out_stride) {
    const int iv = I / VEC;
    const int64_t total = n * iv;
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < total; e += (int64_t)gridDim.x * kNT) {
        const int64_t row = e / iv;
        const int c = (int)(e - row * iv) * VEC;
        const T* g = gu + row * gu_stride + c;
        if constexpr (VEC == 4) {
            const float4 a = ld4(g), b = ld4(g + I);
            st4(out + row * out_stride + c,
                make_float4(gated(a.x, b.x, f), gated(a.y, b.y, f), gated(a.z, b.z, f), gated(a.w, b.w, f)));
        } else {
            st(out + row * out_stride + c, gated(ld(g), ld(g + I), f));
        }
    }
}

// xIELU with the learned pair (p, q): ap = softplus(p), an = 1/2 + softplus(q).
template <typename T>
__device__ __forceinline__ float xielu(float z, float ap, float an) {
    const float zn = fminf(z, 0.f);
    float em;
    if constexpr (sizeof(T) == 2) em = exp_<T>(zn) - 1.f;
    else em = expm1f(zn);
    return (z > 0.f ? ap * z * z : an * (em - zn)) + 0.5f * z;
}

template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void xielu_kernel(const T* __restrict__ x, int64_t stride, int64_t n, int I,
                                                    const T* __restrict__ pq, T* __restrict__ out,
                                                    int64_t out_stride) {
    const float ap = softplusf_(ld(pq)), an = 0.5f + softplusf_(ld(pq + 1));
    const int iv = I / VEC;
    const int64_t total = n * iv;
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < total; e += (int64_t)gridDim.x * kNT) {
        const int64_t row = e / iv;
        const int c = (int)(e - row * iv) * VEC;
        float v[VEC];
        ldv<T, VEC>(x + row * stride + c, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = xielu<T>(v[j], ap, an);
        stv(out + row * out_stride + c, v);
    }
}

// Sine and cosine of pos * turns revolutions: the revolution's fraction is formed in f64.
__device__ __forceinline__ void position_pair(int64_t pos, double turns, float& s, float& c) {
    const double x = (double)pos * turns;
    sincospif(2.f * (float)(x - rint(x)), &s, &c);
}

// out[row] = scale * table[tokens[row]] (+ the position's vector), f32; x the same as T.
template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void embed_kernel(const int64_t* __restrict__ tokens, const T* __restrict__ table,
                                                    int64_t n, int H, float scale,
                                                    const int64_t* __restrict__ positions,
                                                    const double* __restrict__ turns, float* __restrict__ out,
                                                    T* __restrict__ x) {
    const int hv = H / VEC;
    const int64_t total = n * hv;
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < total; e += (int64_t)gridDim.x * kNT) {
        const int64_t row = e / hv;
        const int c = (int)(e - row * hv) * VEC;
        const T* src = table + tokens[row] * H + c;
        if constexpr (VEC == 4) {
            const float4 a = ld4(src);
            float4 v = make_float4(a.x * scale, a.y * scale, a.z * scale, a.w * scale);
            if (turns) {
                const int64_t pos = positions[row];
                float s, k;
                position_pair(pos, turns[c / 2], s, k);
                v.x += s;
                v.y += k;
                position_pair(pos, turns[c / 2 + 1], s, k);
                v.z += s;
                v.w += k;
            }
            st4(out + row * H + c, v);
            if (x) st4(x + row * H + c, v);
        } else {
            float v = ld(src) * scale;
            if (turns) {
                float s, k;
                position_pair(positions[row], turns[c / 2], s, k);
                v += c & 1 ? k : s;
            }
            out[row * H + c] = v;
            if (x) st(x + row * H + c, v);
        }
    }
}

// The last inputs of every sequence's convolutions into its ring. grid (channels / kNT, sequences).
template <typename T>
__global__ __launch_bounds__(kNT) void conv_save_kernel(const T* __restrict__ x, int64_t stride, int channels, int taps,
                                                        const int32_t* __restrict__ cu,
                                                        const int32_t* __restrict__ rows,
                                                        const int64_t* __restrict__ positions, T* __restrict__ ring) {
    const int s = blockIdx.y, row = rows[s];
    if (row < 0) return;
    const int t0 = cu[s], t1 = cu[s + 1];
    const int ch = blockIdx.x * kNT + threadIdx.x;
    if (ch >= channels || t0 >= t1) return;
    const int64_t pos0 = positions[t0];
    for (int t = max(t0, t1 - taps); t < t1; ++t)
        ring[((int64_t)row * taps + (pos0 + t - t0) % taps) * channels + ch] = x[(int64_t)t * stride + ch];
}

template <typename T>
__global__ __launch_bounds__(kNT) void softcap_kernel(const T* __restrict__ x, float* __restrict__ out, int64_t n,
                                                      float cap) {
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < n; e += (int64_t)gridDim.x * kNT) {
        const float v = ld(x + e);
        out[e] = cap > 0.f ? cap * tanhf(v / cap) : v;
    }
}

// ---- out = rms over each of `groups` equal parts of y silu(z), times w; one workgroup per (token, part) ----
// Up to kMax groups of VEC values per thread in registers; HOLD false: any length, formed twice.
template <typename T, int NT, int VEC, int kMax, bool HOLD>
__global__ __launch_bounds__(NT) void gated_norm_kernel(const T* __restrict__ y, int64_t y_stride,
                                                        const T* __restrict__ z, int64_t z_stride,
                                                        const T* __restrict__ w, int groups, int len, float eps,
                                                        T* __restrict__ out, int64_t out_stride) {
    __shared__ float s_red[NT / kWave];
    const int64_t t = blockIdx.x / groups;
    const int c0 = (int)(blockIdx.x % groups) * len, nv = len / VEC;
    const T* yp = y + t * y_stride + c0;
    const T* zp = z + t * z_stride + c0;
    float a[HOLD ? kMax : 1][VEC];
    auto form = [&](int v, float (&o)[VEC]) {
        float zz[VEC];
        ldv<T, VEC>(yp + VEC * v, o);
        ldv<T, VEC>(zp + VEC * v, zz);
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] *= zz[j] * sigmoid_<T>(zz[j]);
    };
    float ss = 0.f;
    if constexpr (HOLD) {
#pragma unroll
        for (int k = 0; k < kMax; ++k) {
            const int v = threadIdx.x + k * NT;
            if (v < nv) {
                form(v, a[k]);
#pragma unroll
                for (int j = 0; j < VEC; ++j) ss += a[k][j] * a[k][j];
            }
        }
    } else {
        for (int v = threadIdx.x; v < nv; v += NT) {
            form(v, a[0]);
#pragma unroll
            for (int j = 0; j < VEC; ++j) ss += a[0][j] * a[0][j];
        }
    }
    const float r = 1.f / sqrtf(block_total<NT>(ss, s_red) / (float)len + eps);
    auto put = [&](int v, float (&o)[VEC]) {
        float ww[VEC];
        ldv<T, VEC>(w + c0 + VEC * v, ww);
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] *= r * ww[j];
        stv(out + t * out_stride + c0 + VEC * v, o);
    };
    if constexpr (HOLD) {
#pragma unroll
        for (int k = 0; k < kMax; ++k) {
            const int v = threadIdx.x + k * NT;
            if (v < nv) put(v, a[k]);
        }
    } else {
        for (int v = threadIdx.x; v < nv; v += NT) {
            form(v, a[0]);
            put(v, a[0]);
        }
    }
}

// ---- a sublayer's result between two norms in equal parts: gated, normed, added to the residual, normed again ----
template <typename T>
struct GateNormAdd {
    const T* a;
    const int64_t* rows;  // row of a (NULL: the output's own)
    int parts;            // consecutive rows of a that are summed
    const T* z;           // gate logits (NULL: no gate) and their bias
    int64_t z_stride;
    const float* zb;
    const T* w;
    int groups;
    float eps, mult;
    float* h;
    int fresh;  // the residual starts at 0
    const T* wn;
    T* out;
    int H;
};

// One block per row, the row in registers: chunks of VEC elements, chunk threadIdx + k NT, each in one group of `per`
// chunks. A group's sum: within L lanes (the power of two in per, at most a wave) by shuffles, then over per / L numbers
// in LDS. PARTS: rows that are summed (0: any number).
template <typename T, int NT, int VEC, int kMaxV, int PARTS>
__global__ __launch_bounds__(NT) void gate_norm_add_kernel(GateNormAdd<T> p, int L) {
    extern __shared__ float s_p[];
    __shared__ float s_red[NT / kWave];
    const int nv = p.H / VEC, per = nv / p.groups, sums = per / L;
    const int64_t base = (int64_t)blockIdx.x * p.H;
    const int64_t row = p.rows ? p.rows[blockIdx.x] : blockIdx.x;
    const float len = (float)(p.H / p.groups);
    const int parts = PARTS ? PARTS : p.parts;
    float y[kMaxV][VEC], h[kMaxV][VEC], r[kMaxV];
    // r: 1 / root mean square of every chunk's group, from the chunks' sums of squares
    auto scales = [&]() {
        if (p.groups == 1) {
            float one = 0.f;
#pragma unroll
            for (int k = 0; k < kMaxV; ++k) one += r[k];
            one = 1.f / sqrtf(block_total<NT>(one, s_red) / len + p.eps);
#pragma unroll
            for (int k = 0; k < kMaxV; ++k) r[k] = one;
            return;
        }
#pragma unroll
        for (int k = 0; k < kMaxV; ++k)
            for (int o = 1; o < L; o <<= 1) r[k] += __shfl_xor(r[k], o, kWave);
        if (sums > 1) {
            __syncthreads();  // the sums before these are read
#pragma unroll
            for (int k = 0; k < kMaxV; ++k) {
                const int v = threadIdx.x + k * NT;
                if (v < nv && v % L == 0) s_p[v / L] = r[k];
            }
            __syncthreads();
#pragma unroll
            for (int k = 0; k < kMaxV; ++k) {
                const int v = threadIdx.x + k * NT;
                if (v >= nv) continue;
                const float* q = s_p + v / per * sums;
                float s = 0.f;
                for (int i = 0; i < sums; ++i) s += q[i];
                r[k] = s;
            }
        }
#pragma unroll
        for (int k = 0; k < kMaxV; ++k) r[k] = 1.f / sqrtf(r[k] / len + p.eps);
    };
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * NT;
        r[k] = 0.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[k][j] = h[k][j] = 0.f;
        if (v < nv) {
            const T* src = p.a + row * parts * p.H + VEC * v;
            ldv<T, VEC>(src, y[k]);
            if (!p.fresh) ldv<float, VEC>(p.h + base + VEC * v, h[k]);
            auto add = [&](int i) {
                float x[VEC];
                ldv<T, VEC>(src + (int64_t)i * p.H, x);
#pragma unroll
                for (int j = 0; j < VEC; ++j) y[k][j] += x[j];
            };
            if constexpr (PARTS > 0) {
#pragma unroll
                for (int i = 1; i < PARTS; ++i) add(i);
            } else {
                for (int i = 1; i < parts; ++i) add(i);
            }
            if (p.z) {
                float z[VEC], b[VEC];
                ldv<T, VEC>(p.z + blockIdx.x * p.z_stride + VEC * v, z);
                ldv<float, VEC>(p.zb + VEC * v, b);
#pragma unroll
                for (int j = 0; j < VEC; ++j) y[k][j] *= sigmoid_<T>(z[j] + b[j]);
            }
#pragma unroll
            for (int j = 0; j < VEC; ++j) r[k] += y[k][j] * y[k][j];
        }
    }
    scales();
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * NT;
        const float rk = r[k];
        r[k] = 0.f;
        if (v < nv) {
            float w[VEC];
            ldv<T, VEC>(p.w + VEC * v, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                h[k][j] += p.mult * (y[k][j] * rk * w[j]);
                r[k] += h[k][j] * h[k][j];
            }
            stv(p.h + base + VEC * v, h[k]);
        }
    }
    scales();
#pragma unroll
    for (int k = 0; k < kMaxV; ++k) {
        const int v = threadIdx.x + k * NT;
        if (v < nv) {
            float w[VEC];
            ldv<T, VEC>(p.wn + VEC * v, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) h[k][j] *= r[k] * w[j];
            stv(p.out + base + VEC * v, h[k]);
        }
    }
}

template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void tanh_kernel(const T* __restrict__ x, int64_t stride, int64_t n, int I,
                                                   T* __restrict__ out) {
    const int iv = I / VEC;
    const int64_t total = n * iv;
    for (int64_t e = (int64_t)blockIdx.x * kNT + threadIdx.x; e < total; e += (int64_t)gridDim.x * kNT) {
        const int64_t row = e / iv;
        const int c = (int)(e - row * iv) * VEC;
        float v[VEC];
        ldv<T, VEC>(x + row * stride + c, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = tanhf(v[j]);
        stv(out + row * I + c, v);
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
    hipLaunchKernelGGL((add_norm_kernel<T, V, K>), dim3(n), dim3(kNT), 0, s, d, hidden, st_, w, w_base, H, eps, \
                       kind, o)

extern "C" int skyrl_add_norm(const void* delta, float* hidden, const void* step, const void* weight, float w_base,
                              int32_t n, int32_t H, float eps, int32_t kind, void* out, int32_t dtype, void* stream) {
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

extern "C" int skyrl_gate_mul(const void* gate_up, int64_t gu_stride, int64_t n, int32_t I, int32_t act, float alpha,
                              float limit, void* out, int64_t out_stride, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gate_mul");
    SKYRL_REQUIRE(n >= 0 && I > 0 && gu_stride >= 2 * (int64_t)I && out_stride >= I, "gate_mul: bad sizes");
    SKYRL_REQUIRE(act == SKYRL_ACT_SILU || act == SKYRL_ACT_GELU_TANH || act == SKYRL_ACT_CLAMPED,
                  "gate_mul: unknown activation");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(gate_up && out, "gate_mul: null pointer");
    const Gate f{act, alpha, limit};
    SKYRL_DISPATCH_T(dtype, {
        const T* g = reinterpret_cast<const T*>(gate_up);
        T* o = reinterpret_cast<T*>(out);
        const uintptr_t mis = (reinterpret_cast<uintptr_t>(g) | reinterpret_cast<uintptr_t>(o)) & (4 * sizeof(T) - 1);
        if (I % 4 == 0 && gu_stride % 4 == 0 && out_stride % 4 == 0 && mis == 0)
            hipLaunchKernelGGL((gate_mul_kernel<T, 4>), dim3(grid_for(n * (I / 4))), dim3(kNT), 0, as_stream(stream),
                               g, gu_stride, n, I, f, o, out_stride);
        else
            hipLaunchKernelGGL((gate_mul_kernel<T, 1>), dim3(grid_for(n * I)), dim3(kNT), 0, as_stream(stream), g,
                               gu_stride, n, I, f, o, out_stride);
    })
    return check_launch("gate_mul_kernel");
}

extern "C" int skyrl_embed(const int64_t* tokens, const void* table, int64_t n, int32_t H, float scale,
                           const int64_t* positions, const double* turns, float* out, void* x, int32_t dtype,
                           void* stream) {
    SKYRL_REQUIRE_T(dtype, "embed");
    SKYRL_REQUIRE(n >= 0 && H > 0, "embed: bad sizes");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(tokens && table && out && (positions || !turns), "embed: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const T* w = reinterpret_cast<const T*>(table);
        T* xo = reinterpret_cast<T*>(x);
        if (H % 4 == 0)
            hipLaunchKernelGGL((embed_kernel<T, 4>), dim3(grid_for(n * (H / 4))), dim3(kNT), 0, as_stream(stream),
                               tokens, w, n, H, scale, positions, turns, out, xo);
        else
            hipLaunchKernelGGL((embed_kernel<T, 1>), dim3(grid_for(n * H)), dim3(kNT), 0, as_stream(stream), tokens, w,
                               n, H, scale, positions, turns, out, xo);
    })
    return check_launch("embed_kernel");
}

#define LAUNCH_NORM_ADD(V, K)                                                                                   if (b) hipLaunchKernelGGL((norm_add_kernel<T, V, K, true>), dim3(n), dim3(kNT), 0, as_stream(stream), p);     else hipLaunchKernelGGL((norm_add_kernel<T, V, K, false>), dim3(n), dim3(kNT), 0, as_stream(stream), p)

extern "C" int skyrl_norm_add(const void* a, const void* wa, const void* b, const void* wb, float share, float* hidden,
                              const void* weight, int32_t weight_n, const void* final_weight, int32_t final_n,
                              int32_t n, int32_t H, float eps, void* out, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "norm_add");
    SKYRL_REQUIRE(n >= 0 && H > 0 && H <= 8192, "norm_add: H must be in [1, 8192]");
    SKYRL_REQUIRE((weight_n == 1 || weight_n == H) && (!final_weight || final_n == 1 || final_n == H),
                  "norm_add: a weight has 1 or H values");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(a && hidden && weight && out && (!b || (wa && wb)), "norm_add: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        auto t = [](const void* q) { return reinterpret_cast<const T*>(q); };
        const NormAdd<T> p{t(a), t(wa), t(b), t(wb), share, hidden, t(weight), weight_n > 1, t(final_weight),
                           final_n > 1, reinterpret_cast<T*>(out), H, eps};
        if (H % 4 == 0) {
            if (H <= 4 * kNT) { LAUNCH_NORM_ADD(4, 1); }
            else if (H <= 8 * kNT) { LAUNCH_NORM_ADD(4, 2); }
            else if (H <= 16 * kNT) { LAUNCH_NORM_ADD(4, 4); }
            else { LAUNCH_NORM_ADD(4, 8); }
        } else {
            if (H <= 4 * kNT) { LAUNCH_NORM_ADD(1, 4); }
            else { LAUNCH_NORM_ADD(1, 32); }
        }
    })
    return check_launch("norm_add_kernel");
}

extern "C" int skyrl_xielu(const void* x, int64_t stride, int64_t n, int32_t I, const void* pq, void* out,
                           int64_t out_stride, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "xielu");
    SKYRL_REQUIRE(n >= 0 && I > 0 && stride >= I && out_stride >= I, "xielu: bad sizes");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && pq && out, "xielu: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const T* in = reinterpret_cast<const T*>(x);
        T* o = reinterpret_cast<T*>(out);
        const T* w = reinterpret_cast<const T*>(pq);
        if (I % 8 == 0 && stride % 8 == 0 && out_stride % 8 == 0 && aligned16(in) && aligned16(o))
            hipLaunchKernelGGL((xielu_kernel<T, 8>), dim3(grid_for(n * (I / 8))), dim3(kNT), 0, as_stream(stream), in,
                               stride, n, I, w, o, out_stride);
        else
            hipLaunchKernelGGL((xielu_kernel<T, 1>), dim3(grid_for(n * I)), dim3(kNT), 0, as_stream(stream), in,
                               stride, n, I, w, o, out_stride);
    })
    return check_launch("xielu_kernel");
}

#define LAUNCH_GNA_(NT, V, K, P) \
    hipLaunchKernelGGL((gate_norm_add_kernel<T, NT, V, K, P>), dim3(n), dim3(NT), lds, as_stream(stream), p, L)
#define LAUNCH_GNA(NT)                              \
    do {                                            \
        if (parts == 1) LAUNCH_GNA_(NT, 8, 1, 1);   \
        else if (parts == 2) LAUNCH_GNA_(NT, 8, 1, 2); \
        else if (parts == 4) LAUNCH_GNA_(NT, 8, 1, 4); \
        else if (parts == 8) LAUNCH_GNA_(NT, 8, 1, 8); \
        else LAUNCH_GNA_(NT, 8, 1, 0);              \
    } while (0)

extern "C" int skyrl_gate_norm_add(const void* a, const int64_t* rows, int32_t parts, const void* gate,
                                   int64_t gate_stride, const float* gate_bias, const void* weight, int32_t groups,
                                   float eps, float mult, float* hidden, int32_t fresh, const void* next, int32_t n,
                                   int32_t H, void* out, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gate_norm_add");
    SKYRL_REQUIRE(n >= 0 && H > 0 && H <= 8192 && parts > 0, "gate_norm_add: H must be in [1, 8192], parts positive");
    SKYRL_REQUIRE(groups > 0 && H % groups == 0, "gate_norm_add: H must be a multiple of groups");
    SKYRL_REQUIRE(!gate || (gate_bias && gate_stride >= H), "gate_norm_add: gate needs a bias and a stride >= H");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(a && weight && hidden && next && out, "gate_norm_add: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        auto t = [](const void* q) { return reinterpret_cast<const T*>(q); };
        const GateNormAdd<T> p{t(a), rows, parts, t(gate), gate_stride, gate_bias, t(weight), groups, eps, mult, hidden,
                               fresh, t(next), reinterpret_cast<T*>(out), H};
        const bool wide = H / groups % 8 == 0 && (!gate || (gate_stride % 8 == 0 && aligned16(gate))) && aligned16(a) &&
                          aligned16(hidden) && aligned16(weight) && aligned16(next) && aligned16(out);
        const int V = wide ? 8 : 1;
        int L = 1;
        while (L < kWave && H / V / groups % (2 * L) == 0) L <<= 1;
        const size_t lds = groups > 1 ? (size_t)(H / V / L) * sizeof(float) : 0;
        if (wide) {
            if (H <= 8 * 256) LAUNCH_GNA(256);
            else if (H <= 8 * 512) LAUNCH_GNA(512);
            else LAUNCH_GNA(1024);
        } else {
            if (H <= 4 * kNT) LAUNCH_GNA_(kNT, 1, 4, 0);
            else LAUNCH_GNA_(kNT, 1, 32, 0);
        }
    })
    return check_launch("gate_norm_add_kernel");
}

extern "C" int skyrl_tanh(const void* x, int64_t stride, int64_t n, int32_t I, void* out, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "tanh");
    SKYRL_REQUIRE(n >= 0 && I > 0 && stride >= I, "tanh: bad sizes");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && out, "tanh: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        const T* in = reinterpret_cast<const T*>(x);
        T* o = reinterpret_cast<T*>(out);
        if (I % 8 == 0 && stride % 8 == 0 && aligned16(in) && aligned16(o))
            hipLaunchKernelGGL((tanh_kernel<T, 8>), dim3(grid_for(n * (I / 8))), dim3(kNT), 0, as_stream(stream), in,
                               stride, n, I, o);
        else
            hipLaunchKernelGGL((tanh_kernel<T, 1>), dim3(grid_for(n * I)), dim3(kNT), 0, as_stream(stream), in, stride, n,
                               I, o);
    })
    return check_launch("tanh_kernel");
}

extern "C" int skyrl_conv_save(const void* x, int64_t stride, int32_t channels, int32_t taps, const int32_t* cu,
                               const int32_t* rows, const int64_t* positions, int32_t nseq, void* ring, int32_t dtype,
                               void* stream) {
    SKYRL_REQUIRE_T(dtype, "conv_save");
    SKYRL_REQUIRE(channels > 0 && taps > 0 && stride >= channels && nseq >= 0 && nseq <= 65535, "conv_save: bad sizes");
    if (nseq == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && cu && rows && positions && ring, "conv_save: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((conv_save_kernel<T>), dim3((channels + kNT - 1) / kNT, nseq), dim3(kNT), 0,
                           as_stream(stream), reinterpret_cast<const T*>(x), stride, channels, taps, cu, rows,
                           positions, reinterpret_cast<T*>(ring));
    })
    return check_launch("conv_save_kernel");
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

#define LAUNCH_GNORM(NT, VEC, K, HOLD)                                                                               \
    hipLaunchKernelGGL((gated_norm_kernel<T, NT, VEC, K, HOLD>), dim3((unsigned)(n * groups)), dim3(NT), 0,          \
                       as_stream(stream), y_, y_stride, z_, z_stride, w_, groups, len, eps, o_, out_stride)

extern "C" int skyrl_gated_norm(const void* y, int64_t y_stride, const void* z, int64_t z_stride, const void* weight,
                                int64_t n, int32_t width, int32_t groups, float eps, void* out, int64_t out_stride,
                                int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "gated_norm");
    SKYRL_REQUIRE(n >= 0 && width > 0 && groups > 0 && width % groups == 0 && n * groups < (1ll << 31) &&
                      y_stride >= width && z_stride >= width && out_stride >= width,
                  "gated_norm: bad sizes");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(y && z && weight && out, "gated_norm: null pointer");
    const int len = width / groups;
    SKYRL_DISPATCH_T(dtype, {
        const T* y_ = reinterpret_cast<const T*>(y);
        const T* z_ = reinterpret_cast<const T*>(z);
        const T* w_ = reinterpret_cast<const T*>(weight);
        T* o_ = reinterpret_cast<T*>(out);
        const bool wide = len % 8 == 0 && y_stride % 8 == 0 && z_stride % 8 == 0 && out_stride % 8 == 0 &&
                          aligned16(y) && aligned16(z) && aligned16(weight) && aligned16(out);
        if (wide && len <= 512) LAUNCH_GNORM(64, 8, 1, true);
        else if (wide && len <= 2048) LAUNCH_GNORM(256, 8, 1, true);
        else if (wide && len <= 8192) LAUNCH_GNORM(256, 8, 4, true);
        else if (wide) LAUNCH_GNORM(256, 8, 1, false);
        else LAUNCH_GNORM(256, 1, 1, false);
    })
    return check_launch("gated_norm_kernel");
}
