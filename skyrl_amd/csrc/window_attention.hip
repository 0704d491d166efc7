// Grouped attention over a paged key / value cache with normed queries and keys, a sliding window and an
// elementwise output gate (include/skyrl_layers.h has the equations and the tensor layouts).
//
// Write (attn_write): norms of q and k, queries to a padded buffer, keys and values into the pages. Eight
// channels per thread; prompts take runs of up to eight tokens, so that the transposed values leave as 16-byte
// pieces.
//
// Decode form (attn_attend): one wave per (share of the window, key / value head and group of 16 of its query
// heads, token). The query heads are the 16 columns of the matrix instructions and the exp'd scores are already
// the operand of O^T += V^T P^T. Shares of a split window are merged by attn_merge, which also applies the gate.
//
// Prompt form (attn_prefill): flash style, waves of 16 QT queries of one head share a tile of 64 keys and
// values in LDS, read straight from the pages, from the window's first tile to the diagonal. A running maximum
// is only raised when the scores outgrow it by kSlack.
#include "paged.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kGroup = 16;  // query heads per decode wave
constexpr int kRun = 8;     // tokens per run of the prompt's write
constexpr float kLow = -1e30f;  // a running maximum before any visible key

struct Dims {
    int H, G, D, V, window;
    float scale, eps;
    __host__ __device__ int dp() const { return (D + 31) / 32 * 32; }
    __host__ __device__ int vp() const { return (V + 15) / 16 * 16; }
    __host__ __device__ int R() const { return H / G; }
    __host__ __device__ int groups() const { return (R() + kGroup - 1) / kGroup; }
    __host__ __device__ int channels() const { return (H + G) * D + G * V; }
    // first position that pos sees
    __device__ int first(int pos) const { return window > 0 ? max(0, pos - window + 1) : 0; }
};

// Run r of the launch: given (first token, count of consecutive slots) or one token each.
struct Runs {
    const int32_t* runs;
    int first;
};

// bf16, dim and vdim multiples of 8. grid (runs, blocks): the first hb blocks take (256 / LG) heads of q and k
// each, LG lanes per head, the others 256 pieces of eight value channels.
__global__ __launch_bounds__(kNT) void attn_write_kernel(Dims d, Runs rn, const uint16_t* __restrict__ proj,
                                                         int64_t stride, const uint16_t* __restrict__ qw,
                                                         const uint16_t* __restrict__ kw_, int LG, int hb,
                                                         const int64_t* __restrict__ slots, uint16_t* __restrict__ q,
                                                         uint16_t* __restrict__ kc, uint16_t* __restrict__ vc) {
    int t0, count;
    if (rn.runs) {
        t0 = rn.runs[2 * blockIdx.x];
        count = rn.runs[2 * blockIdx.x + 1];
    } else {
        t0 = rn.first + blockIdx.x;
        count = 1;
    }
    const int64_t slot = slots[t0], blk = slot / kBS;
    const int off = (int)(slot % kBS), dp = d.dp();
    const bool heads = (int)blockIdx.y < hb;
    int col, h = 0, e = 0;
    bool on;
    if (heads) {
        h = blockIdx.y * (kNT / LG) + threadIdx.x / LG;
        e = (threadIdx.x % LG) * 8;
        on = h < d.H + d.G && e < d.D;
        col = h * d.D + e;
    } else {
        const int pc = ((int)blockIdx.y - hb) * kNT + threadIdx.x;
        on = pc < d.G * d.V / 8;
        h = on ? pc * 8 / d.V : 0;
        e = pc * 8 - h * d.V;
        col = (d.H + d.G) * d.D + pc * 8;
    }
    if (!on) col = 0;
    uint4 x[kRun];
#pragma unroll
    for (int j = 0; j < kRun; ++j)
        if (j < count) x[j] = *reinterpret_cast<const uint4*>(proj + (int64_t)(t0 + j) * stride + col);
    if (heads) {
        float w[8];
        ldv<uint16_t, 8>((h < d.H ? qw : kw_) + (on ? e : 0), w);
#pragma unroll
        for (int j = 0; j < kRun; ++j) {
            if (j >= count) break;
            float y[8], ss = 0.f;
            unpack8(x[j], y);
#pragma unroll
            for (int i = 0; i < 8; ++i) ss += y[i] * y[i];
            if (!on) ss = 0.f;
            for (int o = 1; o < LG; o <<= 1) ss += __shfl_xor(ss, o, kWave);
            const float r = 1.f / sqrtf(ss / (float)d.D + d.eps);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] *= r * w[i];
            if (!on) continue;
            if (h < d.H) st8(q + ((int64_t)(t0 + j) * d.H + h) * dp + e, y);
            else if (slot >= 0) st8(kc + ((blk * d.G + h - d.H) * kBS + off + j) * dp + e, y);
        }
        return;
    }
    if (!on || slot < 0) return;
    uint16_t* dst = vc + ((blk * d.G + h) * d.vp() + e) * kBS + off;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        uint16_t v[kRun];
#pragma unroll
        for (int j = 0; j < kRun; ++j) {
            const uint32_t wd = i < 2 ? x[j].x : i < 4 ? x[j].y : i < 6 ? x[j].z : x[j].w;
            v[j] = (uint16_t)(i & 1 ? wd >> 16 : wd);
        }
        if (count == kRun) {
            *reinterpret_cast<uint4*>(dst + i * kBS) = make_uint4(v[0] | (uint32_t)v[1] << 16, v[2] | (uint32_t)v[3] << 16,
                                                                  v[4] | (uint32_t)v[5] << 16, v[6] | (uint32_t)v[7] << 16);
        } else {
#pragma unroll
            for (int j = 0; j < kRun; ++j)
                if (j < count) dst[i * kBS + j] = v[j];
        }
    }
}

// Any sizes and types: grid (tokens, ceil((H + G + ceil(G V / 64)) / 4)), a wave per head of q and k or 64 value channels.
template <typename T>
__global__ __launch_bounds__(kNT) void attn_write_plain_kernel(Dims d, int first, const T* __restrict__ proj,
                                                               int64_t stride, const T* __restrict__ qw,
                                                               const T* __restrict__ kw_,
                                                               const int64_t* __restrict__ slots, T* __restrict__ q,
                                                               T* __restrict__ kc, T* __restrict__ vc) {
    const int t = first + blockIdx.x, lane = threadIdx.x & 63;
    const int item = blockIdx.y * (kNT / kWave) + (threadIdx.x >> 6);
    const int64_t slot = slots[t], blk = slot / kBS;
    const int off = (int)(slot % kBS), dp = d.dp();
    const T* p = proj + (int64_t)t * stride;
    if (item < d.H + d.G) {
        const T* src = p + item * d.D;
        float ss = 0.f;
        for (int i = lane; i < d.D; i += kWave) ss += ld(src + i) * ld(src + i);
        const float r = 1.f / sqrtf(wave_sum(ss) / (float)d.D + d.eps);
        const bool query = item < d.H;
        if (!query && slot < 0) return;
        const T* w = query ? qw : kw_;
        T* dst = query ? q + ((int64_t)t * d.H + item) * dp : kc + ((blk * d.G + item - d.H) * kBS + off) * dp;
        for (int i = lane; i < d.D; i += kWave) st(dst + i, ld(src + i) * r * ld(w + i));
        return;
    }
    const int e = (item - d.H - d.G) * kWave + lane;
    if (e >= d.G * d.V || slot < 0) return;
    const int h = e / d.V;
    vc[((blk * d.G + h) * d.vp() + e - h * d.V) * kBS + off] = p[(d.H + d.G) * d.D + e];
}

// ---- plain form: one workgroup per (token, head), f32 or bf16, vdim <= 1024 ------------------------
template <typename T>
__global__ __launch_bounds__(kNT) void attn_plain_kernel(Dims d, const T* __restrict__ q, const T* __restrict__ gate,
                                                         int64_t gate_stride, const T* __restrict__ kc,
                                                         const T* __restrict__ vc, const int32_t* __restrict__ tables,
                                                         int64_t bt_stride, const int32_t* __restrict__ bt_row,
                                                         const int64_t* __restrict__ positions, T* __restrict__ out,
                                                         int64_t out_stride) {
    extern __shared__ float s_q[];  // dp
    __shared__ float s_p[kWave];
    constexpr int kAcc = 4;
    const int t = blockIdx.x, h = blockIdx.y, kvh = h / d.R();
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int pos = (int)positions[t], dp = d.dp(), vp = d.vp();
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride;
    for (int i = threadIdx.x; i < d.D; i += kNT) s_q[i] = ld(q + ((int64_t)t * d.H + h) * dp + i);
    __syncthreads();
    float acc[kAcc] = {0.f, 0.f, 0.f, 0.f}, m = -INFINITY, l = 0.f;
    for (int j0 = d.first(pos); j0 <= pos; j0 += kWave) {
        const int nk = min(kWave, pos + 1 - j0);
        for (int jj = wave; jj < nk; jj += kNT / kWave) {
            const int j = j0 + jj;
            const T* key = kc + (((int64_t)bt[j / kBS] * d.G + kvh) * kBS + j % kBS) * dp;
            float s = 0.f;
            for (int i = lane; i < d.D; i += kWave) s += s_q[i] * ld(key + i);
            s = wave_sum(s);
            if (lane == 0) s_p[jj] = s * d.scale;
        }
        __syncthreads();
        const float sv = lane < nk ? s_p[lane] : -INFINITY;
        const float mn = fmaxf(m, wave_max(sv));
        const float alpha = expf(m - mn), p = lane < nk ? expf(sv - mn) : 0.f;
        l = l * alpha + wave_sum(p);
        m = mn;
        __syncthreads();
        if (wave == 0) s_p[lane] = p;
        __syncthreads();
#pragma unroll
        for (int a = 0; a < kAcc; ++a) acc[a] *= alpha;
        for (int jj = 0; jj < nk; ++jj) {
            const int j = j0 + jj;
            const T* val = vc + (((int64_t)bt[j / kBS] * d.G + kvh) * vp) * kBS + j % kBS;
#pragma unroll
            for (int a = 0; a < kAcc; ++a) {
                const int e = threadIdx.x + a * kNT;
                if (e < d.V) acc[a] += s_p[jj] * ld(val + (int64_t)e * kBS);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int a = 0; a < kAcc; ++a) {
        const int e = threadIdx.x + a * kNT;
        if (e < d.V) {
            const int64_t o = (int64_t)h * d.V + e;
            st(out + (int64_t)t * out_stride + o, acc[a] / l * sigmoidf_(ld(gate + (int64_t)t * gate_stride + o)));
        }
    }
}

// Four consecutive gated outputs of a head from column e on (f: a factor of them all).
__device__ __forceinline__ void gated_store4(uint16_t* orow, const uint16_t* grow, int e, int V, bool vec,
                                             const f32x4& o, float f) {
    float v[4];
    if (vec && e + 4 <= V) {
        const float4 g = ld4(grow + e);
        v[0] = o[0] * f * sigmoid_<uint16_t>(g.x);
        v[1] = o[1] * f * sigmoid_<uint16_t>(g.y);
        v[2] = o[2] * f * sigmoid_<uint16_t>(g.z);
        v[3] = o[3] * f * sigmoid_<uint16_t>(g.w);
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = e + i < V ? o[i] * f * sigmoid_<uint16_t>(ld(grow + e + i)) : 0.f;
    }
    store4(orow, e, V, vec, v);
}
__device__ __forceinline__ bool gate_vec(const uint16_t* out, int64_t out_stride, const uint16_t* gate,
                                         int64_t gate_stride, int V) {
    return out_vec(out, out_stride, V) && out_vec(gate, gate_stride, V);
}

// A token's window as shares of pages: positions [base, pos], base on a page.
struct Span {
    int lo, base, part, np;
};
__device__ __forceinline__ Span span_of(const Dims& d, int pos, int part_min, int nparts) {
    Span s;
    s.lo = d.first(pos);
    s.base = s.lo / kBS * kBS;
    ctx_split(pos + 1 - s.base, part_min, nparts, s.part, s.np);
    return s;
}

// ---- decode form ----------------------------------------------------------------------------------
// grid (nparts, G groups, tokens), one wave. Lane (c, g): column c = query head of the group. KS: 32-wide steps
// of the key row, NT: 16-wide tiles of the values, both at least the shape's own (EXACT: equal).
template <int KS, int NT, int PF, bool EXACT>
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, 8))) void attn_attend_kernel(
    Dims d, const uint16_t* __restrict__ q, const uint16_t* __restrict__ gate, int64_t gate_stride,
    const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, const int32_t* __restrict__ tables,
    int64_t bt_stride, const int32_t* __restrict__ bt_row, const int64_t* __restrict__ positions, float scale_log2,
    int part_min, int nparts, uint16_t* __restrict__ out, int64_t out_stride, float* __restrict__ ws_o,
    float* __restrict__ ws_ml) {
    const int t = blockIdx.z, part = blockIdx.x;
    const int ng = d.groups(), kvh = blockIdx.y / ng, hg = blockIdx.y - kvh * ng;
    const int pos = (int)positions[t];
    const Span sp = span_of(d, pos, part_min, nparts);
    if (part >= sp.np) return;
    const int tk0 = sp.base + part * sp.part, tk1 = min(pos + 1, tk0 + sp.part);
    const int lane = threadIdx.x, c = lane & 15, g = lane >> 4;
    const int dp = d.dp(), vp = d.vp();
    const int ks = EXACT ? KS : dp / 32, nt = EXACT ? NT : vp / 16;
    const int r = hg * kGroup + c, h = kvh * d.R() + r;
    const bool hv = r < d.R();

    s16x8 qf[KS];
    const uint16_t* qrow = q + ((int64_t)t * d.H + (hv ? h : 0)) * dp;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
        const int col = 32 * s + 8 * g;
        qf[s] = *reinterpret_cast<const s16x8*>(qrow + min(col, dp - 8));
        if (!hv || col >= dp) qf[s] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
    f32x4 o[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;

    // up to 64 block ids at a time, one per lane
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride + tk0 / kBS;
    const int nb = (tk1 - tk0 + kBS - 1) / kBS;
    int tbl = lane < nb ? bt[lane] : 0;
    const uint16_t* kbase = kc + (int64_t)kvh * kBS * dp + c * dp + 8 * g;
    const uint16_t* vbase = vc + (int64_t)kvh * kBS * vp + c * kBS + 4 * g;
    const int64_t kblk = (int64_t)d.G * kBS * dp, vblk = (int64_t)d.G * kBS * vp;
    auto load = [&](int jb, s16x8 (&kd)[KS], s16x4 (&vd)[NT]) {
        const int64_t blk = __builtin_amdgcn_readlane(tbl, jb & 63);
#pragma unroll
        for (int s = 0; s < KS; ++s)
            kd[s] = *reinterpret_cast<const s16x8*>(kbase + blk * kblk + 32 * (EXACT ? s : min(s, ks - 1)));
#pragma unroll
        for (int n = 0; n < NT; ++n)
            vd[n] = *reinterpret_cast<const s16x4*>(vbase + blk * vblk + 16 * (EXACT ? n : min(n, nt - 1)) * kBS);
    };
    auto step = [&](int j, const s16x8 (&kf)[KS], s16x4 (&vf)[NT]) {
        const int k0 = tk0 + j * kBS + 4 * g;  // this lane's first key
        const int nv = tk1 - k0, below = sp.lo - k0;
        f32x4 sa = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[s], qf[s], sa, 0, 0, 0);
        float sv[4], bm = -INFINITY;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            sv[i] = i < nv && i >= below ? sa[i] * scale_log2 : -INFINITY;
            bm = fmaxf(bm, sv[i]);
        }
        bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
        bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
        const float mn = fmaxf(m, bm);  // finite: every page of a share has a visible key
        const float alpha = fast_exp2(m - mn);
        float p[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) p[i] = fast_exp2(sv[i] - mn);
        l = l * alpha + ((p[0] + p[1]) + (p[2] + p[3]));
        m = mn;
        if (nv < 4) {  // a slot past the end may hold anything: 0 * NaN must not reach the sums
#pragma unroll
            for (int n = 0; n < NT; ++n)
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (i >= nv) vf[n][i] = 0;
        }
        const uint2 pk = make_uint2(pack_bf16x2(p[0], p[1]), pack_bf16x2(p[2], p[3]));
        const s16x4 pf = __builtin_bit_cast(s16x4, pk);
#pragma unroll
        for (int n = 0; n < NT; ++n) {
            o[n] = o[n] * alpha;
            o[n] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(vf[n], pf, o[n], 0, 0, 0);
        }
    };
    s16x8 kb[PF][KS];
    s16x4 vb[PF][NT];
#pragma unroll
    for (int i = 0; i < PF - 1; ++i)
        if (i < nb) load(i, kb[i], vb[i]);
    for (int j0 = 0; j0 < nb; j0 += PF) {
#pragma unroll
        for (int u = 0; u < PF; ++u) {
            const int j = j0 + u;
            if (j < nb) {
                const int jn = j + PF - 1;
                if (jn < nb) {
                    if ((jn & 63) == 0) tbl = (jn + lane < nb) ? bt[jn + lane] : 0;
                    load(jn, kb[(u + PF - 1) % PF], vb[(u + PF - 1) % PF]);
                }
                step(j, kb[u], vb[u]);
            }
        }
    }
    l += __shfl_xor(l, 16, kWave);
    l += __shfl_xor(l, 32, kWave);
    if (!hv) return;
    if (sp.np > 1) {
        const int64_t rec = ((int64_t)t * d.H + h) * nparts + part;
#pragma unroll
        for (int n = 0; n < NT; ++n)
            if (EXACT || n < nt) *reinterpret_cast<f32x4*>(ws_o + rec * vp + 16 * n + 4 * g) = o[n];
        if (g == 0) {
            ws_ml[rec * 2] = m;
            ws_ml[rec * 2 + 1] = l;
        }
        return;
    }
    const float inv = 1.f / l;
    uint16_t* orow = out + (int64_t)t * out_stride + (int64_t)h * d.V;
    const uint16_t* grow = gate + (int64_t)t * gate_stride + (int64_t)h * d.V;
    const bool vec = gate_vec(out, out_stride, gate, gate_stride, d.V);
#pragma unroll
    for (int n = 0; n < NT; ++n)
        if (EXACT || n < nt) gated_store4(orow, grow, 16 * n + 4 * g, d.V, vec, o[n], inv);
}

// Merge of a split window: grid (heads, tokens), one wave, four columns per lane.
__global__ __launch_bounds__(kWave) void attn_merge_kernel(Dims d, const float* __restrict__ ws_o,
                                                           const float* __restrict__ ws_ml,
                                                           const uint16_t* __restrict__ gate, int64_t gate_stride,
                                                           const int64_t* __restrict__ positions, int part_min,
                                                           int nparts, uint16_t* __restrict__ out, int64_t out_stride) {
    const int h = blockIdx.x, t = blockIdx.y, lane = threadIdx.x;
    const Span sp = span_of(d, (int)positions[t], part_min, nparts);
    if (sp.np == 1) return;  // written by the attention kernel
    const int64_t rec = ((int64_t)t * d.H + h) * nparts;
    const int vp = d.vp(), e = 4 * lane;
    float M = -INFINITY, L = 0.f;
    for (int p = lane; p < sp.np; p += kWave) M = fmaxf(M, ws_ml[(rec + p) * 2]);
    M = wave_max(M);
    for (int p = lane; p < sp.np; p += kWave) L += fast_exp2(ws_ml[(rec + p) * 2] - M) * ws_ml[(rec + p) * 2 + 1];
    const float inv = 1.f / wave_sum(L);
    if (e >= vp) return;
    f32x4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int p = 0; p < sp.np; ++p)
        a += *reinterpret_cast<const f32x4*>(ws_o + (rec + p) * vp + e) * fast_exp2(ws_ml[(rec + p) * 2] - M);
    gated_store4(out + (int64_t)t * out_stride + (int64_t)h * d.V, gate + (int64_t)t * gate_stride + (int64_t)h * d.V, e,
                 d.V, gate_vec(out, out_stride, gate, gate_stride, d.V), a, inv);
}

// ---- prompt form ----------------------------------------------------------------------------------
constexpr int kKT = 64;         // keys per LDS tile
constexpr int kQueries = 128;   // per workgroup
constexpr float kSlack = 8.f;   // a running maximum may lag by this (base 2): weights stay below 2^8

// KM: 32-wide steps of the key row, NV: 16-wide tiles of the values, at least the shape's own; QT: 16-query
// tiles per wave.
template <int KM, int NV, int QT, bool EXACT>
__global__ __launch_bounds__(kQueries / 16 / QT * kWave) __attribute__((amdgpu_waves_per_eu(2))) void attn_prefill_kernel(
    Dims d, const uint16_t* __restrict__ q, const uint16_t* __restrict__ gate, int64_t gate_stride,
    const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, const int32_t* __restrict__ tables,
    int64_t bt_stride, const int32_t* __restrict__ tiles, float scale_log2, uint16_t* __restrict__ out,
    int64_t out_stride) {
    constexpr int NTH = kQueries / 16 / QT * kWave;
    constexpr int LDK = KM * 32 + 8, LDV = kKT + 8;
    constexpr int KPT = (KM * 256 + NTH - 1) / NTH, VPT = (NV * 128 + NTH - 1) / NTH;  // 16-byte pieces per thread
    __shared__ __attribute__((aligned(16))) uint16_t s_k[kKT * LDK];
    __shared__ __attribute__((aligned(16))) uint16_t s_v[NV * 16 * LDV];
    const int H = d.H, b = blockIdx.x % H;
    const int h = H % 8 == 0 ? (b & 7) * (H / 8) + b / 8 : b;  // an XCD's heads share their keys
    const int32_t* tl = tiles + 4 * (blockIdx.x / H);
    const int tok0 = tl[0], ntok = tl[1], pos0 = tl[2];
    const int32_t* bt = tables + (int64_t)tl[3] * bt_stride;
    const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int kvh = h / d.R();
    const int dp = EXACT ? KM * 32 : d.dp(), vp = EXACT ? NV * 16 : d.vp();
    const int km = EXACT ? KM : dp / 32, nv = EXACT ? NV : vp / 16;

    const int qi0 = 16 * QT * wave + c;  // query of tile 0; tile x: + 16 x
    s16x8 qf[QT][KM];
#pragma unroll
    for (int x = 0; x < QT; ++x) {
        const uint16_t* qrow = q + ((int64_t)(tok0 + min(qi0 + 16 * x, ntok - 1)) * H + h) * dp;
#pragma unroll
        for (int s = 0; s < KM; ++s)
            if (EXACT || s < km) qf[x][s] = *reinterpret_cast<const s16x8*>(qrow + 32 * s + 8 * g);
    }
    f32x4 o[QT][NV];
    float m[QT], l[QT];
#pragma unroll
    for (int x = 0; x < QT; ++x) {
        m[x] = kLow;
        l[x] = 0.f;
#pragma unroll
        for (int n = 0; n < NV; ++n) o[x][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int last = pos0 + ntok - 1;  // the tile's last position
    const int last_page = last / kBS, j0 = d.first(pos0) / kKT, jn = last / kKT;
    const int wq0 = pos0 + 16 * QT * wave, wq1 = min(wq0 + 16 * QT - 1, last), wlo = d.first(wq0);
    // this thread's pieces of a tile: page within the tile, offset within the page, place in LDS
    int kpage[KPT], koff[KPT], kdst[KPT], vpage[VPT], voff[VPT], vdst[VPT];
    const int nkc = 2 * dp, nvc = 2 * vp, kr8 = dp / 8;  // pieces per page, per key row
#pragma unroll
    for (int i = 0; i < KPT; ++i) {
        const int e = min(tid + NTH * i, 4 * nkc - 1), w = e % nkc;
        kpage[i] = e / nkc;
        koff[i] = 8 * w;
        kdst[i] = (kpage[i] * kBS + w / kr8) * LDK + (w % kr8) * 8;
    }
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int e = min(tid + NTH * i, 4 * nvc - 1), w = e % nvc;
        vpage[i] = e / nvc;
        voff[i] = 8 * w;
        vdst[i] = (w >> 1) * LDV + vpage[i] * kBS + (w & 1) * 8;
    }
    const uint16_t* kh = kc + (int64_t)kvh * kBS * dp;
    const uint16_t* vh = vc + (int64_t)kvh * kBS * vp;
    const int64_t kblk = (int64_t)d.G * kBS * dp, vblk = (int64_t)d.G * kBS * vp;
    s16x8 kr[KPT], vr[VPT];
    int tbl = 0;
    auto fetch = [&](int j) {
        if (j == j0 || (j & 15) == 0) tbl = bt[min(4 * (j & ~15) + lane, last_page)];  // block ids of 16 tiles
        const int p0 = 4 * (j & 15);
#pragma unroll
        for (int i = 0; i < KPT; ++i)
            kr[i] = *reinterpret_cast<const s16x8*>(kh + (int64_t)__shfl(tbl, p0 + kpage[i], kWave) * kblk + koff[i]);
#pragma unroll
        for (int i = 0; i < VPT; ++i)
            vr[i] = *reinterpret_cast<const s16x8*>(vh + (int64_t)__shfl(tbl, p0 + vpage[i], kWave) * vblk + voff[i]);
    };
    fetch(j0);
    for (int j = j0; j <= jn; ++j) {
        const int kp0 = j * kKT, kp1 = kp0 + kKT - 1;
        if (kp1 > last) {  // slots after the last token may hold anything: 0 * NaN must not reach the sums
#pragma unroll
            for (int i = 0; i < VPT; ++i) {
                const int key = kp0 + vpage[i] * kBS + ((voff[i] >> 3) & 1) * 8;
#pragma unroll
                for (int x = 0; x < 8; ++x)
                    if (key + x > last) vr[i][x] = 0;
            }
        }
        __syncthreads();  // the previous tile is consumed
#pragma unroll
        for (int i = 0; i < KPT; ++i) *reinterpret_cast<s16x8*>(&s_k[kdst[i]]) = kr[i];
#pragma unroll
        for (int i = 0; i < VPT; ++i) *reinterpret_cast<s16x8*>(&s_v[vdst[i]]) = vr[i];
        __syncthreads();
        if (j < jn) fetch(j + 1);
        if (kp0 > wq1 || wq0 > last || kp1 < wlo) continue;  // no key of this tile for this wave
        const bool edge = kp1 > wq0, low = kp0 < d.first(wq1);
        f32x4 sc[QT][4];
#pragma unroll
        for (int x = 0; x < QT; ++x)
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) sc[x][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KM; ++s) {
            if (EXACT || s < km) {
#pragma unroll
                for (int tt = 0; tt < 4; ++tt) {
                    const s16x8 kf = *reinterpret_cast<const s16x8*>(&s_k[(16 * tt + c) * LDK + 32 * s + 8 * g]);
#pragma unroll
                    for (int x = 0; x < QT; ++x)
                        sc[x][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[x][s], sc[x][tt], 0, 0, 0);
                }
            }
        }
        float top[QT];
        bool grown = false;
#pragma unroll
        for (int x = 0; x < QT; ++x) {
            const int qpos = pos0 + qi0 + 16 * x;
            if (edge || low) {
                const int seen = qpos - kp0 - 4 * g;              // keys up to this one, counted from the lane's first
                const int from = d.first(qpos) - kp0 - 4 * g;     // and from this one on
#pragma unroll
                for (int tt = 0; tt < 4; ++tt)
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        if (16 * tt + i > seen || 16 * tt + i < from) sc[x][tt][i] = -INFINITY;
            }
            float bm = -INFINITY;
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)
                bm = fmaxf(bm, fmaxf(fmaxf(sc[x][tt][0], sc[x][tt][1]), fmaxf(sc[x][tt][2], sc[x][tt][3])));
            bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
            bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
            top[x] = bm * scale_log2;  // scale > 0
            grown |= top[x] > m[x] + kSlack;
        }
        if (__any(grown)) {  // at the first tile; later seldom
#pragma unroll
            for (int x = 0; x < QT; ++x) {
                const float mn = fmaxf(m[x], top[x]), alpha = fast_exp2(m[x] - mn);
                m[x] = mn;
                l[x] = l[x] * alpha;
#pragma unroll
                for (int n = 0; n < NV; ++n) o[x][n] = o[x][n] * alpha;
            }
        }
        s16x8 pf[QT][2];  // [32-key step]
#pragma unroll
        for (int x = 0; x < QT; ++x) {
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                uint32_t pk[4];
#pragma unroll
                for (int bb = 0; bb < 2; ++bb) {
                    float p[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        p[i] = fast_exp2(fmaf(sc[x][2 * kk + bb][i], scale_log2, -m[x]));
                        l[x] += p[i];
                    }
                    pk[2 * bb] = pack_bf16x2(p[0], p[1]);
                    pk[2 * bb + 1] = pack_bf16x2(p[2], p[3]);
                }
                pf[x][kk] = __builtin_bit_cast(s16x8, make_uint4(pk[0], pk[1], pk[2], pk[3]));
            }
        }
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            if (EXACT || n < nv) {
#pragma unroll
                for (int kk = 0; kk < 2; ++kk) {
                    const uint16_t* vp_ = &s_v[(16 * n + c) * LDV + 32 * kk + 4 * g];
                    const s16x4 v0 = *reinterpret_cast<const s16x4*>(vp_);
                    const s16x4 v1 = *reinterpret_cast<const s16x4*>(vp_ + 16);
                    const s16x8 vf = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
                    for (int x = 0; x < QT; ++x)
                        o[x][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[x][kk], o[x][n], 0, 0, 0);
                }
            }
        }
    }
    const bool vec = gate_vec(out, out_stride, gate, gate_stride, d.V);
#pragma unroll
    for (int x = 0; x < QT; ++x) {
        float s = l[x];
        s += __shfl_xor(s, 16, kWave);
        s += __shfl_xor(s, 32, kWave);
        const int qi = qi0 + 16 * x;
        if (qi >= ntok) continue;
        const float inv = 1.f / s;
        uint16_t* orow = out + (int64_t)(tok0 + qi) * out_stride + (int64_t)h * d.V;
        const uint16_t* grow = gate + (int64_t)(tok0 + qi) * gate_stride + (int64_t)h * d.V;
#pragma unroll
        for (int n = 0; n < NV; ++n)
            if (EXACT || n < nv) gated_store4(orow, grow, 16 * n + 4 * g, d.V, vec, o[x][n], inv);
    }
}

// ---- host -----------------------------------------------------------------------------------------
const char* bad_shape(const skyrl_attn_shape* sh) {
    if (!sh) return "attn: null shape";
    if (sh->heads <= 0 || sh->kv_heads <= 0 || sh->heads % sh->kv_heads) return "attn: heads must be a multiple of kv_heads";
    if (sh->dim <= 0 || sh->vdim <= 0 || sh->dim > 1024 || sh->vdim > 1024) return "attn: dim and vdim must be in [1, 1024]";
    return nullptr;
}
Dims dims_of(const skyrl_attn_shape* s) {
    return Dims{s->heads, s->kv_heads, s->dim, s->vdim, s->window, s->scale, s->eps};
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

extern "C" int skyrl_attn_write(const skyrl_attn_shape* shape, const void* proj, int64_t proj_stride, const void* q_norm,
                                const void* k_norm, const int64_t* slots, const int32_t* runs, int32_t first,
                                int32_t count, void* q, void* k_cache, void* v_cache, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "attn_write");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(first >= 0 && count >= 0 && proj_stride >= d.channels(), "attn_write: bad sizes");
    if (count == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && q_norm && k_norm && slots && q && k_cache && v_cache, "attn_write: null pointer");
    SKYRL_REQUIRE(aligned16(q) && aligned16(k_cache) && aligned16(v_cache), "attn_write: 16-byte alignment");
    const bool wide = dtype == SKYRL_BF16 && d.D % 8 == 0 && d.D <= 512 && d.V % 8 == 0 && proj_stride % 8 == 0 &&
                      aligned16(proj) && aligned16(q_norm) && aligned16(k_norm);
    SKYRL_REQUIRE(wide || !runs, "attn_write: runs need bf16 and sizes, strides and pointers in multiples of 8");
    if (wide) {
        int LG = 1;
        while (8 * LG < d.D) LG <<= 1;
        const int hb = ((d.H + d.G) * LG + kNT - 1) / kNT, vb = (d.G * d.V / 8 + kNT - 1) / kNT;
        hipLaunchKernelGGL(attn_write_kernel, dim3(count, hb + vb), dim3(kNT), 0, as_stream(stream), d,
                           Runs{runs, first}, reinterpret_cast<const uint16_t*>(proj), proj_stride,
                           reinterpret_cast<const uint16_t*>(q_norm), reinterpret_cast<const uint16_t*>(k_norm), LG,
                           hb, slots, reinterpret_cast<uint16_t*>(q), reinterpret_cast<uint16_t*>(k_cache),
                           reinterpret_cast<uint16_t*>(v_cache));
        return check_launch("attn_write_kernel");
    }
    const int items = d.H + d.G + (d.G * d.V + kWave - 1) / kWave;
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((attn_write_plain_kernel<T>), dim3(count, (items + 3) / 4), dim3(kNT), 0, as_stream(stream),
                           d, first, reinterpret_cast<const T*>(proj), proj_stride, reinterpret_cast<const T*>(q_norm),
                           reinterpret_cast<const T*>(k_norm), slots, reinterpret_cast<T*>(q),
                           reinterpret_cast<T*>(k_cache), reinterpret_cast<T*>(v_cache));
    })
    return check_launch("attn_write_plain_kernel");
}

extern "C" int skyrl_attn_mfma(const skyrl_attn_shape* shape, int32_t dtype) {
    return dtype == SKYRL_BF16 && !bad_shape(shape) && shape->dim <= 256 && shape->vdim <= 256 && shape->scale > 0.f;
}

extern "C" size_t skyrl_attn_attend_workspace_bytes(const skyrl_attn_shape* shape, int32_t T_, int32_t nparts) {
    if (bad_shape(shape) || T_ <= 0 || nparts <= 1) return 0;
    return (size_t)T_ * shape->heads * nparts * ((size_t)dims_of(shape).vp() + 2) * sizeof(float);
}

#define LAUNCH_ATTEND_(KS, NT, PF, EX)                                                                                  \
    hipLaunchKernelGGL((attn_attend_kernel<KS, NT, PF, EX>), dim3(nparts, d.G * d.groups(), T_), dim3(64), 0, s, d, q_, \
                       g_, gate_stride, k_, v_, block_tables, bt_stride, bt_row, positions, d.scale * kLog2e, part_min, \
                       nparts, o_, out_stride, ws_o, ws_ml)
#define LAUNCH_ATTEND(KS, NT, PF)                               \
    if (ks == KS && nt == NT) LAUNCH_ATTEND_(KS, NT, PF, true); \
    else LAUNCH_ATTEND_(KS, NT, PF, false)

extern "C" int skyrl_attn_attend(const skyrl_attn_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                                 const void* k_cache, const void* v_cache, const int32_t* block_tables,
                                 int64_t bt_stride, const int32_t* bt_row, const int64_t* positions, int32_t T_,
                                 int32_t part_min, int32_t nparts, void* out, int64_t out_stride, void* workspace,
                                 int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "attn_attend");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    const int64_t ow = (int64_t)d.H * d.V;
    SKYRL_REQUIRE(T_ >= 0 && T_ <= 65535 && d.H <= 65535 && gate_stride >= ow && out_stride >= ow,
                  "attn_attend: bad sizes (T <= 65535)");
    if (T_ == 0) return SKYRL_OK;
    SKYRL_REQUIRE(q && gate && k_cache && v_cache && block_tables && bt_row && positions && out,
                  "attn_attend: null pointer");
    hipStream_t s = as_stream(stream);
    if (!skyrl_attn_mfma(shape, dtype)) {
        SKYRL_DISPATCH_T(dtype, {
            hipLaunchKernelGGL((attn_plain_kernel<T>), dim3(T_, d.H), dim3(kNT), d.dp() * sizeof(float), s, d,
                               reinterpret_cast<const T*>(q), reinterpret_cast<const T*>(gate), gate_stride,
                               reinterpret_cast<const T*>(k_cache), reinterpret_cast<const T*>(v_cache), block_tables,
                               bt_stride, bt_row, positions, reinterpret_cast<T*>(out), out_stride);
        })
        return check_launch("attn_plain_kernel");
    }
    SKYRL_REQUIRE(nparts >= 1 && part_min >= kBS && part_min % kBS == 0,
                  "attn_attend: nparts >= 1 and part_min a positive multiple of 16");
    SKYRL_REQUIRE(nparts == 1 || workspace, "attn_attend: nparts > 1 needs a workspace");
    SKYRL_REQUIRE(aligned16(q) && aligned16(k_cache) && aligned16(v_cache) && aligned16(workspace),
                  "attn_attend: 16-byte alignment");
    const uint16_t* q_ = reinterpret_cast<const uint16_t*>(q);
    const uint16_t* g_ = reinterpret_cast<const uint16_t*>(gate);
    const uint16_t* k_ = reinterpret_cast<const uint16_t*>(k_cache);
    const uint16_t* v_ = reinterpret_cast<const uint16_t*>(v_cache);
    uint16_t* o_ = reinterpret_cast<uint16_t*>(out);
    float* ws_o = reinterpret_cast<float*>(workspace);
    float* ws_ml = ws_o ? ws_o + (size_t)T_ * d.H * nparts * d.vp() : nullptr;
    const int ks = d.dp() / 32, nt = d.vp() / 16;
    if (ks <= 2) {
        if (nt <= 4) LAUNCH_ATTEND(2, 4, 4);
        else if (nt <= 8) LAUNCH_ATTEND(2, 8, 4);
        else LAUNCH_ATTEND_(2, 16, 3, false);
    } else if (ks <= 4) {
        if (nt <= 8) LAUNCH_ATTEND(4, 8, 4);
        else LAUNCH_ATTEND(4, 16, 3);
    } else {
        LAUNCH_ATTEND(8, 16, 2);
    }
    const int rc = check_launch("attn_attend_kernel");
    if (rc != SKYRL_OK || nparts == 1) return rc;
    hipLaunchKernelGGL(attn_merge_kernel, dim3(d.H, T_), dim3(kWave), 0, s, d, ws_o, ws_ml, g_, gate_stride, positions,
                       part_min, nparts, o_, out_stride);
    return check_launch("attn_merge_kernel");
}

#define LAUNCH_PROMPT_(KM, NV, QT, EX)                                                                                 \
    hipLaunchKernelGGL((attn_prefill_kernel<KM, NV, QT, EX>), dim3((unsigned)ntiles * d.H),                            \
                       dim3(kQueries / 16 / QT * kWave), 0, as_stream(stream), d, reinterpret_cast<const uint16_t*>(q), \
                       reinterpret_cast<const uint16_t*>(gate), gate_stride,                                           \
                       reinterpret_cast<const uint16_t*>(k_cache), reinterpret_cast<const uint16_t*>(v_cache),         \
                       block_tables, bt_stride, tiles, d.scale * kLog2e, reinterpret_cast<uint16_t*>(out), out_stride)
#define LAUNCH_PROMPT(KM, NV, QT)                               \
    if (km == KM && nt == NV) LAUNCH_PROMPT_(KM, NV, QT, true); \
    else LAUNCH_PROMPT_(KM, NV, QT, false)

extern "C" int skyrl_attn_prefill(const skyrl_attn_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                                  const void* k_cache, const void* v_cache, const int32_t* block_tables,
                                  int64_t bt_stride, const int32_t* tiles, int32_t ntiles, void* out,
                                  int64_t out_stride, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    const int64_t ow = (int64_t)d.H * d.V;
    SKYRL_REQUIRE(skyrl_attn_mfma(shape, SKYRL_BF16), "attn_prefill: dim, vdim <= 256 and scale > 0");
    SKYRL_REQUIRE(ntiles >= 0 && (int64_t)ntiles * d.H < (1 << 30) && gate_stride >= ow && out_stride >= ow,
                  "attn_prefill: bad sizes");
    if (ntiles == 0) return SKYRL_OK;
    SKYRL_REQUIRE(q && gate && k_cache && v_cache && block_tables && tiles && out, "attn_prefill: null pointer");
    SKYRL_REQUIRE(aligned16(q) && aligned16(k_cache) && aligned16(v_cache), "attn_prefill: 16-byte alignment");
    const int km = d.dp() / 32, nt = d.vp() / 16;
    if (km <= 2) {
        if (nt <= 4) LAUNCH_PROMPT(2, 4, 2);
        else if (nt <= 8) LAUNCH_PROMPT(2, 8, 2);
        else LAUNCH_PROMPT_(2, 16, 1, false);
    } else if (km <= 4) {
        if (nt <= 8) LAUNCH_PROMPT(4, 8, 2);
        else LAUNCH_PROMPT(4, 16, 1);
    } else {
        LAUNCH_PROMPT_(8, 16, 1, false);
    }
    return check_launch("attn_prefill_kernel");
}
