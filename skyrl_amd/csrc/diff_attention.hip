// Differential attention over a paged key / value cache (include/skyrl_layers.h has the equations and the
// tensor layouts): two softmax maps per query head over the same values, their difference normed and gated.
//
// Write (diff_write, diff_write_runs): short convolution of the projected q, k and v, rotation, queries to a
// padded buffer, keys and values into the pages, one pass. Prompts take runs of up to eight tokens per
// thread: a channel's inputs are read once per run, and the transposed values leave as 16-byte pieces.
//
// Decode form (diff_attend): one wave per (share of the context, key / value head and group of eight of its
// query heads, token). The 16 columns of the matrix instructions are (map, query head): a page's keys
// [16 x 2 dp] meet queries that are zero outside their own map, so one product gives both maps' scores, and
// the exp'd scores are already the operand of O^T += V^T P^T, both maps sharing the value registers. Keys and
// values stream from HBM to registers, PF pages in flight. The maps meet by one lane exchange at the end;
// shares of a split context are merged, and the maps combined, by diff_merge.
//
// Prompt form (diff_prefill): flash style, eight waves of 16 queries of one head share a tile of 64 keys and
// values in LDS, read straight from the pages; each wave keeps both maps' sums and combines them in registers.
// A map's running maximum is only raised when the scores outgrow it by kSlack, so that the sums are rescaled
// at the first tile and seldom after.
#include "conv.h"
#include "paged.h"

namespace skyrl {
namespace {

constexpr int kNT = 256;
constexpr int kGroup = 8;  // query heads per decode wave
constexpr int kRun = 8;    // tokens per thread of the prompt's write

struct Dims {
    int H, G, D, V, rot, taps, kv;
    float scale, diff, eps;
    __host__ __device__ int dp() const { return (D + 15) / 16 * 16; }
    __host__ __device__ int vp() const { return (V + 15) / 16 * 16; }
    __host__ __device__ int qch() const { return H * 2 * D; }
    __host__ __device__ int kch() const { return kv ? G * 2 * D : 0; }
    __host__ __device__ int channels() const { return qch() + (kv ? G * (2 * D + V) : 0); }
    __host__ __device__ int R() const { return H / G; }
    __host__ __device__ int groups() const { return (R() + kGroup - 1) / kGroup; }
};

// Where a channel goes: 0 query, 1 key, 2 value; head; column d of map `map`.
struct Place {
    int kind, head, map, d;
};
__device__ __forceinline__ Place place_of(const Dims& d, int ch) {
    Place p;
    const int q = d.qch(), k = d.kch();
    if (ch < q + k) {
        p.kind = ch < q ? 0 : 1;
        const int e = ch < q ? ch : ch - q;
        p.head = e / (2 * d.D);
        const int r = e - p.head * 2 * d.D;
        p.map = r >= d.D;
        p.d = r - p.map * d.D;
    } else {
        p.kind = 2;
        p.head = (ch - q - k) / d.V;
        p.map = 0;
        p.d = ch - q - k - p.head * d.V;
    }
    return p;
}

// Rotates the pairs among eight consecutive columns d.. of a map.
__device__ __forceinline__ void rotate8(float (&y)[8], int d, int rot, const float* __restrict__ cs) {
    const int h2 = rot / 2;
#pragma unroll
    for (int i = 0; i < 8; i += 2) {
        if (d + i < rot) {
            const float c = cs[(d + i) / 2], s = cs[h2 + (d + i) / 2], u = y[i], v = y[i + 1];
            y[i] = u * c - v * s;
            y[i + 1] = v * c + u * s;
        }
    }
}

// grid (tokens, ceil(channels / (VEC kNT))).
template <typename T, int VEC>
__global__ __launch_bounds__(kNT) void diff_write_kernel(
    Dims d, const T* __restrict__ proj, int64_t stride, const float* __restrict__ conv_t,
    const int32_t* __restrict__ cu, const int32_t* __restrict__ rows, const int32_t* __restrict__ bt_row,
    const int64_t* __restrict__ positions, const int64_t* __restrict__ slots, const float* __restrict__ cos_sin,
    T* __restrict__ ring_base, int save, int first, T* __restrict__ q, T* __restrict__ kc, T* __restrict__ vc) {
    const int t = first + blockIdx.x;
    const int ch = (blockIdx.y * kNT + threadIdx.x) * VEC, n = d.channels();
    if (ch >= n) return;
    const int seq = bt_row[t], t0 = cu[seq], row = rows[seq];
    const int pos = (int)positions[t];
    const int64_t slot = slots[t];
    // an idle row has one token at position 0, whose convolution reads no ring
    T* ring = ring_base + (int64_t)max(row, 0) * d.taps * n;
    const Place p = place_of(d, ch);
    float y[VEC], x0[VEC];
    conv_at<T, VEC>(proj, stride, conv_t, ring, n, d.taps, ch, t, t0, pos, y, x0);
    if (p.kind < 2 && p.d < d.rot) {
        const float* cs = cos_sin + (int64_t)pos * d.rot;
        if constexpr (VEC == 8) {
            rotate8(y, p.d, d.rot, cs);
        } else {  // the other half of the pair is a convolution of its own
            const int odd = p.d & 1;
            float z[VEC], unused[VEC];
            conv_at<T, VEC>(proj, stride, conv_t, ring, n, d.taps, odd ? ch - 1 : ch + 1, t, t0, pos, z, unused);
            const float c = cs[p.d / 2], s = cs[d.rot / 2 + p.d / 2];
            y[0] = odd ? y[0] * c + z[0] * s : y[0] * c - z[0] * s;
        }
    }
    if (save && row >= 0) {
        T* dst = ring + (int64_t)(pos % d.taps) * n + ch;
        if constexpr (VEC == 8) st8(dst, x0);
        else st(dst, x0[0]);
    }
    const int kw = 2 * d.dp();
    const int64_t blk = slot / kBS;
    const int off = (int)(slot % kBS);
    if (p.kind == 0) {
        T* dst = q + ((int64_t)t * d.H + p.head) * kw + p.map * d.dp() + p.d;
        if constexpr (VEC == 8) st8(dst, y);
        else st(dst, y[0]);
    } else if (slot < 0) {
        return;
    } else if (p.kind == 1) {
        T* dst = kc + ((blk * d.G + p.head) * kBS + off) * kw + p.map * d.dp() + p.d;
        if constexpr (VEC == 8) st8(dst, y);
        else st(dst, y[0]);
    } else {
        T* dst = vc + ((blk * d.G + p.head) * d.vp() + p.d) * kBS + off;
#pragma unroll
        for (int i = 0; i < VEC; ++i) st(dst + i * kBS, y[i]);
    }
}

// bf16, eight channels and a run of up to eight tokens per thread. grid (ceil(channels / (8 kNT)), runs). TW >= taps.
template <int TW>
__global__ __launch_bounds__(kNT) void diff_write_runs_kernel(
    Dims d, const uint16_t* __restrict__ proj, int64_t stride, const float* __restrict__ conv_t,
    const int32_t* __restrict__ cu, const int32_t* __restrict__ rows, const int32_t* __restrict__ bt_row,
    const int64_t* __restrict__ positions, const int64_t* __restrict__ slots, const float* __restrict__ cos_sin,
    const uint16_t* __restrict__ ring_base, const int32_t* __restrict__ runs, uint16_t* __restrict__ q,
    uint16_t* __restrict__ kc, uint16_t* __restrict__ vc) {
    const int ch = (blockIdx.x * kNT + threadIdx.x) * 8, n = d.channels();
    if (ch >= n) return;
    const int t_first = runs[2 * blockIdx.y], count = runs[2 * blockIdx.y + 1];
    const int seq = bt_row[t_first], t0 = cu[seq], row = rows[seq];
    const int pos0 = (int)positions[t_first];
    const int64_t slot = slots[t_first];
    const uint16_t* ring = ring_base + (int64_t)max(row, 0) * d.taps * n;
    const int r0 = pos0 % d.taps;
    uint4 x[TW - 1 + kRun];  // x[TW - 1 + j]: token t_first + j
#pragma unroll
    for (int i = 0; i < TW - 1 + kRun; ++i) {
        const int j = i - (TW - 1);
        x[i] = make_uint4(0, 0, 0, 0);
        if (j >= 0 ? j < count : (-j < d.taps && -j <= pos0)) {
            const uint16_t* src = proj + (int64_t)(t_first + j) * stride + ch;
            if (j < 0 && t_first + j < t0) src = ring + (int64_t)(r0 + j < 0 ? r0 + j + d.taps : r0 + j) * n + ch;
            x[i] = *reinterpret_cast<const uint4*>(src);
        }
    }
    float f[TW][8];  // f[k]: the tap on the token TW - 1 - k back
#pragma unroll
    for (int k = 0; k < TW; ++k) {
        const int tap = k - (TW - d.taps);
        if (tap >= 0) {
            ldv<float, 8>(conv_t + (int64_t)tap * n + ch, f[k]);
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) f[k][i] = 0.f;
        }
    }
    const Place p = place_of(d, ch);
    const int kw = 2 * d.dp();
    const int64_t blk = slot / kBS;
    const int off = (int)(slot % kBS);
    uint32_t vt[8][kRun / 2];
#pragma unroll
    for (int j = 0; j < kRun; ++j) {
        float y[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) y[i] = 0.f;
#pragma unroll
        for (int k = 0; k < TW; ++k) {
            float u[8];
            unpack8(x[j + k], u);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] += u[i] * f[k][i];
        }
        if (p.kind < 2) {
            if (j >= count) break;
            if (p.d < d.rot) rotate8(y, p.d, d.rot, cos_sin + (int64_t)(pos0 + j) * d.rot);
            if (p.kind == 0) st8(q + ((int64_t)(t_first + j) * d.H + p.head) * kw + p.map * d.dp() + p.d, y);
            else if (slot >= 0) st8(kc + ((blk * d.G + p.head) * kBS + off + j) * kw + p.map * d.dp() + p.d, y);
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const uint32_t b = f32_to_bf16(y[i]);
                if (j & 1) vt[i][j / 2] |= b << 16;
                else vt[i][j / 2] = b;
            }
        }
    }
    if (p.kind == 2 && slot >= 0) {
        uint16_t* dst = vc + ((blk * d.G + p.head) * d.vp() + p.d) * kBS + off;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            if (count == kRun) {
                *reinterpret_cast<uint4*>(dst + i * kBS) = make_uint4(vt[i][0], vt[i][1], vt[i][2], vt[i][3]);
            } else {
#pragma unroll
                for (int j = 0; j < kRun; ++j)
                    if (j < count) dst[i * kBS + j] = (uint16_t)(vt[i][j / 2] >> (16 * (j & 1)));
            }
        }
    }
}

// ---- plain form: one workgroup per (token, head), f32 or bf16, vdim <= 1024 ------------------------
template <typename T>
__global__ __launch_bounds__(kNT) void diff_attend_plain_kernel(
    Dims d, const T* __restrict__ q, const T* __restrict__ gate, int64_t gate_stride, const T* __restrict__ kc,
    const T* __restrict__ vc, const int32_t* __restrict__ tables, int64_t bt_stride,
    const int32_t* __restrict__ bt_row, const int64_t* __restrict__ positions, const float* __restrict__ lambda,
    T* __restrict__ out, int64_t out_stride) {
    extern __shared__ float s_q[];  // 2 dp
    __shared__ float s_p[2][kWave];
    __shared__ float s_red[kNT / kWave];
    constexpr int kAcc = 4;
    const int t = blockIdx.x, h = blockIdx.y, kvh = h / d.R();
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int pos = (int)positions[t], dp = d.dp(), kw = 2 * dp, vp = d.vp();
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride;
    for (int i = threadIdx.x; i < kw; i += kNT) s_q[i] = ld(q + ((int64_t)t * d.H + h) * kw + i);
    __syncthreads();
    float acc[2][kAcc], m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
    for (int k = 0; k < kAcc; ++k) acc[0][k] = acc[1][k] = 0.f;
    for (int j0 = 0; j0 <= pos; j0 += kWave) {
        const int nk = min(kWave, pos + 1 - j0);
        for (int jj = wave; jj < nk; jj += kNT / kWave) {
            const int j = j0 + jj;
            const T* key = kc + (((int64_t)bt[j / kBS] * d.G + kvh) * kBS + j % kBS) * kw;
            float s0 = 0.f, s1 = 0.f;
            for (int i = lane; i < dp; i += kWave) {
                s0 += s_q[i] * ld(key + i);
                s1 += s_q[dp + i] * ld(key + dp + i);
            }
            s0 = wave_sum(s0);
            s1 = wave_sum(s1);
            if (lane == 0) {
                s_p[0][jj] = s0 * d.scale;
                s_p[1][jj] = s1 * d.scale;
            }
        }
        __syncthreads();
        float p[2];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const float sv = lane < nk ? s_p[k][lane] : -INFINITY;
            const float mn = fmaxf(m[k], wave_max(sv));
            const float alpha = expf(m[k] - mn);
            p[k] = lane < nk ? expf(sv - mn) : 0.f;
            l[k] = l[k] * alpha + wave_sum(p[k]);
            m[k] = mn;
#pragma unroll
            for (int a = 0; a < kAcc; ++a) acc[k][a] *= alpha;
        }
        __syncthreads();
        if (wave == 0) {
            s_p[0][lane] = p[0];
            s_p[1][lane] = p[1];
        }
        __syncthreads();
        for (int jj = 0; jj < nk; ++jj) {
            const int j = j0 + jj;
            const T* val = vc + (((int64_t)bt[j / kBS] * d.G + kvh) * vp) * kBS + j % kBS;
            const float p0 = s_p[0][jj], p1 = s_p[1][jj];
#pragma unroll
            for (int a = 0; a < kAcc; ++a) {
                const int e = threadIdx.x + a * kNT;
                if (e < d.V) {
                    const float v = ld(val + (int64_t)e * kBS);
                    acc[0][a] += p0 * v;
                    acc[1][a] += p1 * v;
                }
            }
        }
        __syncthreads();
    }
    const float lam = lambda[0];
    float ss = 0.f;
#pragma unroll
    for (int a = 0; a < kAcc; ++a) {
        const float o = acc[0][a] / l[0] - lam * (acc[1][a] / l[1]);
        acc[0][a] = o;
        if ((int)threadIdx.x + a * kNT < d.V) ss += o * o;
    }
    const float r = 1.f / sqrtf(block_total<kNT>(ss, s_red) / (float)d.V + d.eps) * (1.f - d.diff) *
                    sigmoidf_(ld(gate + (int64_t)t * gate_stride + h));
#pragma unroll
    for (int a = 0; a < kAcc; ++a) {
        const int e = threadIdx.x + a * kNT;
        if (e < d.V) st(out + (int64_t)t * out_stride + (int64_t)h * d.V + e, acc[0][a] * r);
    }
}

// ---- decode form ----------------------------------------------------------------------------------
// grid (nparts, G groups, tokens), one wave. Lane (c, g): column c = map * 8 + query head of the group.
// KS: 32-wide steps of the key row, NT: 16-wide tiles of the values, both at least the shape's own (EXACT:
// equal; otherwise the last step or tile is loaded again and its queries are zero, its sums not used).
template <int KS, int NT, int PF, bool EXACT>
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, 8))) void diff_attend_kernel(
    Dims d, const uint16_t* __restrict__ q, const uint16_t* __restrict__ gate, int64_t gate_stride,
    const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, const int32_t* __restrict__ tables,
    int64_t bt_stride, const int32_t* __restrict__ bt_row, const int64_t* __restrict__ positions,
    const float* __restrict__ lambda, float scale_log2, int part_min, int nparts, uint16_t* __restrict__ out,
    int64_t out_stride, float* __restrict__ ws_o, float* __restrict__ ws_ml) {
    const int t = blockIdx.z, part = blockIdx.x;
    const int ng = d.groups(), kvh = blockIdx.y / ng, hg = blockIdx.y - kvh * ng;
    const int ctx = (int)positions[t] + 1;
    int part_tokens, np;
    ctx_split(ctx, part_min, nparts, part_tokens, np);
    if (part >= np) return;
    const int tk0 = part * part_tokens, tk1 = min(ctx, tk0 + part_tokens);
    const int lane = threadIdx.x, c = lane & 15, g = lane >> 4;
    const int dp = d.dp(), kw = 2 * dp, vp = d.vp();
    const int ks = EXACT ? KS : kw / 32, nt = EXACT ? NT : vp / 16;
    const int map = c >> 3, r = hg * kGroup + (c & 7), h = kvh * d.R() + r;
    const bool hv = r < d.R();

    s16x8 qf[KS];
    const uint16_t* qrow = q + ((int64_t)t * d.H + (hv ? h : 0)) * kw;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
        const int col = 32 * s + 8 * g;
        qf[s] = *reinterpret_cast<const s16x8*>(qrow + min(col, kw - 8));
        if (!hv || col >= kw || (col >= dp) != map) qf[s] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
    f32x4 o[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;

    // up to 64 block ids at a time, one per lane
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride + tk0 / kBS;
    const int nb = (tk1 - tk0 + kBS - 1) / kBS;
    int tbl = lane < nb ? bt[lane] : 0;
    const uint16_t* kbase = kc + (int64_t)kvh * kBS * kw + c * kw + 8 * g;
    const uint16_t* vbase = vc + (int64_t)kvh * kBS * vp + c * kBS + 4 * g;
    const int64_t kblk = (int64_t)d.G * kBS * kw, vblk = (int64_t)d.G * kBS * vp;
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
        const int nv = tk1 - (tk0 + j * kBS + 4 * g);  // visible among this lane's four keys
        f32x4 sa = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[s], qf[s], sa, 0, 0, 0);
        float sv[4], bm = -INFINITY;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            sv[i] = i < nv ? sa[i] * scale_log2 : -INFINITY;
            bm = fmaxf(bm, sv[i]);
        }
        bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
        bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
        const float mn = fmaxf(m, bm);
        const float alpha = fast_exp2(m - mn);  // first block: 0; every share starts with a visible key
        float p[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) p[i] = fast_exp2(sv[i] - mn);
        l = l * alpha + ((p[0] + p[1]) + (p[2] + p[3]));
        m = mn;
        if (nv < 4) {  // a masked slot may hold anything: 0 * NaN must not reach the sums
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
    if (np > 1) {
        if (!hv) return;
        const int64_t rec = (((int64_t)t * d.H + h) * 2 + map) * nparts + part;
#pragma unroll
        for (int n = 0; n < NT; ++n)
            if (EXACT || n < nt) *reinterpret_cast<f32x4*>(ws_o + rec * vp + 16 * n + 4 * g) = o[n];
        if (g == 0) {
            ws_ml[rec * 2] = m;
            ws_ml[rec * 2 + 1] = l;
        }
        return;
    }
    // the maps are eight lanes apart; afterwards both lanes hold the difference
    const float inv = 1.f / l, lam = lambda[0];
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        if (EXACT || n < nt) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float a = o[n][i] * inv, b = __shfl_xor(a, 8, kWave);
                o[n][i] = map ? b - lam * a : a - lam * b;
                ss += o[n][i] * o[n][i];
            }
        }
    }
    ss += __shfl_xor(ss, 16, kWave);
    ss += __shfl_xor(ss, 32, kWave);
    if (!hv) return;
    const float f = 1.f / sqrtf(ss / (float)d.V + d.eps) * (1.f - d.diff) *
                    sigmoidf_(bf16_to_f32(gate[(int64_t)t * gate_stride + h]));
    uint16_t* orow = out + (int64_t)t * out_stride + (int64_t)h * d.V;
    const bool vec = out_vec(out, out_stride, d.V);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        if ((n & 1) == map && (EXACT || n < nt)) {
            const float v[4] = {o[n][0] * f, o[n][1] * f, o[n][2] * f, o[n][3] * f};
            store4(orow, 16 * n + 4 * g, d.V, vec, v);
        }
    }
}

// Merge of a split context and combination of the maps: grid (heads, tokens), one wave per map.
__global__ __launch_bounds__(2 * kWave) void diff_merge_kernel(Dims d, const float* __restrict__ ws_o,
                                                               const float* __restrict__ ws_ml,
                                                               const uint16_t* __restrict__ gate, int64_t gate_stride,
                                                               const int64_t* __restrict__ positions,
                                                               const float* __restrict__ lambda, int part_min,
                                                               int nparts, uint16_t* __restrict__ out,
                                                               int64_t out_stride) {
    __shared__ __attribute__((aligned(16))) float s_a[256];
    const int h = blockIdx.x, t = blockIdx.y, lane = threadIdx.x & 63;
    const int map = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    int part_tokens, np;
    ctx_split((int)positions[t] + 1, part_min, nparts, part_tokens, np);
    if (np == 1) return;  // written by the attention kernel
    const int64_t rec = (((int64_t)t * d.H + h) * 2 + map) * nparts;
    const int vp = d.vp(), e = 4 * lane;
    float M = -INFINITY, L = 0.f;
    for (int p = lane; p < np; p += kWave) M = fmaxf(M, ws_ml[(rec + p) * 2]);
    M = wave_max(M);
    for (int p = lane; p < np; p += kWave) L += fast_exp2(ws_ml[(rec + p) * 2] - M) * ws_ml[(rec + p) * 2 + 1];
    const float inv = 1.f / wave_sum(L);
    float a[4] = {0.f, 0.f, 0.f, 0.f};
    if (e < vp) {
#pragma unroll 8
        for (int p = 0; p < np; ++p) {
            const float w = fast_exp2(ws_ml[(rec + p) * 2] - M) * inv;
            const float4 x = ld4(ws_o + (rec + p) * vp + e);
            a[0] += w * x.x; a[1] += w * x.y; a[2] += w * x.z; a[3] += w * x.w;
        }
    }
    if (map == 1) st4(s_a + e, make_float4(a[0], a[1], a[2], a[3]));
    __syncthreads();
    if (map == 1) return;
    const float lam = lambda[0];
    const float4 b = ld4(s_a + e);
    a[0] -= lam * b.x; a[1] -= lam * b.y; a[2] -= lam * b.z; a[3] -= lam * b.w;
    const float ss = wave_sum(a[0] * a[0] + a[1] * a[1] + a[2] * a[2] + a[3] * a[3]);  // the padding is zero
    const float f = 1.f / sqrtf(ss / (float)d.V + d.eps) * (1.f - d.diff) *
                    sigmoidf_(bf16_to_f32(gate[(int64_t)t * gate_stride + h]));
    const float v[4] = {a[0] * f, a[1] * f, a[2] * f, a[3] * f};
    if (e < vp) store4(out + (int64_t)t * out_stride + (int64_t)h * d.V, e, d.V, out_vec(out, out_stride, d.V), v);
}

// ---- prompt form ----------------------------------------------------------------------------------
constexpr int kKT = 64;        // keys per LDS tile
constexpr float kSlack = 8.f;  // a running maximum may lag by this (base 2): weights stay below 2^8
constexpr int kPNT = 512;

// KM: 32-wide steps of one map's key columns (with dp % 32 == 16 the middle step belongs to both maps, the
// queries zero outside their own), NV: 16-wide tiles of the values; both at least the shape's own.
template <int KM, int NV, bool EXACT>
__global__ __launch_bounds__(kPNT) __attribute__((amdgpu_waves_per_eu(2))) void diff_prefill_kernel(
    Dims d, const uint16_t* __restrict__ q, const uint16_t* __restrict__ gate, int64_t gate_stride,
    const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, const int32_t* __restrict__ tables,
    int64_t bt_stride, const int32_t* __restrict__ tiles, const float* __restrict__ lambda, float scale_log2,
    uint16_t* __restrict__ out, int64_t out_stride) {
    constexpr int LDK = KM * 64 + 8, LDV = kKT + 8;
    constexpr int KPT = KM, VPT = (NV * 128 + kPNT - 1) / kPNT;  // 16-byte pieces per thread
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
    const int dp = EXACT ? KM * 32 : d.dp(), kw = 2 * dp, vp = EXACT ? NV * 16 : d.vp();
    const int km = EXACT ? KM : (dp + 31) / 32, nv = EXACT ? NV : vp / 16;
    const int ks1 = dp / 32;  // first step of map 2

    const int qi = 16 * wave + c, qpos = pos0 + qi;
    s16x8 qf[2][KM];
    const uint16_t* qrow = q + ((int64_t)(tok0 + min(qi, ntok - 1)) * H + h) * kw;
#pragma unroll
    for (int s = 0; s < KM; ++s) {
#pragma unroll
        for (int mp = 0; mp < 2; ++mp) {
            const int col = 32 * ((mp ? ks1 : 0) + s) + 8 * g;
            qf[mp][s] = *reinterpret_cast<const s16x8*>(qrow + min(col, kw - 8));
            if (!EXACT && (col >= kw || (col >= dp) != mp)) qf[mp][s] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
        }
    }
    f32x4 o[2][NV];
#pragma unroll
    for (int n = 0; n < NV; ++n) o[0][n] = o[1][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};

    const int last = pos0 + ntok - 1;  // the tile's last position
    const int last_page = last / kBS, jn = last / kKT;
    const int wq0 = pos0 + 16 * wave, wq1 = min(wq0 + 15, last);
    // this thread's pieces of a tile: page within the tile, offset within the page, place in LDS
    int kpage[KPT], koff[KPT], kdst[KPT], vpage[VPT], voff[VPT], vdst[VPT];
    const int nkc = 2 * kw, nvc = 2 * vp, kr8 = kw / 8;  // pieces per page, per key row
#pragma unroll
    for (int i = 0; i < KPT; ++i) {
        const int e = min(tid + kPNT * i, 4 * nkc - 1), w = e % nkc;
        kpage[i] = e / nkc;
        koff[i] = 8 * w;
        kdst[i] = (kpage[i] * kBS + w / kr8) * LDK + (w % kr8) * 8;
    }
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int e = min(tid + kPNT * i, 4 * nvc - 1), w = e % nvc;
        vpage[i] = e / nvc;
        voff[i] = 8 * w;
        vdst[i] = (w >> 1) * LDV + vpage[i] * kBS + (w & 1) * 8;
    }
    const uint16_t* kh = kc + (int64_t)kvh * kBS * kw;
    const uint16_t* vh = vc + (int64_t)kvh * kBS * vp;
    const int64_t kblk = (int64_t)d.G * kBS * kw, vblk = (int64_t)d.G * kBS * vp;
    s16x8 kr[KPT], vr[VPT];
    int tbl = 0;
    auto fetch = [&](int j) {
        if ((j & 15) == 0) tbl = bt[min(4 * j + lane, last_page)];  // block ids of the next 16 tiles
        const int p0 = 4 * (j & 15);
#pragma unroll
        for (int i = 0; i < KPT; ++i)
            kr[i] = *reinterpret_cast<const s16x8*>(kh + (int64_t)__shfl(tbl, p0 + kpage[i], kWave) * kblk + koff[i]);
#pragma unroll
        for (int i = 0; i < VPT; ++i)
            vr[i] = *reinterpret_cast<const s16x8*>(vh + (int64_t)__shfl(tbl, p0 + vpage[i], kWave) * vblk + voff[i]);
    };
    fetch(0);
    for (int j = 0; j <= jn; ++j) {
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
        if (kp0 > wq1 || wq0 > last) continue;  // no key of this tile for this wave
        const bool edge = kp1 > wq0;
        s16x8 pf[2][2];  // [map][32-key step]
        f32x4 sc[2][4];
        float top[2];
        bool grown = false;
#pragma unroll
        for (int mp = 0; mp < 2; ++mp) {
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) sc[mp][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < KM; ++s) {
                if (EXACT || s < km) {
                    const int col = 32 * ((mp ? ks1 : 0) + s) + 8 * g;
#pragma unroll
                    for (int tt = 0; tt < 4; ++tt) {
                        const s16x8 kf = *reinterpret_cast<const s16x8*>(&s_k[(16 * tt + c) * LDK + col]);
                        sc[mp][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[mp][s], sc[mp][tt], 0, 0, 0);
                    }
                }
            }
            if (edge) {
                const int seen = qpos - kp0 - 4 * g;  // keys up to this one, counted from the lane's first
#pragma unroll
                for (int tt = 0; tt < 4; ++tt)
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        if (16 * tt + i > seen) sc[mp][tt][i] = -INFINITY;
            }
            float bm = -INFINITY;
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)
                bm = fmaxf(bm, fmaxf(fmaxf(sc[mp][tt][0], sc[mp][tt][1]), fmaxf(sc[mp][tt][2], sc[mp][tt][3])));
            bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
            bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
            top[mp] = bm * scale_log2;  // scale > 0
            grown |= top[mp] > m[mp] + kSlack;
        }
        if (__any(grown)) {  // at the first tile; later seldom
#pragma unroll
            for (int mp = 0; mp < 2; ++mp) {
                const float mn = fmaxf(m[mp], top[mp]), alpha = fast_exp2(m[mp] - mn);
                m[mp] = mn;
                l[mp] = l[mp] * alpha;
#pragma unroll
                for (int n = 0; n < NV; ++n) o[mp][n] = o[mp][n] * alpha;
            }
        }
#pragma unroll
        for (int mp = 0; mp < 2; ++mp) {
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                uint32_t pk[4];
#pragma unroll
                for (int bb = 0; bb < 2; ++bb) {
                    float p[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        p[i] = fast_exp2(fmaf(sc[mp][2 * kk + bb][i], scale_log2, -m[mp]));
                        l[mp] += p[i];
                    }
                    pk[2 * bb] = pack_bf16x2(p[0], p[1]);
                    pk[2 * bb + 1] = pack_bf16x2(p[2], p[3]);
                }
                pf[mp][kk] = __builtin_bit_cast(s16x8, make_uint4(pk[0], pk[1], pk[2], pk[3]));
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
                    o[0][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[0][kk], o[0][n], 0, 0, 0);
                    o[1][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[1][kk], o[1][n], 0, 0, 0);
                }
            }
        }
    }
    float inv[2];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
        float s = l[mp];
        s += __shfl_xor(s, 16, kWave);
        s += __shfl_xor(s, 32, kWave);
        inv[mp] = 1.f / s;
    }
    const float i2 = inv[1] * lambda[0];
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NV; ++n) {
        if (EXACT || n < nv) {
            o[0][n] = o[0][n] * inv[0] - o[1][n] * i2;
#pragma unroll
            for (int i = 0; i < 4; ++i) ss += o[0][n][i] * o[0][n][i];
        }
    }
    ss += __shfl_xor(ss, 16, kWave);
    ss += __shfl_xor(ss, 32, kWave);
    if (qi >= ntok) return;
    const float f = 1.f / sqrtf(ss / (float)d.V + d.eps) * (1.f - d.diff) *
                    sigmoidf_(bf16_to_f32(gate[(int64_t)(tok0 + qi) * gate_stride + h]));
    uint16_t* orow = out + (int64_t)(tok0 + qi) * out_stride + (int64_t)h * d.V;
    const bool vec = out_vec(out, out_stride, d.V);
#pragma unroll
    for (int n = 0; n < NV; ++n) {
        if (EXACT || n < nv) {
            const float v[4] = {o[0][n][0] * f, o[0][n][1] * f, o[0][n][2] * f, o[0][n][3] * f};
            store4(orow, 16 * n + 4 * g, d.V, vec, v);
        }
    }
}

// ---- host -----------------------------------------------------------------------------------------
const char* bad_shape(const skyrl_diff_shape* sh) {
    if (!sh) return "diff: null shape";
    if (sh->heads <= 0 || sh->kv_heads <= 0 || sh->heads % sh->kv_heads) return "diff: heads must be a multiple of kv_heads";
    if (sh->dim <= 0 || sh->vdim <= 0 || sh->dim > 1024 || sh->vdim > 1024) return "diff: dim and vdim must be in [1, 1024]";
    if (sh->rot_dims < 0 || sh->rot_dims % 2 || sh->rot_dims > sh->dim) return "diff: rot_dims must be even and at most dim";
    if (sh->taps <= 0 || sh->taps > 64) return "diff: taps must be in [1, 64]";
    return nullptr;
}
Dims dims_of(const skyrl_diff_shape* s) {
    return Dims{s->heads, s->kv_heads, s->dim, s->vdim, s->rot_dims, s->taps, s->kv, s->scale, s->diff, s->eps};
}

bool wide(const Dims& d, const void* proj, int64_t stride) {  // every piece of eight channels is one head's and aligned
    return d.D % 8 == 0 && d.V % 8 == 0 && stride % 8 == 0 && aligned16(proj);
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

extern "C" int skyrl_diff_write(const skyrl_diff_shape* shape, const void* proj, int64_t proj_stride,
                                const float* conv_t, const int32_t* cu, const int32_t* rows, const int32_t* bt_row,
                                const int64_t* positions, const int64_t* slots, const float* cos_sin, void* ring,
                                int32_t save_conv, int32_t first, int32_t count, void* q, void* k_cache,
                                void* v_cache, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "diff_write");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(first >= 0 && count >= 0 && proj_stride >= d.channels(), "diff_write: bad sizes");
    if (count == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_t && cu && rows && bt_row && positions && slots && ring && q &&
                      (cos_sin || d.rot == 0) && (!d.kv || (k_cache && v_cache)),
                  "diff_write: null pointer");
    SKYRL_REQUIRE(aligned16(conv_t) && aligned16(ring) && aligned16(q) && aligned16(k_cache) && aligned16(v_cache),
                  "diff_write: 16-byte alignment");
#define LAUNCH_WRITE(VEC)                                                                                             \
    hipLaunchKernelGGL((diff_write_kernel<T, VEC>), dim3(count, (d.channels() / VEC + kNT - 1) / kNT), dim3(kNT), 0,  \
                       as_stream(stream), d, reinterpret_cast<const T*>(proj), proj_stride, conv_t, cu, rows, bt_row, \
                       positions, slots, cos_sin, reinterpret_cast<T*>(ring), save_conv, first,                       \
                       reinterpret_cast<T*>(q), reinterpret_cast<T*>(k_cache), reinterpret_cast<T*>(v_cache))
    SKYRL_DISPATCH_T(dtype, {
        if (wide(d, proj, proj_stride)) LAUNCH_WRITE(8);
        else LAUNCH_WRITE(1);
    })
    return check_launch("diff_write_kernel");
}

extern "C" int skyrl_diff_write_runs(const skyrl_diff_shape* shape, const void* proj, int64_t proj_stride,
                                     const float* conv_t, const int32_t* cu, const int32_t* rows,
                                     const int32_t* bt_row, const int64_t* positions, const int64_t* slots,
                                     const float* cos_sin, const void* ring, const int32_t* runs, int32_t nruns,
                                     void* q, void* k_cache, void* v_cache, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(nruns >= 0 && nruns <= 65535 && proj_stride >= d.channels(), "diff_write_runs: bad sizes");
    SKYRL_REQUIRE(wide(d, proj, proj_stride) && d.taps <= kConvWindow,
                  "diff_write_runs: dim, vdim and proj_stride must be multiples of 8, proj aligned, taps <= 8");
    if (nruns == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && conv_t && cu && rows && bt_row && positions && slots && ring && runs && q &&
                      (cos_sin || d.rot == 0) && (!d.kv || (k_cache && v_cache)),
                  "diff_write_runs: null pointer");
    SKYRL_REQUIRE(aligned16(conv_t) && aligned16(ring) && aligned16(q) && aligned16(k_cache) && aligned16(v_cache),
                  "diff_write_runs: 16-byte alignment");
#define LAUNCH_RUNS(TW)                                                                                                \
    hipLaunchKernelGGL((diff_write_runs_kernel<TW>), dim3((d.channels() / 8 + kNT - 1) / kNT, nruns), dim3(kNT), 0,    \
                       as_stream(stream), d, reinterpret_cast<const uint16_t*>(proj), proj_stride, conv_t, cu, rows,   \
                       bt_row, positions, slots, cos_sin, reinterpret_cast<const uint16_t*>(ring), runs,               \
                       reinterpret_cast<uint16_t*>(q), reinterpret_cast<uint16_t*>(k_cache),                           \
                       reinterpret_cast<uint16_t*>(v_cache))
    if (d.taps <= 4) LAUNCH_RUNS(4);
    else LAUNCH_RUNS(8);
    return check_launch("diff_write_runs_kernel");
}

extern "C" int skyrl_diff_mfma(const skyrl_diff_shape* shape, int32_t dtype) {
    return dtype == SKYRL_BF16 && !bad_shape(shape) && shape->dim <= 128 && shape->vdim <= 256 && shape->scale > 0.f;
}

extern "C" size_t skyrl_diff_attend_workspace_bytes(const skyrl_diff_shape* shape, int32_t T_, int32_t nparts) {
    if (bad_shape(shape) || T_ <= 0 || nparts <= 1) return 0;
    const size_t recs = (size_t)T_ * shape->heads * 2 * nparts;
    return recs * ((size_t)dims_of(shape).vp() + 2) * sizeof(float);
}

#define LAUNCH_DIFF_(KS, NT, PF, EX)                                                                                    \
    hipLaunchKernelGGL((diff_attend_kernel<KS, NT, PF, EX>), dim3(nparts, d.G * d.groups(), T_), dim3(64), 0, s, d, q_, \
                       g_, gate_stride, k_, v_, block_tables, bt_stride, bt_row, positions, lambda, d.scale * kLog2e,   \
                       part_min, nparts, o_, out_stride, ws_o, ws_ml)
#define LAUNCH_DIFF(KS, NT, PF)                             \
    if (ks == KS && nt == NT) LAUNCH_DIFF_(KS, NT, PF, true); \
    else LAUNCH_DIFF_(KS, NT, PF, false)

extern "C" int skyrl_diff_attend(const skyrl_diff_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                                 const void* k_cache, const void* v_cache, const int32_t* block_tables,
                                 int64_t bt_stride, const int32_t* bt_row, const int64_t* positions, int32_t T_,
                                 const float* lambda, int32_t part_min, int32_t nparts, void* out, int64_t out_stride,
                                 void* workspace, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "diff_attend");
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(T_ >= 0 && T_ <= 65535 && d.H <= 65535 && gate_stride >= d.H && out_stride >= (int64_t)d.H * d.V,
                  "diff_attend: bad sizes (T <= 65535)");
    if (T_ == 0) return SKYRL_OK;
    SKYRL_REQUIRE(q && gate && k_cache && v_cache && block_tables && bt_row && positions && lambda && out,
                  "diff_attend: null pointer");
    hipStream_t s = as_stream(stream);
    if (!skyrl_diff_mfma(shape, dtype)) {
        SKYRL_DISPATCH_T(dtype, {
            hipLaunchKernelGGL((diff_attend_plain_kernel<T>), dim3(T_, d.H), dim3(kNT), 2 * d.dp() * sizeof(float), s,
                               d, reinterpret_cast<const T*>(q), reinterpret_cast<const T*>(gate), gate_stride,
                               reinterpret_cast<const T*>(k_cache), reinterpret_cast<const T*>(v_cache), block_tables,
                               bt_stride, bt_row, positions, lambda, reinterpret_cast<T*>(out), out_stride);
        })
        return check_launch("diff_attend_plain_kernel");
    }
    SKYRL_REQUIRE(nparts >= 1 && part_min >= kBS && part_min % kBS == 0,
                  "diff_attend: nparts >= 1 and part_min a positive multiple of 16");
    SKYRL_REQUIRE(nparts == 1 || workspace, "diff_attend: nparts > 1 needs a workspace");
    SKYRL_REQUIRE(aligned16(q) && aligned16(k_cache) && aligned16(v_cache) && aligned16(workspace),
                  "diff_attend: 16-byte alignment");
    const uint16_t* q_ = reinterpret_cast<const uint16_t*>(q);
    const uint16_t* g_ = reinterpret_cast<const uint16_t*>(gate);
    const uint16_t* k_ = reinterpret_cast<const uint16_t*>(k_cache);
    const uint16_t* v_ = reinterpret_cast<const uint16_t*>(v_cache);
    uint16_t* o_ = reinterpret_cast<uint16_t*>(out);
    float* ws_o = reinterpret_cast<float*>(workspace);
    float* ws_ml = ws_o ? ws_o + (size_t)T_ * d.H * 2 * nparts * d.vp() : nullptr;
    const int ks = d.dp() / 16, nt = d.vp() / 16;
    if (ks <= 2) {
        if (nt <= 4) LAUNCH_DIFF(2, 4, 4);
        else if (nt <= 8) LAUNCH_DIFF_(2, 8, 4, false);
        else LAUNCH_DIFF_(2, 16, 3, false);
    } else if (ks <= 4) {
        if (nt <= 4) LAUNCH_DIFF(4, 4, 4);
        else if (nt <= 8) LAUNCH_DIFF(4, 8, 4);
        else LAUNCH_DIFF_(4, 16, 3, false);
    } else {
        if (nt <= 8) LAUNCH_DIFF(8, 8, 3);
        else LAUNCH_DIFF(8, 16, 2);
    }
    const int rc = check_launch("diff_attend_kernel");
    if (rc != SKYRL_OK || nparts == 1) return rc;
    hipLaunchKernelGGL(diff_merge_kernel, dim3(d.H, T_), dim3(2 * kWave), 0, s, d, ws_o, ws_ml, g_, gate_stride,
                       positions, lambda, part_min, nparts, o_, out_stride);
    return check_launch("diff_merge_kernel");
}

#define LAUNCH_PROMPT_(KM, NV, EX)                                                                                     \
    hipLaunchKernelGGL((diff_prefill_kernel<KM, NV, EX>), dim3((unsigned)ntiles * d.H), dim3(kPNT), 0,                 \
                       as_stream(stream), d, reinterpret_cast<const uint16_t*>(q),                                     \
                       reinterpret_cast<const uint16_t*>(gate), gate_stride,                                           \
                       reinterpret_cast<const uint16_t*>(k_cache), reinterpret_cast<const uint16_t*>(v_cache),         \
                       block_tables, bt_stride, tiles, lambda, d.scale * kLog2e, reinterpret_cast<uint16_t*>(out),     \
                       out_stride)
#define LAUNCH_PROMPT(KM, NV)                                         \
    if (d.dp() == 32 * KM && nt == NV) LAUNCH_PROMPT_(KM, NV, true);  \
    else LAUNCH_PROMPT_(KM, NV, false)

extern "C" int skyrl_diff_prefill(const skyrl_diff_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                                  const void* k_cache, const void* v_cache, const int32_t* block_tables,
                                  int64_t bt_stride, const int32_t* tiles, int32_t ntiles, const float* lambda,
                                  void* out, int64_t out_stride, void* stream) {
    const char* bad = bad_shape(shape);
    SKYRL_REQUIRE(!bad, bad);
    const Dims d = dims_of(shape);
    SKYRL_REQUIRE(skyrl_diff_mfma(shape, SKYRL_BF16), "diff_prefill: dim <= 128, vdim <= 256 and scale > 0");
    SKYRL_REQUIRE(ntiles >= 0 && (int64_t)ntiles * d.H < (1 << 30) && gate_stride >= d.H &&
                      out_stride >= (int64_t)d.H * d.V,
                  "diff_prefill: bad sizes");
    if (ntiles == 0) return SKYRL_OK;
    SKYRL_REQUIRE(q && gate && k_cache && v_cache && block_tables && tiles && lambda && out,
                  "diff_prefill: null pointer");
    SKYRL_REQUIRE(aligned16(q) && aligned16(k_cache) && aligned16(v_cache), "diff_prefill: 16-byte alignment");
    const int km = (d.dp() + 31) / 32, nt = d.vp() / 16;
    if (km <= 1) {
        if (nt <= 4) LAUNCH_PROMPT(1, 4);
        else if (nt <= 8) LAUNCH_PROMPT_(1, 8, false);
        else LAUNCH_PROMPT_(1, 16, false);
    } else if (km <= 2) {
        if (nt <= 8) LAUNCH_PROMPT(2, 8);
        else LAUNCH_PROMPT_(2, 16, false);
    } else {
        if (nt <= 8) LAUNCH_PROMPT_(4, 8, false);
        else LAUNCH_PROMPT(4, 16);
    }
    return check_launch("diff_prefill_kernel");
}
