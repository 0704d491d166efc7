// Latent attention (low-rank shared keys/values) over a paged latent cache.
//
// Per token only the normed latent c (rank) and one rotated key part (rot_dim) shared by every head
// are cached. A head's score against token j is q_n . (W_uk c_j) + q_r . kr_j, its value W_uv c_j.
//
// Decode form (latent_attend): the up-projections are moved to the query and the output, so that all
// heads share one key row [c | kr] and one value row c: q_n . (W_uk c) = (W_uk^T q_n) . c, and the sum
// over keys of p_j W_uv c_j = W_uv (sum p_j c_j). The cache is streamed once for up to 16 heads.
// A workgroup takes a share of a token's pages, four pages (64 keys) at a time: each wave scores one
// page, S^T[token x head] = K[16 x row] . Q^T[row x 16] (mfma_f32_16x16x32_bf16, K straight from HBM to
// registers, the next tile's loads in flight), scores and latents go to LDS, and each wave sums a quarter of the rank over all 64 keys, O^T[rank x head] +=
// C^T[rank x keys] . P^T[keys x head], C^T by transposing LDS reads.
//
// Prompt form (latent_gather + two library products + latent_prefill): a long portion pays the
// up-projection once per key instead of once per query, and the scores cost dim + rot_dim instead of
// rank + rot_dim per pair. latent_prefill is a windowed flash-style kernel: four waves share a K and
// a V^T tile of 64 keys in LDS, each wave owns 32 queries of one head.
#include "elem.h"

namespace skyrl {
namespace {

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kBS = 16;  // tokens per cache block
constexpr int kNT = 256;

// Dimension pairs of the rotation: neighbours, or i with i + rot / 2 (halves).
struct Pairs {
    int rot, halves;
    __device__ __forceinline__ int first(int i) const { return halves ? i : 2 * i; }
    __device__ __forceinline__ int second(int i) const { return halves ? i + rot / 2 : 2 * i + 1; }
};

// One workgroup per token. Parts of the row p that are there: the rotated parts of `heads` queries at its start, or
// (q_rank > 0) a query latent that is normed in place; the key latent and its rotated part at lat_at (rank > 0).
template <typename T>
__global__ __launch_bounds__(kNT) void latent_write_kernel(T* __restrict__ proj, int64_t stride, int heads, int dim,
                                                           Pairs pr, int q_rank, const T* __restrict__ q_norm,
                                                           int rank, int lat_at, const T* __restrict__ norm_w,
                                                           float eps, const int64_t* __restrict__ positions,
                                                           const int64_t* __restrict__ slots,
                                                           const float* __restrict__ cos_sin, T* __restrict__ cache,
                                                           int row) {
    __shared__ float s_red[kNT / kWave];
    const int t = blockIdx.x;
    T* p = proj + (int64_t)t * stride;
    const int rot = pr.rot, qd = dim + rot, h2 = rot / 2;
    const float* cs = cos_sin + positions[t] * rot;
    if (q_rank > 0) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < q_rank; i += kNT) {
            const float v = ld(p + i);
            ss += v * v;
        }
        const float r = 1.f / sqrtf(block_total<kNT>(ss, s_red) / (float)q_rank + eps);
        for (int i = threadIdx.x; i < q_rank; i += kNT) st(p + i, ld(p + i) * r * ld(q_norm + i));
    }
    if (rank > 0) {
        const T* lat = p + lat_at;
        float ss = 0.f;
        for (int i = threadIdx.x; i < rank; i += kNT) {
            const float v = ld(lat + i);
            ss += v * v;
        }
        const float r = 1.f / sqrtf(block_total<kNT>(ss, s_red) / (float)rank + eps);
        const int64_t slot = slots[t];
        if (slot >= 0) {
            T* c = cache + slot * row;
            for (int i = threadIdx.x; i < rank; i += kNT) st(c + i, ld(lat + i) * r * ld(norm_w + i));
            for (int i = threadIdx.x; i < h2; i += kNT) {
                const int a = pr.first(i), b = pr.second(i);
                const float u = ld(lat + rank + a), v = ld(lat + rank + b);
                st(c + rank + a, u * cs[i] - v * cs[h2 + i]);
                st(c + rank + b, v * cs[i] + u * cs[h2 + i]);
            }
        }
    }
    for (int e = threadIdx.x; e < heads * h2; e += kNT) {
        const int h = e / h2, i = e - h * h2;
        T* q = p + (int64_t)h * qd + dim;
        const int a = pr.first(i), b = pr.second(i);
        const float u = ld(q + a), v = ld(q + b);
        st(q + a, u * cs[i] - v * cs[h2 + i]);
        st(q + b, v * cs[i] + u * cs[h2 + i]);
    }
}

// What ends a head's softmax: a learned sink in the denominator and a sigmoid gate on the output, each optional.
template <typename T>
struct HeadEnd {
    const float* sinks;  // [heads]
    const T* gate;       // logits [token][head]
    int64_t gate_stride;
    __device__ __forceinline__ float sink(int h) const { return sinks ? sinks[h] : -INFINITY; }
    __device__ __forceinline__ float gated(int t, int h) const {
        return gate ? sigmoidf_(ld(gate + (int64_t)t * gate_stride + h)) : 1.f;
    }
};
// Factor of the value sums with running maximum m and denominator l, all in powers of two; sink in the same units.
__device__ __forceinline__ float sum_factor(float m, float l, float sink) {
    const float mm = fmaxf(m, sink), a = fast_exp2(m - mm);
    return a / (l * a + fast_exp2(sink - mm));
}

// ---- decode form, plain: one workgroup per (token, head), any rank up to 2048, f32 or bf16 ----
template <typename T>
__global__ __launch_bounds__(kNT) void latent_attend_plain_kernel(
    const T* __restrict__ qa, const T* __restrict__ q_rot, int64_t q_stride, int64_t q_head,
    const T* __restrict__ cache, int row, const int32_t* __restrict__ tables, int64_t bt_stride,
    const int32_t* __restrict__ bt_row, const int64_t* __restrict__ positions, int ntok, int heads, int rank, int rot,
    float scale, int window, HeadEnd<T> end, T* __restrict__ out) {
    extern __shared__ float s_q[];  // rank + rot
    __shared__ float s_p[kWave];
    constexpr int kAcc = 8;
    const int h = blockIdx.x, t = blockIdx.y;
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int pos = (int)positions[t];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride;
    const int n = rank + rot;
    for (int i = threadIdx.x; i < n; i += kNT)
        s_q[i] = i < rank ? ld(qa + ((int64_t)h * ntok + t) * rank + i)
                          : ld(q_rot + (int64_t)t * q_stride + (int64_t)h * q_head + (i - rank));
    __syncthreads();
    float acc[kAcc], m = -INFINITY, l = 0.f;
#pragma unroll
    for (int k = 0; k < kAcc; ++k) acc[k] = 0.f;
    for (int j0 = lo; j0 <= pos; j0 += kWave) {
        const int nk = min(kWave, pos + 1 - j0);
        for (int jj = wave; jj < nk; jj += kNT / kWave) {
            const int j = j0 + jj;
            const T* key = cache + ((int64_t)bt[j / kBS] * kBS + j % kBS) * row;
            float s = 0.f;
            for (int i = lane; i < n; i += kWave) s += s_q[i] * ld(key + i);
            s = wave_sum(s);
            if (lane == 0) s_p[jj] = s * scale;
        }
        __syncthreads();
        const float sv = lane < nk ? s_p[lane] : -INFINITY;
        const float mn = fmaxf(m, wave_max(sv));
        const float alpha = expf(m - mn);
        const float p = lane < nk ? expf(sv - mn) : 0.f;
        l = l * alpha + wave_sum(p);
        m = mn;
        __syncthreads();
        if (threadIdx.x < kWave) s_p[threadIdx.x] = p;
        __syncthreads();
#pragma unroll
        for (int k = 0; k < kAcc; ++k) acc[k] *= alpha;
        for (int jj = 0; jj < nk; ++jj) {
            const int j = j0 + jj;
            const T* key = cache + ((int64_t)bt[j / kBS] * kBS + j % kBS) * row;
            const float pj = s_p[jj];
#pragma unroll
            for (int k = 0; k < kAcc; ++k) {
                const int d = threadIdx.x + k * kNT;
                if (d < rank) acc[k] += pj * ld(key + d);
            }
        }
        __syncthreads();
    }
    const float sink = end.sink(h), mm = fmaxf(m, sink), a = expf(m - mm);
    const float f = a / (l * a + expf(sink - mm)) * end.gated(t, h);
#pragma unroll
    for (int k = 0; k < kAcc; ++k) {
        const int d = threadIdx.x + k * kNT;
        if (d < rank) st(out + ((int64_t)h * ntok + t) * rank + d, acc[k] * f);
    }
}

// Pages [p0, p0 + np) of a token's context cut into shares of `per` pages; parts = number of shares.
struct PageSplit {
    int p0, per, parts, np;
};
__device__ __forceinline__ PageSplit page_split(int lo, int pos, int part_min, int nparts) {
    PageSplit s;
    s.p0 = lo / kBS;
    s.np = pos / kBS - s.p0 + 1;
    s.per = max((s.np + nparts - 1) / nparts, part_min / kBS);
    s.parts = (s.np + s.per - 1) / s.per;
    return s;
}

// Transposing LDS read: within each group of 16 lanes, lane 4 k + q supplies the address of row k's
// elements 4 q .. 4 q + 3, and lane i receives element i of the four rows.
__device__ __forceinline__ s16x4 lds_read_tr(const uint16_t* p) {
    typedef __attribute__((address_space(3))) s16x4* lds_ptr;
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)p);
}

// ---- decode form, MFMA ------------------------------------------------------------------------
// grid (nparts, ceil(heads / (16 HG)), tokens), four waves per group of 16 heads. A tile is four pages, staged
// through registers into LDS in whole 1 KB pieces (a page is contiguous; row-by-row operand loads from
// HBM ran at half the rate), one page per wave, the next tile's loads in flight. Each wave scores one
// page for its head group; for the values it takes a quarter of the rank over all 64 keys. With HG = 2
// two head groups share the tile and each stages half of it. NV: 16-wide tiles of the rank,
// NK: 32-wide steps of the cache row; EXACT when both equal the shape's own.
template <int NV, int NK, bool EXACT, int HG>
__global__ __launch_bounds__(kNT * HG) __attribute__((amdgpu_waves_per_eu(1, 2))) void latent_attend_mfma_kernel(
    const uint16_t* __restrict__ qa, const uint16_t* __restrict__ q_rot, int64_t q_stride, int64_t q_head,
    const uint16_t* __restrict__ cache, int row, const int32_t* __restrict__ tables, int64_t bt_stride,
    const int32_t* __restrict__ bt_row, const int64_t* __restrict__ positions, int ntok, int heads, int rank, int rot,
    float scale_log2, int window, int part_min, int nparts, HeadEnd<uint16_t> end, uint16_t* __restrict__ out,
    float* __restrict__ ws_o, float* __restrict__ ws_ml) {
    constexpr int LDR = NK * 32 + 8;  // padded LDS row
    constexpr int LDS_ = 64 + 4, NW = NV / 4, NT = kNT * HG;
    constexpr int NL = (NK + HG - 1) / HG;  // 16-byte pieces of its page per lane
    __shared__ __attribute__((aligned(16))) uint16_t s_c[64 * LDR];  // first the query, then the tile
    __shared__ __attribute__((aligned(16))) float s_scores[HG * 16 * LDS_];  // scores [head][key of the tile]
    const int t = blockIdx.z;
    const int pos = (int)positions[t];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const PageSplit sp = page_split(lo, pos, part_min, nparts);
    const int part = blockIdx.x;
    if (part >= sp.parts) return;
    const int nk = EXACT ? NK : row / 32;
    const int nv = EXACT ? NV : (rank + 15) / 16;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6) & 3, hg = __builtin_amdgcn_readfirstlane(tid >> 8);
    const int c = lane & 15, g = lane >> 4;
    const int h0 = blockIdx.y * 16 * HG;  // the workgroup's first head
    float* s_s = s_scores + hg * 16 * LDS_;

    const int first = sp.p0 + part * sp.per;
    const int np = min(sp.per, sp.np - part * sp.per);
    const int32_t* bt = tables + (int64_t)bt_row[t] * bt_stride + first;
    // Pages come in windows of 64, whose block ids a wave holds by lane (no table load ahead of a page's).
    // Loads are unconditional, the last page again past the end: a branch around them would turn every
    // wait into one for all loads in flight.
    const int rc = EXACT ? NK * 4 : nk * 4;  // pieces per row
    auto piece = [&](int k) { return min(lane + 64 * (hg + HG * k), 16 * rc - 1); };
    int lds_at[NL];
#pragma unroll
    for (int k = 0; k < NL; ++k) {
        const int e = piece(k), r = e / rc;
        lds_at[k] = (16 * wave + r) * LDR + (e - r * rc) * 8;
    }
    s16x8 st_[NL];
    int tbl = 0, npw = 0;
    auto window_at = [&](int w0) {
        npw = min(64, np - w0);
        tbl = bt[w0 + min(lane, npw - 1)];
    };
    auto load_page = [&](int j) {
        const uint16_t* p = cache + (int64_t)__builtin_amdgcn_readlane(tbl, min(j, npw - 1)) * kBS * row;
#pragma unroll
        for (int k = 0; k < NL; ++k) st_[k] = *reinterpret_cast<const s16x8*>(p + piece(k) * 8);
    };
    window_at(0);
    load_page(wave);

    // the query rows of this head group, [latent | rotated | 0], through LDS into MFMA operands
    const bool vec = rank % 8 == 0;
    for (int e = tid; e < HG * 16 * NK * 4; e += NT) {
        const int hh = e / (NK * 4), d = (e - hh * (NK * 4)) * 8, h = h0 + hh;
        s16x8 f = {0, 0, 0, 0, 0, 0, 0, 0};
        if (h < heads && d < row) {
            const uint16_t* qrow = qa + ((int64_t)h * ntok + t) * rank;
            const uint16_t* rrow = q_rot + (int64_t)t * q_stride + (int64_t)h * q_head;
            if (vec && d + 8 <= rank) {
                f = *reinterpret_cast<const s16x8*>(qrow + d);
            } else {
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int dd = d + j;
                    const uint16_t* src = dd < rank ? qrow + dd : dd < rank + rot ? rrow + (dd - rank) : qrow;
                    const uint16_t x = *src;
                    f[j] = (short)(dd < rank + rot ? x : 0);
                }
            }
        }
        *reinterpret_cast<s16x8*>(&s_c[hh * LDR + d]) = f;
    }
    __syncthreads();
    s16x8 qf[NK];
#pragma unroll
    for (int s = 0; s < NK; ++s) qf[s] = *reinterpret_cast<const s16x8*>(&s_c[(16 * hg + c) * LDR + 32 * s + 8 * g]);

    f32x4 o[NW];
#pragma unroll
    for (int n = 0; n < NW; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    auto tile = [&](int w0, int j0) {
        const int tb = (first + w0 + j0 + wave) * kBS;  // this wave's page
        const bool edge = j0 + wave >= npw || tb < lo || tb + kBS - 1 > pos;
        if (edge) {  // a masked slot may hold anything: 0 * NaN must not reach the sums
#pragma unroll
            for (int k = 0; k < NL; ++k) {
                const int tok = tb + piece(k) / rc;
                if (!(j0 + wave < npw && tok >= lo && tok <= pos)) st_[k] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
            }
        }
        __syncthreads();  // the query operands, or the previous tile, are consumed
#pragma unroll
        for (int k = 0; k < NL; ++k) *reinterpret_cast<s16x8*>(&s_c[lds_at[k]]) = st_[k];
        load_page(j0 + 4 + wave);
        __syncthreads();
        f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = sa;
#pragma unroll
        for (int s = 0; s < NK; ++s) {
            if (EXACT || s < nk) {
                const s16x8 kf = *reinterpret_cast<const s16x8*>(&s_c[(16 * wave + c) * LDR + 32 * s + 8 * g]);
                if (s & 1) sb = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], sb, 0, 0, 0);
                else sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], sa, 0, 0, 0);
            }
        }
        f32x4 sv = (sa + sb) * scale_log2;  // token tb + 4 g + i, head c
        if (edge) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int tok = tb + 4 * g + i;
                if (!(j0 + wave < npw && tok >= lo && tok <= pos)) sv[i] = -INFINITY;
            }
        }
        *reinterpret_cast<f32x4*>(&s_s[c * LDS_ + 16 * wave + 4 * g]) = sv;
        __syncthreads();
        // every wave: weights of all 64 keys, the lane's own 16 in the order of the MFMA operand
        f32x4 x[4];
#pragma unroll
        for (int w = 0; w < 4; ++w) x[w] = *reinterpret_cast<const f32x4*>(&s_s[c * LDS_ + 16 * w + 4 * g]);
        float bm = -INFINITY;
#pragma unroll
        for (int w = 0; w < 4; ++w) bm = fmaxf(bm, fmaxf(fmaxf(x[w][0], x[w][1]), fmaxf(x[w][2], x[w][3])));
        bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
        bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
        const float mn = fmaxf(m, bm);
        const float alpha = fast_exp2(m - mn);  // first tile: m = -inf, 0; every share starts with a visible key
        float sum = 0.f;
        s16x8 pf[2];
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            uint32_t pk[4];
#pragma unroll
            for (int b = 0; b < 2; ++b) {
                float p[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    p[i] = fast_exp2(x[2 * kk + b][i] - mn);
                    sum += p[i];
                }
                pk[2 * b] = pack_bf16x2(p[0], p[1]);
                pk[2 * b + 1] = pack_bf16x2(p[2], p[3]);
            }
            pf[kk] = __builtin_bit_cast(s16x8, make_uint4(pk[0], pk[1], pk[2], pk[3]));
        }
        l = l * alpha + sum;
        m = mn;
#pragma unroll
        for (int n = 0; n < NW; ++n) {
            const int vt = wave * NW + n;
            if (EXACT || vt < nv) {
                o[n] = o[n] * alpha;
#pragma unroll
                for (int kk = 0; kk < 2; ++kk) {
                    const uint16_t* vp = &s_c[(32 * kk + 4 * g + (c >> 2)) * LDR + 16 * vt + 4 * (c & 3)];
                    const s16x4 a = lds_read_tr(vp), b = lds_read_tr(vp + 16 * LDR);
                    const s16x8 vf = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
                    o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[kk], o[n], 0, 0, 0);
                }
            }
        }
    };
    for (int w0 = 0; w0 < np; w0 += 64) {
        if (w0 > 0) {
            window_at(w0);
            load_page(wave);
        }
        for (int j0 = 0; j0 < npw; j0 += 4) tile(w0, j0);
    }
    l += __shfl_xor(l, 16, kWave);  // the sum over all keys, the same in every wave
    l += __shfl_xor(l, 32, kWave);
    const int h = h0 + 16 * hg + c;
    if (h >= heads) return;
    if (sp.parts == 1) {
        const float inv = sum_factor(m, l, end.sink(h) * kLog2e) * end.gated(t, h);
        uint16_t* orow = out + ((int64_t)h * ntok + t) * rank;
#pragma unroll
        for (int n = 0; n < NW; ++n) {
            const int d = 16 * (wave * NW + n) + 4 * g;
            if (EXACT || (rank % 4 == 0 && d + 4 <= rank)) {
                *reinterpret_cast<uint2*>(orow + d) =
                    make_uint2(pack_bf16x2(o[n][0] * inv, o[n][1] * inv), pack_bf16x2(o[n][2] * inv, o[n][3] * inv));
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (d + i < rank) orow[d + i] = f32_to_bf16(o[n][i] * inv);
            }
        }
    } else {
        const int64_t rec = ((int64_t)t * heads + h) * nparts + part;
        float* wo = ws_o + rec * (((rank + 15) / 16) * 16);
#pragma unroll
        for (int n = 0; n < NW; ++n)
            if (EXACT || wave * NW + n < nv) *reinterpret_cast<f32x4*>(wo + 16 * (wave * NW + n) + 4 * g) = o[n];
        if (wave == 0 && g == 0) {
            ws_ml[rec * 2] = m;
            ws_ml[rec * 2 + 1] = l;
        }
    }
}

// Merge of the shares of one (token, head): grid (heads, tokens), one wave per 256 dimensions.
__global__ __launch_bounds__(kWave * 2) void latent_merge_kernel(const float* __restrict__ ws_o,
                                                                 const float* __restrict__ ws_ml,
                                                                 const int64_t* __restrict__ positions, int ntok,
                                                                 int heads, int rank, int window, int part_min,
                                                                 int nparts, HeadEnd<uint16_t> end,
                                                                 uint16_t* __restrict__ out) {
    const int h = blockIdx.x, t = blockIdx.y, lane = threadIdx.x & 63;
    const int pos = (int)positions[t];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const PageSplit sp = page_split(lo, pos, part_min, nparts);
    if (sp.parts == 1) return;
    const int64_t rec = ((int64_t)t * heads + h) * nparts;
    const int rp = ((rank + 15) / 16) * 16;
    float M = -INFINITY;
    for (int p = lane; p < sp.parts; p += kWave) M = fmaxf(M, ws_ml[(rec + p) * 2]);
    M = wave_max(M);
    float L = 0.f;
    for (int p = lane; p < sp.parts; p += kWave) L += fast_exp2(ws_ml[(rec + p) * 2] - M) * ws_ml[(rec + p) * 2 + 1];
    const float inv = sum_factor(M, wave_sum(L), end.sink(h) * kLog2e) * end.gated(t, h);
    uint16_t* orow = out + ((int64_t)h * ntok + t) * rank;
    for (int d = threadIdx.x * 4; d < rp; d += kWave * 8) {
        float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
        for (int p = 0; p < sp.parts; ++p) {
            const float w = fast_exp2(ws_ml[(rec + p) * 2] - M) * inv;
            const float4 x = ld4(ws_o + (rec + p) * rp + d);
            acc.x += w * x.x; acc.y += w * x.y; acc.z += w * x.z; acc.w += w * x.w;
        }
        if (rank % 4 == 0 && d + 4 <= rank) {
            st4(orow + d, acc);
        } else {
            const float v[4] = {acc.x, acc.y, acc.z, acc.w};
            for (int i = 0; i < 4; ++i)
                if (d + i < rank) orow[d + i] = f32_to_bf16(v[i]);
        }
    }
}

// ---- prompt form --------------------------------------------------------------------------------
// grid (ceil(max rows / 16), nseg): 16 packed rows per workgroup; rows past the segment's count up to the next
// multiple of 64 are zeroed.
template <typename T>
__global__ __launch_bounds__(kNT) void latent_gather_kernel(const T* __restrict__ cache, int row,
                                                            const int32_t* __restrict__ tables, int64_t bt_stride,
                                                            const int32_t* __restrict__ seg, int rank, int rot,
                                                            T* __restrict__ latent, T* __restrict__ k_rot) {
    const int32_t* sg = seg + 4 * blockIdx.y;
    const int count = sg[2], padded = (count + 63) / 64 * 64;
    const int r0 = blockIdx.x * 16;
    if (r0 >= padded) return;
    const int32_t* bt = tables + (int64_t)sg[0] * bt_stride;
    const int n = rank + rot;
    if (rank % 4 == 0 && rot % 4 == 0) {
        const int n4 = n / 4;
        for (int e = threadIdx.x; e < 16 * n4; e += kNT) {
            const int rr = e / n4, d = (e - rr * n4) * 4, r = r0 + rr;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (r < count) {
                const int p = sg[1] + r;
                v = ld4(cache + ((int64_t)bt[p / kBS] * kBS + p % kBS) * row + d);
            }
            const int64_t dst = sg[3] + r;
            if (d < rank) st4(latent + dst * rank + d, v);
            else st4(k_rot + dst * rot + (d - rank), v);
        }
        return;
    }
    for (int e = threadIdx.x; e < 16 * n; e += kNT) {
        const int rr = e / n, d = e - rr * n, r = r0 + rr;
        float v = 0.f;
        if (r < count) {
            const int p = sg[1] + r;
            v = ld(cache + ((int64_t)bt[p / kBS] * kBS + p % kBS) * row + d);
        }
        const int64_t dst = sg[3] + r;
        if (d < rank) st(latent + dst * rank + d, v);
        else st(k_rot + dst * rot + (d - rank), v);
    }
}

constexpr int kKT = 64;   // keys per LDS tile

// 8 consecutive elements starting at column d of a key row assembled from [nope | rot | 0].
template <bool VEC>
__device__ __forceinline__ s16x8 key_chunk(const uint16_t* nope, const uint16_t* rotp, int d, int dim, int rot) {
    s16x8 f = {0, 0, 0, 0, 0, 0, 0, 0};
    if constexpr (VEC) {
        if (d < dim) f = *reinterpret_cast<const s16x8*>(nope + d);
        else if (d < dim + rot) f = *reinterpret_cast<const s16x8*>(rotp + (d - dim));
        return f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int dd = d + j;
        f[j] = (short)(dd < dim ? nope[dd] : dd < dim + rot ? rotp[dd - dim] : (uint16_t)0);
    }
    return f;
}

// QT: 16-query tiles per wave, 128 queries per workgroup. VEC: every row piece is 16-byte aligned.
template <int NK, int NV, int QT, bool VEC>
__global__ __launch_bounds__(512 / QT) __attribute__((amdgpu_waves_per_eu(2))) void latent_prefill_kernel(
    const uint16_t* __restrict__ q, int64_t q_stride, const uint16_t* __restrict__ k_nope, int64_t k_stride,
    const uint16_t* __restrict__ k_rot, const uint16_t* __restrict__ v_t, int64_t vt_stride,
    const int32_t* __restrict__ tiles, int heads, int dim, int rot, int vdim, float scale_log2, int window,
    HeadEnd<uint16_t> end, uint16_t* __restrict__ out, int64_t out_stride) {
    constexpr int NT = 512 / QT, QW = 16 * QT;
    constexpr int LDK = NK * 32 + 8, LDV = kKT + 8;
    constexpr int TPK = NT / kKT, KPT = NK * 4 / TPK;     // threads per key row, 16-byte chunks per thread
    constexpr int VPT = NV * 16 * (kKT / 8) / NT, VROWS = NT / 8;
    __shared__ __attribute__((aligned(16))) uint16_t s_k[kKT * LDK];
    __shared__ __attribute__((aligned(16))) uint16_t s_v[NV * 16 * LDV];
    const int h = blockIdx.x % heads;  // one head's tiles stay on one XCD when heads is a multiple of 8
    const int32_t* tl = tiles + 8 * (blockIdx.x / heads);
    const int tok0 = tl[0], ntok = tl[1], pos0 = tl[2], seg_row = tl[3], seg_pos = tl[4];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = lane & 15, g = lane >> 4;
    const int dk = dim + rot;
    const int w = window > 0 ? window : 0x3fffffff;

    // this wave's queries: QW * wave + 16 qq + c
    s16x8 qf[QT][NK];
    int qpos[QT];
#pragma unroll
    for (int qq = 0; qq < QT; ++qq) {
        const int qi = QW * wave + 16 * qq + c;
        const bool ok = qi < ntok;
        qpos[qq] = pos0 + qi;
        const uint16_t* qr = q + (int64_t)(tok0 + (ok ? qi : 0)) * q_stride + (int64_t)h * dk;
#pragma unroll
        for (int s = 0; s < NK; ++s) {
            s16x8 f = {0, 0, 0, 0, 0, 0, 0, 0};
            if (ok) f = key_chunk<VEC>(qr, qr + dim, 32 * s + 8 * g, dim, rot);
            qf[qq][s] = f;
        }
    }
    f32x4 o[NV][QT];
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
        for (int qq = 0; qq < QT; ++qq) o[n][qq] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m[QT], l[QT];
#pragma unroll
    for (int qq = 0; qq < QT; ++qq) {
        m[qq] = -INFINITY;
        l[qq] = 0.f;
    }

    const int lo = max(0, pos0 - w + 1);
    const int j0 = (lo - seg_pos) / kKT, j1 = (pos0 + ntok - 1 - seg_pos) / kKT;
    const int wq0 = pos0 + QW * wave;                                // the wave's first query
    const int wq1 = min(wq0 + QW - 1, pos0 + ntok - 1);                  // and its last
    s16x8 kr[KPT], vr[VPT];
    const int ktok = threadIdx.x / TPK, kd = (threadIdx.x % TPK) * 8;   // key row and first column of this thread
    const int vd = threadIdx.x >> 3, vtok = (threadIdx.x & 7) * 8;      // value row and first key
    auto fetch = [&](int j) {
        const int64_t r0 = seg_row + (int64_t)j * kKT;
        const uint16_t* kp = k_nope + (r0 + ktok) * k_stride + (int64_t)h * dim;
        const uint16_t* rp = k_rot + (r0 + ktok) * rot;
#pragma unroll
        for (int i = 0; i < KPT; ++i) kr[i] = key_chunk<VEC>(kp, rp, kd + 8 * TPK * i, dim, rot);
        const uint16_t* vp = v_t + ((int64_t)h * vdim + vd) * vt_stride + r0 + vtok;
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            vr[i] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
            if (vd + VROWS * i < vdim) vr[i] = *reinterpret_cast<const s16x8*>(vp + (int64_t)VROWS * i * vt_stride);
        }
    };
    fetch(j0);
    for (int j = j0; j <= j1; ++j) {
        __syncthreads();  // the previous tile is consumed
#pragma unroll
        for (int i = 0; i < KPT; ++i) *reinterpret_cast<s16x8*>(&s_k[ktok * LDK + kd + 8 * TPK * i]) = kr[i];
#pragma unroll
        for (int i = 0; i < VPT; ++i) *reinterpret_cast<s16x8*>(&s_v[(vd + VROWS * i) * LDV + vtok]) = vr[i];
        __syncthreads();
        if (j < j1) fetch(j + 1);
        const int kp0 = seg_pos + j * kKT, kp1 = kp0 + kKT - 1;
        if (kp0 > wq1 || kp1 < wq0 - w + 1 || wq0 > wq1) continue;  // no key of this tile for this wave
        const bool edge = kp1 > wq0 || kp0 < wq1 - w + 1 || wq1 != wq0 + QW - 1;
        f32x4 sc[4][QT];
#pragma unroll
        for (int tt = 0; tt < 4; ++tt)
#pragma unroll
            for (int qq = 0; qq < QT; ++qq) sc[tt][qq] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < NK; ++s) {
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) {
                const s16x8 kf = *reinterpret_cast<const s16x8*>(&s_k[(16 * tt + c) * LDK + 32 * s + 8 * g]);
#pragma unroll
                for (int qq = 0; qq < QT; ++qq)
                    sc[tt][qq] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qq][s], sc[tt][qq], 0, 0, 0);
            }
        }
        s16x8 pf[QT][2];  // [query tile][32-key step]
        float alpha[QT];
#pragma unroll
        for (int qq = 0; qq < QT; ++qq) {
            float bm = -INFINITY;
            const unsigned dist = qpos[qq] - kp0 - 4 * g;  // to the lane's first key
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    float v = sc[tt][qq][i] * scale_log2;
                    if (edge && dist - (16 * tt + i) >= (unsigned)w) v = -INFINITY;  // after the query, or too far back
                    sc[tt][qq][i] = v;
                    bm = fmaxf(bm, v);
                }
            bm = fmaxf(bm, __shfl_xor(bm, 16, kWave));
            bm = fmaxf(bm, __shfl_xor(bm, 32, kWave));
            const float mn = fmaxf(m[qq], bm);
            const float base = mn == -INFINITY ? 0.f : mn;  // no key seen yet: every weight is 0
            alpha[qq] = fast_exp2(m[qq] - base);
            float sum = 0.f;
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                uint32_t pk[4];
#pragma unroll
                for (int b = 0; b < 2; ++b) {
                    float p[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        p[i] = fast_exp2(sc[2 * kk + b][qq][i] - base);
                        sum += p[i];
                    }
                    pk[2 * b] = pack_bf16x2(p[0], p[1]);
                    pk[2 * b + 1] = pack_bf16x2(p[2], p[3]);
                }
                pf[qq][kk] = __builtin_bit_cast(s16x8, make_uint4(pk[0], pk[1], pk[2], pk[3]));
            }
            l[qq] = l[qq] * alpha[qq] + sum;
            m[qq] = mn;
        }
#pragma unroll
        for (int n = 0; n < NV; ++n) {
#pragma unroll
            for (int qq = 0; qq < QT; ++qq) o[n][qq] = o[n][qq] * alpha[qq];
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                const uint16_t* vp = &s_v[(16 * n + c) * LDV + 32 * kk + 4 * g];
                const s16x4 v0 = *reinterpret_cast<const s16x4*>(vp);
                const s16x4 v1 = *reinterpret_cast<const s16x4*>(vp + 16);
                const s16x8 vf = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
                for (int qq = 0; qq < QT; ++qq)
                    o[n][qq] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[qq][kk], o[n][qq], 0, 0, 0);
            }
        }
    }
#pragma unroll
    for (int qq = 0; qq < QT; ++qq) {
        float s = l[qq];
        s += __shfl_xor(s, 16, kWave);
        s += __shfl_xor(s, 32, kWave);
        const int qi = QW * wave + 16 * qq + c;
        if (qi >= ntok) continue;
        const float inv = sum_factor(m[qq], s, end.sink(h) * kLog2e) * end.gated(tok0 + qi, h);
        uint16_t* orow = out + (int64_t)(tok0 + qi) * out_stride + (int64_t)h * vdim;
        const bool ovec = vdim % 4 == 0 && out_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & 7) == 0;
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const int d = 16 * n + 4 * g;
            if (ovec && d + 4 <= vdim) {
                *reinterpret_cast<uint2*>(orow + d) = make_uint2(pack_bf16x2(o[n][qq][0] * inv, o[n][qq][1] * inv),
                                                                 pack_bf16x2(o[n][qq][2] * inv, o[n][qq][3] * inv));
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (d + i < vdim) orow[d + i] = f32_to_bf16(o[n][qq][i] * inv);
            }
        }
    }
}


}  // namespace
}  // namespace skyrl

using namespace skyrl;

extern "C" int skyrl_latent_write(void* proj, int64_t proj_stride, int32_t T_, int32_t heads, int32_t dim,
                                  int32_t rot_dim, int32_t halves, int32_t q_rank, const void* q_norm, int32_t rank,
                                  int32_t latent_at, const void* norm_weight, float eps, const int64_t* positions,
                                  const int64_t* slots, const float* cos_sin, void* cache, int32_t row, int32_t dtype,
                                  void* stream) {
    SKYRL_REQUIRE_T(dtype, "latent_write");
    SKYRL_REQUIRE(T_ >= 0 && heads >= 0 && dim >= 0 && rot_dim >= 0 && rot_dim % 2 == 0 && rank >= 0 && q_rank >= 0,
                  "latent_write: bad sizes");
    SKYRL_REQUIRE(heads == 0 || q_rank == 0, "latent_write: queries or their latent, not both");
    SKYRL_REQUIRE(rank == 0 || (row % 32 == 0 && row >= rank + rot_dim),
                  "latent_write: row must be a multiple of 32 >= rank + rot_dim");
    const int64_t qw = q_rank > 0 ? q_rank : (int64_t)heads * (dim + rot_dim);
    SKYRL_REQUIRE(proj_stride >= qw && (rank == 0 || (latent_at >= qw && proj_stride >= (int64_t)latent_at + rank + rot_dim)),
                  "latent_write: proj_stride");
    if (T_ == 0) return SKYRL_OK;
    SKYRL_REQUIRE(proj && positions && cos_sin && (q_rank == 0 || q_norm) && (rank == 0 || (norm_weight && slots && cache)),
                  "latent_write: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((latent_write_kernel<T>), dim3(T_), dim3(kNT), 0, as_stream(stream),
                           reinterpret_cast<T*>(proj), proj_stride, heads, dim, Pairs{rot_dim, halves}, q_rank,
                           reinterpret_cast<const T*>(q_norm), rank, latent_at, reinterpret_cast<const T*>(norm_weight),
                           eps, positions, slots, cos_sin, reinterpret_cast<T*>(cache), row);
    })
    return check_launch("latent_write_kernel");
}

extern "C" int skyrl_latent_attend_mfma(int32_t rank, int32_t rot_dim, int32_t row, int32_t dtype) {
    return dtype == SKYRL_BF16 && rank > 0 && rot_dim >= 0 && rank <= 512 && row % 32 == 0 && row >= rank + rot_dim &&
           row <= 640;
}

extern "C" size_t skyrl_latent_attend_workspace_bytes(int32_t T_, int32_t heads, int32_t rank, int32_t nparts) {
    const size_t recs = (size_t)(T_ > 0 ? T_ : 0) * heads * nparts;
    return recs * ((size_t)((rank + 15) / 16) * 16 + 2) * sizeof(float) + 16;
}

#define LAUNCH_ATTEND_(NV, NK, EX, HG)                                                                               \
    hipLaunchKernelGGL((latent_attend_mfma_kernel<NV, NK, EX, HG>), dim3(nparts, (heads + 16 * HG - 1) / (16 * HG), T_), \
                       dim3(kNT * HG), 0, s, q_, r_, q_stride, q_head, c_, row, block_tables, bt_stride, bt_row,     \
                       positions, T_, heads, rank, rot_dim, scale * kLog2e, window, part_min, nparts, end_, o_,  \
                       ws_o, ws_ml)
#define LAUNCH_ATTEND(NV, NK, EX)                    \
    if (heads > 16) LAUNCH_ATTEND_(NV, NK, EX, 2);   \
    else LAUNCH_ATTEND_(NV, NK, EX, 1)

extern "C" int skyrl_latent_attend(const void* qa, const void* q_rot, int64_t q_stride, int64_t q_head,
                                   const void* cache, int32_t row, const int32_t* block_tables, int64_t bt_stride,
                                   const int32_t* bt_row, const int64_t* positions, int32_t T_, int32_t heads,
                                   int32_t rank, int32_t rot_dim, float scale, int32_t window, int32_t part_min,
                                   int32_t nparts, const float* sinks, const void* gate, int64_t gate_stride, void* out,
                                   void* workspace, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "latent_attend");
    SKYRL_REQUIRE(!gate || gate_stride >= heads, "latent_attend: gate_stride");
    SKYRL_REQUIRE(T_ >= 0 && T_ <= 65535 && heads > 0 && rank > 0 && rank <= 2048 && rot_dim >= 0,
                  "latent_attend: bad sizes (T <= 65535, rank <= 2048)");
    SKYRL_REQUIRE(row % 32 == 0 && row >= rank + rot_dim, "latent_attend: row must be a multiple of 32 >= rank + rot_dim");
    if (T_ == 0) return SKYRL_OK;
    SKYRL_REQUIRE(qa && q_rot && cache && block_tables && bt_row && positions && out, "latent_attend: null pointer");
    hipStream_t s = as_stream(stream);
    if (!skyrl_latent_attend_mfma(rank, rot_dim, row, dtype)) {
        SKYRL_DISPATCH_T(dtype, {
            hipLaunchKernelGGL((latent_attend_plain_kernel<T>), dim3(heads, T_), dim3(kNT),
                               (rank + rot_dim) * sizeof(float), s, reinterpret_cast<const T*>(qa),
                               reinterpret_cast<const T*>(q_rot), q_stride, q_head, reinterpret_cast<const T*>(cache),
                               row, block_tables, bt_stride, bt_row, positions, T_, heads, rank, rot_dim, scale,
                               window, HeadEnd<T>{sinks, reinterpret_cast<const T*>(gate), gate_stride},
                               reinterpret_cast<T*>(out));
        })
        return check_launch("latent_attend_plain_kernel");
    }
    SKYRL_REQUIRE(nparts >= 1 && part_min >= kBS && part_min % kBS == 0,
                  "latent_attend: nparts >= 1 and part_min a positive multiple of 16");
    SKYRL_REQUIRE(nparts == 1 || workspace, "latent_attend: nparts > 1 needs a workspace");
    SKYRL_REQUIRE(aligned16(qa) && aligned16(cache) && aligned16(workspace), "latent_attend: 16-byte alignment");
    const uint16_t* q_ = reinterpret_cast<const uint16_t*>(qa);
    const uint16_t* r_ = reinterpret_cast<const uint16_t*>(q_rot);
    const uint16_t* c_ = reinterpret_cast<const uint16_t*>(cache);
    uint16_t* o_ = reinterpret_cast<uint16_t*>(out);
    const HeadEnd<uint16_t> end_{sinks, reinterpret_cast<const uint16_t*>(gate), gate_stride};
    float* ws_o = reinterpret_cast<float*>(workspace);
    float* ws_ml = ws_o ? ws_o + (size_t)T_ * heads * nparts * (((rank + 15) / 16) * 16) : nullptr;
    const int nk = row / 32, nv = (rank + 15) / 16;
    if (nv <= 4 && nk <= 4) {
        LAUNCH_ATTEND(4, 4, false);
    } else if (nv <= 8 && nk <= 6) {
        LAUNCH_ATTEND(8, 6, false);
    } else if (nv <= 16 && nk <= 10) {
        LAUNCH_ATTEND(16, 10, false);
    } else if (rank == 512 && nk == 18) {
        LAUNCH_ATTEND(32, 18, true);
    } else {
        LAUNCH_ATTEND(32, 20, false);
    }
    int rc = check_launch("latent_attend_mfma_kernel");
    if (rc != SKYRL_OK || nparts == 1) return rc;
    hipLaunchKernelGGL(latent_merge_kernel, dim3(heads, T_), dim3(kWave * 2), 0, s, ws_o, ws_ml, positions, T_, heads, rank,
                       window, part_min, nparts, end_, o_);
    return check_launch("latent_merge_kernel");
}

extern "C" int skyrl_latent_gather(const void* cache, int32_t row, const int32_t* block_tables, int64_t bt_stride,
                                   const int32_t* seg, int32_t nseg, int32_t max_count, int32_t rank, int32_t rot_dim,
                                   void* latent, void* k_rot, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "latent_gather");
    SKYRL_REQUIRE(nseg >= 0 && nseg <= 65535 && max_count > 0 && rank > 0 && rot_dim >= 0 && row >= rank + rot_dim &&
                      row % 32 == 0,
                  "latent_gather: bad sizes");
    if (nseg == 0) return SKYRL_OK;
    SKYRL_REQUIRE(cache && block_tables && seg && latent && k_rot, "latent_gather: null pointer");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((latent_gather_kernel<T>), dim3((max_count + 63) / 64 * 4, nseg), dim3(kNT), 0,
                           as_stream(stream), reinterpret_cast<const T*>(cache), row, block_tables, bt_stride, seg,
                           rank, rot_dim, reinterpret_cast<T*>(latent), reinterpret_cast<T*>(k_rot));
    })
    return check_launch("latent_gather_kernel");
}

#define LAUNCH_PREFILL(NK, NV, QT)                                                                                    \
    if (vec) LAUNCH_PREFILL_(NK, NV, QT, true);                                                                       \
    else LAUNCH_PREFILL_(NK, NV, QT, false)
#define LAUNCH_PREFILL_(NK, NV, QT, VEC)                                                                              \
    hipLaunchKernelGGL((latent_prefill_kernel<NK, NV, QT, VEC>), dim3((unsigned)ntiles * heads), dim3(512 / QT), 0,   \
                       as_stream(stream), reinterpret_cast<const uint16_t*>(q), q_stride,                             \
                       reinterpret_cast<const uint16_t*>(k_nope), k_stride, reinterpret_cast<const uint16_t*>(k_rot), \
                       reinterpret_cast<const uint16_t*>(v_t), vt_stride, tiles, heads, dim, rot_dim, vdim,           \
                       scale * kLog2e, window, end_, reinterpret_cast<uint16_t*>(out), out_stride)

extern "C" int skyrl_latent_prefill(const void* q, int64_t q_stride, const void* k_nope, int64_t k_stride,
                                    const void* k_rot, const void* v_t, int64_t vt_stride, const int32_t* tiles,
                                    int32_t ntiles, int32_t heads, int32_t dim, int32_t rot_dim, int32_t vdim,
                                    float scale, int32_t window, const float* sinks, const void* gate,
                                    int64_t gate_stride, void* out, int64_t out_stride, void* stream) {
    SKYRL_REQUIRE(ntiles >= 0 && heads > 0 && dim >= 0 && rot_dim >= 0 && dim + rot_dim > 0 && dim + rot_dim <= 256 &&
                      vdim > 0 && vdim <= 256,
                  "latent_prefill: dim + rot_dim and vdim must be in [1, 256]");
    SKYRL_REQUIRE((int64_t)ntiles * heads < (1 << 30), "latent_prefill: grid too large");
    SKYRL_REQUIRE(vt_stride % 64 == 0, "latent_prefill: vt_stride must be a multiple of 64");
    if (ntiles == 0) return SKYRL_OK;
    SKYRL_REQUIRE(q && k_nope && k_rot && v_t && tiles && out, "latent_prefill: null pointer");
    SKYRL_REQUIRE(aligned16(k_nope) && aligned16(k_rot) && aligned16(v_t), "latent_prefill: 16-byte alignment");
    SKYRL_REQUIRE(!gate || gate_stride >= heads, "latent_prefill: gate_stride");
    const HeadEnd<uint16_t> end_{sinks, reinterpret_cast<const uint16_t*>(gate), gate_stride};
    const int nk = (dim + rot_dim + 31) / 32, nv = (vdim + 15) / 16;
    const bool vec = dim % 8 == 0 && rot_dim % 8 == 0 && k_stride % 8 == 0 && q_stride % 8 == 0 && aligned16(q);
    if (nk <= 2 && nv <= 8) {
        LAUNCH_PREFILL(2, 8, 2);
    } else if (nk <= 4 && nv <= 8) {
        LAUNCH_PREFILL(4, 8, 2);
    } else if (nk <= 6 && nv <= 8) {
        LAUNCH_PREFILL(6, 8, 2);
    } else {
        LAUNCH_PREFILL(8, 16, 1);
    }
    return check_launch("latent_prefill_kernel");
}
