// Routed experts: of many small gated feed-forwards every token runs a few (include/skyrl_layers.h has the equations and
// the tensor layouts).
//
//   route    f32 logits (one workgroup per 16 tokens on the matrix instructions, bf16 products are exact in f32; any
//            size and f32: a workgroup per token), then a wave per token picks groups and experts.
//   sort     counts the (token, expert) pairs by expert (many pairs: in a launch of its own) and lists them in tiles of
//            TM rows that belong to one expert; the grids of the products are sized for the most tiles there can be, so that nothing comes
//            back to the host and a step can be captured.
//   gate_up  per tile and 64 or 128 hidden columns: both products of the gathered token rows and act(gate) * up.
//   down     per tile and 128 or 256 output columns, scaled by the pair's weight, to the pair's own row: a token's rows are
//            consecutive and are summed where they are read (skyrl_gate_norm_add).
//
// The products stage pieces of the rows and of the weight rows through LDS (16-byte direct loads, chunk index
// xor-swizzled by the row so that the reads of 16 rows do not conflict), weights as the left operand: a lane holds
// four consecutive columns of a token. Small tiles (decode) keep several stages in flight: they stream weights.
#include "elem.h"

namespace skyrl {
namespace {

typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) void lds_void;
typedef __attribute__((address_space(1))) void gbl_void;

constexpr int kNT = 256;
constexpr int kMaxExperts = 1024;

struct Router {
    int experts, top, groups, keep;
};

// ---- routing --------------------------------------------------------------------------------------
// A wave picks a token's experts from its logits in LDS. s_s and s_c (scores, corrected scores) and s_g are the wave's own.
__device__ __forceinline__ void wave_lds_sync() {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
    __builtin_amdgcn_wave_barrier();
}
// EP: experts per lane, consecutive ones.
template <int EP>
__device__ __forceinline__ void pick(const Router& ro, const float* z, const float* __restrict__ correction, float* s_s,
                                     float* s_c, float* s_g, int lane, int32_t* __restrict__ idx,
                                     float* __restrict__ weight) {
    const int E = ro.experts, per = E / ro.groups;
    float ch[EP];
#pragma unroll
    for (int j = 0; j < EP; ++j) {
        const int e = lane * EP + j;
        ch[j] = -INFINITY;
        if (e < E) {
            const float s = sigmoidf_(z[e]);
            ch[j] = s + correction[e];
            s_s[e] = s;
            s_c[e] = ch[j];
        }
    }
    wave_lds_sync();
    if (EP == 1 && ro.keep < ro.groups && (per & (per - 1)) == 0) {  // an expert per lane, a group in neighbouring lanes
        float a = ch[0], b = -INFINITY;  // the two largest
        for (int o = 1; o < per; o <<= 1) {
            const float x = __shfl_xor(a, o, kWave), y = __shfl_xor(b, o, kWave);
            b = fmaxf(fminf(a, x), fmaxf(b, y));
            a = fmaxf(a, x);
        }
        const float score = per > 1 ? a + b : a;
        const int q = lane / per;
        int better = 0;
        for (int i = 0; i < ro.groups; ++i) {
            const float x = __shfl(score, i * per, kWave);
            better += x > score || (x == score && i < q);
        }
        if (better >= ro.keep) ch[0] = -INFINITY;
    } else if (ro.keep < ro.groups) {
        for (int q = lane; q < ro.groups; q += kWave) {
            float a = -INFINITY, b = -INFINITY;  // the two largest
            for (int i = 0; i < per; ++i) {
                const float x = s_c[q * per + i];
                b = fmaxf(b, fminf(a, x));
                a = fmaxf(a, x);
            }
            s_g[q] = per > 1 ? a + b : a;
        }
        wave_lds_sync();
        for (int q = lane; q < ro.groups; q += kWave) {
            const float x = s_g[q];
            int better = 0;
            for (int i = 0; i < ro.groups; ++i) better += s_g[i] > x || (s_g[i] == x && i < q);
            s_c[q] = better < ro.keep ? 1.f : 0.f;  // the corrected scores are in registers
        }
        wave_lds_sync();
#pragma unroll
        for (int j = 0; j < EP; ++j) {
            const int e = lane * EP + j;
            if (e < E && s_c[e / per] == 0.f) ch[j] = -INFINITY;
        }
    }
    int mine = 0;
    for (int k = 0; k < ro.top; ++k) {
        float best = ch[0];
        int at = 0;
#pragma unroll
        for (int j = 1; j < EP; ++j)
            if (ch[j] > best) {
                best = ch[j];
                at = j;
            }
        const float m = wave_max_uniform(best);
        const int who = __builtin_ctzll(__ballot(best == m));  // the lowest lane, whose experts come first
        const int e = min(__builtin_amdgcn_readlane(lane * EP + at, who), E - 1);
        if (lane == who) {
#pragma unroll
            for (int j = 0; j < EP; ++j)
                if (j == at) ch[j] = -INFINITY;
        }
        if (lane == k % kWave) mine = e;
        if (k % kWave == kWave - 1 || k == ro.top - 1) {  // 64 at a time
            const int k0 = k / kWave * kWave;
            if (k0 + lane <= k) {
                idx[k0 + lane] = mine;
                weight[k0 + lane] = s_s[mine];
            }
        }
    }
    wave_lds_sync();  // the buffers are written again for the next token
}

// Any size: one workgroup per token.
template <typename T>
__global__ __launch_bounds__(kNT) void moe_route_plain_kernel(Router ro, const T* __restrict__ x, int width,
                                                              const T* __restrict__ w,
                                                              const float* __restrict__ correction,
                                                              int32_t* __restrict__ idx, float* __restrict__ weight) {
    __shared__ float s_z[kMaxExperts], s_s[kMaxExperts], s_c[kMaxExperts], s_g[kMaxExperts];
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const T* row = x + t * width;
    for (int e = wave; e < ro.experts; e += kNT / kWave) {
        float s = 0.f;
        for (int i = lane; i < width; i += kWave) s += ld(row + i) * ld(w + (int64_t)e * width + i);
        s = wave_sum(s);
        if (lane == 0) s_z[e] = s;
    }
    __syncthreads();
    if (wave == 0) pick<kMaxExperts / kWave>(ro, s_z, correction, s_s, s_c, s_g, lane, idx + t * ro.top, weight + t * ro.top);
}

// bf16, width a multiple of 8, at most 16 NE experts (rows past the last: the last again): 16 tokens per workgroup, the
// width in shares of NWV waves, U steps of 32 in flight.
template <int NE, int NWV, int U>
__global__ __launch_bounds__(NWV * kWave) void moe_route_kernel(Router ro, const uint16_t* __restrict__ x, int n,
                                                                int width, const uint16_t* __restrict__ w,
                                                                const float* __restrict__ correction,
                                                                int32_t* __restrict__ idx, float* __restrict__ weight) {
    constexpr int E16 = NE * 16, LZ = E16 + 4, EP = (E16 + kWave - 1) / kWave;
    __shared__ __attribute__((aligned(16))) float s_z[NWV][16 * LZ];
    float* own = s_z[1] + (threadIdx.x >> 6) * 3 * E16;  // a wave's scores, once the shares are summed
    static_assert((NWV - 1) * 16 * LZ >= NWV * 3 * E16, "room for the scores");
    const int t0 = blockIdx.x * 16;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c = lane & 15, g = lane >> 4;
    f32x4 acc[NE];
#pragma unroll
    for (int k = 0; k < NE; ++k) acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint16_t* xr = x + (int64_t)min(t0 + c, n - 1) * width;
    const uint16_t* wr[NE];
#pragma unroll
    for (int k = 0; k < NE; ++k) wr[k] = w + (int64_t)min(16 * k + c, ro.experts - 1) * width;
    const int steps = (width + 31) / 32, share = (steps + NWV - 1) / NWV;
    const int s1 = min(steps, (wave + 1) * share);
    for (int s = wave * share; s < s1; s += U) {
        s16x8 xf[U], wf[U][NE];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k0 = 32 * (s + u) + 8 * g, at = min(k0, width - 8);
            xf[u] = *reinterpret_cast<const s16x8*>(xr + at);
#pragma unroll
            for (int k = 0; k < NE; ++k) wf[u][k] = *reinterpret_cast<const s16x8*>(wr[k] + at);
            if (k0 >= width || s + u >= s1) xf[u] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};  // the router's weights are finite
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int k = 0; k < NE; ++k) acc[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u][k], xf[u], acc[k], 0, 0, 0);
    }
#pragma unroll
    for (int k = 0; k < NE; ++k) *reinterpret_cast<f32x4*>(&s_z[wave][c * LZ + 16 * k + 4 * g]) = acc[k];
    __syncthreads();
    for (int e = threadIdx.x; e < 16 * E16; e += NWV * kWave) {
        const int at = e / E16 * LZ + e % E16;
        float z = 0.f;
#pragma unroll
        for (int i = 0; i < NWV; ++i) z += s_z[i][at];
        s_z[0][at] = z;
    }
    __syncthreads();
#pragma unroll 1
    for (int i = wave; i < 16; i += NWV) {
        const int t = t0 + i;
        if (t >= n) break;
        pick<EP>(ro, &s_z[0][i * LZ], correction, own, own + E16, own + 2 * E16, lane, idx + (int64_t)t * ro.top,
                 weight + (int64_t)t * ro.top);
    }
}

// Pairs by expert, in tiles of tm rows: order[tile * tm + r] = pair or -1, tile_expert[tile] = expert or -1 past the
// last, tile_expert[ntiles] = tiles in use. A workgroup lists `span` pairs; with several, counts [workgroup][expert]
// (moe_count_kernel) say where its own begin.
constexpr int kSpan = 2048;  // pairs per workgroup
__global__ __launch_bounds__(1024) void moe_count_kernel(const int32_t* __restrict__ idx, int npairs, int experts,
                                                         int32_t* __restrict__ counts) {
    __shared__ int s_n[kMaxExperts];
    for (int e = threadIdx.x; e < experts; e += 1024) s_n[e] = 0;
    __syncthreads();
    const int p1 = min(npairs, ((int)blockIdx.x + 1) * kSpan);
    for (int p = blockIdx.x * kSpan + threadIdx.x; p < p1; p += 1024) atomicAdd(&s_n[idx[p]], 1);
    __syncthreads();
    for (int e = threadIdx.x; e < experts; e += 1024) counts[blockIdx.x * experts + e] = s_n[e];
}
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int32_t* __restrict__ idx, int npairs, int experts, int tm,
                                                        int ntiles, int span, const int32_t* __restrict__ counts,
                                                        int32_t* __restrict__ order, int32_t* __restrict__ tile_expert) {
    __shared__ int s_n[kMaxExperts], s_at[kMaxExperts], s_sum[16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int p0 = blockIdx.x * span, p1 = min(npairs, p0 + span);
    int cnt = 0, ahead = 0;  // of this thread's expert: all pairs, those of the workgroups before
    if (counts) {
        if (tid < experts)
#pragma unroll 8
            for (int b = 0; b < (int)gridDim.x; ++b) {
                const int c = counts[b * experts + tid];
                if (b < (int)blockIdx.x) ahead += c;
                cnt += c;
            }
    } else {
        if (tid < experts) s_n[tid] = 0;
        __syncthreads();
        for (int p = p0 + tid; p < p1; p += 1024) atomicAdd(&s_n[idx[p]], 1);
        __syncthreads();
        if (tid < experts) cnt = s_n[tid];
    }
    // tiles before each expert: a scan over at most 1024 experts
    const int tiles = (cnt + tm - 1) / tm;
    int x = tiles;
#pragma unroll
    for (int o = 1; o < kWave; o <<= 1) {
        const int y = __shfl_up(x, o, kWave);
        if (lane >= o) x += y;
    }
    if (lane == kWave - 1) s_sum[wave] = x;
    __syncthreads();
    int before = x - tiles, total = 0;
    for (int i = 0; i < 16; ++i) {
        if (i < wave) before += s_sum[i];
        total += s_sum[i];
    }
    if (tid < experts) {
        s_at[tid] = before * tm + ahead;
        if (blockIdx.x == 0) {
            for (int i = 0; i < tiles && before + i < ntiles; ++i) tile_expert[before + i] = tid;
            for (int i = cnt; i < tiles * tm; ++i) order[before * tm + i] = -1;
        }
    }
    if (blockIdx.x == 0) {
        for (int i = total + tid; i < ntiles; i += 1024) tile_expert[i] = -1;
        if (tid == 0) tile_expert[ntiles] = total;
    }
    __syncthreads();
    for (int p = p0 + tid; p < p1; p += 1024) order[atomicAdd(&s_at[idx[p]], 1)] = p;
}

// ---- products, any size and type: 16 rows x 64 columns per workgroup ---------------------------------
struct Product {
    int K, N;                 // depth, output columns
    const int32_t* order;
    const int32_t* tile_expert;
    int tm;
    int row_div;              // row of x: pair / row_div (the token), or 0: the sorted place itself
    const float* weight;      // of the pair, NULL: 1
    int out_pairs;            // rows of the output: the pair's, or the sorted place
};

// GATED: two weight matrices of N rows per expert, out = silu(gate) * up.
template <typename T, bool GATED>
__global__ __launch_bounds__(kNT) void moe_plain_kernel(Product p, const T* __restrict__ x, const T* __restrict__ w,
                                                        T* __restrict__ out) {
    constexpr int KT = 32;
    __shared__ float s_x[16][KT + 1], s_w[GATED ? 2 : 1][64][KT + 1];
    const int64_t place0 = (int64_t)blockIdx.y * 16;
    const int e = p.tile_expert[place0 / p.tm];
    if (e < 0) return;
    const int n0 = blockIdx.x * 64, tid = threadIdx.x, col = tid & 63, r0 = (tid >> 6) * 4;
    const T* we = w + (int64_t)e * (GATED ? 2 : 1) * p.N * p.K;
    float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < p.K; k0 += KT) {
        for (int i = tid; i < 16 * KT; i += kNT) {
            const int r = i / KT, k = i % KT;
            const int pair = p.order[place0 + r];
            const int64_t row = p.row_div ? pair / p.row_div : place0 + r;
            s_x[r][k] = pair >= 0 && k0 + k < p.K ? ld(x + row * p.K + k0 + k) : 0.f;
        }
        for (int i = tid; i < 64 * KT; i += kNT) {
            const int r = i / KT, k = i % KT;
            const bool on = n0 + r < p.N && k0 + k < p.K;
            s_w[0][r][k] = on ? ld(we + (int64_t)(n0 + r) * p.K + k0 + k) : 0.f;
            if constexpr (GATED) s_w[1][r][k] = on ? ld(we + (int64_t)(p.N + n0 + r) * p.K + k0 + k) : 0.f;
        }
        __syncthreads();
        for (int k = 0; k < KT; ++k) {
            const float u = s_w[0][col][k];
#pragma unroll
            for (int i = 0; i < 4; ++i) a[i] += s_x[r0 + i][k] * u;
            if constexpr (GATED) {
                const float v = s_w[1][col][k];
#pragma unroll
                for (int i = 0; i < 4; ++i) b[i] += s_x[r0 + i][k] * v;
            }
        }
        __syncthreads();
    }
    if (n0 + col >= p.N) return;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int pair = p.order[place0 + r0 + i];
        if (pair < 0) continue;
        const int64_t row = p.out_pairs ? pair : place0 + r0 + i;
        float y = a[i];
        if constexpr (GATED) y = siluf_(a[i]) * b[i];
        if (p.weight) y *= p.weight[pair];
        st(out + row * p.N + n0 + col, y);
    }
}

// ---- products, bf16, depth and columns multiples of 8 ------------------------------------------------
// All but the N latest loads have landed, all LDS reads have returned.
template <int N>
__device__ __forceinline__ void wait_loads() {
    asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"(N) : "memory");
}
__device__ __forceinline__ void lds_read(s16x8& v, uint32_t at, int offset) {
    asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(v) : "v"(at), "n"(offset));
}
__device__ const uint4 kZero16 = {0u, 0u, 0u, 0u};

// A workgroup: one tile of TM rows and TN weight rows (GATED: half of each matrix, the same columns), WM x WN waves. S
// stages of 64-deep pieces. Tiles of one expert share its weights and a tile's columns its rows: with several tiles per
// expert (TM > 16) an XCD takes a run of tiles, a tile's columns together. The output leaves through LDS, whole rows.
template <int TM, int TN, int WM, int WN, int S, bool GATED>
__global__ __launch_bounds__(WM* WN* kWave) void moe_gemm_kernel(Product p, const uint16_t* __restrict__ x,
                                                                 const uint16_t* __restrict__ w,
                                                                 uint16_t* __restrict__ out, int ncols, int ntiles) {
    constexpr int BK = 64, NWV = WM * WN, CH = BK / 8, RP = 64 / CH;  // 16-byte chunks of a row, rows of a 1 KB piece
    constexpr int XP = TM / RP, WP = TN / RP;             // pieces of a stage
    constexpr int MT = TM / WM / 16, NTL = TN / WN / 16;  // 16-wide tiles per wave
    constexpr int XL = (XP + NWV - 1) / NWV, WL = WP / NWV;  // pieces per wave
    constexpr int kStage = (TM + TN) * BK;                // elements
    constexpr int OC = GATED ? TN / 2 : TN, LO = OC + 8;  // output columns and their row in LDS
    constexpr int kLds = S * kStage > TM * LO ? S * kStage : TM * LO;
    static_assert(WP % NWV == 0 && (XP % NWV == 0 || XP < NWV), "staging split");
    __shared__ __attribute__((aligned(16))) uint16_t smem[kLds];
    __shared__ int s_pair[TM];
    __shared__ float s_wt[TM];
    int tile = blockIdx.x / ncols, nb = blockIdx.x % ncols;
    if constexpr (TM > 16) {
        const int used = p.tile_expert[ntiles], per = (used + 7) / 8, i = blockIdx.x / 8;
        tile = i / ncols;
        if (tile >= per) return;
        tile += blockIdx.x % 8 * per;
        nb = i % ncols;
        if (tile >= used) return;
    }
    const int e = p.tile_expert[tile];
    if (e < 0) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int n0 = nb * OC;
    const uint16_t* we = w + (int64_t)e * (GATED ? 2 : 1) * p.N * p.K;
    const int64_t place0 = (int64_t)tile * TM;
    const int nk = (p.K + BK - 1) / BK;

    if (tid < TM) {  // what the end needs of the rows
        const int pair = p.order[place0 + tid];
        s_pair[tid] = pair;
        s_wt[tid] = p.weight && pair >= 0 ? p.weight[pair] : 1.f;
    }
    // global sources of this lane's 16 bytes per piece: row RP piece + lane / CH, chunk (lane % CH) ^ swizzle, so that the
    // 16 rows a matrix operand reads at a time lie in different banks
    auto swz = [](int r) { return r / (128 / BK) % CH; };
    const uint16_t* xs[XL];
    const uint16_t* ws[WL];
    int xk[XL], wk[WL];
#pragma unroll
    for (int i = 0; i < XL; ++i) {
        const int r = min(wave * XL + i, XP - 1) * RP + lane / CH;
        const int pair = p.order[place0 + r];
        const int64_t row = pair < 0 ? 0 : p.row_div ? pair / p.row_div : place0 + r;
        xk[i] = (lane % CH ^ swz(r)) * 8;
        xs[i] = x + row * p.K;
    }
#pragma unroll
    for (int i = 0; i < WL; ++i) {
        const int r = (wave * WL + i) * RP + lane / CH;
        const int col = n0 + (GATED ? r % OC : r);
        const int64_t row = (GATED && r >= OC ? p.N : 0) + min(col, p.N - 1);
        wk[i] = (lane % CH ^ swz(r)) * 8;
        ws[i] = we + row * p.K;
    }
    auto fetch = [&](int t) {  // piece t (the last again past the end) into stage t % S
        uint16_t* dst = smem + (t % S) * kStage;
        const int k0 = min(t, nk - 1) * BK;
#pragma unroll
        for (int i = 0; i < XL; ++i) {
            const int k = k0 + xk[i], piece = min(wave * XL + i, XP - 1);
            const void* src = k < p.K ? (const void*)(xs[i] + k) : (const void*)&kZero16;
            __builtin_amdgcn_global_load_lds((gbl_void*)src, (lds_void*)(dst + piece * 512), 16, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < WL; ++i) {
            const int k = k0 + wk[i];
            const void* src = k < p.K ? (const void*)(ws[i] + k) : (const void*)&kZero16;
            __builtin_amdgcn_global_load_lds((gbl_void*)src, (lds_void*)(dst + TM * BK + (wave * WL + i) * 512), 16, 0, 0);
        }
    };
    const int wm = wave / WN, wn = wave % WN;
    f32x4 acc[MT][NTL];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NTL; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    // weight row of this wave's tile n: with GATED the first half of the tiles are gate rows, the others the same columns' up rows
    auto wrow = [&](int n) {
        if (!GATED) return (wn * NTL + n) * 16;
        return n < NTL / 2 ? (wn * (NTL / 2) + n) * 16 : OC + (wn * (NTL / 2) + n - NTL / 2) * 16;
    };
    // Matrix operands of a 32-deep half, read while the other half's products run. The reads are not the compiler's: it
    // would wait for every load into LDS under way before one.
    s16x8 xf[2][MT], wf[2][NTL];
    const uint32_t lds0 = (uint32_t)(uintptr_t)(lds_void*)smem;
    const uint32_t xat = lds0 + (wm * MT * 16 + c) * BK * 2;
    const uint32_t wat = lds0 + (TM + wn * (GATED ? NTL / 2 : NTL) * 16 + c) * BK * 2;
    auto operands = [&](int t, int ks) {
        const uint32_t at = (t % S) * kStage * 2 + ((ks * 4 + g) ^ swz(c)) * 16;  // swz(16 j + c) = swz(c)
#pragma unroll
        for (int n = 0; n < NTL; ++n)
            lds_read(wf[ks][n], wat + at, (n < NTL / 2 || !GATED ? n * 16 : OC + (n - NTL / 2) * 16) * BK * 2);
#pragma unroll
        for (int m = 0; m < MT; ++m) lds_read(xf[ks][m], xat + at, m * 16 * BK * 2);
    };
    auto hold = [&](int ks) {  // the operands' registers are in use up to here
#pragma unroll
        for (int n = 0; n < NTL; ++n) asm volatile("" : "+v"(wf[ks][n]));
#pragma unroll
        for (int m = 0; m < MT; ++m) asm volatile("" : "+v"(xf[ks][m]));
    };
    auto ready = [&](int ks) {  // all but the reads of the other half have returned
        asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(MT + NTL) : "memory");
        hold(ks);
    };
    auto products = [&](int ks) {
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int n = 0; n < NTL; ++n)
                acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[ks][n], xf[ks][m], acc[m][n], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
    };
#pragma unroll
    for (int t = 0; t < S; ++t) fetch(t);
    wait_loads<(S - 1) * (XL + WL)>();
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    operands(0, 0);
    for (int t = 0; t < nk; ++t) {
        operands(t, 1);
        ready(0);
        products(0);
        wait_loads<(S - 2) * (XL + WL)>();  // this wave's loads of piece t + 1 have landed, its reads of piece t too
        __builtin_amdgcn_s_barrier();       // and everyone's
        asm volatile("" ::: "memory");
        fetch(t + S);
        operands(t + 1, 0);
        ready(1);
        products(1);
    }
    wait_loads<0>();  // nothing is under way, into LDS or into the registers of the last reads
    hold(0);
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int r = (wm * MT + m) * 16 + c;
        const float scale = s_wt[r];
#pragma unroll
        for (int n = 0; n < (GATED ? NTL / 2 : NTL); ++n) {
            const int col = (GATED ? (wn * (NTL / 2) + n) * 16 : wrow(n)) + 4 * g;
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if constexpr (GATED) v[i] = acc[m][n][i] * sigmoid_<uint16_t>(acc[m][n][i]) * acc[m][n + NTL / 2][i];
                else v[i] = acc[m][n][i] * scale;
            }
            *reinterpret_cast<uint2*>(&smem[r * LO + col]) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
        }
    }
    __syncthreads();
    for (int i = tid; i < TM * (OC / 8); i += NWV * kWave) {
        const int r = i / (OC / 8), col = i % (OC / 8) * 8, pair = s_pair[r];
        if (pair < 0 || n0 + col >= p.N) continue;  // N is a multiple of 8
        *reinterpret_cast<uint4*>(out + (p.out_pairs ? (int64_t)pair : place0 + r) * p.N + n0 + col) =
            *reinterpret_cast<const uint4*>(&smem[r * LO + col]);
    }
}

bool fast_form(int K, int N, int tm, int dtype, const void* x, const void* w, const void* out) {
    return dtype == SKYRL_BF16 && K % 8 == 0 && N % 8 == 0 && (tm == 16 || tm == 64 || tm == 128 || tm == 256) && aligned16(x) &&
           aligned16(w) && aligned16(out);
}

template <bool GATED>
int launch_product(const Product& p, const void* x, const void* w, void* out, int ntiles, int dtype, hipStream_t s) {
    if (fast_form(p.K, p.N, p.tm, dtype, x, w, out)) {
        const uint16_t* x_ = reinterpret_cast<const uint16_t*>(x);
        const uint16_t* w_ = reinterpret_cast<const uint16_t*>(w);
        uint16_t* o_ = reinterpret_cast<uint16_t*>(out);
#define LAUNCH_GEMM(TM, TN, WM, WN, S)                                                                                \
    do {                                                                                                              \
        constexpr int kCols = GATED ? TN / 2 : TN;                                                                    \
        const int ncols = (p.N + kCols - 1) / kCols;                                                                  \
        const int64_t grid = (int64_t)ncols * ((ntiles + 7) / 8 * 8);  /* a run of tiles per XCD */                   \
        SKYRL_REQUIRE(grid < (1ll << 31), "moe: grid too large");                                                     \
        hipLaunchKernelGGL((moe_gemm_kernel<TM, TN, WM, WN, S, GATED>), dim3((unsigned)(TM > 16 ? grid : (int64_t)ncols * ntiles)), \
                           dim3(WM * WN * kWave), 0, s, p, x_, w_, o_, ncols, ntiles);                                \
    } while (0)
        if (p.tm == 256) LAUNCH_GEMM(256, 256, 2, 4, 2);
        else if (p.tm == 128) LAUNCH_GEMM(128, 128, 2, 2, 2);
        else if (p.tm == 64) LAUNCH_GEMM(64, 128, 2, 2, 3);
        else LAUNCH_GEMM(16, 128, 1, 4, 4);
        return check_launch("moe_gemm_kernel");
    }
    const int64_t rows = (int64_t)ntiles * p.tm / 16;
    SKYRL_REQUIRE(p.tm % 16 == 0 && rows <= 65535, "moe: too many rows for the plain form in one call");
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((moe_plain_kernel<T, GATED>), dim3((p.N + 63) / 64, (unsigned)rows), dim3(kNT), 0, s, p,
                           reinterpret_cast<const T*>(x), reinterpret_cast<const T*>(w), reinterpret_cast<T*>(out));
    })
    return check_launch("moe_plain_kernel");
}

const char* bad_router(const skyrl_moe_shape* sh) {
    if (!sh) return "moe: null shape";
    if (sh->experts <= 0 || sh->experts > kMaxExperts) return "moe: experts must be in [1, 1024]";
    if (sh->groups <= 0 || sh->experts % sh->groups) return "moe: experts must be a multiple of groups";
    if (sh->keep <= 0 || sh->keep > sh->groups) return "moe: keep must be in [1, groups]";
    if (sh->top <= 0 || sh->top > sh->experts / sh->groups * sh->keep) return "moe: top must be in [1, experts of the kept groups]";
    if (sh->width <= 0 || sh->ff <= 0) return "moe: width and ff must be positive";
    return nullptr;
}

}  // namespace
}  // namespace skyrl

using namespace skyrl;

extern "C" int skyrl_moe_route(const skyrl_moe_shape* shape, const void* x, int32_t n, const void* router,
                               const float* correction, int32_t* idx, float* weight, int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "moe_route");
    const char* bad = bad_router(shape);
    SKYRL_REQUIRE(!bad, bad);
    SKYRL_REQUIRE(n >= 0, "moe_route: bad n");
    if (n == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && router && correction && idx && weight, "moe_route: null pointer");
    const Router ro{shape->experts, shape->top, shape->groups, shape->keep};
    const int W = shape->width;
    hipStream_t s = as_stream(stream);
    if (dtype == SKYRL_BF16 && W % 8 == 0 && ro.experts <= 256 && aligned16(x) && aligned16(router)) {
        const uint16_t* x_ = reinterpret_cast<const uint16_t*>(x);
        const uint16_t* w_ = reinterpret_cast<const uint16_t*>(router);
        const dim3 grid((n + 15) / 16);
#define LAUNCH_ROUTE(NE, NWV, U)                                                                                     \
    hipLaunchKernelGGL((moe_route_kernel<NE, NWV, U>), grid, dim3(NWV * kWave), 0, s, ro, x_, n, W, w_, correction, idx, \
                       weight)
        if (ro.experts <= 16) LAUNCH_ROUTE(1, 16, 4);
        else if (ro.experts <= 32) LAUNCH_ROUTE(2, 16, 4);
        else if (ro.experts <= 64) LAUNCH_ROUTE(4, 16, 4);
        else if (ro.experts <= 128) LAUNCH_ROUTE(8, 8, 4);
        else LAUNCH_ROUTE(16, 4, 4);
        return check_launch("moe_route_kernel");
    }
    SKYRL_DISPATCH_T(dtype, {
        hipLaunchKernelGGL((moe_route_plain_kernel<T>), dim3(n), dim3(kNT), 0, s, ro, reinterpret_cast<const T*>(x), W,
                           reinterpret_cast<const T*>(router), correction, idx, weight);
    })
    return check_launch("moe_route_plain_kernel");
}

extern "C" int32_t skyrl_moe_tiles(int32_t experts, int32_t npairs, int32_t tm) {
    return npairs <= 0 || tm <= 0 ? 0 : npairs / tm + (experts < npairs ? experts : npairs);
}

extern "C" int32_t skyrl_moe_counts(int32_t experts, int32_t npairs) {
    return npairs <= 2 * kSpan ? 0 : (npairs + kSpan - 1) / kSpan * experts;
}

extern "C" int skyrl_moe_sort(const int32_t* idx, int32_t npairs, int32_t experts, int32_t tm, int32_t ntiles,
                              int32_t* counts, int32_t* order, int32_t* tile_expert, void* stream) {
    SKYRL_REQUIRE(npairs >= 0 && experts > 0 && experts <= kMaxExperts && tm > 0 && tm % 16 == 0, "moe_sort: bad sizes");
    SKYRL_REQUIRE(ntiles >= skyrl_moe_tiles(experts, npairs, tm), "moe_sort: too few tiles");
    if (npairs == 0) return SKYRL_OK;
    SKYRL_REQUIRE(idx && order && tile_expert, "moe_sort: null pointer");
    const bool several = skyrl_moe_counts(experts, npairs) > 0;
    SKYRL_REQUIRE(!several || counts, "moe_sort: this many pairs need counts");
    const int grid = several ? (npairs + kSpan - 1) / kSpan : 1;
    if (several) {
        hipLaunchKernelGGL(moe_count_kernel, dim3(grid), dim3(1024), 0, as_stream(stream), idx, npairs, experts, counts);
        const int rc = check_launch("moe_count_kernel");
        if (rc != SKYRL_OK) return rc;
    }
    hipLaunchKernelGGL(moe_sort_kernel, dim3(grid), dim3(1024), 0, as_stream(stream), idx, npairs, experts, tm, ntiles,
                       several ? kSpan : npairs, several ? counts : nullptr, order, tile_expert);
    return check_launch("moe_sort_kernel");
}

extern "C" int skyrl_moe_gate_up(const skyrl_moe_shape* shape, const void* x, const void* w, const int32_t* order,
                                 const int32_t* tile_expert, int32_t tm, int32_t ntiles, void* act, int32_t dtype,
                                 void* stream) {
    SKYRL_REQUIRE_T(dtype, "moe_gate_up");
    const char* bad = bad_router(shape);
    SKYRL_REQUIRE(!bad, bad);
    SKYRL_REQUIRE(tm > 0 && ntiles >= 0, "moe_gate_up: bad sizes");
    if (ntiles == 0) return SKYRL_OK;
    SKYRL_REQUIRE(x && w && order && tile_expert && act, "moe_gate_up: null pointer");
    const Product p{shape->width, shape->ff, order, tile_expert, tm, shape->top, nullptr, 0};
    return launch_product<true>(p, x, w, act, ntiles, dtype, as_stream(stream));
}

extern "C" int skyrl_moe_down(const skyrl_moe_shape* shape, const void* act, const void* w, const int32_t* order,
                              const int32_t* tile_expert, int32_t tm, int32_t ntiles, const float* weight, void* out,
                              int32_t dtype, void* stream) {
    SKYRL_REQUIRE_T(dtype, "moe_down");
    const char* bad = bad_router(shape);
    SKYRL_REQUIRE(!bad, bad);
    SKYRL_REQUIRE(tm > 0 && ntiles >= 0, "moe_down: bad sizes");
    if (ntiles == 0) return SKYRL_OK;
    SKYRL_REQUIRE(act && w && order && tile_expert && weight && out, "moe_down: null pointer");
    const Product p{shape->ff, shape->width, order, tile_expert, tm, 0, weight, 1};
    return launch_product<false>(p, act, w, out, ntiles, dtype, as_stream(stream));
}
