// Routed experts: of many small gated feed-forwards every token runs a few (include/skyrl_layers.h has the equations and
// the tensor layouts).
//
//   route    f32 logits (one workgroup per 16 tokens on the matrix instructions, bf16 products are exact in f32; any
//            size and f32: a workgroup per token), then a wave per token picks groups and experts.
//   sort     one workgroup counts the (token, expert) pairs by expert and lists them in tiles of TM rows that belong to
//            one expert; the grids of the products are sized for the most tiles there can be, so that nothing comes
//            back to the host and a step can be captured.
//   gate_up  per tile and 64 hidden columns: both products of the gathered token rows and act(gate) * up.
//   down     per tile and 128 output columns, scaled by the pair's weight, to the pair's own row: a token's rows are
//            consecutive and are summed where they are read (skyrl_gate_norm_add).
//
// The products stage 64-deep pieces of the rows and of 128 weight rows through LDS (16-byte direct loads, chunk index
// xor-swizzled by (row / 2) % 8 so that the reads of 16 rows do not conflict), weights as the left operand: a lane holds
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
__device__ void pick(const Router& ro, const float* z, const float* __restrict__ correction, float* s_s, float* s_c,
                     float* s_g, int lane, int32_t* __restrict__ idx, float* __restrict__ weight) {
    const int E = ro.experts, per = E / ro.groups;
    for (int e = lane; e < E; e += kWave) {
        const float s = sigmoidf_(z[e]);
        s_s[e] = s;
        s_c[e] = s + correction[e];
    }
    wave_lds_sync();
    if (ro.keep < ro.groups) {
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
            if (better >= ro.keep)
                for (int i = 0; i < per; ++i) s_c[q * per + i] = -INFINITY;
        }
        wave_lds_sync();
    }
    for (int k = 0; k < ro.top; ++k) {
        float best = -INFINITY;
        int at = E;
        for (int e = lane; e < E; e += kWave)
            if (s_c[e] > best) {
                best = s_c[e];
                at = e;
            }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float x = __shfl_xor(best, o, kWave);
            const int i = __shfl_xor(at, o, kWave);
            if (x > best || (x == best && i < at)) {
                best = x;
                at = i;
            }
        }
        at = min(at, E - 1);
        if (lane == 0) {
            idx[k] = at;
            weight[k] = s_s[at];
            s_c[at] = -INFINITY;
        }
        wave_lds_sync();
    }
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
    if (wave == 0) pick(ro, s_z, correction, s_s, s_c, s_g, lane, idx + t * ro.top, weight + t * ro.top);
}

// bf16, width a multiple of 8, at most 16 NE experts (rows past the last: the last again): 16 tokens per workgroup, a
// quarter of the width per wave.
template <int NE>
__global__ __launch_bounds__(kNT) void moe_route_kernel(Router ro, const uint16_t* __restrict__ x, int n, int width,
                                                        const uint16_t* __restrict__ w,
                                                        const float* __restrict__ correction, int32_t* __restrict__ idx,
                                                        float* __restrict__ weight) {
    constexpr int E16 = NE * 16, LZ = E16 + 4;
    __shared__ __attribute__((aligned(16))) float s_z[4][16 * LZ];
    __shared__ float s_s[4][E16], s_c[4][E16], s_g[4][E16];
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
    const int steps = (width + 31) / 32, share = (steps + 3) / 4;
    const int s1 = min(steps, (wave + 1) * share);
#pragma unroll 4
    for (int s = wave * share; s < s1; ++s) {
        const int k0 = 32 * s + 8 * g;
        const bool on = k0 < width;
        const int at = on ? k0 : 0;
        s16x8 xf = *reinterpret_cast<const s16x8*>(xr + at);
        if (!on) xf = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
        for (int k = 0; k < NE; ++k) {
            s16x8 wf = *reinterpret_cast<const s16x8*>(wr[k] + at);
            if (!on) wf = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
            acc[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, xf, acc[k], 0, 0, 0);
        }
    }
#pragma unroll
    for (int k = 0; k < NE; ++k) *reinterpret_cast<f32x4*>(&s_z[wave][c * LZ + 16 * k + 4 * g]) = acc[k];
    __syncthreads();
    for (int e = threadIdx.x; e < 16 * E16; e += kNT) {
        const int at = e / E16 * LZ + e % E16;
        s_z[0][at] = s_z[0][at] + s_z[1][at] + s_z[2][at] + s_z[3][at];
    }
    __syncthreads();
    for (int i = 0; i < 4; ++i) {
        const int t = t0 + 4 * wave + i;
        if (t >= n) break;
        pick(ro, &s_z[0][(4 * wave + i) * LZ], correction, s_s[wave], s_c[wave], s_g[wave], lane, idx + (int64_t)t * ro.top,
             weight + (int64_t)t * ro.top);
    }
}

// Pairs by expert, in tiles of tm rows: order[tile * tm + r] = pair or -1, tile_expert[tile] = expert or -1 past the last.
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int32_t* __restrict__ idx, int npairs, int experts, int tm,
                                                        int ntiles, int32_t* __restrict__ order,
                                                        int32_t* __restrict__ tile_expert) {
    __shared__ int s_n[kMaxExperts], s_at[kMaxExperts], s_sum[16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    if (tid < experts) s_n[tid] = 0;
    __syncthreads();
    for (int p = tid; p < npairs; p += 1024) atomicAdd(&s_n[idx[p]], 1);
    __syncthreads();
    // tiles before each expert: a scan over at most 1024 experts
    const int cnt = tid < experts ? s_n[tid] : 0, tiles = (cnt + tm - 1) / tm;
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
        s_at[tid] = before * tm;
        for (int i = 0; i < tiles && before + i < ntiles; ++i) tile_expert[before + i] = tid;
        for (int i = cnt; i < tiles * tm; ++i) order[before * tm + i] = -1;
    }
    for (int i = total + tid; i < ntiles; i += 1024) tile_expert[i] = -1;
    __syncthreads();
    for (int p = tid; p < npairs; p += 1024) order[atomicAdd(&s_at[idx[p]], 1)] = p;
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
__device__ const uint4 kZero16 = {0u, 0u, 0u, 0u};

// A workgroup: one tile of TM rows and 128 weight rows (GATED: 64 of each matrix, the same columns). Four waves: TM 128
// as 2 x 2 of 64 rows x 64 weight rows, TM 64 of 32 x 64, TM 16: each wave 32 weight rows. S stages of 64-deep pieces.
template <int TM, int S, bool GATED>
__global__ __launch_bounds__(kNT) void moe_gemm_kernel(Product p, const uint16_t* __restrict__ x,
                                                       const uint16_t* __restrict__ w, uint16_t* __restrict__ out,
                                                       int ncols) {
    constexpr int BK = 64, TN = 128;
    constexpr int XP = TM / 8, WP = TN / 8;             // 1 KB pieces (8 rows) of a stage
    constexpr int WM = TM >= 64 ? 2 : 1, WN = 4 / WM;   // waves along rows, along weight rows
    constexpr int MT = TM / WM / 16, NTL = TN / WN / 16;  // 16-wide tiles per wave
    constexpr int XL = (XP + 3) / 4, WL = WP / 4;       // pieces per wave
    constexpr int kStage = (TM + TN) * BK;              // elements
    __shared__ __attribute__((aligned(16))) uint16_t smem[S * kStage];
    // tiles of one expert share its weights: a column of tiles at a time, consecutive workgroups of an XCD along it
    const int tile = blockIdx.x / ncols, nb = blockIdx.x % ncols;
    const int e = p.tile_expert[tile];
    if (e < 0) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int n0 = nb * (GATED ? 64 : 128);
    const uint16_t* we = w + (int64_t)e * (GATED ? 2 : 1) * p.N * p.K;
    const int64_t place0 = (int64_t)tile * TM;
    const int nk = (p.K + BK - 1) / BK;

    // global sources of this lane's 16 bytes per piece: row 8 piece + lane / 8, chunk (lane % 8) ^ swizzle
    const uint16_t* xs[XL];
    const uint16_t* ws[WL];
    int xk[XL], wk[WL];
#pragma unroll
    for (int i = 0; i < XL; ++i) {
        const int r = min(wave * XL + i, XP - 1) * 8 + (lane >> 3);
        const int pair = p.order[place0 + r];
        const int64_t row = pair < 0 ? 0 : p.row_div ? pair / p.row_div : place0 + r;
        xk[i] = ((lane & 7) ^ ((r >> 1) & 7)) * 8;
        xs[i] = x + row * p.K;
    }
#pragma unroll
    for (int i = 0; i < WL; ++i) {
        const int r = (wave * WL + i) * 8 + (lane >> 3);
        const int col = GATED ? n0 + (r & 63) : n0 + r;
        const int64_t row = (GATED && r >= 64 ? p.N : 0) + min(col, p.N - 1);
        wk[i] = ((lane & 7) ^ ((r >> 1) & 7)) * 8;
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
        return n < NTL / 2 ? (wn * (NTL / 2) + n) * 16 : 64 + (wn * (NTL / 2) + n - NTL / 2) * 16;
    };
#pragma unroll
    for (int t = 0; t < S - 1; ++t) fetch(t);
    for (int t = 0; t < nk; ++t) {
        wait_loads<(S - 2) * (XL + WL)>();  // this wave's loads of piece t have landed
        __builtin_amdgcn_s_barrier();       // and everyone's; everyone is done with piece t - 1
        asm volatile("" ::: "memory");
        fetch(t + S - 1);
        const uint16_t* sx = smem + (t % S) * kStage;
        const uint16_t* sw = sx + TM * BK;
#pragma unroll
        for (int ks = 0; ks < BK / 32; ++ks) {
            s16x8 xf[MT], wf[NTL];
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                const int r = (wm * MT + m) * 16 + c;
                xf[m] = *reinterpret_cast<const s16x8*>(sx + r * BK + (((ks * 4 + g) ^ ((r >> 1) & 7)) * 8));
            }
#pragma unroll
            for (int n = 0; n < NTL; ++n) {
                const int r = wrow(n) + c;
                wf[n] = *reinterpret_cast<const s16x8*>(sw + r * BK + (((ks * 4 + g) ^ ((r >> 1) & 7)) * 8));
            }
#pragma unroll
            for (int m = 0; m < MT; ++m)
#pragma unroll
                for (int n = 0; n < NTL; ++n)
                    acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[n], xf[m], acc[m][n], 0, 0, 0);
        }
    }
    wait_loads<0>();  // nothing is under way into LDS when the workgroup ends
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int64_t place = place0 + (wm * MT + m) * 16 + c;
        const int pair = p.order[place];
        if (pair < 0) continue;
        const float scale = p.weight ? p.weight[pair] : 1.f;
        uint16_t* orow = out + (p.out_pairs ? (int64_t)pair : place) * p.N;
#pragma unroll
        for (int n = 0; n < (GATED ? NTL / 2 : NTL); ++n) {
            const int col = n0 + (GATED ? (wn * (NTL / 2) + n) * 16 : wrow(n)) + 4 * g;
            if (col >= p.N) continue;  // N is a multiple of 8
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if constexpr (GATED) v[i] = acc[m][n][i] * sigmoid_<uint16_t>(acc[m][n][i]) * acc[m][n + NTL / 2][i];
                else v[i] = acc[m][n][i] * scale;
            }
            *reinterpret_cast<uint2*>(orow + col) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
        }
    }
}

bool fast_form(int K, int N, int tm, int dtype, const void* x, const void* w, const void* out) {
    return dtype == SKYRL_BF16 && K % 8 == 0 && N % 8 == 0 && (tm == 16 || tm == 64 || tm == 128) && aligned16(x) &&
           aligned16(w) && aligned16(out);
}

template <bool GATED>
int launch_product(const Product& p, const void* x, const void* w, void* out, int ntiles, int dtype, hipStream_t s) {
    if (fast_form(p.K, p.N, p.tm, dtype, x, w, out)) {
        const int ncols = (p.N + (GATED ? 63 : 127)) / (GATED ? 64 : 128);
        SKYRL_REQUIRE((int64_t)ncols * ntiles < (1ll << 31), "moe: grid too large");
        const dim3 grid((unsigned)(ncols * ntiles)), block(kNT);
        const uint16_t* x_ = reinterpret_cast<const uint16_t*>(x);
        const uint16_t* w_ = reinterpret_cast<const uint16_t*>(w);
        uint16_t* o_ = reinterpret_cast<uint16_t*>(out);
        if (p.tm == 128) hipLaunchKernelGGL((moe_gemm_kernel<128, 2, GATED>), grid, block, 0, s, p, x_, w_, o_, ncols);
        else if (p.tm == 64) hipLaunchKernelGGL((moe_gemm_kernel<64, 3, GATED>), grid, block, 0, s, p, x_, w_, o_, ncols);
        else hipLaunchKernelGGL((moe_gemm_kernel<16, 4, GATED>), grid, block, 0, s, p, x_, w_, o_, ncols);
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
        const dim3 grid((n + 15) / 16), block(kNT);
#define LAUNCH_ROUTE(NE) \
    hipLaunchKernelGGL((moe_route_kernel<NE>), grid, block, 0, s, ro, x_, n, W, w_, correction, idx, weight)
        if (ro.experts <= 16) LAUNCH_ROUTE(1);
        else if (ro.experts <= 32) LAUNCH_ROUTE(2);
        else if (ro.experts <= 64) LAUNCH_ROUTE(4);
        else if (ro.experts <= 128) LAUNCH_ROUTE(8);
        else LAUNCH_ROUTE(16);
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

extern "C" int skyrl_moe_sort(const int32_t* idx, int32_t npairs, int32_t experts, int32_t tm, int32_t ntiles,
                              int32_t* order, int32_t* tile_expert, void* stream) {
    SKYRL_REQUIRE(npairs >= 0 && experts > 0 && experts <= kMaxExperts && tm > 0 && tm % 16 == 0, "moe_sort: bad sizes");
    SKYRL_REQUIRE(ntiles >= skyrl_moe_tiles(experts, npairs, tm), "moe_sort: too few tiles");
    if (npairs == 0) return SKYRL_OK;
    SKYRL_REQUIRE(idx && order && tile_expert, "moe_sort: null pointer");
    hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024), 0, as_stream(stream), idx, npairs, experts, tm, ntiles, order,
                       tile_expert);
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
