// Mixture-of-experts feed-forward on gfx950: router, grouping of tokens by expert, grouped matrix products.
//
// Every token of a step chooses `top` of E experts; a (token, choice) is a pair, numbered token * top + choice.
//   route   logits in fp32 (bf16 operands on MFMA, or fp32 throughout), the largest `top` of them, softmax over those
//   group   pairs sorted by expert: order[], and offsets[e] = first place of expert e's pairs in it
//   gate_up act[i] = silu(Wg h_i) * (Wu h_i) for place i of the order, h_i the pair's token
//   down    out[pair] = weight[pair] * (Wd act[i])
// The products are tiled per expert.  Tiles of expert e start at number offsets[e] / BM + e, so the tile -> expert search
// needs the offsets alone, and a launch of n_pairs / BM + E row tiles covers every distribution of the tokens.  A row of a
// product depends on its own token only, so neither the order inside an expert nor the tiling shows in a result.
//   moe_gemm_kernel    128 x 128 tiles through LDS: prompts
//   moe_skinny_kernel  16 rows x 16 (+ 16) weight rows, weights straight to registers, k dealt to the wavefronts: decoding
//   moe_f32_kernel     fp32 on the vector unit
#include "common.hpp"
#include "launch.hpp"

namespace mi355 {

constexpr int kMaxExperts = 1024;
constexpr int kMaxTop = 64;

__device__ __forceinline__ float moe_wave_sum(float v) {
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}

// ---- router -------------------------------------------------------------------------------------
struct RouteParams {
    const void* h;
    const void* w;               // (E + extra, k) rows of h's type, stride w_stride
    const float* bias;           // (E + extra)
    int32_t* ids;                // (T, top)
    float* weights;              // (T, top)
    float* extra_logit;          // (T): the logit of row E, or null
    int64_t T, h_stride, w_stride;
    int k, E, n_logits, top;
};

// One wavefront: the `top` largest of the E logits at z (LDS; overwritten), their softmax.  Ties go to the lower index.
__device__ __forceinline__ void choose_experts(const RouteParams& p, float* z, int64_t token, int lane) {
    float mine = -INFINITY;                       // logit of choice `lane`
    int mine_id = 0;
    for (int c = 0; c < p.top; ++c) {
        float best = -INFINITY;
        int id = 0x7fffffff;
        for (int e = lane; e < p.E; e += 64) {
            const float v = z[e];
            if (v > best || (v == best && e < id && v > -INFINITY)) {
                best = v;
                id = e;
            }
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) {
            const float v = __shfl_xor(best, off, 64);
            const int i = __shfl_xor(id, off, 64);
            if (v > best || (v == best && i < id)) {
                best = v;
                id = i;
            }
        }
        id = min(id, p.E - 1);                    // (logits that are not numbers: some valid expert)
        if (lane == id % 64) z[id] = -INFINITY;
        if (lane == c) {
            mine = best;
            mine_id = id;
        }
    }
    const float top1 = __shfl(mine, 0, 64);
    const float e = lane < p.top ? expf(mine - top1) : 0.f;
    const float sum = moe_wave_sum(e);
    if (lane < p.top) {
        p.ids[token * p.top + lane] = mine_id;
        p.weights[token * p.top + lane] = e / sum;
    }
}

// 16 tokens per workgroup; the wavefronts take the 32-wide steps of k in turn and meet in LDS.
constexpr int kRouteWaves = 8;
__global__ __launch_bounds__(64 * kRouteWaves) void moe_route_kernel(RouteParams p) {
    extern __shared__ __attribute__((aligned(16))) float route_lds[];
    constexpr int kTiles = 4, kBatch = 4;         // 16 logits each
    f32x4* part = reinterpret_cast<f32x4*>(route_lds);                         // [wave][tile][lane]
    float* z = route_lds + kRouteWaves * kTiles * 64 * 4;                              // [16][n_logits]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, kg = lane >> 4;
    const int64_t t0 = (int64_t)blockIdx.x * 16;
    const __bf16* h = (const __bf16*)p.h + min(t0 + r, p.T - 1) * p.h_stride;
    for (int l0 = 0; l0 < p.n_logits; l0 += 16 * kTiles) {
        f32x4 acc[kTiles];
        const __bf16* w[kTiles];
#pragma unroll
        for (int j = 0; j < kTiles; ++j) {
            acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
            w[j] = (const __bf16*)p.w + (int64_t)min(l0 + 16 * j + r, p.n_logits - 1) * p.w_stride;
        }
        for (int k0 = 32 * wave; k0 < p.k; k0 += 32 * kRouteWaves * kBatch) {       // kBatch steps' loads, then their products
            u32x4 hv[kBatch], wv[kTiles][kBatch];
#pragma unroll
            for (int i = 0; i < kBatch; ++i) {
                const int col = k0 + 32 * kRouteWaves * i + 8 * kg;
                const bool in = col < p.k;
                hv[i] = u32x4{0u, 0u, 0u, 0u};
                if (in) hv[i] = *reinterpret_cast<const u32x4*>(h + col);
#pragma unroll
                for (int j = 0; j < kTiles; ++j) {
                    wv[j][i] = u32x4{0u, 0u, 0u, 0u};
                    if (in && l0 + 16 * j < p.n_logits) wv[j][i] = *reinterpret_cast<const u32x4*>(w[j] + col);
                }
            }
#pragma unroll
            for (int j = 0; j < kTiles; ++j)
                if (l0 + 16 * j < p.n_logits)
#pragma unroll
                    for (int i = 0; i < kBatch; ++i) acc[j] = mfma16(as_bf16x8(wv[j][i]), as_bf16x8(hv[i]), acc[j]);      // column r: token, rows 4 kg + i: logits
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < kTiles; ++j) part[(wave * kTiles + j) * 64 + lane] = acc[j];
        __syncthreads();
        // wavefront j sums tile j
        if (wave < kTiles) {
            f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int w8 = 0; w8 < kRouteWaves; ++w8) s += part[(w8 * kTiles + wave) * 64 + lane];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int l = l0 + 16 * wave + 4 * kg + i;
                if (l < p.n_logits) z[r * p.n_logits + l] = s[i] + p.bias[l];
            }
        }
    }
    __syncthreads();
    for (int t = wave; t < 16; t += kRouteWaves) {
        if (t0 + t >= p.T) break;
        float* zt = z + t * p.n_logits;
        if (p.extra_logit && lane == 0) p.extra_logit[t0 + t] = zt[p.E];
        choose_experts(p, zt, t0 + t, lane);
    }
}

// fp32: one wavefront per token
__global__ __launch_bounds__(256) void moe_route_f32_kernel(RouteParams p) {
    extern __shared__ __attribute__((aligned(16))) float route_lds[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int64_t t = (int64_t)blockIdx.x * 4 + wave;
    if (t >= p.T) return;
    float* z = route_lds + wave * p.n_logits;
    const float* h = (const float*)p.h + t * p.h_stride;
    for (int l = 0; l < p.n_logits; ++l) {
        const float* w = (const float*)p.w + (int64_t)l * p.w_stride;
        float s = 0.f;
        for (int c = lane; c < p.k; c += 64) s = fmaf(w[c], h[c], s);
        s = moe_wave_sum(s) + p.bias[l];
        if (lane == l % 64) z[l] = s;             // (the lane that reads it below)
    }
    if (p.extra_logit && lane == p.E % 64) p.extra_logit[t] = z[p.E];
    choose_experts(p, z, t, lane);
}

// ---- pairs sorted by expert -----------------------------------------------------------------------
// Workgroup e lists expert e's pairs: each of its 16 wavefronts counts the pairs of lower experts and of its own expert in
// its share of the ids, the shares are summed, and a second pass writes.
__global__ __launch_bounds__(1024) void moe_group_kernel(const int32_t* ids, int n_pairs, int E, int32_t* offsets, int32_t* order) {
    __shared__ int below[16], equal[16];
    const int e = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int share = ((n_pairs + 15) / 16 + 63) / 64 * 64;
    const int i0 = min(n_pairs, wave * share), i1 = min(n_pairs, i0 + share);
    int n_below = 0, n_equal = 0;
    for (int i = i0; i < i1; i += 64) {
        const int id = i + lane < i1 ? ids[i + lane] : E;
        n_below += __popcll(__builtin_amdgcn_ballot_w64(id < e));
        n_equal += __popcll(__builtin_amdgcn_ballot_w64(id == e));
    }
    if (lane == 0) {
        below[wave] = n_below;
        equal[wave] = n_equal;
    }
    __syncthreads();
    int at = 0;
    for (int w = 0; w < 16; ++w) at += below[w] + (w < wave ? equal[w] : 0);
    if (threadIdx.x == 0) {
        offsets[e] = at;
        if (e == E - 1) offsets[E] = n_pairs;
    }
    for (int i = i0; i < i1; i += 64) {
        const bool mine = i + lane < i1 && ids[i + lane] == e;
        const uint64_t m = __builtin_amdgcn_ballot_w64(mine);
        if (mine) order[at + __popcll(m & ((1ull << lane) - 1))] = i + lane;
        at += __popcll(m);
    }
}

// ---- grouped products -------------------------------------------------------------------------------
struct MoeParams {
    const void* a;               // rows of the left operand: tokens (gather) or places of the order
    const void* w;               // (E, rows of w, k)
    void* out;
    const int32_t *offsets, *order;
    const float* weights;        // down: per pair
    int64_t a_stride, a_rows, out_stride, out_rows;
    int n_pairs, E, k, n;        // n: output columns (gate_up: w has 2 n rows, gates first)
    int top;
};

// expert and first place of row tile `tile`; false: the tile has no rows
template <int BM>
__device__ __forceinline__ bool find_tile(const MoeParams& p, int tile, int& e, int& first, int& end) {
    int lo = 0, hi = p.E - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (p.offsets[mid] / BM + mid <= tile) lo = mid;
        else hi = mid - 1;
    }
    e = __builtin_amdgcn_readfirstlane(lo);
    const int start = __builtin_amdgcn_readfirstlane(p.offsets[e]);
    end = min(__builtin_amdgcn_readfirstlane(p.offsets[e + 1]), p.n_pairs);
    first = start + (tile - (start / BM + e)) * BM;
    return first >= start && first < end;
}

// row of the left operand for place i of the order
template <bool GATE_UP>
__device__ __forceinline__ int64_t left_row(const MoeParams& p, int i) {
    const int64_t row = GATE_UP ? p.order[i] / p.top : i;
    return min(max(row, (int64_t)0), p.a_rows - 1);
}

__device__ __forceinline__ float silu_fast(float x) { return x * __builtin_amdgcn_rcpf(1.0f + fast_exp2(-kLog2e * x)); }

// Four adjacent columns of one row into the output; out_row: place (gate_up) or pair (down)
__device__ __forceinline__ void store4(const MoeParams& p, int64_t out_row, int col, const float (&v)[4]) {
    __bf16* o = (__bf16*)p.out + out_row * p.out_stride + col;
    if (col + 4 <= p.n) {
        *reinterpret_cast<u32x2*>(o) = u32x2{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (col + i < p.n) o[i] = (__bf16)v[i];
    }
}

// 128 rows x 128 rows of w per workgroup (gate_up: 64 gates and the 64 ups of the same columns), k in steps of 64 through two
// LDS buffers filled by direct loads.  A 128-byte LDS row holds its eight 16-byte pieces in the order piece ^ (row % 8).
// Wavefront (wm, wn) computes 64 x 64; weights are the MFMA's first operand, so that a lane ends with adjacent columns.
template <bool GATE_UP>
__global__ __launch_bounds__(256, 2) void moe_gemm_kernel(MoeParams p, int n_tiles, int m_tiles) {
    constexpr int BM = 128, BK = 64, kTile = 128 * BK * 2;
    __shared__ __attribute__((aligned(1024))) unsigned char lds[4 * kTile];          // [buffer][rows | w]
    const int id = xcd_chunked_id(blockIdx.x, n_tiles * m_tiles, n_tiles);
    const int n_tile = id % n_tiles;
    int e, first, end;
    if (!find_tile<BM>(p, id / n_tiles, e, first, end)) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave >> 1, wn = wave & 1, r = lane & 15, kg = lane >> 4;
    const int n0 = n_tile * (GATE_UP ? 64 : 128);
    const __bf16* a_base = (const __bf16*)p.a;
    const __bf16* w_base = (const __bf16*)p.w + (int64_t)e * (GATE_UP ? 2 : 1) * p.n * p.k;
    // wavefront w fills rows 32 w .. 32 w + 31 of both tiles, 8 rows per load
    uint32_t a_off[4], w_off[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int row = 32 * wave + 8 * j + (lane >> 3), piece = (lane & 7) ^ (row & 7);
        a_off[j] = (uint32_t)((left_row<GATE_UP>(p, min(first + row, end - 1)) * p.a_stride + piece * 8) * 2);
        int64_t wr = GATE_UP ? (row < 64 ? min(n0 + row, p.n - 1) : p.n + min(n0 + row - 64, p.n - 1)) : min(n0 + row, p.n - 1);
        w_off[j] = (uint32_t)((wr * p.k + piece * 8) * 2);
    }
    const uint32_t lds0 = lds_address(lds);
    const auto issue = [&](int k0, int buf) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            dma_to_lds_16(a_base + k0, a_off[j], lds0 + (2 * buf) * kTile + (32 * wave + 8 * j) * 128);
            dma_to_lds_16(w_base + k0, w_off[j], lds0 + (2 * buf + 1) * kTile + (32 * wave + 8 * j) * 128);
        }
    };
    f32x4 acc[4][4];                              // [16 rows of w][16 rows]
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    // 16-row groups of w of this wavefront: gate_up: gates 32 wn, 32 wn + 16, then the ups of these columns
    const auto w_group = [&](int i) { return GATE_UP ? (i >> 1) * 64 + 32 * wn + (i & 1) * 16 : 64 * wn + 16 * i; };
    issue(0, 0);
    for (int k0 = 0, buf = 0; k0 < p.k; k0 += BK, buf ^= 1) {
        wait_vmcnt<0>();
        __syncthreads();                          // the tile has landed, and everybody has read the other buffer
        if (k0 + BK < p.k) issue(k0 + BK, buf ^ 1);
        const unsigned char* at = lds + (2 * buf) * kTile;
        const unsigned char* wt = at + kTile;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const int piece = ((4 * s + kg) ^ (r & 7)) * 16;
            bf16x8 wf[4], af[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                wf[i] = as_bf16x8(*reinterpret_cast<const u32x4*>(wt + (w_group(i) + r) * 128 + piece));
                af[i] = as_bf16x8(*reinterpret_cast<const u32x4*>(at + (64 * wm + 16 * i + r) * 128 + piece));
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = mfma16(wf[i], af[j], acc[i][j]);
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int place = first + 64 * wm + 16 * j + r;
        if (place >= end) continue;
        if constexpr (GATE_UP) {
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                float v[4];
#pragma unroll
                for (int q = 0; q < 4; ++q) v[q] = silu_fast(acc[i][j][q]) * acc[i + 2][j][q];
                store4(p, place, n0 + 32 * wn + 16 * i + 4 * kg, v);
            }
        } else {
            const int pair = min(max(p.order[place], 0), p.n_pairs - 1);
            const float wgt = p.weights[pair];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                float v[4];
#pragma unroll
                for (int q = 0; q < 4; ++q) v[q] = wgt * acc[i][j][q];
                store4(p, pair, n0 + 64 * wn + 16 * i + 4 * kg, v);
            }
        }
    }
}

// 16 rows x 16 rows of w (gate_up: 16 gates and their 16 ups).  The four wavefronts take the 64-wide steps of k in turn, read
// their operands straight from memory and meet in LDS.
template <bool GATE_UP>
__global__ __launch_bounds__(256) void moe_skinny_kernel(MoeParams p, int n_tiles, int m_tiles) {
    constexpr int BM = 16, NW = GATE_UP ? 2 : 1, kBatch = 4;        // steps of k whose loads are in flight together
    __shared__ f32x4 part[4][NW][64];
    const int id = xcd_chunked_id(blockIdx.x, n_tiles * m_tiles, n_tiles);
    const int n0 = id % n_tiles * 16;
    int e, first, end;
    if (!find_tile<BM>(p, id / n_tiles, e, first, end)) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, kg = lane >> 4;
    const __bf16* a = (const __bf16*)p.a + left_row<GATE_UP>(p, min(first + r, end - 1)) * p.a_stride + 8 * kg;
    const __bf16* w = (const __bf16*)p.w + ((int64_t)e * NW * p.n + min(n0 + r, p.n - 1)) * p.k + 8 * kg;
    const int64_t up = (int64_t)p.n * p.k;
    f32x4 acc[NW];
#pragma unroll
    for (int i = 0; i < NW; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 64 * wave; k0 < p.k; k0 += 256 * kBatch) {
        u32x4 av[kBatch][2], wv[NW][kBatch][2];
#pragma unroll
        for (int t = 0; t < kBatch; ++t)
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                const int col = k0 + 256 * t + 32 * s;
                av[t][s] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
                for (int i = 0; i < NW; ++i) wv[i][t][s] = av[t][s];
                if (k0 + 256 * t < p.k) {
#pragma unroll
                    for (int i = 0; i < NW; ++i) wv[i][t][s] = *reinterpret_cast<const u32x4*>(w + i * up + col);
                    av[t][s] = *reinterpret_cast<const u32x4*>(a + col);
                }
            }
#pragma unroll
        for (int t = 0; t < kBatch; ++t)
#pragma unroll
            for (int s = 0; s < 2; ++s)
#pragma unroll
                for (int i = 0; i < NW; ++i) acc[i] = mfma16(as_bf16x8(wv[i][t][s]), as_bf16x8(av[t][s]), acc[i]);
    }
#pragma unroll
    for (int i = 0; i < NW; ++i) part[wave][i][lane] = acc[i];
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
        for (int w4 = 1; w4 < 4; ++w4) acc[i] += part[w4][i][lane];
    const int place = first + r;
    if (place >= end) return;
    float v[4];
    if constexpr (GATE_UP) {
#pragma unroll
        for (int q = 0; q < 4; ++q) v[q] = silu_fast(acc[0][q]) * acc[1][q];
        store4(p, place, n0 + 4 * kg, v);
    } else {
        const int pair = min(max(p.order[place], 0), p.n_pairs - 1);
        const float wgt = p.weights[pair];
#pragma unroll
        for (int q = 0; q < 4; ++q) v[q] = wgt * acc[0][q];
        store4(p, pair, n0 + 4 * kg, v);
    }
}

// fp32: 16 rows x 64 columns per workgroup, a thread owns four rows of one column
template <bool GATE_UP>
__global__ __launch_bounds__(256) void moe_f32_kernel(MoeParams p, int n_tiles, int m_tiles) {
    constexpr int BM = 16, BK = 16, NW = GATE_UP ? 2 : 1;
    __shared__ float a_lds[BM][BK + 1], w_lds[NW][64][BK + 1];
    const int n0 = blockIdx.x % n_tiles * 64;
    int e, first, end;
    if (!find_tile<BM>(p, blockIdx.x / n_tiles, e, first, end)) return;
    const int tid = threadIdx.x, col = tid & 63, rows = (tid >> 6) * 4;
    const float* w = (const float*)p.w + (int64_t)e * NW * p.n * p.k;
    const int ar = tid / BK, ac = tid % BK;
    const float* a = (const float*)p.a + left_row<GATE_UP>(p, min(first + ar, end - 1)) * p.a_stride;
    float acc[NW][4];
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
    for (int k0 = 0; k0 < p.k; k0 += BK) {
        __syncthreads();
        a_lds[ar][ac] = k0 + ac < p.k ? a[k0 + ac] : 0.f;
#pragma unroll
        for (int i = 0; i < NW; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int64_t row = (int64_t)i * p.n + min(n0 + 16 * j + ar, p.n - 1);
                w_lds[i][16 * j + ar][ac] = k0 + ac < p.k ? w[row * p.k + k0 + ac] : 0.f;
            }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; ++k)
#pragma unroll
            for (int i = 0; i < NW; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(w_lds[i][col][k], a_lds[rows + j][k], acc[i][j]);
    }
    if (n0 + col >= p.n) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int place = first + rows + j;
        if (place >= end) continue;
        float v;
        int64_t row = place;
        if constexpr (GATE_UP) {
            v = acc[0][j] / (1.0f + expf(-acc[0][j])) * acc[1][j];
        } else {
            row = min(max(p.order[place], 0), p.n_pairs - 1);
            v = p.weights[row] * acc[0][j];
        }
        ((float*)p.out)[row * p.out_stride + n0 + col] = v;
    }
}

template <bool GATE_UP>
static int launch_moe(const MoeParams& p, int dtype, int tiling, hipStream_t s) {
    const bool large = tiling == MI355_TILING_LARGE || (tiling == MI355_TILING_AUTO && p.n_pairs > 32 * (int64_t)p.E);
    const int bm = dtype == MI355_BF16 && large ? 128 : 16;
    const int bn = dtype == MI355_FP32 ? 64 : (!large ? 16 : (GATE_UP ? 64 : 128));
    const int n_tiles = (p.n + bn - 1) / bn, m_tiles = p.n_pairs / bm + p.E;
    if ((int64_t)n_tiles * m_tiles > 0x7fffffffLL) return (int)hipErrorInvalidValue;
    const dim3 grid((unsigned)(n_tiles * m_tiles)), block(256);
    if (dtype == MI355_FP32) hipLaunchKernelGGL(moe_f32_kernel<GATE_UP>, grid, block, 0, s, p, n_tiles, m_tiles);
    else if (large) hipLaunchKernelGGL(moe_gemm_kernel<GATE_UP>, grid, block, 0, s, p, n_tiles, m_tiles);
    else hipLaunchKernelGGL(moe_skinny_kernel<GATE_UP>, grid, block, 0, s, p, n_tiles, m_tiles);
    return (int)hipGetLastError();
}

static int moe_product(bool gate_up, const void* a, const void* w, void* out, const int32_t* offsets, const int32_t* order,
                       const float* weights, int64_t a_stride, int64_t a_rows, int64_t out_stride, int64_t out_rows, int64_t n_pairs,
                       int E, int top, int k, int n, int dtype, int tiling, void* stream) {
    if (!a || !w || !out || !offsets || !order || (!gate_up && !weights)) return set_error(MI355_EINVAL, "moe: null pointer argument");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "moe: dtype must be MI355_BF16 or MI355_FP32");
    if (E <= 0 || E > kMaxExperts || top <= 0 || k <= 0 || n <= 0 || n_pairs < 0 || n_pairs > 0x3fffffffLL)
        return set_error(MI355_EINVAL, "moe: experts, top, k, n, n_pairs out of range");
    if (tiling < MI355_TILING_AUTO || tiling > MI355_TILING_LARGE) return set_error(MI355_EINVAL, "moe: unknown tiling");
    if (a_stride < k || out_stride < n) return set_error(MI355_EINVAL, "moe: row strides shorter than a row");
    if (a_rows < (gate_up ? (n_pairs + top - 1) / top : n_pairs) || out_rows < n_pairs) return set_error(MI355_EINVAL, "moe: too few rows");
    if (dtype == MI355_BF16) {
        if (k % 64 || a_stride % 8 || out_stride % 4 || (reinterpret_cast<uintptr_t>(a) & 15) || (reinterpret_cast<uintptr_t>(w) & 15) ||
            (reinterpret_cast<uintptr_t>(out) & 7))
            return set_error(MI355_EINVAL, "moe: bf16 operands need k in multiples of 64 and 16-byte aligned rows");
        if (a_rows * a_stride > 0x7fffffffLL || 2LL * n * k > 0x7fffffffLL)
            return set_error(MI355_EINVAL, "moe: an operand is too large for 32-bit byte offsets");
    }
    if (n_pairs == 0) return MI355_OK;
    MoeParams p;
    p.a = a;
    p.w = w;
    p.out = out;
    p.offsets = offsets;
    p.order = order;
    p.weights = weights;
    p.a_stride = a_stride;
    p.a_rows = a_rows;
    p.out_stride = out_stride;
    p.out_rows = out_rows;
    p.n_pairs = (int)n_pairs;
    p.E = E;
    p.k = k;
    p.n = n;
    p.top = top;
    const int rc = gate_up ? launch_moe<true>(p, dtype, tiling, (hipStream_t)stream) : launch_moe<false>(p, dtype, tiling, (hipStream_t)stream);
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

}  // namespace mi355

using namespace mi355;

extern "C" int mi355_moe_route(const void* h, const void* w, const float* bias, int32_t* ids, float* weights, float* extra_logit,
                               int64_t n_tokens, int64_t h_row_stride, int64_t w_row_stride, int k, int n_experts, int top, int dtype,
                               void* stream) {
    if (!h || !w || !bias || !ids || !weights) return set_error(MI355_EINVAL, "moe_route: null pointer argument");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "moe_route: dtype must be MI355_BF16 or MI355_FP32");
    if (n_tokens < 0 || k <= 0 || n_experts <= 0 || n_experts > kMaxExperts || top <= 0 || top > n_experts || top > kMaxTop)
        return set_error(MI355_EINVAL, "moe_route: n_tokens, k, n_experts (up to 1024), top (up to 64) out of range");
    if (h_row_stride < k || w_row_stride < k) return set_error(MI355_EINVAL, "moe_route: row strides shorter than a row");
    if (dtype == MI355_BF16 && (k % 8 || h_row_stride % 8 || w_row_stride % 8 || (reinterpret_cast<uintptr_t>(h) & 15) ||
                                (reinterpret_cast<uintptr_t>(w) & 15)))
        return set_error(MI355_EINVAL, "moe_route: bf16 rows must be 16-byte aligned and k a multiple of 8");
    if (n_tokens > 0x7fffff00LL) return set_error(MI355_EINVAL, "moe_route: too many tokens");
    if (n_tokens == 0) return MI355_OK;
    RouteParams p;
    p.h = h;
    p.w = w;
    p.bias = bias;
    p.ids = ids;
    p.weights = weights;
    p.extra_logit = extra_logit;
    p.T = n_tokens;
    p.h_stride = h_row_stride;
    p.w_stride = w_row_stride;
    p.k = k;
    p.E = n_experts;
    p.n_logits = n_experts + (extra_logit ? 1 : 0);
    p.top = top;
    hipStream_t s = (hipStream_t)stream;
    if (dtype == MI355_BF16)
        hipLaunchKernelGGL(moe_route_kernel, dim3((unsigned)((n_tokens + 15) / 16)), dim3(64 * kRouteWaves),
                           (kRouteWaves * 4 * 64 * 4 + 16 * p.n_logits) * sizeof(float), s, p);
    else
        hipLaunchKernelGGL(moe_route_f32_kernel, dim3((unsigned)((n_tokens + 3) / 4)), dim3(256), 4 * p.n_logits * sizeof(float), s, p);
    const int rc = (int)hipGetLastError();
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

extern "C" int mi355_moe_group(const int32_t* ids, int64_t n_pairs, int n_experts, int32_t* offsets, int32_t* order, void* stream) {
    if (!ids || !offsets || !order) return set_error(MI355_EINVAL, "moe_group: null pointer argument");
    if (n_pairs < 0 || n_pairs > 0x3fffffffLL || n_experts <= 0 || n_experts > kMaxExperts)
        return set_error(MI355_EINVAL, "moe_group: n_pairs, n_experts (up to 1024) out of range");
    hipLaunchKernelGGL(moe_group_kernel, dim3((unsigned)n_experts), dim3(1024), 0, (hipStream_t)stream, ids, (int)n_pairs, n_experts, offsets, order);
    const int rc = (int)hipGetLastError();
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

extern "C" int mi355_moe_gate_up(const void* h, const void* w, void* act, const int32_t* offsets, const int32_t* order, int64_t n_tokens,
                                 int64_t h_row_stride, int64_t act_row_stride, int n_experts, int top, int k, int ff, int dtype,
                                 int tiling, void* stream) {
    return moe_product(true, h, w, act, offsets, order, nullptr, h_row_stride, n_tokens, act_row_stride, n_tokens * top,
                       n_tokens * top, n_experts, top, k, ff, dtype, tiling, stream);
}

extern "C" int mi355_moe_down(const void* act, const void* w, const float* weights, void* out, const int32_t* offsets, const int32_t* order,
                              int64_t n_tokens, int64_t act_row_stride, int64_t out_row_stride, int n_experts, int top, int ff, int n,
                              int dtype, int tiling, void* stream) {
    return moe_product(false, act, w, out, offsets, order, weights, act_row_stride, n_tokens * top, out_row_stride, n_tokens * top,
                       n_tokens * top, n_experts, top, ff, n, dtype, tiling, stream);
}
