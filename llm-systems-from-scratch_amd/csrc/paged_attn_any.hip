// Paged attention for any head size and for fp32: the general path beside the MFMA kernels.
//
// One workgroup of four wavefronts per (query row, query head); it serves prompts and decode steps alike (a query row is
// any token of a sequence whose keys and values already sit in the paged cache, its own included).  The keys are dealt to
// the wavefronts in tiles of 64: a lane takes one key's dot product with the query, the wavefront runs an online softmax
// over its tiles, and the lanes then own value columns while the tile's weights come from LDS.  The four partial results
// meet in LDS.  With a sliding window only the blocks that hold visible keys are walked.  Scores, weights and sums are fp32; keys and values are read as stored (bf16 or fp32).
#include "common.hpp"
#include "launch.hpp"

namespace mi355 {

constexpr int kAnyWaves = 4;
constexpr int kAnyMaxDim = 512;

struct PagedAnyParams {
    const void *q, *k_cache, *v_cache;
    void* out;
    const int32_t* cu_q;              // (B + 1), or null: sequence b owns query row b
    const int32_t* block_tables;
    const int32_t* context_lens;
    const float *head_scale, *sink;   // optional, per query head
    int64_t q_stride, out_stride, bt_stride;      // elements between query rows / output rows / table rows
    int64_t rows;
    int B, Hq, Hkv, Dk, Dv, num_blocks, max_blocks;
    int window, keep_first;           // window 0: every earlier key is visible
    float scale_log2;
};

// NV: value columns per lane (Dv <= 64 * NV)
template <typename T, int NV>
__global__ __launch_bounds__(kAnyWaves * 64) void paged_attn_any_kernel(PagedAnyParams p) {
    __shared__ __attribute__((aligned(16))) float q_lds[kAnyMaxDim];
    __shared__ float w_lds[kAnyWaves][64];
    __shared__ float acc_lds[kAnyWaves][64 * NV];
    __shared__ float m_lds[kAnyWaves], l_lds[kAnyWaves];
    const int lane = threadIdx.x & 63;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int64_t row = blockIdx.x / p.Hq;
    const int h = (int)(blockIdx.x % p.Hq), hk = h / (p.Hq / p.Hkv);
    // the row's sequence: the last b with cu_q[b] <= row
    int b = (int)row, q_start = (int)row, q_end = (int)row + 1;
    if (p.cu_q) {
        int lo = 0, hi = p.B - 1;
        while (lo < hi) {
            const int mid = (lo + hi + 1) / 2;
            if (p.cu_q[mid] <= row) lo = mid;
            else hi = mid - 1;
        }
        b = lo;
        q_start = p.cu_q[b];
        q_end = p.cu_q[b + 1];
        if (row < q_start || row >= q_end) return;         // (a row that no sequence owns; uniform over the workgroup)
    }
    // keys 0 .. n_keys - 1 are visible: the row is token (context - chunk length + row - q_start) of its sequence
    const int ctx = min(p.context_lens[b], 16 * p.max_blocks);
    const VisibleKeys vis = visible_keys(min(ctx, ctx - (q_end - q_start) + (int)(row - q_start) + 1), p.window, p.keep_first);
    const int n_keys = vis.n;
    const T* q = (const T*)p.q + row * p.q_stride + (int64_t)h * p.Dk;
    for (int d = threadIdx.x; d < p.Dk; d += kAnyWaves * 64) q_lds[d] = (float)q[d];
    __syncthreads();

    const float scale = p.head_scale ? p.scale_log2 * p.head_scale[h] : p.scale_log2;
    const int32_t* bt = p.block_tables + (int64_t)b * p.bt_stride;
    const T* kc = (const T*)p.k_cache;
    const T* vc = (const T*)p.v_cache;
    float m = -INFINITY, l = 0.f, acc[NV];
#pragma unroll
    for (int e = 0; e < NV; ++e) acc[e] = 0.f;
    for (int k0 = 64 * wave; k0 < n_keys; k0 += 64 * kAnyWaves) {
        const int key = k0 + lane;
        float x = -INFINITY;
        // a block id outside the pool (a corrupted table) is clamped into it
        const int my_blk = min(max(bt[vis.logical_block(min(key, n_keys - 1) >> 4)], 0), p.num_blocks - 1);
        if (key < n_keys && !vis.hidden(key)) {
            const T* kr = kc + (((int64_t)my_blk * p.Hkv + hk) * 16 + (key & 15)) * p.Dk;
            float dot = 0.f;
            for (int d = 0; d < p.Dk; d += 8) {             // rows are multiples of 8 elements, 16-byte aligned
                float kv[8];
                if constexpr (sizeof(T) == 2) {
                    const bf16x8 t = as_bf16x8(*reinterpret_cast<const u32x4*>(kr + d));
#pragma unroll
                    for (int e = 0; e < 8; ++e) kv[e] = (float)t[e];
                } else {
                    const f32x4 a = *reinterpret_cast<const f32x4*>(kr + d), c = *reinterpret_cast<const f32x4*>(kr + d + 4);
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        kv[e] = a[e];
                        kv[4 + e] = c[e];
                    }
                }
#pragma unroll
                for (int e = 0; e < 8; ++e) dot = fmaf(q_lds[d + e], kv[e], dot);
            }
            x = dot * scale;
        }
        float mx = x;
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
        const float m_new = fmaxf(m, mx);                   // finite: at most 30 keys of a tile are hidden, and the last key is visible
        const float alpha = fast_exp2(m - m_new);           // 0 the first time
        m = m_new;
        const float w = fast_exp2(x - m);
        l = l * alpha + w;
#pragma unroll
        for (int e = 0; e < NV; ++e) acc[e] *= alpha;
        w_lds[wave][lane] = w;                              // (read by this wavefront only, whose LDS operations are in order)
        const int n = min(64, n_keys - k0);
        for (int j0 = 0; j0 < n; j0 += 16) {
            const int64_t slab = ((int64_t)__builtin_amdgcn_readlane(my_blk, j0) * p.Hkv + hk) * 16;
            const int jn = min(16, n - j0);
            for (int j = 0; j < jn; ++j) {
                const T* vr = vc + (slab + j) * p.Dv;
                const float wj = w_lds[wave][j0 + j];
#pragma unroll
                for (int e = 0; e < NV; ++e) {
                    const int d = 64 * e + lane;
                    if (d < p.Dv) acc[e] = fmaf(wj, (float)vr[d], acc[e]);
                }
            }
        }
    }
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) l += __shfl_xor(l, off, 64);
#pragma unroll
    for (int e = 0; e < NV; ++e) acc_lds[wave][64 * e + lane] = acc[e];
    if (lane == 0) {
        m_lds[wave] = m;
        l_lds[wave] = l;
    }
    __syncthreads();
    float M = -INFINITY;
#pragma unroll
    for (int w = 0; w < kAnyWaves; ++w) M = fmaxf(M, m_lds[w]);
    float f[kAnyWaves], den = 0.f;
#pragma unroll
    for (int w = 0; w < kAnyWaves; ++w) {
        f[w] = fast_exp2(m_lds[w] - M);                     // a wavefront without keys has m = -inf -> 0
        den += f[w] * l_lds[w];
    }
    if (p.sink) den += fast_exp2(fmaf(p.sink[h], kLog2e, -M));
    const float inv = 1.0f / den;
    T* out = (T*)p.out + row * p.out_stride + (int64_t)h * p.Dv;
    for (int d = threadIdx.x; d < p.Dv; d += kAnyWaves * 64) {
        float num = 0.f;
#pragma unroll
        for (int w = 0; w < kAnyWaves; ++w) num += f[w] * acc_lds[w][d];
        out[d] = (T)(num * inv);
    }
}

template <typename T>
static int launch_any(const PagedAnyParams& p, hipStream_t s) {
    const dim3 grid((unsigned)(p.rows * p.Hq)), block(kAnyWaves * 64);
    if (p.Dv <= 64) hipLaunchKernelGGL((paged_attn_any_kernel<T, 1>), grid, block, 0, s, p);
    else if (p.Dv <= 128) hipLaunchKernelGGL((paged_attn_any_kernel<T, 2>), grid, block, 0, s, p);
    else if (p.Dv <= 256) hipLaunchKernelGGL((paged_attn_any_kernel<T, 4>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((paged_attn_any_kernel<T, 8>), grid, block, 0, s, p);
    return (int)hipGetLastError();
}

}  // namespace mi355

using namespace mi355;

static int paged_attn_any_common(const void* q, const void* k_cache, const void* v_cache, void* out, int64_t q_row_stride,
                                        int64_t out_row_stride, int64_t n_rows, const int32_t* cu_seqlens_q,
                                        const int32_t* block_tables, int64_t bt_row_stride, int64_t max_blocks,
                                        const int32_t* context_lens, const float* head_scale, const float* sink, int B, int Hq,
                                        int Hkv, int Dk, int Dv, int block_size, int64_t num_blocks, float softmax_scale,
                                        int window, int keep_first, int dtype, void* stream) {
    if (!q || !k_cache || !v_cache || !out || !block_tables || !context_lens)
        return set_error(MI355_EINVAL, "paged_attn_any: null pointer argument");
    if (dtype != MI355_BF16 && dtype != MI355_FP32)
        return set_error(MI355_EDTYPE, "paged_attn_any: dtype must be MI355_BF16 or MI355_FP32");
    if (B <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || n_rows < 0)
        return set_error(MI355_EINVAL, "paged_attn_any: B, Hq, Hkv and n_rows out of range (Hq a multiple of Hkv)");
    if (!cu_seqlens_q && n_rows != B) return set_error(MI355_EINVAL, "paged_attn_any: one query row per sequence without cu_seqlens_q");
    if (block_size != 16) return set_error(MI355_EINVAL, "paged_attn_any: block_size must be 16");
    if (Dk <= 0 || Dv <= 0 || Dk > kAnyMaxDim || Dv > kAnyMaxDim || Dk % 8 || Dv % 8)
        return set_error(MI355_EINVAL, "paged_attn_any: head sizes must be multiples of 8 up to 512");
    if (num_blocks <= 0 || num_blocks > 0x7fffffffLL || max_blocks <= 0 || max_blocks > bt_row_stride || max_blocks > 0x7ffffff)
        return set_error(MI355_EINVAL, "paged_attn_any: num_blocks, max_blocks out of range");
    if (((uintptr_t)k_cache | (uintptr_t)v_cache) & 15)
        return set_error(MI355_EINVAL, "paged_attn_any: the caches must be 16-byte aligned");
    if (q_row_stride < (int64_t)Hq * Dk || out_row_stride < (int64_t)Hq * Dv)
        return set_error(MI355_EINVAL, "paged_attn_any: row strides shorter than a row");
    if (window < 0 || keep_first < 0) return set_error(MI355_EINVAL, "paged_attn_any: window and keep_first must not be negative");
    if (n_rows * Hq > 0x7fffffffLL) return set_error(MI355_EINVAL, "paged_attn_any: too many rows");
    if (n_rows == 0) return MI355_OK;
    PagedAnyParams p;
    p.q = q;
    p.k_cache = k_cache;
    p.v_cache = v_cache;
    p.out = out;
    p.cu_q = cu_seqlens_q;
    p.block_tables = block_tables;
    p.context_lens = context_lens;
    p.head_scale = head_scale;
    p.sink = sink;
    p.q_stride = q_row_stride;
    p.out_stride = out_row_stride;
    p.bt_stride = bt_row_stride;
    p.rows = n_rows;
    p.B = B;
    p.Hq = Hq;
    p.Hkv = Hkv;
    p.Dk = Dk;
    p.Dv = Dv;
    p.num_blocks = (int)num_blocks;
    p.max_blocks = (int)max_blocks;
    p.window = window;
    p.keep_first = keep_first;
    p.scale_log2 = softmax_scale * kLog2e;
    const int rc = dtype == MI355_BF16 ? launch_any<__bf16>(p, (hipStream_t)stream) : launch_any<float>(p, (hipStream_t)stream);
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

extern "C" int mi355_paged_attn_any_fwd(const void* q, const void* k_cache, const void* v_cache, void* out, int64_t q_row_stride,
                                        int64_t out_row_stride, int64_t n_rows, const int32_t* cu_seqlens_q,
                                        const int32_t* block_tables, int64_t bt_row_stride, int64_t max_blocks,
                                        const int32_t* context_lens, const float* head_scale, const float* sink, int B, int Hq,
                                        int Hkv, int Dk, int Dv, int block_size, int64_t num_blocks, float softmax_scale,
                                        int dtype, void* stream) {
    return paged_attn_any_common(q, k_cache, v_cache, out, q_row_stride, out_row_stride, n_rows, cu_seqlens_q, block_tables,
                                 bt_row_stride, max_blocks, context_lens, head_scale, sink, B, Hq, Hkv, Dk, Dv, block_size, num_blocks,
                                 softmax_scale, 0, 0, dtype, stream);
}

extern "C" int mi355_paged_attn_any_fwd_window(const void* q, const void* k_cache, const void* v_cache, void* out, int64_t q_row_stride,
                                               int64_t out_row_stride, int64_t n_rows, const int32_t* cu_seqlens_q,
                                               const int32_t* block_tables, int64_t bt_row_stride, int64_t max_blocks,
                                               const int32_t* context_lens, const float* head_scale, const float* sink, int B, int Hq,
                                               int Hkv, int Dk, int Dv, int block_size, int64_t num_blocks, float softmax_scale,
                                               int window, int keep_first, int dtype, void* stream) {
    return paged_attn_any_common(q, k_cache, v_cache, out, q_row_stride, out_row_stride, n_rows, cu_seqlens_q, block_tables,
                                 bt_row_stride, max_blocks, context_lens, head_scale, sink, B, Hq, Hkv, Dk, Dv, block_size, num_blocks,
                                 softmax_scale, window, keep_first, dtype, stream);
}
