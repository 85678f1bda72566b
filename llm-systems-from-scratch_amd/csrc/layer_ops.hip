// The fused elementwise/normalisation ops that sit next to attention in a transformer
// block: RMSNorm forward (optionally fused with the residual add in front of it),
// silu(gate) * up, the end of a sublayer in a model with Dynamic Tanh norms and gated
// residuals, the PolyNorm activation, the token + position embedding, the RMS norm of an
// fp32 residual stream with everything that is added to the stream in front of it, gated
// and plain feed-forward activations, and the gated norm behind a recurrent mixer.  All are
// streaming kernels: HBM-bound, 16-byte accesses, fp32 math, one rounding to bf16 per
// stored value (all but the first two also exist with fp32 values throughout).
#include "common.hpp"
#include "launch.hpp"

namespace mi355 {

struct RmsNormParams {
    const __bf16* x;
    const __bf16* residual;      // optional: h = bf16(x + residual) is normalised instead of x
    const void* weight;          // bf16 or fp32 (n_cols)
    __bf16* y;
    __bf16* sum_out;             // optional (with residual): receives h
    float* rstd_out;             // optional (n_rows)
    int64_t n_rows;
    int64_t xs, rs, ys, ss;      // row strides in elements
    int n_cols;
    float eps;
    bool weight_fp32;
};

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}

__device__ __forceinline__ void load_weight8(const RmsNormParams& p, int col, float (&w)[8]) {
    if (p.weight_fp32) {
        const f32x4* wp = reinterpret_cast<const f32x4*>(static_cast<const float*>(p.weight) + col);
        const f32x4 a = wp[0], b = wp[1];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            w[e] = a[e];
            w[4 + e] = b[e];
        }
    } else {
        const bf16x8 a = as_bf16x8(*reinterpret_cast<const u32x4*>(static_cast<const __bf16*>(p.weight) + col));
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = (float)a[e];
    }
}

// One wavefront per row, the row held in registers: NCHUNK chunks of 512 elements (8 per lane).
// Requires n_cols % 8 == 0, n_cols <= 512 * NCHUNK, 16-byte aligned rows.
// The occupancy attribute caps the registers at 128: without it the compiler hoists every weight load
// of the 8-chunk instance (232 registers, two wavefronts per SIMD) and the kernel streams 15 % slower.
template <int NCHUNK>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(4, 8))) void rms_norm_rows_kernel(RmsNormParams p) {
    const int lane = threadIdx.x & 63;
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= p.n_rows) return;
    const __bf16* xr = p.x + row * p.xs;
    const __bf16* rr = p.residual ? p.residual + row * p.rs : nullptr;
    u32x4 raw[NCHUNK];
    float ssq = 0.f;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * 512 + lane * 8;
        raw[c] = u32x4{0u, 0u, 0u, 0u};
        if (col < p.n_cols) {
            raw[c] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(xr + col));
            if (rr) {
                const u32x4 rw = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(rr + col));
                const bf16x8 a = as_bf16x8(raw[c]), b = as_bf16x8(rw);
                u32x4 s;
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    s[e] = pack_bf16((float)a[2 * e] + (float)b[2 * e], (float)a[2 * e + 1] + (float)b[2 * e + 1]);
                raw[c] = s;
                if (p.sum_out) __builtin_nontemporal_store(s, reinterpret_cast<u32x4*>(p.sum_out + row * p.ss + col));
            }
            const bf16x8 v = as_bf16x8(raw[c]);
#pragma unroll
            for (int e = 0; e < 8; ++e) ssq += (float)v[e] * (float)v[e];
        }
    }
    ssq = wave_sum(ssq);
    const float rstd = 1.0f / sqrtf(ssq / (float)p.n_cols + p.eps);
    if (p.rstd_out && lane == 0) p.rstd_out[row] = rstd;
    __bf16* yr = p.y + row * p.ys;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * 512 + lane * 8;
        if (col < p.n_cols) {
            float w[8];
            load_weight8(p, col, w);
            const bf16x8 v = as_bf16x8(raw[c]);
            u32x4 o;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                o[e] = pack_bf16(w[2 * e] * ((float)v[2 * e] * rstd), w[2 * e + 1] * ((float)v[2 * e + 1] * rstd));
            __builtin_nontemporal_store(o, reinterpret_cast<u32x4*>(yr + col));
        }
    }
}

// Any n_cols, any alignment: one wavefront per row, two passes over the row, scalar accesses.
__global__ __launch_bounds__(256) void rms_norm_generic_kernel(RmsNormParams p) {
    const int lane = threadIdx.x & 63;
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= p.n_rows) return;
    const __bf16* xr = p.x + row * p.xs;
    const __bf16* rr = p.residual ? p.residual + row * p.rs : nullptr;
    __bf16* sr = (rr && p.sum_out) ? p.sum_out + row * p.ss : nullptr;
    float ssq = 0.f;
    for (int col = lane; col < p.n_cols; col += 64) {
        float v = (float)xr[col];
        if (rr) {
            v = (float)(__bf16)(v + (float)rr[col]);
            if (sr) sr[col] = (__bf16)v;
        }
        ssq += v * v;
    }
    ssq = wave_sum(ssq);
    const float rstd = 1.0f / sqrtf(ssq / (float)p.n_cols + p.eps);
    if (p.rstd_out && lane == 0) p.rstd_out[row] = rstd;
    __bf16* yr = p.y + row * p.ys;
    for (int col = lane; col < p.n_cols; col += 64) {
        float v = (float)xr[col];
        if (rr) v = (float)(__bf16)(v + (float)rr[col]);
        const float w = p.weight_fp32 ? static_cast<const float*>(p.weight)[col]
                                      : (float)static_cast<const __bf16*>(p.weight)[col];
        yr[col] = (__bf16)(w * (v * rstd));
    }
}

struct SiluMulParams {
    const __bf16* gate;
    const __bf16* up;
    __bf16* out;
    int64_t n_rows;
    int64_t gs, us, os;          // row strides in elements
    int n_cols;
};

// silu in fp32, rounded to bf16, then multiplied by `up` (product rounded to bf16): the order of
// roundings of a bf16 tensor program silu(gate).to(bf16) * up.
__device__ __forceinline__ float silu_mul_one(float g, float u) {
    const float s = g / (1.0f + __expf(-g));
    return (float)(__bf16)s * u;
}

// One thread per 8 adjacent elements of a row.  Requires n_cols % 8 == 0 and 16-byte aligned rows.
// The grid covers the tensor once (the loop only runs again beyond 2^31 workgroups): workgroups are
// dispatched in order, so the accesses in flight at any time form one window that moves through the
// tensor, which DRAM serves faster than the scattered windows of a small persistent grid (measured:
// 6.4 against 4.9 TB/s for a two-reads-one-write stream of this size).
__global__ __launch_bounds__(256) void silu_mul_vec8_kernel(SiluMulParams p) {
    const int groups = p.n_cols / 8;
    const int64_t total = p.n_rows * groups;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total;
         idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / groups;
        const int col = (int)(idx % groups) * 8;
        const bf16x8 g = as_bf16x8(__builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p.gate + row * p.gs + col)));
        const bf16x8 u = as_bf16x8(__builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p.up + row * p.us + col)));
        u32x4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e)
            o[e] = pack_bf16(silu_mul_one((float)g[2 * e], (float)u[2 * e]),
                             silu_mul_one((float)g[2 * e + 1], (float)u[2 * e + 1]));
        __builtin_nontemporal_store(o, reinterpret_cast<u32x4*>(p.out + row * p.os + col));
    }
}

__global__ __launch_bounds__(256) void silu_mul_generic_kernel(SiluMulParams p) {
    const int64_t total = p.n_rows * p.n_cols;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total;
         idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / p.n_cols;
        const int col = (int)(idx % p.n_cols);
        p.out[row * p.os + col] = (__bf16)silu_mul_one((float)p.gate[row * p.gs + col], (float)p.up[row * p.us + col]);
    }
}

// ---- element access shared by the kernels that serve bf16 and fp32 tensors ----------------------
template <typename T>
__device__ __forceinline__ void load8(const T* p, float (&v)[8]) {
    if constexpr (sizeof(T) == 2) {
        const bf16x8 a = as_bf16x8(__builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p)));
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (float)a[e];
    } else {
        const f32x4 a = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(p));
        const f32x4 b = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(p) + 1);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = a[e];
            v[4 + e] = b[e];
        }
    }
}
template <typename T>
__device__ __forceinline__ void store8(T* p, const float (&v)[8]) {
    if constexpr (sizeof(T) == 2) {
        u32x4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = pack_bf16(v[2 * e], v[2 * e + 1]);
        __builtin_nontemporal_store(o, reinterpret_cast<u32x4*>(p));
    } else {
        __builtin_nontemporal_store(f32x4{v[0], v[1], v[2], v[3]}, reinterpret_cast<f32x4*>(p));
        __builtin_nontemporal_store(f32x4{v[4], v[5], v[6], v[7]}, reinterpret_cast<f32x4*>(p) + 1);
    }
}
// parameter vectors: small, read by every workgroup, kept in the caches; null = the given constant
__device__ __forceinline__ void load_param8(const float* p, int col, float none, float (&v)[8]) {
    if (p) {
        const f32x4* q = reinterpret_cast<const f32x4*>(p + col);
        const f32x4 a = q[0], b = q[1];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = a[e];
            v[4 + e] = b[e];
        }
    } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = none;
    }
}

// tanh and the logistic function.  FAST (results that go to bf16, or to the residual of a bf16 model): through one
// hardware exponential and one reciprocal, absolute error about 2e-7; both saturate cleanly (exp -> 0 or inf).
template <bool FAST>
__device__ __forceinline__ float tanh_of(float x) {
    if constexpr (FAST) return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(2.0f * kLog2e * x));
    else return tanhf(x);
}
template <bool FAST>
__device__ __forceinline__ float sigmoid_of(float x) {
    if constexpr (FAST) return __builtin_amdgcn_rcpf(1.0f + fast_exp2(-kLog2e * x));
    else return 1.0f / (1.0f + expf(-x));
}

// ---- end of a sublayer with Dynamic Tanh norms and a gated residual ------------------------------
//   s = (sub + sub_bias) * sigmoid(gate + gate_bias)          (no gate: s = sub + sub_bias)
//   x = resid + (post ? tanh(post_alpha * s) * post_w + post_b : s)      (no sub: x = resid)
//   y = tanh(next_alpha * x) * next_w + next_b                (the norm in front of the next sublayer)
// The norm has no statistics, so the whole chain is one pass over the elements.
template <typename T>
struct DytResidualParams {
    const T* sub;
    const T* gate;
    const float *sub_bias, *gate_bias;
    const float *post_w, *post_b;
    const float* resid_in;
    float* resid_out;            // may be resid_in; null: x is not kept
    const float *next_w, *next_b;
    T* y;
    float post_alpha, next_alpha;
    int64_t n_rows, sub_stride, gate_stride, y_stride;      // resid rows are contiguous
    int n_cols;
};

template <typename T, bool FAST>
__device__ __forceinline__ float dyt_sublayer(const DytResidualParams<T>& p, float sub, float gate, float sb, float gb, float pw,
                                              float pb) {
    float s = sub + sb;
    if (p.gate) s *= sigmoid_of<FAST>(gate + gb);
    return p.post_w ? fmaf(tanh_of<FAST>(p.post_alpha * s), pw, pb) : s;
}

// A thread owns 8 adjacent columns of ROWS rows, so that the six parameter vectors -- more bytes than the tensors
// themselves -- are fetched once for all of them, and asks for all of its rows before it computes.  Adjacent threads own
// adjacent columns.
template <typename T, int ROWS>
__global__ __launch_bounds__(256) void dyt_residual_vec8_kernel(DytResidualParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int groups = p.n_cols / 8;
    const int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x;
    const int64_t row0 = idx / groups * ROWS;
    const int col = (int)(idx % groups) * 8;
    if (row0 >= p.n_rows) return;
    float x[ROWS][8], s[ROWS][8], g[ROWS][8];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int64_t row = min(row0 + r, p.n_rows - 1);       // (rows past the end re-read the last one and store nothing)
        load8(p.resid_in + row * p.n_cols + col, x[r]);
        if (p.sub) load8(p.sub + row * p.sub_stride + col, s[r]);
        if (p.gate) load8(p.gate + row * p.gate_stride + col, g[r]);
    }
    if (p.sub) {
        float sb[8], gb[8], pw[8], pb[8];
        load_param8(p.sub_bias, col, 0.f, sb);
        load_param8(p.gate_bias, col, 0.f, gb);
        load_param8(p.post_w, col, 1.f, pw);
        load_param8(p.post_b, col, 0.f, pb);
#pragma unroll
        for (int r = 0; r < ROWS; ++r)
#pragma unroll
            for (int e = 0; e < 8; ++e) x[r][e] += dyt_sublayer<T, FAST>(p, s[r][e], g[r][e], sb[e], gb[e], pw[e], pb[e]);
    }
    if (p.resid_out) {
#pragma unroll
        for (int r = 0; r < ROWS; ++r)
            if (row0 + r < p.n_rows) store8(p.resid_out + (row0 + r) * p.n_cols + col, x[r]);
    }
    if (p.y) {
        float nw[8], nb[8];
        load_param8(p.next_w, col, 1.f, nw);
        load_param8(p.next_b, col, 0.f, nb);
#pragma unroll
        for (int r = 0; r < ROWS; ++r) {
            float y[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] = fmaf(tanh_of<FAST>(p.next_alpha * x[r][e]), nw[e], nb[e]);
            if (row0 + r < p.n_rows) store8(p.y + (row0 + r) * p.y_stride + col, y);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void dyt_residual_generic_kernel(DytResidualParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int64_t total = p.n_rows * p.n_cols;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / p.n_cols;
        const int col = (int)(idx % p.n_cols);
        float x = p.resid_in[idx];
        if (p.sub)
            x += dyt_sublayer<T, FAST>(p, (float)p.sub[row * p.sub_stride + col], p.gate ? (float)p.gate[row * p.gate_stride + col] : 0.f,
                                       p.sub_bias ? p.sub_bias[col] : 0.f, p.gate && p.gate_bias ? p.gate_bias[col] : 0.f,
                                       p.post_w ? p.post_w[col] : 1.f, p.post_b ? p.post_b[col] : 0.f);
        if (p.resid_out) p.resid_out[idx] = x;
        if (p.y)
            p.y[row * p.y_stride + col] = (T)fmaf(tanh_of<FAST>(p.next_alpha * x), p.next_w ? p.next_w[col] : 1.f,
                                                  p.next_b ? p.next_b[col] : 0.f);
    }
}

// ---- PolyNorm: out = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3, N(v) = v / sqrt(mean(v^2) + eps) over the row ----
template <typename T>
struct PolyNormParams {
    const T* z;
    T* out;
    int64_t n_rows, zs, os;
    int n_cols;
    float eps, c0, c1, c2, c3;
};

// factors of z, z^2 and z^3 from the row's sums of squares of the three powers
template <typename T>
__device__ __forceinline__ void polynorm_factors(const PolyNormParams<T>& p, float s1, float s2, float s3, float& f1, float& f2,
                                                 float& f3) {
    const float n = (float)p.n_cols;
    f1 = p.c0 / sqrtf(s1 / n + p.eps);
    f2 = p.c1 / sqrtf(s2 / n + p.eps);
    f3 = p.c2 / sqrtf(s3 / n + p.eps);
}

// WAVES wavefronts per row (1: four rows per workgroup, 4: one), the row held in registers as NCHUNK chunks of
// 512 * WAVES elements.  Requires n_cols % 8 == 0, n_cols <= 512 * WAVES * NCHUNK, 16-byte aligned rows.
template <typename T, int WAVES, int NCHUNK>
__global__ __launch_bounds__(256) void polynorm_rows_kernel(PolyNormParams<T> p) {
    __shared__ float part[4][3];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int64_t row = WAVES == 4 ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + wave;
    if (row >= p.n_rows) return;
    const int first = (WAVES == 4 ? (int)threadIdx.x : lane) * 8;
    const T* zr = p.z + row * p.zs;
    float z[NCHUNK][8];
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
        if (col < p.n_cols) load8(zr + col, z[c]);
        else
#pragma unroll
            for (int e = 0; e < 8; ++e) z[c][e] = 0.f;
    }
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float v2 = z[c][e] * z[c][e], v3 = v2 * z[c][e];
            s1 += v2;
            s2 = fmaf(v2, v2, s2);
            s3 = fmaf(v3, v3, s3);
        }
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    s3 = wave_sum(s3);
    if constexpr (WAVES == 4) {
        if (lane == 0) {
            part[wave][0] = s1;
            part[wave][1] = s2;
            part[wave][2] = s3;
        }
        __syncthreads();
        s1 = part[0][0] + part[1][0] + part[2][0] + part[3][0];
        s2 = part[0][1] + part[1][1] + part[2][1] + part[3][1];
        s3 = part[0][2] + part[1][2] + part[2][2] + part[3][2];
    }
    float f1, f2, f3;
    polynorm_factors(p, s1, s2, s3, f1, f2, f3);
    T* orow = p.out + row * p.os;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
        if (col < p.n_cols) {
            float o[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = fmaf(fmaf(fmaf(f3, z[c][e], f2), z[c][e], f1), z[c][e], p.c3);
            store8(orow + col, o);
        }
    }
}

// Any n_cols, any alignment: one wavefront per row, two passes.
template <typename T>
__global__ __launch_bounds__(256) void polynorm_generic_kernel(PolyNormParams<T> p) {
    const int lane = threadIdx.x & 63;
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= p.n_rows) return;
    const T* zr = p.z + row * p.zs;
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
    for (int col = lane; col < p.n_cols; col += 64) {
        const float v = (float)zr[col], v2 = v * v, v3 = v2 * v;
        s1 += v2;
        s2 = fmaf(v2, v2, s2);
        s3 = fmaf(v3, v3, s3);
    }
    float f1, f2, f3;
    polynorm_factors(p, wave_sum(s1), wave_sum(s2), wave_sum(s3), f1, f2, f3);
    T* orow = p.out + row * p.os;
    for (int col = lane; col < p.n_cols; col += 64) {
        const float v = (float)zr[col];
        orow[col] = (T)fmaf(fmaf(fmaf(f3, v, f2), v, f1), v, p.c3);
    }
}

// ---- token embedding + learned position vector -> fp32 residual -----------------------------------
template <typename T>
struct EmbedPosParams {
    const T* embed;
    const T* pos;
    const int64_t* tokens;
    const int32_t* positions;
    float* out;
    int64_t n_rows, vocab, n_positions;
    int n_cols;
};

// Ids outside their table are clamped into it (the host checks what it can).
// One thread per 8 elements: n_cols % 8 == 0, aligned tables.
template <typename T>
__global__ __launch_bounds__(256) void embed_pos_vec8_kernel(EmbedPosParams<T> p) {
    const int groups = p.n_cols / 8;
    const int64_t total = p.n_rows * groups;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / groups;
        const int col = (int)(idx % groups) * 8;
        const int64_t tok = min(max(p.tokens[row], (int64_t)0), p.vocab - 1);
        const int64_t pos = min(max((int64_t)p.positions[row], (int64_t)0), p.n_positions - 1);
        float a[8], b[8];
        load8(p.embed + tok * p.n_cols + col, a);
        load8(p.pos + pos * p.n_cols + col, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) a[e] += b[e];
        store8(p.out + row * p.n_cols + col, a);
    }
}

// One thread per element: any shape.
template <typename T>
__global__ __launch_bounds__(256) void embed_pos_kernel(EmbedPosParams<T> p) {
    const int64_t total = p.n_rows * p.n_cols;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / p.n_cols;
        const int col = (int)(idx % p.n_cols);
        const int64_t tok = min(max(p.tokens[row], (int64_t)0), p.vocab - 1);
        const int64_t pos = min(max((int64_t)p.positions[row], (int64_t)0), p.n_positions - 1);
        p.out[idx] = (float)p.embed[tok * p.n_cols + col] + (float)p.pos[pos * p.n_cols + col];
    }
}

// ---- fp32 residual stream + what a layer adds to it + RMS norm ------------------------------------
//   x = resid + sub + sum_k routed[row * top + k] + embed[token]        (each term optional; no resid: zero)
//   y = x / sqrt(mean(x^2) + eps) * (w_offset + w)
// embed: the embedding output itself at the start of a model, or added again in front of a repeated pass.
template <typename T>
struct ResidualRmsParams {
    const T* sub;
    const T* routed;
    const T* embed;
    const int64_t* tokens;
    const float* resid_in;
    float* resid_out;            // may be resid_in; null: x is not kept
    const float* w;
    T* y;
    int64_t n_rows, vocab, sub_stride, routed_stride, y_stride;      // resid and embed rows are contiguous
    int n_cols, y_cols, top;     // columns n_cols .. y_cols - 1 of y are set to zero
    float w_offset, eps;
};

template <typename T>
__device__ __forceinline__ int64_t embed_row(const ResidualRmsParams<T>& p, int64_t row) {
    return min(max(p.tokens[row], (int64_t)0), p.vocab - 1);           // (an id outside the table is clamped into it)
}

// WAVES wavefronts per row (1: four rows per workgroup, 4: one), the row held in registers as NCHUNK chunks of
// 512 * WAVES elements.  Requires n_cols % 8 == 0, n_cols <= 512 * WAVES * NCHUNK, 16-byte aligned rows.
template <typename T, int WAVES, int NCHUNK>
__global__ __launch_bounds__(256) void residual_rms_rows_kernel(ResidualRmsParams<T> p) {
    __shared__ float part[4];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int64_t row = WAVES == 4 ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + wave;
    if (row >= p.n_rows) return;                                       // (uniform over the wavefronts that share a row)
    const int first = (WAVES == 4 ? (int)threadIdx.x : lane) * 8;
    const int64_t tok = p.embed ? embed_row(p, row) : 0;
    float x[NCHUNK][8];
    float ssq = 0.f;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[c][e] = 0.f;
        if (col < p.n_cols) {
            if (p.resid_in) load8(p.resid_in + row * p.n_cols + col, x[c]);
            float t[8];
            if (p.sub) {
                load8(p.sub + row * p.sub_stride + col, t);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[c][e] += t[e];
            }
            if (p.embed) {
                load8(p.embed + tok * p.n_cols + col, t);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[c][e] += t[e];
            }
            for (int k = 0; k < (p.routed ? p.top : 0); ++k) {
                load8(p.routed + (row * p.top + k) * p.routed_stride + col, t);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[c][e] += t[e];
            }
            if (p.resid_out) store8(p.resid_out + row * p.n_cols + col, x[c]);
#pragma unroll
            for (int e = 0; e < 8; ++e) ssq = fmaf(x[c][e], x[c][e], ssq);
        }
    }
    if (!p.y) return;
    ssq = wave_sum(ssq);
    if constexpr (WAVES == 4) {
        if (lane == 0) part[wave] = ssq;
        __syncthreads();
        ssq = part[0] + part[1] + part[2] + part[3];
    }
    const float rstd = 1.0f / sqrtf(ssq / (float)p.n_cols + p.eps);
    T* yr = p.y + row * p.y_stride;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
        if (col < p.n_cols) {
            float w[8], o[8];
            load_param8(p.w, col, 0.f, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = x[c][e] * rstd * (p.w_offset + w[e]);
            store8(yr + col, o);
        }
    }
    for (int col = p.n_cols + first / 8; col < p.y_cols; col += 64 * WAVES) yr[col] = (T)0.f;
}

// Any n_cols, any alignment: one wavefront per row, two passes.
template <typename T>
__global__ __launch_bounds__(256) void residual_rms_generic_kernel(ResidualRmsParams<T> p) {
    const int lane = threadIdx.x & 63;
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= p.n_rows) return;
    const int64_t tok = p.embed ? embed_row(p, row) : 0;
    const auto value = [&](int col) {
        float x = p.resid_in ? p.resid_in[row * p.n_cols + col] : 0.f;
        if (p.sub) x += (float)p.sub[row * p.sub_stride + col];
        if (p.embed) x += (float)p.embed[tok * p.n_cols + col];
        for (int k = 0; k < (p.routed ? p.top : 0); ++k) x += (float)p.routed[(row * p.top + k) * p.routed_stride + col];
        return x;
    };
    float ssq = 0.f;
    for (int col = lane; col < p.n_cols; col += 64) {
        const float x = value(col);
        ssq = fmaf(x, x, ssq);
    }
    const float rstd = 1.0f / sqrtf(wave_sum(ssq) / (float)p.n_cols + p.eps);
    for (int col = lane; col < p.n_cols; col += 64) {
        const float x = value(col);                                    // (before resid_out, which may be resid_in, is written)
        if (p.resid_out) p.resid_out[row * p.n_cols + col] = x;
        if (p.y) p.y[row * p.y_stride + col] = (T)(x * rstd * (p.w_offset + (p.w ? p.w[col] : 0.f)));
    }
    if (p.y)
        for (int col = p.n_cols + lane; col < p.y_cols; col += 64) p.y[row * p.y_stride + col] = (T)0.f;
}

// ---- feed-forward activations: out = silu(a) * b, or gelu(a) in its tanh form; times sigmoid(row_gate) per row ----
template <typename T>
struct FfActParams {
    const T* a;
    const T* b;                  // null: gelu(a)
    const float* row_gate;       // optional, one logit per row
    T* out;
    int64_t n_rows, as, bs, os;
    int n_cols;
};

template <bool FAST>
__device__ __forceinline__ float gelu_tanh_of(float z) {
    const float u = 0.7978845608028654f * fmaf(0.044715f * z * z, z, z);
    // 1 + tanh(u) = 2 sigmoid(2u)
    if constexpr (FAST) return z * sigmoid_of<true>(2.0f * u);
    else return 0.5f * z * (1.0f + tanhf(u));
}

template <typename T>
__global__ __launch_bounds__(256) void ff_act_vec8_kernel(FfActParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int groups = p.n_cols / 8;
    const int64_t total = p.n_rows * groups;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / groups;
        const int col = (int)(idx % groups) * 8;
        float a[8], b[8];
        load8(p.a + row * p.as + col, a);
        if (p.b) load8(p.b + row * p.bs + col, b);
        const float f = p.row_gate ? sigmoid_of<FAST>(p.row_gate[row]) : 1.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) a[e] = f * (p.b ? a[e] * sigmoid_of<FAST>(a[e]) * b[e] : gelu_tanh_of<FAST>(a[e]));
        store8(p.out + row * p.os + col, a);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void ff_act_generic_kernel(FfActParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int64_t total = p.n_rows * p.n_cols;
    for (int64_t idx = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = idx / p.n_cols;
        const int col = (int)(idx % p.n_cols);
        const float a = (float)p.a[row * p.as + col];
        const float f = p.row_gate ? sigmoid_of<FAST>(p.row_gate[row]) : 1.0f;
        p.out[row * p.os + col] = (T)(f * (p.b ? a * sigmoid_of<FAST>(a) * (float)p.b[row * p.bs + col] : gelu_tanh_of<FAST>(a)));
    }
}

// ---- gated norm: v = y * silu(z); each of `groups` equal parts of a row divided by its root mean square; times w ----
template <typename T>
struct GatedNormParams {
    const T* y;
    const T* z;
    const float* w;
    T* out;
    int64_t n_rows, ys, zs, os;
    int part, groups;            // columns of a part, parts of a row
    float eps;
};

// WAVES wavefronts per part of a row, as in residual_rms_rows_kernel.
template <typename T, int WAVES, int NCHUNK>
__global__ __launch_bounds__(256) void gated_norm_rows_kernel(GatedNormParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    __shared__ float sums[4];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int64_t item = WAVES == 4 ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + wave;
    if (item >= p.n_rows * p.groups) return;
    const int64_t row = item / p.groups;
    const int base = (int)(item % p.groups) * p.part;
    const int first = (WAVES == 4 ? (int)threadIdx.x : lane) * 8;
    float v[NCHUNK][8];
    float ssq = 0.f;
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
#pragma unroll
        for (int e = 0; e < 8; ++e) v[c][e] = 0.f;
        if (col < p.part) {
            float z[8];
            load8(p.y + row * p.ys + base + col, v[c]);
            load8(p.z + row * p.zs + base + col, z);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                v[c][e] *= z[e] * sigmoid_of<FAST>(z[e]);
                ssq = fmaf(v[c][e], v[c][e], ssq);
            }
        }
    }
    ssq = wave_sum(ssq);
    if constexpr (WAVES == 4) {
        if (lane == 0) sums[wave] = ssq;
        __syncthreads();
        ssq = sums[0] + sums[1] + sums[2] + sums[3];
    }
    const float rstd = 1.0f / sqrtf(ssq / (float)p.part + p.eps);
#pragma unroll
    for (int c = 0; c < NCHUNK; ++c) {
        const int col = c * (512 * WAVES) + first;
        if (col < p.part) {
            float w[8];
            load_param8(p.w, base + col, 1.f, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[c][e] *= rstd * w[e];
            store8(p.out + row * p.os + base + col, v[c]);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void gated_norm_generic_kernel(GatedNormParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int lane = threadIdx.x & 63;
    const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= p.n_rows * p.groups) return;
    const int64_t row = item / p.groups;
    const int base = (int)(item % p.groups) * p.part;
    const auto value = [&](int col) {
        const float z = (float)p.z[row * p.zs + base + col];
        return (float)p.y[row * p.ys + base + col] * (z * sigmoid_of<FAST>(z));
    };
    float ssq = 0.f;
    for (int col = lane; col < p.part; col += 64) {
        const float v = value(col);
        ssq = fmaf(v, v, ssq);
    }
    const float rstd = 1.0f / sqrtf(wave_sum(ssq) / (float)p.part + p.eps);
    for (int col = lane; col < p.part; col += 64)
        p.out[row * p.os + base + col] = (T)(value(col) * rstd * (p.w ? p.w[base + col] : 1.f));
}

}  // namespace mi355

using namespace mi355;

static bool aligned16(const void* ptr) { return (reinterpret_cast<uintptr_t>(ptr) & 15) == 0; }

extern "C" int mi355_rms_norm_fwd(const void* x, const void* residual, const void* weight, void* y, void* sum_out,
                                  float* rstd_out, int64_t n_rows, int n_cols, int64_t x_row_stride,
                                  int64_t residual_row_stride, int64_t y_row_stride, int64_t sum_row_stride, float eps,
                                  int weight_dtype, void* stream) {
    if (!x || !weight || !y) return set_error(MI355_EINVAL, "rms_norm: null pointer argument");
    if (sum_out && !residual) return set_error(MI355_EINVAL, "rms_norm: sum_out given without residual");
    if (n_rows < 0 || n_cols <= 0) return set_error(MI355_EINVAL, "rms_norm: n_rows, n_cols out of range");
    if (weight_dtype != MI355_BF16 && weight_dtype != MI355_FP32)
        return set_error(MI355_EDTYPE, "rms_norm: weight dtype must be MI355_BF16 or MI355_FP32");
    if (!(eps >= 0.f)) return set_error(MI355_EINVAL, "rms_norm: eps must be >= 0");
    if (n_rows == 0) return MI355_OK;
    RmsNormParams p;
    p.x = (const __bf16*)x;
    p.residual = (const __bf16*)residual;
    p.weight = weight;
    p.y = (__bf16*)y;
    p.sum_out = (__bf16*)sum_out;
    p.rstd_out = rstd_out;
    p.n_rows = n_rows;
    p.xs = x_row_stride;
    p.rs = residual_row_stride;
    p.ys = y_row_stride;
    p.ss = sum_row_stride;
    p.n_cols = n_cols;
    p.eps = eps;
    p.weight_fp32 = weight_dtype == MI355_FP32;
    const int64_t wgs = (n_rows + 3) / 4;
    if (wgs > 0x7fffffffLL) return set_error(MI355_EINVAL, "rms_norm: too many rows");
    const bool vec = n_cols % 8 == 0 && n_cols <= 8192 && aligned16(x) && aligned16(y) && aligned16(weight) &&
                     (!residual || aligned16(residual)) && (!sum_out || aligned16(sum_out)) &&
                     ((x_row_stride | y_row_stride) & 7) == 0 && (!residual || (residual_row_stride & 7) == 0) &&
                     (!sum_out || (sum_row_stride & 7) == 0);
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)wgs), block(256);
    if (!vec) hipLaunchKernelGGL(rms_norm_generic_kernel, grid, block, 0, s, p);
    else if (n_cols <= 512) hipLaunchKernelGGL(rms_norm_rows_kernel<1>, grid, block, 0, s, p);
    else if (n_cols <= 1024) hipLaunchKernelGGL(rms_norm_rows_kernel<2>, grid, block, 0, s, p);
    else if (n_cols <= 2048) hipLaunchKernelGGL(rms_norm_rows_kernel<4>, grid, block, 0, s, p);
    else if (n_cols <= 4096) hipLaunchKernelGGL(rms_norm_rows_kernel<8>, grid, block, 0, s, p);
    else hipLaunchKernelGGL(rms_norm_rows_kernel<16>, grid, block, 0, s, p);
    const int rc = (int)hipGetLastError();
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

extern "C" int mi355_silu_mul_fwd(const void* gate, const void* up, void* out, int64_t n_rows, int n_cols,
                                  int64_t gate_row_stride, int64_t up_row_stride, int64_t out_row_stride, void* stream) {
    if (!gate || !up || !out) return set_error(MI355_EINVAL, "silu_mul: null pointer argument");
    if (n_rows < 0 || n_cols <= 0) return set_error(MI355_EINVAL, "silu_mul: n_rows, n_cols out of range");
    if (n_rows == 0) return MI355_OK;
    SiluMulParams p;
    p.gate = (const __bf16*)gate;
    p.up = (const __bf16*)up;
    p.out = (__bf16*)out;
    p.n_rows = n_rows;
    p.gs = gate_row_stride;
    p.us = up_row_stride;
    p.os = out_row_stride;
    p.n_cols = n_cols;
    const bool vec = n_cols % 8 == 0 && aligned16(gate) && aligned16(up) && aligned16(out) &&
                     ((gate_row_stride | up_row_stride | out_row_stride) & 7) == 0;
    const int64_t total = vec ? n_rows * (n_cols / 8) : n_rows * (int64_t)n_cols;
    const int64_t blocks = (total + 255) / 256;
    const unsigned grid = (unsigned)(blocks < 0x7fffffffLL ? blocks : 0x7fffffffLL);
    hipStream_t s = (hipStream_t)stream;
    if (vec) hipLaunchKernelGGL(silu_mul_vec8_kernel, dim3(grid), dim3(256), 0, s, p);
    else hipLaunchKernelGGL(silu_mul_generic_kernel, dim3(grid), dim3(256), 0, s, p);
    const int rc = (int)hipGetLastError();
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

static unsigned grid_1d(int64_t threads) {
    const int64_t blocks = (threads + 255) / 256;
    return (unsigned)(blocks < 0x7fffffffLL ? blocks : 0x7fffffffLL);
}

static int launch_status() {
    const int rc = (int)hipGetLastError();
    return rc != 0 ? set_error(rc, hipGetErrorString((hipError_t)rc)) : MI355_OK;
}

template <typename T>
static int dyt_residual(const void* sub, const float* sub_bias, const void* gate, const float* gate_bias, float post_alpha,
                        const float* post_w, const float* post_b, const float* resid_in, float* resid_out, float next_alpha,
                        const float* next_w, const float* next_b, void* y, int64_t n_rows, int n_cols, int64_t sub_stride,
                        int64_t gate_stride, int64_t y_stride, hipStream_t s) {
    DytResidualParams<T> p;
    p.sub = (const T*)sub;
    p.gate = (const T*)gate;
    p.sub_bias = sub_bias;
    p.gate_bias = gate_bias;
    p.post_w = post_w;
    p.post_b = post_b;
    p.resid_in = resid_in;
    p.resid_out = resid_out;
    p.next_w = next_w;
    p.next_b = next_b;
    p.y = (T*)y;
    p.post_alpha = post_alpha;
    p.next_alpha = next_alpha;
    p.n_rows = n_rows;
    p.n_cols = n_cols;
    p.sub_stride = sub_stride;
    p.gate_stride = gate_stride;
    p.y_stride = y_stride;
    bool vec = n_cols % 8 == 0 && ((sub_stride | gate_stride | y_stride) & 7) == 0;
    for (const void* ptr : {sub, gate, (const void*)sub_bias, (const void*)gate_bias, (const void*)post_w, (const void*)post_b,
                            (const void*)resid_in, (const void*)resid_out, (const void*)next_w, (const void*)next_b, (const void*)y})
        vec = vec && aligned16(ptr);
    if (vec) {
        // rows per thread: as many as leave the GPU several workgroups per compute unit
        const int64_t groups = n_cols / 8, work = n_rows * groups;
        const int r = work >= 4 * 256 * 2048 ? 4 : work >= 2 * 256 * 2048 ? 2 : 1;
        const int64_t threads = (n_rows + r - 1) / r * groups;
        if ((threads + 255) / 256 > 0x7fffffffLL) return set_error(MI355_EINVAL, "dyt_residual: too many elements");
        const dim3 grid(grid_1d(threads)), block(256);
        if (r == 4) hipLaunchKernelGGL((dyt_residual_vec8_kernel<T, 4>), grid, block, 0, s, p);
        else if (r == 2) hipLaunchKernelGGL((dyt_residual_vec8_kernel<T, 2>), grid, block, 0, s, p);
        else hipLaunchKernelGGL((dyt_residual_vec8_kernel<T, 1>), grid, block, 0, s, p);
    } else {
        hipLaunchKernelGGL(dyt_residual_generic_kernel<T>, dim3(grid_1d(n_rows * (int64_t)n_cols)), dim3(256), 0, s, p);
    }
    return launch_status();
}

extern "C" int mi355_dyt_residual_fwd(const void* sub, const float* sub_bias, const void* gate, const float* gate_bias,
                                      float post_alpha, const float* post_weight, const float* post_bias,
                                      const float* resid_in, float* resid_out, float next_alpha, const float* next_weight,
                                      const float* next_bias, void* y, int64_t n_rows, int n_cols, int64_t sub_row_stride,
                                      int64_t gate_row_stride, int64_t y_row_stride, int dtype, void* stream) {
    if (!resid_in || (!resid_out && !y)) return set_error(MI355_EINVAL, "dyt_residual: null pointer argument");
    if (!sub && (gate || post_weight || sub_bias)) return set_error(MI355_EINVAL, "dyt_residual: gate, post norm or bias given without a sublayer result");
    if ((post_weight == nullptr) != (post_bias == nullptr) || (next_weight == nullptr) != (next_bias == nullptr))
        return set_error(MI355_EINVAL, "dyt_residual: a norm's weight and bias go together");
    if (gate_bias && !gate) return set_error(MI355_EINVAL, "dyt_residual: gate_bias given without a gate");
    if (n_rows < 0 || n_cols <= 0) return set_error(MI355_EINVAL, "dyt_residual: n_rows, n_cols out of range");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "dyt_residual: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16
               ? dyt_residual<__bf16>(sub, sub_bias, gate, gate_bias, post_alpha, post_weight, post_bias, resid_in, resid_out, next_alpha,
                                      next_weight, next_bias, y, n_rows, n_cols, sub_row_stride, gate_row_stride, y_row_stride, s)
               : dyt_residual<float>(sub, sub_bias, gate, gate_bias, post_alpha, post_weight, post_bias, resid_in, resid_out, next_alpha,
                                     next_weight, next_bias, y, n_rows, n_cols, sub_row_stride, gate_row_stride, y_row_stride, s);
}

template <typename T>
static int polynorm(const void* z, void* out, int64_t n_rows, int n_cols, int64_t zs, int64_t os, const float* c, float eps,
                    hipStream_t s) {
    PolyNormParams<T> p;
    p.z = (const T*)z;
    p.out = (T*)out;
    p.n_rows = n_rows;
    p.n_cols = n_cols;
    p.zs = zs;
    p.os = os;
    p.eps = eps;
    p.c0 = c[0];
    p.c1 = c[1];
    p.c2 = c[2];
    p.c3 = c[3];
    const bool vec = n_cols % 8 == 0 && n_cols <= 16384 && aligned16(z) && aligned16(out) && ((zs | os) & 7) == 0;
    const bool wide = vec && n_cols > 1024;
    const int64_t wgs = wide ? n_rows : (n_rows + 3) / 4;
    if (wgs > 0x7fffffffLL) return set_error(MI355_EINVAL, "polynorm: too many rows");
    const dim3 grid((unsigned)wgs), block(256);
    if (!vec) hipLaunchKernelGGL(polynorm_generic_kernel<T>, grid, block, 0, s, p);
    else if (n_cols <= 512) hipLaunchKernelGGL((polynorm_rows_kernel<T, 1, 1>), grid, block, 0, s, p);
    else if (n_cols <= 1024) hipLaunchKernelGGL((polynorm_rows_kernel<T, 1, 2>), grid, block, 0, s, p);
    else if (n_cols <= 2048) hipLaunchKernelGGL((polynorm_rows_kernel<T, 4, 1>), grid, block, 0, s, p);
    else if (n_cols <= 4096) hipLaunchKernelGGL((polynorm_rows_kernel<T, 4, 2>), grid, block, 0, s, p);
    else if (n_cols <= 8192) hipLaunchKernelGGL((polynorm_rows_kernel<T, 4, 4>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((polynorm_rows_kernel<T, 4, 8>), grid, block, 0, s, p);
    return launch_status();
}

extern "C" int mi355_polynorm_fwd(const void* z, void* out, int64_t n_rows, int n_cols, int64_t z_row_stride,
                                  int64_t out_row_stride, const float coeffs[4], float eps, int dtype, void* stream) {
    if (!z || !out || !coeffs) return set_error(MI355_EINVAL, "polynorm: null pointer argument");
    if (n_rows < 0 || n_cols <= 0) return set_error(MI355_EINVAL, "polynorm: n_rows, n_cols out of range");
    if (!(eps >= 0.f)) return set_error(MI355_EINVAL, "polynorm: eps must be >= 0");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "polynorm: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16 ? polynorm<__bf16>(z, out, n_rows, n_cols, z_row_stride, out_row_stride, coeffs, eps, s)
                               : polynorm<float>(z, out, n_rows, n_cols, z_row_stride, out_row_stride, coeffs, eps, s);
}

template <typename T>
static int embed_pos(const void* embed, const void* pos, const int64_t* tokens, const int32_t* positions, float* out, int64_t n_rows,
                     int n_cols, int64_t vocab, int64_t n_positions, hipStream_t s) {
    EmbedPosParams<T> p;
    p.embed = (const T*)embed;
    p.pos = (const T*)pos;
    p.tokens = tokens;
    p.positions = positions;
    p.out = out;
    p.n_rows = n_rows;
    p.n_cols = n_cols;
    p.vocab = vocab;
    p.n_positions = n_positions;
    if (n_cols % 8 == 0 && aligned16(embed) && aligned16(pos) && aligned16(out))
        hipLaunchKernelGGL(embed_pos_vec8_kernel<T>, dim3(grid_1d(n_rows * (int64_t)(n_cols / 8))), dim3(256), 0, s, p);
    else
        hipLaunchKernelGGL(embed_pos_kernel<T>, dim3(grid_1d(n_rows * (int64_t)n_cols)), dim3(256), 0, s, p);
    return launch_status();
}

extern "C" int mi355_embed_pos_fwd(const void* embed, const void* pos, const int64_t* tokens, const int32_t* positions, float* out,
                                   int64_t n_rows, int n_cols, int64_t vocab, int64_t n_positions, int dtype, void* stream) {
    if (!embed || !pos || !tokens || !positions || !out) return set_error(MI355_EINVAL, "embed_pos: null pointer argument");
    if (n_rows < 0 || n_cols <= 0 || vocab <= 0 || n_positions <= 0)
        return set_error(MI355_EINVAL, "embed_pos: n_rows, n_cols, vocab, n_positions out of range");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "embed_pos: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16 ? embed_pos<__bf16>(embed, pos, tokens, positions, out, n_rows, n_cols, vocab, n_positions, s)
                               : embed_pos<float>(embed, pos, tokens, positions, out, n_rows, n_cols, vocab, n_positions, s);
}

template <typename T>
static int residual_rms(const ResidualRmsParams<T>& p, bool vec, hipStream_t s) {
    const bool wide = vec && p.n_cols > 1024;
    const int64_t wgs = wide ? p.n_rows : (p.n_rows + 3) / 4;
    if (wgs > 0x7fffffffLL) return set_error(MI355_EINVAL, "residual_rms: too many rows");
    const dim3 grid((unsigned)wgs), block(256);
    if (!vec) hipLaunchKernelGGL(residual_rms_generic_kernel<T>, grid, block, 0, s, p);
    else if (p.n_cols <= 512) hipLaunchKernelGGL((residual_rms_rows_kernel<T, 1, 1>), grid, block, 0, s, p);
    else if (p.n_cols <= 1024) hipLaunchKernelGGL((residual_rms_rows_kernel<T, 1, 2>), grid, block, 0, s, p);
    else if (p.n_cols <= 2048) hipLaunchKernelGGL((residual_rms_rows_kernel<T, 4, 1>), grid, block, 0, s, p);
    else if (p.n_cols <= 4096) hipLaunchKernelGGL((residual_rms_rows_kernel<T, 4, 2>), grid, block, 0, s, p);
    else if (p.n_cols <= 8192) hipLaunchKernelGGL((residual_rms_rows_kernel<T, 4, 4>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((residual_rms_rows_kernel<T, 4, 8>), grid, block, 0, s, p);
    return launch_status();
}

template <typename T>
static int residual_rms_args(const float* resid_in, float* resid_out, const void* sub, const void* routed, int top, const void* embed,
                             const int64_t* tokens, int64_t vocab, const float* weight, float weight_offset, float eps, void* y,
                             int64_t n_rows, int n_cols, int y_cols, int64_t sub_stride, int64_t routed_stride, int64_t y_stride,
                             hipStream_t s) {
    ResidualRmsParams<T> p;
    p.sub = (const T*)sub;
    p.routed = (const T*)routed;
    p.embed = (const T*)embed;
    p.tokens = tokens;
    p.resid_in = resid_in;
    p.resid_out = resid_out;
    p.w = weight;
    p.y = (T*)y;
    p.n_rows = n_rows;
    p.vocab = vocab;
    p.sub_stride = sub_stride;
    p.routed_stride = routed_stride;
    p.y_stride = y_stride;
    p.n_cols = n_cols;
    p.y_cols = y_cols;
    p.top = top;
    p.w_offset = weight_offset;
    p.eps = eps;
    bool vec = n_cols % 8 == 0 && n_cols <= 16384 && ((sub_stride | routed_stride | y_stride) & 7) == 0;
    for (const void* ptr : {sub, routed, embed, (const void*)resid_in, (const void*)resid_out, (const void*)weight, (const void*)y})
        vec = vec && aligned16(ptr);
    return residual_rms(p, vec, s);
}

extern "C" int mi355_residual_rms_fwd(const float* resid_in, float* resid_out, const void* sub, const void* routed, int top,
                                      const void* embed, const int64_t* tokens, int64_t vocab, const float* weight,
                                      float weight_offset, float eps, void* y, int64_t n_rows, int n_cols, int y_cols,
                                      int64_t sub_row_stride, int64_t routed_row_stride, int64_t y_row_stride, int dtype,
                                      void* stream) {
    if (!resid_out && !y) return set_error(MI355_EINVAL, "residual_rms: no output");
    if (!resid_in && !sub && !routed && !embed) return set_error(MI355_EINVAL, "residual_rms: no input");
    if (embed && (!tokens || vocab <= 0)) return set_error(MI355_EINVAL, "residual_rms: an embedding table needs token ids and its row count");
    if (routed && top <= 0) return set_error(MI355_EINVAL, "residual_rms: routed rows need top >= 1");
    if (n_rows < 0 || n_cols <= 0 || (y && (y_cols < n_cols || y_row_stride < y_cols)))
        return set_error(MI355_EINVAL, "residual_rms: n_rows, n_cols, y_cols out of range");
    if (!(eps >= 0.f)) return set_error(MI355_EINVAL, "residual_rms: eps must be >= 0");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "residual_rms: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16
               ? residual_rms_args<__bf16>(resid_in, resid_out, sub, routed, top, embed, tokens, vocab, weight, weight_offset, eps, y,
                                           n_rows, n_cols, y_cols, sub_row_stride, routed_row_stride, y_row_stride, s)
               : residual_rms_args<float>(resid_in, resid_out, sub, routed, top, embed, tokens, vocab, weight, weight_offset, eps, y,
                                          n_rows, n_cols, y_cols, sub_row_stride, routed_row_stride, y_row_stride, s);
}

template <typename T>
static int ff_act(const void* a, const void* b, const float* row_gate, void* out, int64_t n_rows, int n_cols, int64_t as, int64_t bs,
                  int64_t os, hipStream_t s) {
    FfActParams<T> p;
    p.a = (const T*)a;
    p.b = (const T*)b;
    p.row_gate = row_gate;
    p.out = (T*)out;
    p.n_rows = n_rows;
    p.as = as;
    p.bs = bs;
    p.os = os;
    p.n_cols = n_cols;
    if (n_cols % 8 == 0 && ((as | bs | os) & 7) == 0 && aligned16(a) && aligned16(b) && aligned16(out))
        hipLaunchKernelGGL(ff_act_vec8_kernel<T>, dim3(grid_1d(n_rows * (int64_t)(n_cols / 8))), dim3(256), 0, s, p);
    else
        hipLaunchKernelGGL(ff_act_generic_kernel<T>, dim3(grid_1d(n_rows * (int64_t)n_cols)), dim3(256), 0, s, p);
    return launch_status();
}

extern "C" int mi355_ff_act_fwd(const void* a, const void* b, const float* row_gate, void* out, int64_t n_rows, int n_cols,
                                int64_t a_row_stride, int64_t b_row_stride, int64_t out_row_stride, int dtype, void* stream) {
    if (!a || !out) return set_error(MI355_EINVAL, "ff_act: null pointer argument");
    if (n_rows < 0 || n_cols <= 0) return set_error(MI355_EINVAL, "ff_act: n_rows, n_cols out of range");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "ff_act: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16 ? ff_act<__bf16>(a, b, row_gate, out, n_rows, n_cols, a_row_stride, b_row_stride, out_row_stride, s)
                               : ff_act<float>(a, b, row_gate, out, n_rows, n_cols, a_row_stride, b_row_stride, out_row_stride, s);
}

template <typename T>
static int gated_norm(const void* y, const void* z, const float* w, void* out, int64_t n_rows, int part, int groups, int64_t ys,
                      int64_t zs, int64_t os, float eps, hipStream_t s) {
    GatedNormParams<T> p;
    p.y = (const T*)y;
    p.z = (const T*)z;
    p.w = w;
    p.out = (T*)out;
    p.n_rows = n_rows;
    p.ys = ys;
    p.zs = zs;
    p.os = os;
    p.part = part;
    p.groups = groups;
    p.eps = eps;
    const bool vec = part % 8 == 0 && part <= 16384 && ((ys | zs | os) & 7) == 0 && aligned16(y) && aligned16(z) && aligned16(out) &&
                     aligned16(w);
    const bool wide = vec && part > 1024;
    const int64_t items = n_rows * groups, wgs = wide ? items : (items + 3) / 4;
    if (wgs > 0x7fffffffLL) return set_error(MI355_EINVAL, "gated_norm: too many rows");
    const dim3 grid((unsigned)wgs), block(256);
    if (!vec) hipLaunchKernelGGL(gated_norm_generic_kernel<T>, grid, block, 0, s, p);
    else if (part <= 512) hipLaunchKernelGGL((gated_norm_rows_kernel<T, 1, 1>), grid, block, 0, s, p);
    else if (part <= 1024) hipLaunchKernelGGL((gated_norm_rows_kernel<T, 1, 2>), grid, block, 0, s, p);
    else if (part <= 2048) hipLaunchKernelGGL((gated_norm_rows_kernel<T, 4, 1>), grid, block, 0, s, p);
    else if (part <= 4096) hipLaunchKernelGGL((gated_norm_rows_kernel<T, 4, 2>), grid, block, 0, s, p);
    else if (part <= 8192) hipLaunchKernelGGL((gated_norm_rows_kernel<T, 4, 4>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((gated_norm_rows_kernel<T, 4, 8>), grid, block, 0, s, p);
    return launch_status();
}

extern "C" int mi355_gated_norm_fwd(const void* y, const void* z, const float* weight, void* out, int64_t n_rows, int n_cols, int groups,
                                    int64_t y_row_stride, int64_t z_row_stride, int64_t out_row_stride, float eps, int dtype,
                                    void* stream) {
    if (!y || !z || !out) return set_error(MI355_EINVAL, "gated_norm: null pointer argument");
    if (n_rows < 0 || n_cols <= 0 || groups <= 0 || n_cols % groups) return set_error(MI355_EINVAL, "gated_norm: n_cols must be a positive multiple of groups");
    if (!(eps >= 0.f)) return set_error(MI355_EINVAL, "gated_norm: eps must be >= 0");
    if (dtype != MI355_BF16 && dtype != MI355_FP32) return set_error(MI355_EDTYPE, "gated_norm: dtype must be MI355_BF16 or MI355_FP32");
    if (n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    return dtype == MI355_BF16 ? gated_norm<__bf16>(y, z, weight, out, n_rows, n_cols / groups, groups, y_row_stride, z_row_stride, out_row_stride, eps, s)
                               : gated_norm<float>(y, z, weight, out, n_rows, n_cols / groups, groups, y_row_stride, z_row_stride, out_row_stride, eps, s);
}
