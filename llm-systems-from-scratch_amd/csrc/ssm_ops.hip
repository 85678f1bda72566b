// Mamba-2 mixers (state-space duality) on gfx950: short causal convolution, selective state recurrence, decode step.
//
// Per head, with log decay a_t = neg_a dt_t (dt after softplus) and channels x | B | C behind a causal convolution and silu:
//     S_t = exp(a_t) S_(t-1) + dt_t B_t x_t^T        y_t = S_t^T C_t + D x_t             S: state x vdim, fp32
//
// What a sequence carries from one call to the next lives in slots of two pools:
//   conv_state (slots, taps, channels)            the convolution's inputs as a ring: position p sits in row p % taps.  A
//                                                 convolution reads the taps - 1 rows in front of a token and writes the
//                                                 token's own row, so a step's reads and writes never meet.
//   ssm_state  (slots, heads, state, vdim_pad)    S in fp32 (vdim_pad: vdim rounded up to 4)
// A sequence's first token is at position 0: its history is zero whatever the slot holds, so slots are never cleared.
//
// Three kernels besides the convolution:
//   ssd_chunk_kernel   bf16 prompts: chunks of 64 tokens on MFMA, the state in accumulators from chunk to chunk; where
//                      that walk leaves the chip idle, segments of a sequence side by side (ssd_carry_kernel between them)
//   ssm_scan_kernel    any sizes and fp32: token by token, the state in registers
//   ... the same kernel with the convolution inside: one decode step of every sequence
#include "common.hpp"
#include "launch.hpp"

namespace mi355 {

constexpr int kConvTile = 16;        // tokens per thread of the convolution
constexpr int kMaxTaps = 16;
constexpr int kScanVecs = 16;        // most 4-wide state pieces per thread of the scan

template <typename T>
struct SsmParams {
    const T* proj;                   // rows of the input projection
    int64_t proj_stride, xbc_at, dt_at;
    const float *conv_w, *conv_b;    // (taps, channels), (channels)
    const float *dt_bias, *neg_a, *d_skip;
    T* conv_state;
    float* ssm_state;
    const int32_t *slots, *positions, *cu;      // cu null: sequence b owns row b
    T* xbc;                          // (rows, channels): the convolution's output
    T* y;
    int64_t y_stride, n_rows;
    int B, H, P, Pp, N, G, taps, channels, n_slots;
    int np4, slices;                 // scan: 4-wide pieces of vdim per workgroup, and workgroups per head
    float *seg_state, *seg_decay;    // segments: (segment, head) states (N x Pp), log2 of the decay across a segment
    int seg_len, n_segs;
};

template <typename T>
__device__ __forceinline__ int state_slot(const SsmParams<T>& p, int b) {
    return min(max(p.slots[b], 0), p.n_slots - 1);
}
// the sequence that unit `unit` of `size` tokens lies in: units of sequence b start at number first_row / size + b
template <typename T>
__device__ __forceinline__ int seq_of_unit(const SsmParams<T>& p, int unit, int size) {
    int lo = 0, hi = p.B - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if ((p.cu ? p.cu[mid] : mid) / size + mid <= unit) lo = mid;
        else hi = mid - 1;
    }
    return lo;
}
// rows of sequence b
template <typename T>
__device__ __forceinline__ void seq_rows(const SsmParams<T>& p, int b, int& first, int& len) {
    first = p.cu ? p.cu[b] : b;
    len = (p.cu ? p.cu[b + 1] : b + 1) - first;
    len = max(0, min(len, (int)p.n_rows - first));
}
__device__ __forceinline__ float softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
template <bool FAST>
__device__ __forceinline__ float silu_of(float x) {
    if constexpr (FAST) return x * __builtin_amdgcn_rcpf(1.0f + fast_exp2(-kLog2e * x));
    else return x / (1.0f + expf(-x));
}

// V adjacent channels (8: 16-byte pieces of bf16, 32-byte pieces of fp32; or 1)
template <typename T, int V>
__device__ __forceinline__ void load_ch(const T* p, float (&v)[V]) {
    if constexpr (V == 1) {
        v[0] = (float)p[0];
    } else if constexpr (sizeof(T) == 2) {
        const bf16x8 a = as_bf16x8(*reinterpret_cast<const u32x4*>(p));
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (float)a[e];
    } else {
        const f32x4 a = reinterpret_cast<const f32x4*>(p)[0], b = reinterpret_cast<const f32x4*>(p)[1];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = a[e];
            v[4 + e] = b[e];
        }
    }
}
template <typename T, int V>
__device__ __forceinline__ void store_ch(T* p, const float (&v)[V]) {
    if constexpr (V == 1) {
        p[0] = (T)v[0];
    } else if constexpr (sizeof(T) == 2) {
        u32x4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = pack_bf16(v[2 * e], v[2 * e + 1]);
        *reinterpret_cast<u32x4*>(p) = o;
    } else {
        reinterpret_cast<f32x4*>(p)[0] = f32x4{v[0], v[1], v[2], v[3]};
        reinterpret_cast<f32x4*>(p)[1] = f32x4{v[4], v[5], v[6], v[7]};
    }
}

// Causal convolution + silu of packed prompts.  A thread owns V adjacent channels of kConvTile tokens of one sequence; the
// inputs it has read slide through registers when the number of taps is known at compile time (TAPS > 0).  The thread of a
// sequence's first tile is the only one that touches the sequence's ring for its channels: it reads the history first and
// writes the last taps - 1 inputs of the portion at its end.
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void causal_conv_silu_kernel(SsmParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    const int taps = TAPS > 0 ? TAPS : p.taps;
    const int ch_groups = p.channels / V;
    const int g_blocks = (ch_groups + 255) / 256;
    const int tile = blockIdx.x / g_blocks;
    const int cg = (blockIdx.x % g_blocks) * 256 + threadIdx.x;
    const int b = seq_of_unit(p, tile, kConvTile);
    int first, len;
    seq_rows(p, b, first, len);
    const int t0 = (tile - (first / kConvTile + b)) * kConvTile;
    if (t0 < 0 || t0 >= len || cg >= ch_groups) return;
    const int c = cg * V;
    const int pos0 = p.positions[first];
    T* ring = p.conv_state + (int64_t)state_slot(p, b) * taps * p.channels + c;
    const T* in = p.proj + (int64_t)first * p.proj_stride + p.xbc_at + c;
    const auto input = [&](int t, float (&v)[V]) {              // token t of the portion, or (t < 0) one before it
        if (t >= 0) {
            load_ch<T, V>(in + (int64_t)t * p.proj_stride, v);
        } else if (pos0 + t >= 0) {
            load_ch<T, V>(ring + (int64_t)((pos0 + t) % taps) * p.channels, v);
        } else {
#pragma unroll
            for (int e = 0; e < V; ++e) v[e] = 0.f;
        }
    };
    float bias[V];
    load_ch<float, V>(p.conv_b + c, bias);
    const int n = min(kConvTile, len - t0);
    T* out = p.xbc + (int64_t)(first + t0) * p.channels + c;
    if constexpr (TAPS > 0) {
        float w[TAPS][V], x[TAPS][V];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) load_ch<float, V>(p.conv_w + (int64_t)j * p.channels + c, w[j]);
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) input(t0 - (TAPS - 1) + j, x[j]);
#pragma unroll
        for (int t = 0; t < kConvTile; ++t) {
            if (t < n) {
                load_ch<T, V>(in + (int64_t)(t0 + t) * p.proj_stride, x[TAPS - 1]);
                float a[V];
#pragma unroll
                for (int e = 0; e < V; ++e) {
                    a[e] = bias[e];
#pragma unroll
                    for (int j = 0; j < TAPS; ++j) a[e] = fmaf(w[j][e], x[j][e], a[e]);
                    a[e] = silu_of<FAST>(a[e]);
                }
                store_ch<T, V>(out + (int64_t)t * p.channels, a);
#pragma unroll
                for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
                    for (int e = 0; e < V; ++e) x[j][e] = x[j + 1][e];
            }
        }
    } else {
        for (int t = 0; t < n; ++t) {
            float a[V];
#pragma unroll
            for (int e = 0; e < V; ++e) a[e] = bias[e];
            for (int j = 0; j < taps; ++j) {
                float w[V], x[V];
                load_ch<float, V>(p.conv_w + (int64_t)j * p.channels + c, w);
                input(t0 + t - (taps - 1) + j, x);
#pragma unroll
                for (int e = 0; e < V; ++e) a[e] = fmaf(w[e], x[e], a[e]);
            }
#pragma unroll
            for (int e = 0; e < V; ++e) a[e] = silu_of<FAST>(a[e]);
            store_ch<T, V>(out + (int64_t)t * p.channels, a);
        }
    }
    if (t0 == 0) {
        for (int t = max(0, len - (taps - 1)); t < len; ++t) {
            float x[V];
            load_ch<T, V>(in + (int64_t)t * p.proj_stride, x);
            store_ch<T, V>(ring + (int64_t)((pos0 + t) % taps) * p.channels, x);
        }
    }
}

// Token-by-token recurrence.  One workgroup per (sequence, head, slice of vdim); a thread owns a fixed 4-wide piece of vdim
// and every (256 / np4)-th row of the state, in registers.  DECODE: one token per sequence, the convolution of the head's
// channels inside (B and C channels, shared by the heads of a group, are convolved by each of them and entered into the ring by
// the group's first).
template <typename T, int NV, bool DECODE>
__global__ __launch_bounds__(256) void ssm_scan_kernel(SsmParams<T> p) {
    constexpr bool FAST = sizeof(T) == 2;
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int np = 4 * p.np4;                                  // columns of the slice
    float* x_l = smem;                                         // np
    float* b_l = x_l + np;                                     // N
    float* c_l = b_l + p.N;                                    // N
    f32x4* red = reinterpret_cast<f32x4*>(smem + (np + 2 * p.N + 3) / 4 * 4);       // rows x np4
    const int slice = blockIdx.x % p.slices;
    const int h = (blockIdx.x / p.slices) % p.H;
    const int b = blockIdx.x / (p.slices * p.H);
    int first, len;
    seq_rows(p, b, first, len);
    if (len <= 0) return;
    const int per_group = p.H / p.G, g = h / per_group;
    const int col0 = slice * np;                               // first column of the slice
    const int tid = threadIdx.x, rows = 256 / p.np4;
    const int p4 = tid % p.np4, r = tid / p.np4;
    const bool mine = r < rows && col0 + 4 * p4 < p.Pp;
    const int slot = state_slot(p, b);
    float* st = p.ssm_state + ((int64_t)slot * p.H + h) * p.N * p.Pp + col0 + 4 * p4;
    const int pos0 = p.positions[first];
    f32x4 S[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int n = r + i * rows;
        if (mine && n < p.N && pos0 > 0) S[i] = *reinterpret_cast<const f32x4*>(st + (int64_t)n * p.Pp);
    }
    const float bias = p.dt_bias[h], na = p.neg_a[h], skip = p.d_skip[h];
    const int inner = p.H * p.P;
    // channel of staged value i: x columns of the slice, then B, then C
    const auto channel = [&](int i) {
        if (i < np) return col0 + i < p.P ? h * p.P + col0 + i : -1;
        return i < np + p.N ? inner + g * p.N + (i - np) : inner + (p.G + g) * p.N + (i - np - p.N);
    };
    for (int t = 0; t < len; ++t) {
        const int64_t row = first + t;
        if (t) __syncthreads();                                // the staged values of the token before have been read
        for (int i = tid; i < np + 2 * p.N; i += 256) {
            const int c = channel(i);
            float v = 0.f;
            if (c >= 0) {
                if constexpr (DECODE) {
                    T* ring = p.conv_state + (int64_t)slot * p.taps * p.channels + c;
                    const T now = p.proj[row * p.proj_stride + p.xbc_at + c];
                    v = p.conv_b[c];
                    for (int j = 0; j + 1 < p.taps; ++j) {
                        const int q = pos0 - (p.taps - 1) + j;
                        if (q >= 0) v = fmaf(p.conv_w[(int64_t)j * p.channels + c], (float)ring[(int64_t)(q % p.taps) * p.channels], v);
                    }
                    v = silu_of<FAST>(fmaf(p.conv_w[(int64_t)(p.taps - 1) * p.channels + c], (float)now, v));
                    if (i < np || (h % per_group == 0 && slice == 0)) ring[(int64_t)(pos0 % p.taps) * p.channels] = now;
                } else {
                    v = (float)p.xbc[row * p.channels + c];
                }
            }
            smem[i] = v;
        }
        const float dt = softplus((float)p.proj[row * p.proj_stride + p.dt_at + h] + bias);
        const float decay = FAST ? fast_exp2(kLog2e * (na * dt)) : expf(na * dt);
        __syncthreads();
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if (mine) {
            f32x4 xd = *reinterpret_cast<const f32x4*>(x_l + 4 * p4);
            xd *= dt;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int n = r + i * rows;
                if (n < p.N) {
                    const float bn = b_l[n], cn = c_l[n];
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        S[i][e] = fmaf(decay, S[i][e], bn * xd[e]);
                        acc[e] = fmaf(S[i][e], cn, acc[e]);
                    }
                }
            }
        }
        if (r < rows) red[r * p.np4 + p4] = acc;
        __syncthreads();
        for (int i = tid; i < np; i += 256) {
            if (col0 + i < p.P) {
                const float* rf = reinterpret_cast<const float*>(red);
                float s = skip * x_l[i];
                for (int k = 0; k < rows; ++k) s += rf[k * np + i];
                p.y[row * p.y_stride + h * p.P + col0 + i] = (T)s;
            }
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int n = r + i * rows;
        if (mine && n < p.N) *reinterpret_cast<f32x4*>(st + (int64_t)n * p.Pp) = S[i];
    }
}

// two values -> their bf16 parts and the bf16 parts of what those leave: v = hi + lo to 16 bits
__device__ __forceinline__ void split_bf16(float a, float b, uint32_t& hi, uint32_t& lo) {
    const __bf16 ha = (__bf16)a, hb = (__bf16)b;
    bf16x2 t;
    t[0] = ha;
    t[1] = hb;
    hi = __builtin_bit_cast(uint32_t, t);
    lo = pack_bf16(a - (float)ha, b - (float)hb);
}

// Chunked form for bf16 prompts.  With c_t = a_1 + .. + a_t inside a chunk of 64 tokens and S the state in front of it:
//     y_t = exp(c_t) S^T C_t + sum_{s <= t} [exp(c_t - c_s) dt_s (C_t . B_s)] x_s + D x_t
//     S  <- exp(c_last) S + sum_s B_s (exp(c_last - c_s) dt_s x_s)^T
// One workgroup of four wavefronts per (sequence, head, 64 columns of vdim) walks the chunks; wavefront w owns 16 columns
// and keeps its part of S, all 32 * NT rows of it, in MFMA accumulators.  v_mfma_f32_16x16x32_bf16 throughout:
//   G^T (s x t)   = B C^T         rows from LDS, wavefront w takes tokens t = 16w .. 16w + 15 and only s tiles up to its own;
//                                 weighted in fp32, it goes to LDS as the row t of bracketed factors
//   Y^T (p x t)   = S^T C^T       S^T is the accumulator itself: the MFMA's k order is that of the accumulator's rows, which
//                                 the reads of C mirror; scaled by exp(c_t), then
//                 + X^T F^T       X^T fragments through the transposed LDS read
//   S   (n x p)  += B^T (w x)     B^T through the transposed read; w x: the X^T fragments again, weighted in registers
// x, B and C are bf16 (the convolution's output); what is computed in fp32 -- S, the bracketed factors, the weighted x -- enters
// the MFMAs as a bf16 pair of leading part and remainder, so nothing of the recurrence is rounded to 8 bits.
//
// kWhole: a workgroup walks its whole sequence.  Few sequences and heads leave most of the chip idle then, so their segments
// of seg_len tokens go side by side: kSegState leaves what each segment but the last adds to the state, ssd_carry_kernel turns
// these into the states in front of the segments, and kSegOut computes every segment's outputs from there.
enum { kWhole, kSegState, kSegOut };
template <int NT, int MODE>
__global__ __launch_bounds__(256) void ssd_chunk_kernel(SsmParams<__bf16> p) {
    constexpr int Q = 64, NP = 32 * NT;
    constexpr int kBRow = NP * 2 + 32, kCRow = NP * 2 + 16, kXRow = 64 * 2 + 32, kFRow = Q * 2 + 16;
    __shared__ __attribute__((aligned(16))) unsigned char b_lds[Q * kBRow];
    __shared__ __attribute__((aligned(16))) unsigned char c_lds[Q * kCRow];
    __shared__ __attribute__((aligned(16))) unsigned char x_lds[Q * kXRow];
    __shared__ __attribute__((aligned(16))) unsigned char f_lds[2][Q * kFRow];        // leading parts, remainders
    __shared__ float cum_lds[Q], dt_lds[Q];

    const int h = blockIdx.x / p.slices % p.H;
    const int col0 = (blockIdx.x % p.slices) * 64;
    const int unit = blockIdx.x / (p.slices * p.H);
    const int b = MODE == kWhole ? unit : seq_of_unit(p, unit, p.seg_len);
    int first, len;
    seq_rows(p, b, first, len);
    if (len <= 0) return;
    bool last = true;
    if constexpr (MODE != kWhole) {
        const int s0 = (unit - (first / p.seg_len + b)) * p.seg_len;
        if (s0 < 0 || s0 >= len) return;
        last = s0 + p.seg_len >= len;
        if (MODE == kSegState && last) return;           // nobody comes after it
        first += s0;
        len = min(p.seg_len, len - s0);
    }
    const int g = h / (p.H / p.G), inner = p.H * p.P;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, kg = lane >> 4;
    const int pc = col0 + 16 * wave;                    // first column of this wavefront
    const bool has_cols = pc < p.P;
    const int slot = state_slot(p, b);
    float* st = p.ssm_state + ((int64_t)slot * p.H + h) * p.N * p.Pp + pc + r;
    float* seg_st = MODE == kWhole ? nullptr : p.seg_state + ((int64_t)unit * p.H + h) * p.N * p.Pp + pc + r;
    const float bias = p.dt_bias[h], na2 = p.neg_a[h] * kLog2e, skip = p.d_skip[h];
    const __bf16* xsrc = p.xbc + h * p.P + col0;
    const __bf16* bsrc = p.xbc + inner + g * p.N;
    const __bf16* csrc = p.xbc + inner + (p.G + g) * p.N;

    // S: lane holds column pc + r, rows 16 j + 4 kg + i
    f32x4 S[2 * NT];
    const float* from = MODE == kWhole ? st : seg_st;
    const bool resumed = MODE == kSegOut || (MODE == kWhole && p.positions[first] > 0);
#pragma unroll
    for (int j = 0; j < 2 * NT; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int n = 16 * j + 4 * kg + i;
            S[j][i] = resumed && n < p.N && pc + r < p.P ? from[(int64_t)n * p.Pp] : 0.f;
        }

    // one chunk's loads: NT 16-byte pieces of B and C and two of x per thread, dt of token `lane`
    u32x4 rb[NT], rc[NT], rx[2];
    float rdt = 0.f, total = 0.f;                        // total: log2 of the decay so far
    const auto fetch = [&](int t0) {
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            const int idx = j * 256 + tid, row = idx / (4 * NT), col = idx % (4 * NT) * 8;
            rb[j] = rc[j] = u32x4{0u, 0u, 0u, 0u};
            if (t0 + row < len && col < p.N) {
                const int64_t at = (int64_t)(first + t0 + row) * p.channels + col;
                rb[j] = *reinterpret_cast<const u32x4*>(bsrc + at);
                if constexpr (MODE != kSegState) rc[j] = *reinterpret_cast<const u32x4*>(csrc + at);
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int idx = j * 256 + tid, row = idx / 8, col = idx % 8 * 8;
            rx[j] = u32x4{0u, 0u, 0u, 0u};
            if (t0 + row < len && col0 + col < p.P)
                rx[j] = *reinterpret_cast<const u32x4*>(xsrc + (int64_t)(first + t0 + row) * p.channels + col);
        }
        rdt = t0 + lane < len ? (float)p.proj[(int64_t)(first + t0 + lane) * p.proj_stride + p.dt_at + h] : 0.f;
    };
    fetch(0);
    for (int t0 = 0; t0 < len; t0 += Q) {
        const float dt = t0 + lane < len ? softplus(rdt + bias) : 0.f;
        float cum = na2 * dt;                            // running sum of the log2 decays, per lane = token
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float up = __shfl_up(cum, off, 64);
            if (lane >= off) cum += up;
        }
        const float cum_last = __shfl(cum, 63, 64);
        total += cum_last;
        __syncthreads();                                 // everybody has read the chunk before
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            const int idx = j * 256 + tid, row = idx / (4 * NT), col = idx % (4 * NT) * 8;
            *reinterpret_cast<u32x4*>(b_lds + row * kBRow + col * 2) = rb[j];
            if constexpr (MODE != kSegState) *reinterpret_cast<u32x4*>(c_lds + row * kCRow + col * 2) = rc[j];
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int idx = j * 256 + tid;
            *reinterpret_cast<u32x4*>(x_lds + (idx / 8) * kXRow + (idx % 8) * 16) = rx[j];
        }
        if (wave == 0) {
            cum_lds[lane] = cum;
            dt_lds[lane] = dt;
        }
        if (t0 + Q < len) fetch(t0 + Q);
        __syncthreads();

        // ---- bracketed factors of tokens 16 wave + r ------------------------------------------
        if constexpr (MODE != kSegState) {
            const int t = 16 * wave + r;
            const float ct = cum_lds[t];
            bf16x8 cf[NT];
#pragma unroll
            for (int u = 0; u < NT; ++u)
                cf[u] = as_bf16x8(*reinterpret_cast<const u32x4*>(c_lds + t * kCRow + (32 * u + 8 * kg) * 2));
            // (tiles behind the wavefront's own come out as zeros: four independent chains are shorter than a branch per tile)
#pragma unroll
            for (int s0 = 0; s0 < 4; ++s0) {
                f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int u = 0; u < NT; ++u)
                    acc = mfma16(as_bf16x8(*reinterpret_cast<const u32x4*>(b_lds + (16 * s0 + r) * kBRow + (32 * u + 8 * kg) * 2)),
                                 cf[u], acc);
                float f[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int s = 16 * s0 + 4 * kg + i;
                    f[i] = s <= t ? acc[i] * (fast_exp2(ct - cum_lds[s]) * dt_lds[s]) : 0.f;
                }
                uint32_t h0, h1, l0, l1;
                split_bf16(f[0], f[1], h0, l0);
                split_bf16(f[2], f[3], h1, l1);
                *reinterpret_cast<u32x2*>(f_lds[0] + t * kFRow + (16 * s0 + 4 * kg) * 2) = u32x2{h0, h1};
                *reinterpret_cast<u32x2*>(f_lds[1] + t * kFRow + (16 * s0 + 4 * kg) * 2) = u32x2{l0, l1};
            }
            __syncthreads();
        }
        if (!has_cols) continue;

        // X^T fragments: row p = r, k = token 32 u + 8 kg + j
        bf16x8 xf[2];
        const int tr_row = 8 * kg + (r >> 2), tr_col = (r & 3) * 8;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const unsigned char* src = x_lds + (32 * u + tr_row) * kXRow + 32 * wave + tr_col;
            xf[u] = join_bf16x8(lds_read_tr16(src), lds_read_tr16(src + 4 * kXRow));
        }
        // ---- Y^T -------------------------------------------------------------------------------
        if constexpr (MODE != kSegState) {
            bf16x8 sh[NT], sl[NT];
#pragma unroll
            for (int u = 0; u < NT; ++u) {
                u32x4 hi, lo;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    uint32_t a, c;
                    split_bf16(S[2 * u + e / 2][2 * (e % 2)], S[2 * u + e / 2][2 * (e % 2) + 1], a, c);
                    hi[e] = a;
                    lo[e] = c;
                }
                sh[u] = as_bf16x8(hi);
                sl[u] = as_bf16x8(lo);
            }
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) {
                const int t = 16 * tt + r;
                f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int u = 0; u < NT; ++u) {
                    const unsigned char* src = c_lds + t * kCRow + (32 * u + 4 * kg) * 2;
                    const u32x2 c0 = *reinterpret_cast<const u32x2*>(src), c1 = *reinterpret_cast<const u32x2*>(src + 32);
                    const bf16x8 cf = as_bf16x8(u32x4{c0[0], c0[1], c1[0], c1[1]});
                    acc = mfma16(sh[u], cf, acc);
                    acc = mfma16(sl[u], cf, acc);
                }
                acc *= fast_exp2(cum_lds[t]);
#pragma unroll
                for (int u = 0; u <= tt / 2; ++u) {
#pragma unroll
                    for (int part = 0; part < 2; ++part)
                        acc = mfma16(xf[u], as_bf16x8(*reinterpret_cast<const u32x4*>(f_lds[part] + t * kFRow + (32 * u + 8 * kg) * 2)), acc);
                }
                if (t0 + t < len && pc + 4 * kg < p.P) {
                    const u32x2 xw = *reinterpret_cast<const u32x2*>(x_lds + t * kXRow + (16 * wave + 4 * kg) * 2);
                    const uint32_t x01 = xw[0], x23 = xw[1];
                    const bf16x2 xa = __builtin_bit_cast(bf16x2, x01), xb = __builtin_bit_cast(bf16x2, x23);
                    u32x2 o;
                    o[0] = pack_bf16(fmaf(skip, (float)xa[0], acc[0]), fmaf(skip, (float)xa[1], acc[1]));
                    o[1] = pack_bf16(fmaf(skip, (float)xb[0], acc[2]), fmaf(skip, (float)xb[1], acc[3]));
                    *reinterpret_cast<u32x2*>(p.y + (int64_t)(first + t0 + t) * p.y_stride + h * p.P + pc + 4 * kg) = o;
                }
            }
        }
        // ---- S --------------------------------------------------------------------------------
        {
            const float decay = fast_exp2(cum_last);
            bf16x8 wh[2], wl[2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                u32x4 hi, lo;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int s = 32 * u + 8 * kg + 2 * e;
                    uint32_t a, c;
                    split_bf16((float)xf[u][2 * e] * (fast_exp2(cum_last - cum_lds[s]) * dt_lds[s]),
                               (float)xf[u][2 * e + 1] * (fast_exp2(cum_last - cum_lds[s + 1]) * dt_lds[s + 1]), a, c);
                    hi[e] = a;
                    lo[e] = c;
                }
                wh[u] = as_bf16x8(hi);
                wl[u] = as_bf16x8(lo);
            }
#pragma unroll
            for (int j = 0; j < 2 * NT; ++j) {
                S[j] *= decay;
#pragma unroll
                for (int u = 0; u < 2; ++u) {
                    const unsigned char* src = b_lds + (32 * u + tr_row) * kBRow + 32 * j + tr_col;
                    const bf16x8 bt = join_bf16x8(lds_read_tr16(src), lds_read_tr16(src + 4 * kBRow));
                    S[j] = mfma16(bt, wh[u], S[j]);
                    S[j] = mfma16(bt, wl[u], S[j]);
                }
            }
        }
    }
    if constexpr (MODE == kSegState) {
        if (tid == 0 && col0 == 0) p.seg_decay[(int64_t)unit * p.H + h] = total;
    }
    if (MODE == kSegOut && !last) return;
    float* to = MODE == kSegState ? seg_st : st;
#pragma unroll
    for (int j = 0; j < 2 * NT; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int n = 16 * j + 4 * kg + i;
            if (n < p.N && pc + r < p.P) to[(int64_t)n * p.Pp] = S[j][i];
        }
}

// What the segments of a sequence add -> the states in front of them, in place: a thread owns four columns of one row.
__global__ __launch_bounds__(256) void ssd_carry_kernel(SsmParams<__bf16> p) {
    constexpr int kAhead = 4;
    const int h = blockIdx.x % p.H, b = blockIdx.x / p.H;
    const int64_t size = (int64_t)p.N * p.Pp, at = 4 * (blockIdx.y * 256LL + threadIdx.x);
    int first, len;
    seq_rows(p, b, first, len);
    if (len <= 0 || at >= size) return;
    f32x4 S = {0.f, 0.f, 0.f, 0.f};
    if (p.positions[first] > 0) S = *reinterpret_cast<const f32x4*>(p.ssm_state + ((int64_t)state_slot(p, b) * p.H + h) * size + at);
    const int64_t seg0 = first / p.seg_len + b;
    const int n = (len + p.seg_len - 1) / p.seg_len;
    float* seg = p.seg_state + (seg0 * p.H + h) * size + at;
    const float* decay = p.seg_decay + seg0 * p.H + h;
    for (int i = 0; i < n; i += kAhead) {
        f32x4 add[kAhead];
        float d[kAhead];
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (i + j < n - 1) {                         // (the last segment's state is nobody's start)
                add[j] = *reinterpret_cast<const f32x4*>(seg + (i + j) * p.H * size);
                d[j] = decay[(i + j) * p.H];
            }
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (i + j < n) {
                *reinterpret_cast<f32x4*>(seg + (i + j) * p.H * size) = S;
                if (i + j < n - 1) {
                    const float f = fast_exp2(d[j]);
#pragma unroll
                    for (int e = 0; e < 4; ++e) S[e] = fmaf(f, S[e], add[j][e]);
                }
            }
    }
}

template <typename T>
static int launch_conv(const SsmParams<T>& p, hipStream_t s) {
    bool vec = p.channels % 8 == 0 && p.xbc_at % 8 == 0 && p.proj_stride % 8 == 0;
    for (const void* ptr : {(const void*)p.proj, (const void*)p.conv_w, (const void*)p.conv_b, (const void*)p.conv_state, (const void*)p.xbc})
        vec = vec && (reinterpret_cast<uintptr_t>(ptr) & 15) == 0;
    const int64_t groups = vec ? p.channels / 8 : p.channels;
    const int64_t wgs = (p.n_rows / kConvTile + p.B) * ((groups + 255) / 256);
    if (wgs > 0x7fffffffLL) return (int)hipErrorInvalidValue;
    const dim3 grid((unsigned)wgs), block(256);
    if (!vec) hipLaunchKernelGGL((causal_conv_silu_kernel<T, 1, 0>), grid, block, 0, s, p);
    else if (p.taps == 2) hipLaunchKernelGGL((causal_conv_silu_kernel<T, 8, 2>), grid, block, 0, s, p);
    else if (p.taps == 3) hipLaunchKernelGGL((causal_conv_silu_kernel<T, 8, 3>), grid, block, 0, s, p);
    else if (p.taps == 4) hipLaunchKernelGGL((causal_conv_silu_kernel<T, 8, 4>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((causal_conv_silu_kernel<T, 8, 0>), grid, block, 0, s, p);
    return (int)hipGetLastError();
}

template <typename T, bool DECODE>
static int launch_scan(SsmParams<T> p, hipStream_t s) {
    // the widest slice of vdim whose state fits the registers of a workgroup
    int np4 = p.Pp / 4 < 64 ? p.Pp / 4 : 64;
    while (np4 > 1 && (p.N + 256 / np4 - 1) / (256 / np4) > kScanVecs) --np4;
    const int rows = 256 / np4, nv = (p.N + rows - 1) / rows;
    if (nv > kScanVecs) return (int)hipErrorInvalidValue;
    p.np4 = np4;
    p.slices = (p.Pp / 4 + np4 - 1) / np4;
    const int64_t wgs = (int64_t)p.B * p.H * p.slices;
    if (wgs > 0x7fffffffLL) return (int)hipErrorInvalidValue;
    const size_t lds = (size_t)((4 * np4 + 2 * p.N + 3) / 4 * 4) * 4 + (size_t)rows * np4 * 16;
    const dim3 grid((unsigned)wgs), block(256);
    if (nv <= 1) hipLaunchKernelGGL((ssm_scan_kernel<T, 1, DECODE>), grid, block, lds, s, p);
    else if (nv <= 2) hipLaunchKernelGGL((ssm_scan_kernel<T, 2, DECODE>), grid, block, lds, s, p);
    else if (nv <= 4) hipLaunchKernelGGL((ssm_scan_kernel<T, 4, DECODE>), grid, block, lds, s, p);
    else if (nv <= 8) hipLaunchKernelGGL((ssm_scan_kernel<T, 8, DECODE>), grid, block, lds, s, p);
    else hipLaunchKernelGGL((ssm_scan_kernel<T, 16, DECODE>), grid, block, lds, s, p);
    return (int)hipGetLastError();
}

static bool chunked_takes(const SsmParams<__bf16>& p) {
    return p.N % 8 == 0 && p.N <= 256 && p.P % 8 == 0 && p.y_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(p.xbc) & 15) == 0 &&
           (reinterpret_cast<uintptr_t>(p.y) & 7) == 0;
}

template <int MODE>
static int launch_chunks(const SsmParams<__bf16>& p, int64_t units, hipStream_t s) {
    const int64_t wgs = units * p.H * p.slices;
    if (wgs > 0x7fffffffLL) return (int)hipErrorInvalidValue;
    const dim3 grid((unsigned)wgs), block(256);
    if (p.N <= 32) hipLaunchKernelGGL((ssd_chunk_kernel<1, MODE>), grid, block, 0, s, p);
    else if (p.N <= 64) hipLaunchKernelGGL((ssd_chunk_kernel<2, MODE>), grid, block, 0, s, p);
    else if (p.N <= 128) hipLaunchKernelGGL((ssd_chunk_kernel<4, MODE>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((ssd_chunk_kernel<8, MODE>), grid, block, 0, s, p);
    return (int)hipGetLastError();
}

static int launch_chunked(SsmParams<__bf16> p, hipStream_t s) {
    p.slices = (p.P + 63) / 64;
    if (p.seg_len == 0) return launch_chunks<kWhole>(p, p.B, s);
    p.n_segs = (int)(p.n_rows / p.seg_len) + p.B;
    if (int e = launch_chunks<kSegState>(p, p.n_segs, s)) return e;
    const int64_t pieces = ((int64_t)p.N * p.Pp / 4 + 255) / 256, heads = (int64_t)p.B * p.H;
    if (pieces > 65535 || heads > 0x7fffffffLL) return (int)hipErrorInvalidValue;
    hipLaunchKernelGGL(ssd_carry_kernel, dim3((unsigned)heads, (unsigned)pieces), dim3(256), 0, s, p);
    if (int e = (int)hipGetLastError()) return e;
    return launch_chunks<kSegOut>(p, p.n_segs, s);
}

template <typename T>
static SsmParams<T> ssm_params(const mi355_ssm_args& a) {
    SsmParams<T> p{};
    p.proj = (const T*)a.proj;
    p.proj_stride = a.proj_row_stride;
    p.xbc_at = a.xbc_col;
    p.dt_at = a.dt_col;
    p.conv_w = a.conv_weight;
    p.conv_b = a.conv_bias;
    p.dt_bias = a.dt_bias;
    p.neg_a = a.neg_a;
    p.d_skip = a.d_skip;
    p.conv_state = (T*)a.conv_state;
    p.ssm_state = a.ssm_state;
    p.slots = a.slots;
    p.positions = a.positions;
    p.cu = a.cu_seqlens;
    p.xbc = (T*)a.xbc;
    p.y = (T*)a.y;
    p.y_stride = a.y_row_stride;
    p.n_rows = a.n_rows;
    p.B = a.batch;
    p.H = a.heads;
    p.P = a.vdim;
    p.Pp = (a.vdim + 3) / 4 * 4;
    p.N = a.state;
    p.G = a.groups;
    p.taps = a.taps;
    p.channels = a.heads * a.vdim + 2 * a.groups * a.state;
    p.n_slots = a.n_slots;
    p.seg_state = a.seg_state;
    p.seg_decay = a.seg_decay;
    p.seg_len = a.seg_len;
    return p;
}

static int ssm_check(const mi355_ssm_args* a) {
    if (!a || !a->proj || !a->conv_weight || !a->conv_bias || !a->dt_bias || !a->neg_a || !a->d_skip || !a->conv_state || !a->ssm_state ||
        !a->slots || !a->positions || !a->y)
        return set_error(MI355_EINVAL, "ssm: null pointer argument");
    if (a->dtype != MI355_BF16 && a->dtype != MI355_FP32) return set_error(MI355_EDTYPE, "ssm: dtype must be MI355_BF16 or MI355_FP32");
    if (a->batch <= 0 || a->heads <= 0 || a->vdim <= 0 || a->state <= 0 || a->groups <= 0 || a->heads % a->groups || a->n_slots <= 0 || a->n_rows < 0)
        return set_error(MI355_EINVAL, "ssm: batch, heads, vdim, state, groups, n_slots, n_rows out of range (heads a multiple of groups)");
    if (a->taps < 1 || a->taps > kMaxTaps) return set_error(MI355_EINVAL, "ssm: taps must be in 1..16");
    if (a->state > 256 * kScanVecs || a->vdim > (1 << 20)) return set_error(MI355_EINVAL, "ssm: state must be at most 4096");
    if ((reinterpret_cast<uintptr_t>(a->ssm_state) & 15) != 0) return set_error(MI355_EINVAL, "ssm: ssm_state must be 16-byte aligned");
    const int64_t channels = (int64_t)a->heads * a->vdim + 2LL * a->groups * a->state;
    if (a->xbc_col < 0 || a->dt_col < 0 || a->xbc_col + channels > a->proj_row_stride || a->dt_col + a->heads > a->proj_row_stride ||
        a->y_row_stride < (int64_t)a->heads * a->vdim)
        return set_error(MI355_EINVAL, "ssm: columns outside the rows of proj or y");
    if (a->n_rows > 0x7fffff00LL || channels > 0x7fffff00LL) return set_error(MI355_EINVAL, "ssm: too many rows or channels");
    return MI355_OK;
}

}  // namespace mi355

using namespace mi355;

extern "C" int mi355_ssm_prefill(const mi355_ssm_args* args, int scan, void* stream) {
    if (int e = ssm_check(args)) return e;
    if (!args->xbc) return set_error(MI355_EINVAL, "ssm_prefill: null xbc buffer");
    if (!args->cu_seqlens && args->n_rows != args->batch) return set_error(MI355_EINVAL, "ssm_prefill: one row per sequence without cu_seqlens");
    if (scan < MI355_SCAN_AUTO || scan > MI355_SCAN_CHUNKED) return set_error(MI355_EINVAL, "ssm_prefill: unknown scan");
    if (args->seg_len < 0 || args->seg_len % 64 ||
        (args->seg_len > 0 && (!args->seg_state || !args->seg_decay || (reinterpret_cast<uintptr_t>(args->seg_state) & 15))))
        return set_error(MI355_EINVAL, "ssm_prefill: segments are multiples of 64 tokens and need their buffers");
    if (args->n_rows == 0) return MI355_OK;
    hipStream_t s = (hipStream_t)stream;
    int rc;
    if (args->dtype == MI355_BF16) {
        const SsmParams<__bf16> p = ssm_params<__bf16>(*args);
        const bool chunked = scan != MI355_SCAN_SERIAL && chunked_takes(p);
        if (scan == MI355_SCAN_CHUNKED && !chunked) return set_error(MI355_EINVAL, "ssm_prefill: the chunked scan needs state and vdim in multiples of 8 and state <= 256");
        rc = launch_conv(p, s);
        if (rc == 0) rc = chunked ? launch_chunked(p, s) : launch_scan<__bf16, false>(p, s);
    } else {
        if (scan == MI355_SCAN_CHUNKED) return set_error(MI355_EDTYPE, "ssm_prefill: the chunked scan is bf16");
        const SsmParams<float> p = ssm_params<float>(*args);
        rc = launch_conv(p, s);
        if (rc == 0) rc = launch_scan<float, false>(p, s);
    }
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}

extern "C" int mi355_ssm_decode(const mi355_ssm_args* args, void* stream) {
    if (int e = ssm_check(args)) return e;
    if (args->cu_seqlens || args->n_rows != args->batch) return set_error(MI355_EINVAL, "ssm_decode: one row per sequence");
    hipStream_t s = (hipStream_t)stream;
    const int rc = args->dtype == MI355_BF16 ? launch_scan<__bf16, true>(ssm_params<__bf16>(*args), s)
                                             : launch_scan<float, true>(ssm_params<float>(*args), s);
    if (rc != 0) return set_error(rc, hipGetErrorString((hipError_t)rc));
    return MI355_OK;
}
