// nl_mfma.h -- dense matrix products of the layer-stack models (nl_stack.hip): weights and activations in MFMA operand order,
// two element types behind one source.
//
//   T = __bf16 : v_mfma_f32_16x16x32_bf16, 32-bit accumulation
//   T = float  : v_mfma_f32_16x16x4_f32, eight of them in place of one: IEEE single-precision products and sums
//
// OPERAND ORDER.  A matrix [rows][K] is cut into tiles of 16 rows x 32 columns; a tile is 64 runs of 8 elements, run
// l = (k % 32) / 8 * 16 + row % 16, tiles of a row group one behind the other.  A wavefront's fragment is therefore one contiguous
// 1 KiB (2 KiB for float) read in lane order, from HBM, L2 or LDS alike, and LDS-DMA copies tiles without touching registers.
// Rows and K are padded with zeros to whole tiles.  Weights [out][in] are the A operand (rows = outputs), activations
// [token][in] the B operand (rows = tokens); the accumulator of a 16 x 16 tile has D[row = 4 (lane / 16) + i][token = lane % 16],
// so a lane ends up with four consecutive outputs of one token.
//
// Two kernels: many_kernel for prompts (a 128 x 128 tile per workgroup, an LDS ring filled by LDS-DMA) and few_kernel for
// decode batches of up to 64 tokens (one row tile per workgroup, K split over its wavefronts, the weights read once straight into
// registers; for a handful of tokens the RMS norm of the layer's input runs in its prologue, together with the norm and residual add
// of the sublayer before where a model has norms behind its sublayers).  Epilogues: plain 32-bit store (+ bias), residual add (+ an
// optional second addend), activation(gate) * up stored as the next product's operand, query rows by head with rotary positions, keys and
// values in the operand order of the attention products.  A launch may carry independent work of single wavefronts behind its own
// workgroups (TAIL).
#pragma once
#include "nl_kernels.h"

namespace nl {

typedef __bf16 bf16;
typedef bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int OPT = 512;          // elements of one operand tile (16 rows x 32 columns)
enum { ST_F32 = 0, ST_RESID = 1, ST_GATED = 2, ST_HEADS = 3, ST_KEYS = 4, ST_VALUES = 5 };   // epilogues

template <typename T> struct Frag;
template <> struct Frag<bf16> { bf16x8 v; };
template <> struct Frag<float> { f32x4 a, b; };

__device__ __forceinline__ void frag_zero(Frag<bf16> &f) { f.v = bf16x8{}; }
__device__ __forceinline__ void frag_zero(Frag<float> &f) { f.a = f32x4{}; f.b = f32x4{}; }
__device__ __forceinline__ float frag_get(const Frag<bf16> &f, int j) { return (float)f.v[j]; }
__device__ __forceinline__ float frag_get(const Frag<float> &f, int j) { return j < 4 ? f.a[j & 3] : f.b[j & 3]; }
__device__ __forceinline__ void frag_set(Frag<bf16> &f, int j, float x) { f.v[j] = (bf16)x; }
__device__ __forceinline__ void frag_set(Frag<float> &f, int j, float x) { if (j < 4) f.a[j & 3] = x; else f.b[j & 3] = x; }

__device__ __forceinline__ f32x4 mma(const Frag<bf16> &A, const Frag<bf16> &B, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(A.v, B.v, c, 0, 0, 0);
}
// the K order inside a fragment is the same permutation on both sides: step j multiplies element j of every lane's run
__device__ __forceinline__ f32x4 mma(const Frag<float> &A, const Frag<float> &B, f32x4 c) {
#pragma unroll
    for (int j = 0; j < 4; j++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(A.a[j], B.a[j], c, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; j++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(A.b[j], B.b[j], c, 0, 0, 0);
    return c;
}

// index of element (row, k) of an operand with nks tiles per row group
__host__ __device__ inline long long op_index(int row, int k, int nks) {
    return (((long long)(row >> 4) * nks + (k >> 5)) * 64 + ((k & 31) >> 3) * 16 + (row & 15)) * 8 + (k & 7);
}
__device__ __forceinline__ void put(bf16 *p, float v) { *p = (bf16)v; }
__device__ __forceinline__ void put(float *p, float v) { *p = v; }
__device__ __forceinline__ void put4(bf16 *p, f32x4 v) {
    bf16x4 o;
#pragma unroll
    for (int i = 0; i < 4; i++) o[i] = (bf16)v[i];
    *reinterpret_cast<bf16x4 *>(p) = o;
}
__device__ __forceinline__ void put4(float *p, f32x4 v) { *reinterpret_cast<f32x4 *>(p) = v; }

// Single-precision functions on the hardware's v_exp_f32 / v_rcp_f32 / v_rsq_f32 (1 ulp each).  exp: the rounding of x log2(e) is
// carried as a correction, so the result stays within a few ulp for large |x| too; x finite.
__device__ __forceinline__ float exp_f32(float x) {
    constexpr float L = 1.44269504f, LLO = 1.92596299e-8f, LN2 = 0.693147181f;      // log2(e) = L + LLO
    const float t = x * L, r = fmaf(x, LLO, fmaf(x, L, -t)), e = __builtin_amdgcn_exp2f(t);
    return fmaf(e, r * LN2, e);
}
__device__ __forceinline__ float rcp_f32(float x) { return __builtin_amdgcn_rcpf(x); }
__device__ __forceinline__ float rsqrt_f32(float x) { return __builtin_amdgcn_rsqf(x); }
__device__ __forceinline__ float sigmoid_f32(float z) {
    const float e = exp_f32(-fminf(fabsf(z), 100.f)), r = rcp_f32(1.f + e);
    return z >= 0.f ? r : e * r;
}
__device__ __forceinline__ float silu_f32(float z) { return z * sigmoid_f32(z); }
__device__ __forceinline__ float gelu_tanh_f32(float z) {
    // 0.5 (1 + tanh u) = sigmoid(2 u)
    return z * sigmoid_f32(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
template <int CTRL> __device__ __forceinline__ float dpp_add(float v) {
    return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float lane_value(float v, int lane) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), lane)); }
// sum over the wavefront, in every lane: rows of 16 lanes by DPP (neighbours, pairs, mirrored halves, mirrored row), then the four rows
__device__ __forceinline__ float wave_sum(float v) {
    v = dpp_add<0x140>(dpp_add<0x141>(dpp_add<0x4E>(dpp_add<0xB1>(v))));
    return (lane_value(v, 0) + lane_value(v, 16)) + (lane_value(v, 32) + lane_value(v, 48));
}

// 16 bytes per lane straight into LDS: lane i lands at lds_base + 16 i (lds_base wave-uniform)
__device__ __forceinline__ void lds_dma16(const void *src_lane, void *lds_base) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)src_lane,
                                     (__attribute__((address_space(3))) void *)lds_base, 16, 0, 0);
}
// until at most N of this wavefront's vector memory operations are in flight (they complete in order)
template <int N> __device__ __forceinline__ void vm_wait() { asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory"); }

// Workgroup barrier for data that passes through LDS only.  __syncthreads() also waits for every global load and store the wavefront
// has in flight, i.e. for exactly the prefetches that are meant to run past it.
__device__ __forceinline__ void lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}

// ------------------------------------------------------------- upload ---

// rows x cols of a source matrix (bf16 bits or float) into operand order: row r goes to destination row
// ((row0 + r) / 16 * tstride + toff) * 16 + (row0 + r) % 16, column c to k0 + c.  The destination was zeroed.
template <typename T>
__global__ void pack_operand_kernel(const void *src, int src_f32, long long rows, long long cols, T *dst, int nks, int row0, int k0,
                                    int tstride, int toff) {
    const long long n = rows * cols;
    for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long long)gridDim.x * blockDim.x) {
        const long long r = i / cols;
        const int c = (int)(i - r * cols), R = row0 + (int)r;
        const float v = src_f32 ? reinterpret_cast<const float *>(src)[i]
                                : __uint_as_float((unsigned)reinterpret_cast<const unsigned short *>(src)[i] << 16);
        put(dst + op_index(((R >> 4) * tstride + toff) * 16 + (R & 15), k0 + c, nks), v);
    }
}
// the same with a place per source row: element (r, c) goes to row rbase[r], column kbase[r] + c, or transposed to row rbase[r] + c,
// column kbase[r]
template <typename T>
__global__ void pack_mapped_kernel(const void *src, int src_f32, long long rows, long long cols, T *dst, int nks, const int *rbase, const int *kbase, int transpose) {
    const long long n = rows * cols;
    for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long long)gridDim.x * blockDim.x) {
        const long long r = i / cols;
        const int c = (int)(i - r * cols);
        const float v = src_f32 ? reinterpret_cast<const float *>(src)[i]
                                : __uint_as_float((unsigned)reinterpret_cast<const unsigned short *>(src)[i] << 16);
        put(dst + op_index(rbase[r] + (transpose ? c : 0), kbase[r] + (transpose ? 0 : c), nks), v);
    }
}
// a vector / small matrix as float, plus a constant (1 where a norm's gain is 1 + w); cols > 1: transposed to [cols][n / cols]
__global__ void widen_kernel(const void *src, int src_f32, long long n, float add, float *dst, int cols) {
    for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long long)gridDim.x * blockDim.x)
        dst[cols > 1 ? i % cols * (n / cols) + i / cols : i] = (src_f32 ? reinterpret_cast<const float *>(src)[i]
                          : __uint_as_float((unsigned)reinterpret_cast<const unsigned short *>(src)[i] << 16)) + add;
}

// ---------------------------------------------------- embedding, norm ---

struct LookupParams {
    const void *table;     // [vocab][dim] in operand order
    const int *tok;
    int nks, dim;
    float scale;
    float *x, *x0;         // x0 (may be null): a second copy for stacks that add the embedding output again
};
template <typename T>
__global__ void __launch_bounds__(256) lookup_kernel(LookupParams P) {
    const int n = blockIdx.x, token = P.tok[n];
    for (int k = threadIdx.x; k < P.dim; k += 256) {
        const float v = (float)reinterpret_cast<const T *>(P.table)[op_index(token, k, P.nks)] * P.scale;
        P.x[(long long)n * P.dim + k] = v;
        if (P.x0) P.x0[(long long)n * P.dim + k] = v;
    }
}

// work that rides in a launch: unit(i, lane) for i < units, one wavefront each, reading and writing nothing that the launch touches
struct NoTail {
    static constexpr bool on = false;
    int units = 0;
    __device__ __forceinline__ void unit(int, int) const {}
};

// RMS norm of rows of the residual stream, stored as a product's operand (columns beyond dim zero).  With d: the rows are first
// x + norm(d) dw (a sublayer's result through the norm behind it), stored to x_out unless that is null.
struct NormParams {
    const float *x, *w;    // w: the factor itself
    const int *rows;       // row of x for output token n; null: n
    void *out;
    int dim, nks, n_tokens;
    float eps;
    int ld;                // floats between rows
    const float *d, *dw;
    float *x_out;
};
// grid (tiles of 16 tokens, splits of K [+ 1 for the tail]): every workgroup sums the squares of its 16 rows and stores its share of the
// k tiles, whole 16-row tiles at a time (contiguous stores)
template <typename T, class TAIL>
__global__ void __launch_bounds__(512) norm_operand_kernel(NormParams P, TAIL tail) {
    __shared__ float inv_s[16], invd_s[16];
    const int n0 = blockIdx.x * 16, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
    const int nsplit = gridDim.y - (TAIL::on ? 1 : 0);
    if constexpr (TAIL::on)
        if ((int)blockIdx.y == nsplit) {
            for (int i = 0; i < 2; i++)
                if (n0 + w * 2 + i < tail.units) tail.unit(n0 + w * 2 + i, lane);
            return;
        }
    const bool vec = (P.dim & 3) == 0;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const int n = min(n0 + w * 2 + i, P.n_tokens - 1);
        const long long at = (long long)(P.rows ? P.rows[n] : n) * P.ld;
        const float *x = P.x + at, *d = P.d + at;
        float ss = 0.f, invd = 0.f;
        if (P.d) {
            if (vec) {
#pragma unroll 4
                for (int k = lane * 4; k < P.dim; k += 256) {
                    const f32x4 v = *reinterpret_cast<const f32x4 *>(d + k);
                    ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
                }
            } else
                for (int k = lane; k < P.dim; k += 64) ss += d[k] * d[k];
            invd = rsqrt_f32(wave_sum(ss) / (float)P.dim + P.eps);
            if (lane == 0) invd_s[w * 2 + i] = invd;
            ss = 0.f;
        }
        if (vec) {
#pragma unroll 4
            for (int k = lane * 4; k < P.dim; k += 256) {
                f32x4 v = *reinterpret_cast<const f32x4 *>(x + k);
                if (P.d) v += *reinterpret_cast<const f32x4 *>(d + k) * invd * *reinterpret_cast<const f32x4 *>(P.dw + k);
                ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
            }
        } else
            for (int k = lane; k < P.dim; k += 64) {
                const float v = P.d ? x[k] + d[k] * invd * P.dw[k] : x[k];
                ss += v * v;
            }
        ss = wave_sum(ss);
        if (lane == 0) inv_s[w * 2 + i] = rsqrt_f32(ss / (float)P.dim + P.eps);
    }
    __syncthreads();
    const int r = lane & 15, n = min(n0 + r, P.n_tokens - 1);
    const long long at = (long long)(P.rows ? P.rows[n] : n) * P.ld;
    const float *x = P.x + at, *d = P.d + at;
    const float inv = inv_s[r], invd = P.d ? invd_s[r] : 0.f;
    const bool keep = P.x_out && n0 + r < P.n_tokens;
    T *out = reinterpret_cast<T *>(P.out) + (long long)blockIdx.x * P.nks * OPT;
    for (int ks = blockIdx.y * 8 + w; ks < P.nks; ks += nsplit * 8) {
        const int k0 = ks * 32 + (lane >> 4) * 8;
        f32x4 a, b;
        if (vec && k0 + 8 <= P.dim) {
            a = *reinterpret_cast<const f32x4 *>(x + k0);
            b = *reinterpret_cast<const f32x4 *>(x + k0 + 4);
            if (P.d) {
                a += *reinterpret_cast<const f32x4 *>(d + k0) * invd * *reinterpret_cast<const f32x4 *>(P.dw + k0);
                b += *reinterpret_cast<const f32x4 *>(d + k0 + 4) * invd * *reinterpret_cast<const f32x4 *>(P.dw + k0 + 4);
            }
            if (keep) {
                *reinterpret_cast<f32x4 *>(P.x_out + at + k0) = a;
                *reinterpret_cast<f32x4 *>(P.x_out + at + k0 + 4) = b;
            }
            a = a * inv * *reinterpret_cast<const f32x4 *>(P.w + k0);
            b = b * inv * *reinterpret_cast<const f32x4 *>(P.w + k0 + 4);
        } else {
#pragma unroll
            for (int j = 0; j < 8; j++) {
                float v = 0.f;
                if (k0 + j < P.dim) {
                    v = P.d ? x[k0 + j] + d[k0 + j] * invd * P.dw[k0 + j] : x[k0 + j];
                    if (keep) P.x_out[at + k0 + j] = v;
                    v *= inv * P.w[k0 + j];
                }
                if (j < 4) a[j] = v; else b[j - 4] = v;
            }
        }
        T *o = out + ks * OPT + lane * 8;
        put4(o, a);
        put4(o + 4, b);
    }
}
// the same for rows that fit a workgroup's registers, read once: RW rows per workgroup, a thread holds NU runs of 8 columns of one row.
// RW 1 spreads a decode batch over the chip; RW 8 stores whole 128-byte lines of the operand.  [+ workgroups for the tail]
template <typename T, int RW, int NU, int NTHR, class TAIL>
__global__ void __launch_bounds__(NTHR) norm_rows_kernel(NormParams P, TAIL tail) {
    constexpr int NW = NTHR / 64;
    __shared__ float red[2][NW][RW];
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, nb = (P.n_tokens + RW - 1) / RW;
    if constexpr (TAIL::on)
        if ((int)blockIdx.x >= nb) {
            const int u = (blockIdx.x - nb) * NW + w;
            if (u < tail.units) tail.unit(u, lane);
            return;
        }
    const int r = tid % RW, n = blockIdx.x * RW + r, row = min(n, P.n_tokens - 1), runs = P.nks * 4;
    const long long at = (long long)(P.rows ? P.rows[row] : row) * P.ld;
    f32x4 v[NU][2] = {}, d[NU][2] = {}, wv[NU][2] = {};
    auto each = [&](auto f) {                              // (run, columns of it that exist)
#pragma unroll
        for (int i = 0; i < NU; i++) {
            const int run = tid / RW + i * (NTHR / RW);
            if (run < runs) f(i, run * 8, P.dim - run * 8);
        }
    };
    auto read = [&](f32x4 *o, const float *p, int k0, int left) {
        if (left >= 8 && (P.dim & 3) == 0) {
            o[0] = *reinterpret_cast<const f32x4 *>(p + k0);
            o[1] = *reinterpret_cast<const f32x4 *>(p + k0 + 4);
        } else
#pragma unroll
            for (int j = 0; j < 8; j++)
                if (j < left) o[j >> 2][j & 3] = p[k0 + j];
    };
    // sum of squares of the thread's values over its row
    auto row_sum = [&](f32x4 (&x)[NU][2], int k) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NU; i++)
#pragma unroll
            for (int j = 0; j < 8; j++) ss += x[i][j >> 2][j & 3] * x[i][j >> 2][j & 3];
        if constexpr (RW == 1) ss = wave_sum(ss);
        else
#pragma unroll
            for (int o = RW; o < 64; o <<= 1) ss += __shfl_xor(ss, o);
        if (lane < RW) red[k][w][lane] = ss;
        lds_barrier();
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < NW; i++) ss += red[k][i][r];
        return rsqrt_f32(ss / (float)P.dim + P.eps);
    };
    each([&](int i, int k0, int left) {
        if (P.d) read(d[i], P.d + at, k0, left);
        read(v[i], P.x + at, k0, left);
    });
    f32x4 dw[NU][2] = {};
    each([&](int i, int k0, int left) {
        if (P.d) read(dw[i], P.dw, k0, left);
        read(wv[i], P.w, k0, left);
    });
    if (P.d) {
        const float inv = row_sum(d, 0);
        each([&](int i, int k0, int left) {
#pragma unroll
            for (int h = 0; h < 2; h++) v[i][h] += d[i][h] * inv * dw[i][h];
            if (!P.x_out || n >= P.n_tokens) return;
            float *o = P.x_out + at + k0;
            if (left >= 8 && (P.dim & 3) == 0) {
                *reinterpret_cast<f32x4 *>(o) = v[i][0];
                *reinterpret_cast<f32x4 *>(o + 4) = v[i][1];
            } else
#pragma unroll
                for (int j = 0; j < 8; j++)
                    if (j < left) o[j] = v[i][j >> 2][j & 3];
        });
    }
    const float inv = row_sum(v, 1);
    if (n >= P.n_tokens) return;
    each([&](int i, int k0, int) {
        T *o = reinterpret_cast<T *>(P.out) + op_index(n, k0, P.nks);
        put4(o, v[i][0] * inv * wv[i][0]);
        put4(o + 4, v[i][1] * inv * wv[i][1]);
    });
}
constexpr int NORM_FEW_ROWS = 256;        // rows up to which every row has a workgroup of its own

template <typename T, class TAIL = NoTail>
hipError_t launch_norm_operand(NormParams P, hipStream_t st, TAIL tail = {}) {
    if (!P.ld) P.ld = P.dim;
    if ((P.ld & 3) == 0 || (P.dim & 3)) {                  // (rows of vectors start at vectors)
        const int runs = P.nks * 4;
        auto go = [&](auto kfn, int rw, int nthr) {
            hipLaunchKernelGGL(kfn, dim3((P.n_tokens + rw - 1) / rw + (TAIL::on ? (tail.units + nthr / 64 - 1) / (nthr / 64) : 0)), dim3(nthr), 0, st, P, tail);
            return hipGetLastError();
        };
        if (P.n_tokens <= NORM_FEW_ROWS) {
            if (runs <= 256) return go(norm_rows_kernel<T, 1, 1, 256, TAIL>, 1, 256);
            if (runs <= 1024) return go(norm_rows_kernel<T, 1, 4, 256, TAIL>, 1, 256);
        } else {
            if (runs <= 128) return go(norm_rows_kernel<T, 8, 1, 1024, TAIL>, 8, 1024);
            if (runs <= 256) return go(norm_rows_kernel<T, 8, 2, 1024, TAIL>, 8, 1024);
            if (runs <= 512) return go(norm_rows_kernel<T, 4, 2, 1024, TAIL>, 4, 1024);
        }
    }
    const int tt = (P.n_tokens + 15) / 16, split = std::max(1, std::min((P.nks + 7) / 8, 256 / tt));
    hipLaunchKernelGGL((norm_operand_kernel<T, TAIL>), dim3(tt, split + (TAIL::on ? 1 : 0)), dim3(512), 0, st, P, tail);
    return hipGetLastError();
}

// ----------------------------------------------------------- products ---

// ST_HEADS: rows [0, split) are hrows[0] rows per head, the others hrows[1] rows per head; the latter's first `pairs` pairs of adjacent
// rows are rotated by the token's position.  A row goes to q [token][head][ld] from column col[0 / 1] on, the first kind to the operand
// xq (column = row) instead if there is one.
struct HeadRows {
    void *q, *xq;
    int xq_nks, heads, ld, split, hrows[2], col[2], pairs;
    const float *rope;     // [position][pairs] cos, sin
    const int *pos;
};
// ST_KEYS / ST_VALUES: row = head * hrows + d, token = key slot; operand tiles [head][slots / 16][nt] (keys: nt tiles of 32 dimensions)
// or [head][slots / 32][nt] (values: nt tiles of 16, the order of nl_winattn.h)
struct KeyRows {
    void *dst;
    int hrows, nt, slots;
};

struct MatParams {
    const void *W;         // [nrt][nks] operand tiles; ST_GATED: gate tile, up tile, gate tile, ...
    const void *X;         // [token tiles][nks]
    int nks, nrt, n_tokens, rows;
    float *out;            // ST_F32: [token][ldo]; ST_RESID: the residual stream, updated in place
    int ldo;
    const float *add2;     // ST_RESID: also added (same layout as out), or null
    void *act;             // ST_GATED: [token tiles][act_nks] operand tiles
    int act_nks, act_silu; // activation: silu or tanh-gelu
    const float *bias, *bias2;   // ST_F32: per row; ST_GATED: of gate and up; whole row tiles long, or null
    int x_nks;             // k tiles per token tile of X (0: nks)
    int group;             // few_kernel: row tiles of a group; group i multiplies X's k tiles from i * nks on (0: one group)
    const int *x_tile;     // many_kernel: which tile of X is token tile t (null: t)
    HeadRows hd;
    KeyRows kr;
    // few_kernel with the norm in its prologue: B = norm(x), or of x + norm(nd) ndw, which workgroup 0 stores to nxo (may be null)
    const float *nx, *nw, *nd, *ndw;
    float *nxo;
    int ndim, nld;         // nld: floats between rows (0: ndim)
    float neps;
    // one token: every row tile's largest result and its row, for the argmax that follows (or null)
    float *amax_val;
    int *amax_idx;
};

__device__ __forceinline__ void store_rows(float *out, int ldo, int rows, int tok, int row, f32x4 v) {
    float *o = out + (long long)tok * ldo + row;
    if (row + 3 < rows && (ldo & 3) == 0) *reinterpret_cast<f32x4 *>(o) = v;
    else
        for (int i = 0; i < 4; i++)
            if (row + i < rows) o[i] = v[i];
}
__device__ __forceinline__ void add_rows(float *out, const float *add2, int ldo, int rows, int tok, int row, f32x4 v) {
    const long long at = (long long)tok * ldo + row;
    if (row + 3 < rows && (ldo & 3) == 0) {
        v += *reinterpret_cast<const f32x4 *>(out + at);
        if (add2) v += *reinterpret_cast<const f32x4 *>(add2 + at);
        *reinterpret_cast<f32x4 *>(out + at) = v;
    } else
        for (int i = 0; i < 4; i++)
            if (row + i < rows) out[at + i] = out[at + i] + v[i] + (add2 ? add2[at + i] : 0.f);
}
// four consecutive feed-forward rows f16 * 16 + 4 g .. + 3 of one token
template <typename T>
__device__ __forceinline__ void store_gated(const MatParams &P, int tok, int f16, int g, f32x4 gate, f32x4 up) {
    f32x4 v;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        if (P.bias) {
            gate[i] += P.bias[f16 * 16 + 4 * g + i];
            up[i] += P.bias2[f16 * 16 + 4 * g + i];
        }
        v[i] = (P.act_silu ? silu_f32(gate[i]) : gelu_tanh_f32(gate[i])) * up[i];
    }
    put4(reinterpret_cast<T *>(P.act) + op_index(tok, f16 * 16 + 4 * g, P.act_nks), v);
}

__device__ __forceinline__ f32x4 with_bias(const float *bias, int row, f32x4 v) {
    if (bias) v += *reinterpret_cast<const f32x4 *>(bias + row);
    return v;
}
// four consecutive rows of one head of one token
template <typename T>
__device__ __forceinline__ void store_heads(const HeadRows &H, int tok, int row, f32x4 v) {
    const int kind = row >= H.split, r0 = kind ? row - H.split : row, h = r0 / H.hrows[kind], d = r0 - h * H.hrows[kind];
    if (h >= H.heads) return;
    if (kind) {
        const float *cs = H.rope + ((long long)H.pos[tok] * H.pairs + (d >> 1)) * 2;
#pragma unroll
        for (int i = 0; i < 2; i++)
            if ((d >> 1) + i < H.pairs) {
                const float c = cs[2 * i], s = cs[2 * i + 1], a = v[2 * i], b = v[2 * i + 1];
                v[2 * i] = a * c - b * s;
                v[2 * i + 1] = b * c + a * s;
            }
    } else if (H.xq) {
        put4(reinterpret_cast<T *>(H.xq) + op_index(tok, row, H.xq_nks), v);
        return;
    }
    put4(reinterpret_cast<T *>(H.q) + ((long long)tok * H.heads + h) * H.ld + H.col[kind] + d, v);
}

// prompts: RTW row tiles x 4 token tiles per wavefront, 2 x 2 wavefronts; the k tiles travel through a ring of LDS stages
template <typename T, int RTW> struct ManyGeom {
    static constexpr int RT = 2 * RTW, NT = 8, UNIT = OPT * sizeof(T), NST = sizeof(T) == 2 ? 4 : 2, STAGE = (RT + NT) * UNIT, LDS = NST * STAGE;   // 48 or 64 KB
};
template <typename T, int EPI, int RTW, class TAIL>
__global__ void __launch_bounds__(256) many_kernel(MatParams P, TAIL tail) {
    using G = ManyGeom<T, RTW>;
    constexpr int RT = G::RT, NT = G::NT, UNIT = G::UNIT, NST = G::NST, STAGE = G::STAGE;
    constexpr int PW = STAGE / 4096;                       // 1 KiB pieces per stage and wavefront
    extern __shared__ __align__(16) char lds[];
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4;
    const int nrb = (P.nrt + RT - 1) / RT, ntt = (P.n_tokens + 15) >> 4, ntb = (ntt + NT - 1) / NT, total = nrb * ntb;
    // blocks b, b + 8, ... run on one XCD: give each XCD a contiguous range of (row block, token block), token blocks fastest, so
    // that the token blocks of a row block share its weights in one L2
    const int per = (total + 7) / 8;
    if constexpr (TAIL::on)
        if ((int)blockIdx.x >= per * 8) {
            const int u = (blockIdx.x - per * 8) * 4 + w;
            if (u < tail.units) tail.unit(u, lane);
            return;
        }
    const int id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || id >= total) return;
    const int rb = id / ntb, tb = id - rb * ntb;
    const int wr = w & 1, wt = w >> 1, nks = P.nks;
    f32x4 acc[RTW][4] = {};
    const char *src[PW];                                   // this wavefront's pieces of k tile 0
#pragma unroll
    for (int i = 0; i < PW; i++) {
        const int u = i * 4 + w, t = u / (UNIT / 1024), piece = u % (UNIT / 1024);
        const int xt = min(tb * NT + t - RT, ntt - 1);
        src[i] = (t < RT ? reinterpret_cast<const char *>(P.W) + (long long)min(rb * RT + t, P.nrt - 1) * nks * UNIT
                         : reinterpret_cast<const char *>(P.X) + (long long)(P.x_tile ? P.x_tile[xt] : xt) * P.x_nks * UNIT) + piece * 1024 + lane * 16;
    }
    auto issue = [&](int ks, int st) {
#pragma unroll
        for (int i = 0; i < PW; i++) lds_dma16(src[i] + (long long)ks * UNIT, lds + st * STAGE + (i * 4 + w) * 1024);
    };
#pragma unroll
    for (int s = 0; s < NST - 1; s++)
        if (s < nks) issue(s, s);
    int st = 0;
    for (int ks = 0; ks < nks; ks++) {
        if (nks - 1 - ks >= NST - 2) vm_wait<PW *(NST - 2)>();
        else vm_wait<0>();
        lds_barrier();
        if (ks + NST - 1 < nks) issue(ks + NST - 1, st == 0 ? NST - 1 : st - 1);
        const char *base = lds + st * STAGE + lane * sizeof(Frag<T>);
        st = st + 1 == NST ? 0 : st + 1;
        Frag<T> b[4];
#pragma unroll
        for (int t = 0; t < 4; t++) b[t] = *reinterpret_cast<const Frag<T> *>(base + (RT + wt * 4 + t) * UNIT);
#pragma unroll
        for (int r = 0; r < RTW; r++) {
            const Frag<T> a = *reinterpret_cast<const Frag<T> *>(base + (wr * RTW + r) * UNIT);
#pragma unroll
            for (int t = 0; t < 4; t++) acc[r][t] = EPI == ST_VALUES ? mma(b[t], a, acc[r][t]) : mma(a, b[t], acc[r][t]);
        }
    }
    if constexpr (EPI == ST_VALUES) {
        // operands the other way round: a lane holds four consecutive keys of one value column, two token tiles are its fragment
        const int tph = P.kr.hrows >> 4;
#pragma unroll
        for (int t = 0; t < 4; t += 2) {
            const int kt = tb * NT + wt * 4 + t;
            if (kt >= ntt) continue;
#pragma unroll
            for (int r = 0; r < RTW; r++) {
                const int rt = rb * RT + wr * RTW + r, h = rt / tph;
                if (rt >= P.nrt) continue;
                T *o = reinterpret_cast<T *>(P.kr.dst) + ((((long long)h * (P.kr.slots >> 5) + (kt >> 1)) * P.kr.nt + rt - h * tph) * 64 + lane) * 8;
                put4(o, acc[r][t]);
                put4(o + 4, acc[r][t + 1]);
            }
        }
        return;
    }
#pragma unroll
    for (int t = 0; t < 4; t++) {
        const int tok = (tb * NT + wt * 4 + t) * 16 + (lane & 15);
        if (tok >= P.n_tokens) continue;
#pragma unroll
        for (int r = 0; r < RTW; r++) {
            const int rt = rb * RT + wr * RTW + r;
            if (rt >= P.nrt) continue;
            const int row = rt * 16 + 4 * g;
            if constexpr (EPI == ST_F32) store_rows(P.out, P.ldo, P.rows, tok, row, with_bias(P.bias, row, acc[r][t]));
            else if constexpr (EPI == ST_HEADS) store_heads<T>(P.hd, tok, row, acc[r][t]);
            else if constexpr (EPI == ST_KEYS) {
                const int h = row / P.kr.hrows;
                put4(reinterpret_cast<T *>(P.kr.dst) + (long long)h * P.kr.slots * P.kr.nt * 32 + op_index(tok, row - h * P.kr.hrows, P.kr.nt), acc[r][t]);
            } else if constexpr (EPI == ST_RESID) add_rows(P.out, P.add2, P.ldo, P.rows, tok, row, acc[r][t]);
            else if constexpr (RTW > 1) {
                if ((r & 1) == 0) store_gated<T>(P, tok, rt >> 1, g, acc[r][t], acc[r + (RTW > 1 ? 1 : 0)][t]);
            }
        }
    }
}

constexpr int FEW_MAX_TOKENS = 64;
constexpr int FEW_NORM_SLOTS = 4;         // (token, 2048 columns) slots up to which few_kernel computes the norm itself

// activations go round the vector L1 (sc1): they are L2-resident and every workgroup streams them once
__device__ __forceinline__ void load_act(Frag<bf16> &f, const __amdgpu_buffer_rsrc_t rs, unsigned byte_off) {
    f.v = __builtin_bit_cast(bf16x8, __builtin_amdgcn_raw_buffer_load_b128(rs, byte_off, 0, 16));
}
__device__ __forceinline__ void load_act(Frag<float> &f, const __amdgpu_buffer_rsrc_t rs, unsigned byte_off) {
    f.a = __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(rs, byte_off, 0, 16));
    f.b = __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(rs, byte_off + 16, 0, 16));
}

// decode batches: one row tile (ST_GATED: a gate and an up tile) x NT token tiles per workgroup, k tiles dealt to its WV wavefronts
// in turn; a round's loads are all in flight together
// NORM: 0 none, 1 norm of nx, 2 norm of nx + norm(nd) ndw; NS: bound of its (token, 2048 columns) slots, four columns per thread and slot
// (kept small: a launch this short is held up by fetching its own instructions)
template <typename T, int EPI, int NT, int WV, int NORM, int NS, class TAIL>
__global__ void __launch_bounds__(WV * 64) few_kernel(MatParams P, TAIL tail) {
    constexpr int RB = EPI == ST_GATED ? 2 : 1;
    constexpr int PRE = (NT == 1 ? 8 : NT == 2 ? 6 : WV == 16 ? 4 : 6) / (sizeof(T) == 4 ? 2 : 1);
    extern __shared__ __align__(16) char lds[];
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, col = lane & 15;
    const int rt = blockIdx.x * RB, tt0 = blockIdx.y * NT, nks = P.nks, n = P.n_tokens;
    if constexpr (TAIL::on)
        if (rt >= P.nrt) {
            const int u = (blockIdx.x - P.nrt / RB) * WV + w;
            if (blockIdx.y == 0 && u < tail.units) tail.unit(u, lane);
            return;
        }
    // NORM: the residual rows are requested ahead of the weights (loads return in order)
    f32x4 xv[NORM ? NS : 1], wv[NORM ? NS : 1], dv[NORM == 2 ? NS : 1], dwv[NORM == 2 ? NS : 1];
    const int ux = NORM && NS > 1 ? (nks * 32 + 2047) >> 11 : 1, nslots = NORM ? (NS == 1 ? 1 : n * ux) : 0;
    if constexpr (NORM) {
        static_assert(WV == 8, "a slot is 512 threads wide");
        int t = 0, u = 0;
#pragma unroll
        for (int s = 0; s < NS; s++)
            if (s < nslots) {
                const int k = u * 2048 + tid * 4;
                const bool in = k < P.ndim;
                if constexpr (NORM == 2) {
                    dv[s] = in ? *reinterpret_cast<const f32x4 *>(P.nd + (long long)t * P.nld + k) : f32x4{};
                    dwv[s] = in ? *reinterpret_cast<const f32x4 *>(P.ndw + k) : f32x4{};
                }
                xv[s] = in ? *reinterpret_cast<const f32x4 *>(P.nx + (long long)t * P.nld + k) : f32x4{};
                wv[s] = in ? *reinterpret_cast<const f32x4 *>(P.nw + k) : f32x4{};
                if (++u == ux) { u = 0; t++; }
            }
    }
    const Frag<T> *W = reinterpret_cast<const Frag<T> *>(P.W) + (long long)rt * nks * 64 + lane;
    const __amdgpu_buffer_rsrc_t X = __builtin_amdgcn_make_buffer_rsrc(const_cast<void *>(P.X), 0, NORM ? 0 : (int)(((n + 15) >> 4) * P.x_nks * OPT * sizeof(T)), 0x00027000);
    const int xk0 = P.group ? rt / P.group * nks : 0;
    f32x4 acc[RB][NT] = {};
    Frag<T> a[RB][PRE], b[PRE][NT];
    auto load = [&](int k0) {
#pragma unroll
        for (int u = 0; u < PRE; u++) {
            const int ks = min(k0 + u * WV, nks - 1);
#pragma unroll
            for (int r = 0; r < RB; r++) a[r][u] = W[((long long)r * nks + ks) * 64];
            if constexpr (!NORM) {
#pragma unroll
                for (int t = 0; t < NT; t++) {
                    frag_zero(b[u][t]);
                    if ((tt0 + t) * 16 + col < n) load_act(b[u][t], X, (unsigned)((((tt0 + t) * P.x_nks + xk0 + ks) * 64 + lane) * 8 * sizeof(T)));
                }
            }
        }
    };
    load(w);
    T *xs = reinterpret_cast<T *>(lds);                    // NORM: [nks][4][n][8]
    if constexpr (NORM) {
        float *red = reinterpret_cast<float *>(lds + (size_t)nks * 32 * n * sizeof(T));      // [NORM][n][WV]
        auto sums = [&](const f32x4 *v, float *to) {         // every wavefront's sums of squares, per token
            int t = 0, u = 0;
            float ss = 0.f;
#pragma unroll
            for (int s = 0; s < NS; s++)
                if (s < nslots) {
                    ss += v[s][0] * v[s][0] + v[s][1] * v[s][1] + v[s][2] * v[s][2] + v[s][3] * v[s][3];
                    if (++u == ux) {
                        ss = wave_sum(ss);
                        if (lane == 0) to[t * WV + w] = ss;
                        ss = 0.f; u = 0; t++;
                    }
                }
            lds_barrier();
        };
        auto inverse = [&](const float *from, int t) {
            const f32x4 q = *reinterpret_cast<const f32x4 *>(from + t * WV) + *reinterpret_cast<const f32x4 *>(from + t * WV + 4);
            return rsqrt_f32(((q[0] + q[1]) + (q[2] + q[3])) / (float)P.ndim + P.neps);
        };
        if constexpr (NORM == 2) {
            float *redd = red + n * WV;
            sums(dv, redd);
            const bool keep = P.nxo && blockIdx.x == 0 && blockIdx.y == 0;
            int t = 0, u = 0;
            float invd = 0.f;
#pragma unroll
            for (int s = 0; s < NS; s++)
                if (s < nslots) {
                    if (u == 0) invd = inverse(redd, t);
                    xv[s] += dv[s] * invd * dwv[s];
                    const int k = u * 2048 + tid * 4;
                    if (keep && k < P.ndim) *reinterpret_cast<f32x4 *>(P.nxo + (long long)t * P.nld + k) = xv[s];
                    if (++u == ux) { u = 0; t++; }
                }
        }
        sums(xv, red);
        int t = 0, u = 0;
        float inv = 0.f;
#pragma unroll
        for (int s = 0; s < NS; s++)
            if (s < nslots) {
                if (u == 0) inv = inverse(red, t);
                const int k = u * 2048 + tid * 4;
                if (k < nks * 32) put4(xs + ((k >> 3) * n + t) * 8 + (k & 7), xv[s] * inv * wv[s]);
                if (++u == ux) { u = 0; t++; }
            }
        lds_barrier();
    }
    for (int k0 = w; k0 < nks; k0 += PRE * WV) {
        if (k0 != w) load(k0);
#pragma unroll
        for (int u = 0; u < PRE; u++) {
            const int ks = k0 + u * WV;
            if (ks >= nks) break;
            if constexpr (NORM) {
                frag_zero(b[u][0]);
                if (col < n) b[u][0] = *reinterpret_cast<const Frag<T> *>(xs + ((ks * 4 + g) * n + col) * 8);
            }
#pragma unroll
            for (int t = 0; t < NT; t++)
#pragma unroll
                for (int r = 0; r < RB; r++) acc[r][t] = mma(a[r][u], b[u][t], acc[r][t]);
        }
    }
    // the wavefronts' partial tiles meet in LDS
    if constexpr (NORM) lds_barrier();                   // (the area held the norm)
    f32x4 *red = reinterpret_cast<f32x4 *>(lds);           // [WV][RB * NT][64]
#pragma unroll
    for (int r = 0; r < RB; r++)
#pragma unroll
        for (int t = 0; t < NT; t++) red[(w * RB * NT + r * NT + t) * 64 + lane] = acc[r][t];
    lds_barrier();
    for (int i = tid; i < NT * 64; i += WV * 64) {
        const int t = i >> 6, l = i & 63, tok = (tt0 + t) * 16 + (l & 15), row = rt * 16 + 4 * (l >> 4);
        f32x4 v[RB] = {};
#pragma unroll
        for (int q = 0; q < WV; q++)
#pragma unroll
            for (int r = 0; r < RB; r++) v[r] += red[(q * RB * NT + r * NT + t) * 64 + l];
        if (EPI == ST_F32 && NT == 1 && P.amax_val) {      // one token: rows of column 0, four lanes with four rows each
            float best = -INFINITY;
            int idx = 0x7fffffff;
            if ((l & 15) == 0)
                for (int j = 0; j < 4; j++)
                    if (row + j < P.rows && v[0][j] > best) { best = v[0][j]; idx = row + j; }
#pragma unroll
            for (int o = 16; o < 64; o <<= 1) {
                const float ov = __shfl_xor(best, o);
                const int oi = __shfl_xor(idx, o);
                if (ov > best || (ov == best && oi < idx)) { best = ov; idx = oi; }
            }
            if (l == 0) { P.amax_val[blockIdx.x] = best; P.amax_idx[blockIdx.x] = idx; }
        }
        if (tok >= n) continue;
        if constexpr (EPI == ST_F32) store_rows(P.out, P.ldo, P.rows, tok, row, with_bias(P.bias, row, v[0]));
        else if constexpr (EPI == ST_HEADS) store_heads<T>(P.hd, tok, row, v[0]);
        else if constexpr (EPI == ST_RESID) add_rows(P.out, P.add2, P.ldo, P.rows, tok, row, v[0]);
        else store_gated<T>(P, tok, rt >> 1, l >> 4, v[0], v[RB - 1]);
    }
}

template <typename T, int EPI, int NT, int WV, int NORM, class TAIL, int NS = 1>
hipError_t launch_few_nt(const MatParams &P, hipStream_t st, TAIL tail) {
    constexpr int RB = EPI == ST_GATED ? 2 : 1;
    const int tt = (P.n_tokens + 15) / 16;
    size_t lds = (size_t)WV * RB * NT * 64 * 16;           // at most 64 KB
    if (NORM) lds = std::max(lds, (size_t)P.nks * 32 * P.n_tokens * sizeof(T) + (size_t)P.n_tokens * WV * 4 * NORM);
    hipLaunchKernelGGL((few_kernel<T, EPI, NT, WV, NORM, NS, TAIL>), dim3(P.nrt / RB + (TAIL::on ? (tail.units + WV - 1) / WV : 0), (tt + NT - 1) / NT), dim3(WV * 64), lds, st, P, tail);
    return hipGetLastError();
}
// is the norm of the product's input (rows of dim values, ld apart) computed inside the launch?
inline int few_norm_slots(int n, int nks) { return n * ((nks * 32 + 2047) / 2048); }
inline bool few_norm_ok(int n, int nks, int dim, int ld) { return few_norm_slots(n, nks) <= FEW_NORM_SLOTS && (dim & 3) == 0 && (ld & 3) == 0; }

template <typename T, int EPI, class TAIL>
hipError_t launch_few(const MatParams &P, hipStream_t st, int norm, TAIL tail) {
    constexpr int RB = EPI == ST_GATED ? 2 : 1;
    const bool one = few_norm_slots(P.n_tokens, P.nks) == 1;
    if constexpr (EPI != ST_HEADS && EPI != ST_RESID)
        if (norm == 2) return one ? launch_few_nt<T, EPI, 1, 8, 2, TAIL, 1>(P, st, tail) : launch_few_nt<T, EPI, 1, 8, 2, TAIL, FEW_NORM_SLOTS>(P, st, tail);
    if constexpr (EPI != ST_RESID)
        if (norm) return one ? launch_few_nt<T, EPI, 1, 8, 1, TAIL, 1>(P, st, tail) : launch_few_nt<T, EPI, 1, 8, 1, TAIL, FEW_NORM_SLOTS>(P, st, tail);
    const int tt = (P.n_tokens + 15) / 16, blocks = P.nrt / RB;
    // few row tiles: sixteen wavefronts to a workgroup, and token tiles on workgroups of their own, until the chip is covered
    const bool deep = RB == 1 && blocks < 256 && P.nks >= 48;
    int nt = tt >= 3 ? 4 : tt;
    while (nt > 1 && blocks * ((tt + nt - 1) / nt) < 192) nt /= 2;
    if constexpr (EPI == ST_HEADS) {
        if (P.nks <= 8) {                                  // (a head's few k tiles)
            if (nt == 1) return launch_few_nt<T, EPI, 1, 4, 0>(P, st, tail);
            if (nt == 2) return launch_few_nt<T, EPI, 2, 4, 0>(P, st, tail);
            return launch_few_nt<T, EPI, 4, 4, 0>(P, st, tail);
        }
    } else if constexpr (RB == 1) {
        if (deep) {
            if (nt == 1) return launch_few_nt<T, EPI, 1, 16, 0>(P, st, tail);
            if (nt == 2) return launch_few_nt<T, EPI, 2, 16, 0>(P, st, tail);
            return launch_few_nt<T, EPI, 4, 16, 0>(P, st, tail);
        }
    }
    if (nt == 1) return launch_few_nt<T, EPI, 1, 8, 0>(P, st, tail);
    if (nt == 2) return launch_few_nt<T, EPI, 2, 8, 0>(P, st, tail);
    return launch_few_nt<T, EPI, 4, 8, 0>(P, st, tail);
}

template <typename T, int EPI, class TAIL = NoTail>
hipError_t launch_many(const MatParams &P, hipStream_t st, TAIL tail = {}) {
    const int ntb = (P.n_tokens + 127) / 128;
    auto go = [&](auto kfn, int rt, int lds) {
        const int total = (P.nrt + rt - 1) / rt * ntb;
        hipLaunchKernelGGL(kfn, dim3((total + 7) / 8 * 8 + (TAIL::on ? (tail.units + 3) / 4 : 0)), dim3(256), lds, st, P, tail);
        return hipGetLastError();
    };
    if ((P.nrt + 7) / 8 * ntb >= 512) return go(many_kernel<T, EPI, 4, TAIL>, 8, ManyGeom<T, 4>::LDS);
    return go(many_kernel<T, EPI, 2, TAIL>, 4, ManyGeom<T, 2>::LDS);
}

// norm: see few_kernel.  A tail rides in decode launches only (launch_few).
template <typename T, int EPI, class TAIL = NoTail>
hipError_t launch_product(MatParams P, hipStream_t st, int norm = 0, TAIL tail = {}) {
    if (P.n_tokens <= 0) return hipSuccess;
    if (!P.x_nks) P.x_nks = P.nks;
    if (!P.nld) P.nld = P.ndim;
    if (P.n_tokens <= FEW_MAX_TOKENS) return launch_few<T, EPI>(P, st, norm, tail);
    return launch_many<T, EPI>(P, st);
}

}  // namespace nl
