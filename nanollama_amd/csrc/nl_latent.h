// nl_latent.h -- latent attention of the layer-stack models: keys and values of all heads are linear images of one latent vector c per
// position, beside a rotated key part r that all heads share:
//
//   score_h(i, j) = scale (qu_h . (Uk_h c_j) + qr_h . r_j)        out_h = sum_j p_h(i, j) Uv_h c_j
//
// softmax over j <= i, optionally with a learned score per head in the denominator alone (sink), optionally a gate sigmoid(g_h) per head.
// The cache holds c and r only.  Scores, softmax and norms are 32-bit; operands are of element type T (nl_mfma.h).
//
// CACHE.  [R / 16][nks tiles][64 lanes][8] per stream: position p is row p % 16 of operand tile row p / 16; columns are c (kvt tiles of
// 32, zero-padded) and r (the remaining tiles).  A layer may read the cache of an earlier one.
//
// PROMPTS expand: keys and values of every head are products of the cache tiles (the cache IS a product's operand) with Uk and Uv, stored
// to scratch in the operand order of win_attn_kernel, which then runs with as many key heads as query heads.  r is copied behind every
// head's key.  2 (dim + rot + vdim) flops per score instead of 2 (2 kv_rank + rot).
//
// DECODE absorbs: qc_h = Uk_h^T qu_h (a product per head), then every head attends the latents themselves,
//   score = scale (qc_h . c_j + qr_h . r_j),    o_h = sum_j p_j c_j,    out_h = Uv_h o_h,
// so a position is read once for all heads.  latent_decode_kernel: one workgroup per (key split, token, 16 heads) -- the heads are the
// columns of the score product, tiles travel through an LDS ring by LDS-DMA, and the second product's A operand is the same tile
// transposed on its way out of LDS.  It leaves (max, sum, unnormalised o) per split; latent_out_kernel merges the splits in the prologue
// of the Uv product and applies sink and gate.
#pragma once
#include "nl_winattn.h"

namespace nl {

constexpr int LT_MAX_TILES = 24;          // k tiles of a cached position (c and r)
constexpr int LT_KEYS = 32;               // keys per stage of the decode launch
constexpr int LT_MAX_SPLITS = 32;

struct LatentParams {
    // store: this step's c and r from the projections
    const float *proj;          // [token][ldp]
    int ldp, off_c, off_r, off_g;
    int kv_rank, rot_dim, pairs, kvt, nks;
    const float *norm;          // [kv_rank]
    float eps;
    const float *rope;          // [position][pairs] cos, sin
    const int *pos, *stream;
    void *cache;                // this layer run, stream 0
    long long stride;           // elements per stream
    // decode
    int heads, dv;
    float scale;
    const void *q;              // [token][heads][nks * 32]
    int nsplit;
    float *part, *ml;           // [token][heads][nsplit][kvt * 32]; [token][heads][nsplit] max, sum (units of log 2)
    const void *W;              // Uv, operand order, tph row tiles per head
    int tph;
    const float *sink;          // [heads] or null
    void *y;
    int y_nks;
};

// one wavefront per token: c = norm(first kv_rank) w, r = rotation of the rest (pairs adjacent), into the cache
template <typename T> struct LatentStore {
    static constexpr bool on = true;
    int units;
    LatentParams P;
    __device__ __forceinline__ void unit(int n, int lane) const {
        const float *src = P.proj + (long long)n * P.ldp;
        const int pos = P.pos[n];
        T *K = reinterpret_cast<T *>(P.cache) + P.stream[n] * P.stride;
        constexpr int NV = LT_MAX_TILES / 2;
        float v[NV], ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            v[i] = lane + 64 * i < P.kv_rank ? src[P.off_c + lane + 64 * i] : 0.f;
            ss += v[i] * v[i];
        }
        const float inv = rsqrt_f32(wave_sum(ss) / (float)P.kv_rank + P.eps);
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int d = lane + 64 * i;
            if (d < P.kvt * 32) put(K + op_index(pos, d, P.nks), d < P.kv_rank ? v[i] * inv * P.norm[d] : 0.f);
        }
        for (int d = lane; d < (P.nks - P.kvt) * 32; d += 64) {
            float o = 0.f;
            if (d < P.rot_dim) {
                o = src[P.off_r + d];
                if (d < 2 * P.pairs) {
                    const float *cs = P.rope + ((long long)pos * P.pairs + (d >> 1)) * 2, other = src[P.off_r + (d ^ 1)];
                    o = d & 1 ? o * cs[0] + other * cs[1] : o * cs[0] - other * cs[1];
                }
            }
            put(K + op_index(pos, P.kvt * 32 + d, P.nks), o);
        }
    }
};

// one wavefront per (key tile of the list, rotated tile): r behind every head's expanded key
template <typename T> struct RotatedKeys {
    static constexpr bool on = true;
    int units;
    const void *cache;
    const int *x_tile;
    int nks, kvt, heads, slots, dt, nt;   // cache tiles and latent tiles per position; scratch: slots, tiles before r, tiles
    void *dst;
    __device__ __forceinline__ void unit(int u, int lane) const {
        const int nr = nks - kvt, t = u / nr, k = u - t * nr;
        const Frag<T> f = reinterpret_cast<const Frag<T> *>(cache)[((long long)x_tile[t] * nks + kvt + k) * 64 + lane];
        for (int h = 0; h < heads; h++) reinterpret_cast<Frag<T> *>(dst)[(((long long)h * (slots >> 4) + t) * nt + dt + k) * 64 + lane] = f;
    }
};

// until at most n (any wave-uniform number; rounded down to what an instruction can say) vector memory operations are in flight
__device__ __forceinline__ void vm_wait_upto(int n) {
    switch (n) {
#define NL_CASE(i) case i: vm_wait<i>(); return;
        NL_CASE(0) NL_CASE(1) NL_CASE(2) NL_CASE(3) NL_CASE(4) NL_CASE(5) NL_CASE(6) NL_CASE(7) NL_CASE(8) NL_CASE(9) NL_CASE(10) NL_CASE(11)
        NL_CASE(12) NL_CASE(13) NL_CASE(14) NL_CASE(15) NL_CASE(16) NL_CASE(17) NL_CASE(18) NL_CASE(19) NL_CASE(20) NL_CASE(21) NL_CASE(22)
        NL_CASE(23) NL_CASE(24)
#undef NL_CASE
    default: vm_wait<24>();
    }
}

// A operand of the value product from two key tiles in LDS (`tile`: bytes of the first one's k tile that holds value tile vt, `next`: from
// there to the second one's): lane (g, c) gets value vt * 16 + c of keys 4 g .. 4 g + 3 of either tile, the accumulator order of two
// score tiles.  bfloat16: ds_read_b64_tr_b16 -- of every 16 lanes, lane i offers 4 values (i % 4) of key i / 4 and receives value i of the 4 keys.
__device__ __forceinline__ Frag<bf16> transposed_frag(const bf16 *tile, int next, int vt, int g, int c) {
    typedef bf16x4 __attribute__((address_space(3))) *LdsPtr;
    const int d = (vt & 1) * 16 + (c & 3) * 4, at = ((d >> 3) * 16 + 4 * g + (c >> 2)) * 8 + (d & 7);
    const bf16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((LdsPtr)(bf16 *)(tile + at)), b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((LdsPtr)(bf16 *)(tile + next + at));
    Frag<bf16> f;
    f.v = __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
    return f;
}
__device__ __forceinline__ Frag<float> transposed_frag(const float *tile, int next, int vt, int g, int c) {
    const int d = (vt & 1) * 16 + c;
    const float *p = tile + ((d >> 3) * 16 + 4 * g) * 8 + (d & 7);
    Frag<float> f;
#pragma unroll
    for (int j = 0; j < 4; j++) { f.a[j] = p[j * 8]; f.b[j] = p[next + j * 8]; }
    return f;
}

constexpr int LT_SC = 36;                 // floats per head of a score buffer (32 keys and a shift of the banks)
template <typename T> inline size_t latent_decode_stage(int nks) { return (size_t)2 * nks * OPT * sizeof(T); }
template <typename T> inline size_t latent_decode_fixed(int nks) { return (size_t)nks * OPT * sizeof(T) + 4 * 16 * LT_SC * 4; }

// grid (key splits, tokens, head tiles); VT: value tiles per wavefront, 4 VT >= 2 kvt; nst: stages of the LDS ring
template <typename T, int VT>
__global__ void __launch_bounds__(256) latent_decode_kernel(LatentParams P, int nst) {
    constexpr int UNIT = OPT * sizeof(T), PK = UNIT / 1024;
    extern __shared__ __align__(16) char lds[];
    const int split = blockIdx.x, n = blockIdx.y, h0 = blockIdx.z * 16, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15;
    const int nks = P.nks, kvt = P.kvt, pieces = 2 * nks * PK, pw = (pieces + 3) / 4, stage = pieces * 1024;
    const int pos = P.pos[n], nb = (pos >> 5) + 1, per = (nb + P.nsplit - 1) / P.nsplit, bf = split * per, bl = min(bf + per, nb);
    const long long row = ((long long)n * P.heads + h0 + c) * P.nsplit + split;
    const bool live = h0 + c < P.heads;
    if (bf >= bl) {
        if (w == 0 && g == 0 && live) { P.ml[row * 2] = -INFINITY; P.ml[row * 2 + 1] = 0.f; }
        return;
    }
    char *ql = lds + nst * stage;
    float *sc = reinterpret_cast<float *>(ql + nks * UNIT);          // [parity][half of the k tiles][16 heads][LT_SC]
    const char *K = reinterpret_cast<const char *>(reinterpret_cast<const T *>(P.cache) + P.stream[n] * P.stride) + lane * 16;
    {
        // the queries as a B operand: 16 bytes per lane and piece, in fragment order
        const T *q = reinterpret_cast<const T *>(P.q) + (long long)n * P.heads * nks * 32;
        for (int u = w; u < nks * PK; u += 4) {
            const int fl = sizeof(T) == 2 ? lane : (u & 1) * 32 + (lane >> 1), k = (u / PK) * 32 + (fl >> 4) * 8 + (sizeof(T) == 2 ? 0 : (lane & 1) * 4);
            lds_dma16(q + (long long)min(h0 + (fl & 15), P.heads - 1) * nks * 32 + k, ql + u * 1024);
        }
    }
    auto issue = [&](int b, int st) {
        const char *src = K + (long long)b * stage;
        for (int i = 0; i < pw; i++) {                               // (the same number for every wavefront: past the end the last piece again)
            const int u = min(i * 4 + w, pieces - 1);
            lds_dma16(src + u * 1024, lds + st * stage + u * 1024);
        }
    };
    for (int i = 0; i < nst - 1; i++)
        if (bf + i < bl) issue(bf + i, i);
    f32x4 o[VT] = {};
    float m = -INFINITY, l = 0.f;
    const float scale = P.scale * LOG2E;
    int st = 0;
    for (int b = bf; b < bl; b++) {
        if (nst == 1) {
            lds_barrier();
            issue(b, 0);
            vm_wait<0>();
            lds_barrier();
        } else {
            vm_wait_upto(pw * min(nst - 2, bl - 1 - b));
            lds_barrier();
            if (b + nst - 1 < bl) issue(b + nst - 1, st == 0 ? nst - 1 : st - 1);
        }
        const char *kb = lds + st * stage;
        st = st + 1 == nst ? 0 : st + 1;
        {
            // scores: a wavefront takes one of the two key tiles and every other k tile
            const int a = w & 1;
            f32x4 s = {};
            for (int k = w >> 1; k < nks; k += 2)
                s = mma(*reinterpret_cast<const Frag<T> *>(kb + (a * nks + k) * UNIT + lane * sizeof(Frag<T>)), *reinterpret_cast<const Frag<T> *>(ql + k * UNIT + lane * sizeof(Frag<T>)), s);
            *reinterpret_cast<f32x4 *>(sc + (((b & 1) * 2 + (w >> 1)) * 16 + c) * LT_SC + a * 16 + 4 * g) = s;
        }
        lds_barrier();
        // every wavefront: the softmax of its 16 heads (a lane has 8 keys of one head), then its own value tiles
        f32x4 s[2];
        float mx = m;
#pragma unroll
        for (int a = 0; a < 2; a++) {
            const float *p = sc + ((b & 1) * 32 + c) * LT_SC + a * 16 + 4 * g;
            s[a] = (*reinterpret_cast<const f32x4 *>(p) + *reinterpret_cast<const f32x4 *>(p + 16 * LT_SC)) * scale;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                if (b * LT_KEYS + a * 16 + 4 * g + i > pos) s[a][i] = -INFINITY;
                mx = fmaxf(mx, s[a][i]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));                          // (finite: key 32 b is visible)
        const float corr = exp2_f32(m - mx);
        m = mx;
        Frag<T> p;
        float add = 0.f;
#pragma unroll
        for (int a = 0; a < 2; a++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float e = exp2_f32(s[a][i] - mx);
                add += e;
                frag_set(p, a * 4 + i, e);
            }
        l = l * corr + add;
#pragma unroll
        for (int t = 0; t < VT; t++) {
            const int vt = w + 4 * t;
            if (vt < 2 * kvt) {
                o[t] *= corr;
                o[t] = mma(transposed_frag(reinterpret_cast<const T *>(kb + (vt >> 1) * UNIT), nks * OPT, vt, g, c), p, o[t]);
            }
        }
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (!live) return;
    if (w == 0 && g == 0) { P.ml[row * 2] = m; P.ml[row * 2 + 1] = l; }
#pragma unroll
    for (int t = 0; t < VT; t++) {
        const int vt = w + 4 * t;
        if (vt < 2 * kvt) *reinterpret_cast<f32x4 *>(P.part + row * kvt * 32 + vt * 16 + 4 * g) = o[t];
    }
}

template <typename T>
hipError_t launch_latent_decode(const LatentParams &P, int n, hipStream_t st) {
    const size_t stage = latent_decode_stage<T>(P.nks), fixed = latent_decode_fixed<T>(P.nks);
    const int nst = (int)std::max<size_t>(1, std::min<size_t>(3, (160 * 1024 - fixed) / stage)), vt = (2 * P.kvt + 3) / 4;
    const size_t lds = nst * stage + fixed;
    auto go = [&](auto kfn) {
        if (lds > 65536)
            if (hipError_t s = hipFuncSetAttribute(reinterpret_cast<const void *>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)) return s;
        hipLaunchKernelGGL(kfn, dim3(P.nsplit, n, (P.heads + 15) / 16), dim3(256), lds, st, P, nst);
        return hipGetLastError();
    };
    if (vt <= 2) return go(latent_decode_kernel<T, 2>);
    if (vt <= 4) return go(latent_decode_kernel<T, 4>);
    if (vt <= 8) return go(latent_decode_kernel<T, 8>);
    return go(latent_decode_kernel<T, 12>);
}

// grid (row tiles of Uv / RB, token tiles): merges the splits of one head for 16 tokens, multiplies, gates, stores y's columns
template <typename T, int RB>
__global__ void __launch_bounds__(256) latent_out_kernel(LatentParams P, int n_tokens) {
    constexpr int NK = LT_MAX_TILES / 4;
    extern __shared__ __align__(16) char lds[];
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15, kvt = P.kvt, ns = P.nsplit;
    const int per = (P.tph + RB - 1) / RB, h = blockIdx.x / per, r0 = (blockIdx.x - h * per) * RB, n0 = blockIdx.y * 16, nt = min(16, n_tokens - n0);
    const Frag<T> *W = reinterpret_cast<const Frag<T> *>(P.W) + (long long)(h * P.tph) * kvt * 64 + lane;
    Frag<T> a[NK];
    auto load = [&](int r) {                               // (row tiles past the head's end repeat its last one)
#pragma unroll
        for (int i = 0; i < NK; i++)
            if (w + 4 * i < kvt) a[i] = W[((long long)min(r0 + r, P.tph - 1) * kvt + w + 4 * i) * 64];
    };
    load(0);
    float *wt = reinterpret_cast<float *>(lds);            // [16][ns]
    T *xs = reinterpret_cast<T *>(lds + ((16 * ns * 4 + 15) & ~15));        // [kvt][4][16 tokens][8]
    f32x4 *red = reinterpret_cast<f32x4 *>(reinterpret_cast<char *>(xs) + kvt * OPT * sizeof(T));    // [4][RB][64]
    {
        const int t = tid >> 4, j = tid & 15;
        const float sk = P.sink ? P.sink[h] * LOG2E : -INFINITY;
        const float *ml = P.ml + ((long long)(n0 + min(t, nt - 1)) * P.heads + h) * ns * 2;
        float mm = -INFINITY, den = 0.f;
        for (int s = j; s < ns; s += 16) mm = fmaxf(mm, ml[s * 2]);
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
        mm = fmaxf(mm, sk);
        for (int s = j; s < ns; s += 16) den += ml[s * 2 + 1] * exp2_f32(ml[s * 2] - mm);
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) den += __shfl_xor(den, o);
        const float inv = 1.f / (den + exp2_f32(sk - mm));
        for (int s = j; s < ns; s += 16) wt[t * ns + s] = exp2_f32(ml[s * 2] - mm) * inv;
    }
    lds_barrier();
    for (int i = tid; i < nt * kvt * 8; i += 256) {
        const int t = i / (kvt * 8), d = (i - t * kvt * 8) * 4;
        const float *p = P.part + ((long long)(n0 + t) * P.heads + h) * ns * kvt * 32 + d;
        f32x4 v = {};
        for (int s0 = 0; s0 < ns; s0 += 8) {
            f32x4 x[8];
#pragma unroll
            for (int s = 0; s < 8; s++) x[s] = *reinterpret_cast<const f32x4 *>(p + (long long)min(s0 + s, ns - 1) * kvt * 32);
#pragma unroll
            for (int s = 0; s < 8; s++)
                if (s0 + s < ns) {
                    const float f = wt[t * ns + s0 + s];   // (an empty split left no values behind)
                    if (f != 0.f) v += f * x[s];
                }
        }
        put4(xs + ((d >> 3) * 16 + t) * 8 + (d & 7), v);
    }
    lds_barrier();
    f32x4 acc[RB] = {};
#pragma unroll
    for (int r = 0; r < RB; r++) {
#pragma unroll
        for (int i = 0; i < NK; i++)
            if (w + 4 * i < kvt) {
                Frag<T> b;
                frag_zero(b);
                if (c < nt) b = *reinterpret_cast<const Frag<T> *>(xs + (((w + 4 * i) * 4 + g) * 16 + c) * 8);
                acc[r] = mma(a[i], b, acc[r]);
            }
        if (r + 1 < RB) load(r + 1);
    }
#pragma unroll
    for (int r = 0; r < RB; r++) red[(w * RB + r) * 64 + lane] = acc[r];
    lds_barrier();
    for (int i = tid; i < RB * 64; i += 256) {
        const int r = i >> 6, l = i & 63, tok = n0 + (l & 15), d = (r0 + r) * 16 + 4 * (l >> 4), k = h * P.dv + d;
        if ((l & 15) >= nt || r0 + r >= P.tph) continue;
        f32x4 v = red[r * 64 + l] + red[(RB + r) * 64 + l] + red[(2 * RB + r) * 64 + l] + red[(3 * RB + r) * 64 + l];
        if (P.off_g >= 0) v *= sigmoid_f32(P.proj[(long long)tok * P.ldp + P.off_g + h]);
        T *y = reinterpret_cast<T *>(P.y);
        if (d + 3 < P.dv && (k & 3) == 0) put4(y + op_index(tok, k, P.y_nks), v);
        else
            for (int x = 0; x < 4; x++)
                if (d + x < P.dv) put(y + op_index(tok, k + x, P.y_nks), v[x]);
    }
}

template <typename T>
hipError_t launch_latent_out(const LatentParams &P, int n, hipStream_t st) {
    const int tt = (n + 15) / 16;
    auto go = [&](auto kfn, int rb) {
        const size_t lds = ((16 * P.nsplit * 4 + 15) & ~15) + (size_t)P.kvt * OPT * sizeof(T) + 4 * rb * 64 * 16;
        if (lds > 65536)
            if (hipError_t s = hipFuncSetAttribute(reinterpret_cast<const void *>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)) return s;
        hipLaunchKernelGGL(kfn, dim3(P.heads * ((P.tph + rb - 1) / rb), tt), dim3(256), lds, st, P, n);
        return hipGetLastError();
    };
    // few tokens: a row tile per workgroup; many: the merged head serves several of them
    return P.tph >= 2 && P.heads * ((P.tph + 3) / 4) * tt >= 128 ? go(latent_out_kernel<T, 4>, 4) : go(latent_out_kernel<T, 1>, 1);
}

}  // namespace nl
