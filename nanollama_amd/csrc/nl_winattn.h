// nl_winattn.h -- grouped-query softmax attention of the layer-stack models: optional per-head RMS norm of queries and keys, a
// linear distance bias slope_h (i - j), an optional sliding window (keys i - window < j <= i), an optional learned score per head in
// the denominator alone (prompts), an output gate sigmoid(g) per value or per head; query / key and value sizes may differ.  Scores, softmax and the norms are 32-bit; keys, values and the softmax
// weights are operands of element type T (nl_mfma.h).
//
// CACHE.  A ring of R positions per (stream, kv head), position p in slot p % R, R a multiple of 64 and at least window - 1 + the
// tokens a step may add, so that a step may write all its keys first and attend afterwards.  Both halves lie in MFMA operand
// order, because both passes read them as the A operand:
//   K  [R / 16][dim tiles of 32][64 lanes][8]       lane = dim-run * 16 + slot % 16                       (scores^T = K q^T)
//   V  [R / 32][value tiles of 16][64 lanes][8]     lane = (slot % 16) / 4 * 16 + value % 16,
//                                                   element j = slot / 16 % 2 * 4 + slot % 4              (out^T = V^T p^T)
// The V order is the accumulator order of two 16-key score tiles, so the softmax weights become the second product's B operand
// without leaving their lanes.  Reset is O(1): slots of another request are never visible (the mask is by position).
//
// PROMPTS: win_prep_kernel (norms, ring store, queries), win_attn_kernel (64 queries x one head per workgroup, keys and values
// through LDS by LDS-DMA, a ring of stages).  DECODE: mix_decode_kernel -- attention heads (optionally split over key ranges, the
// last split to arrive merges) and the linear-attention heads of a parallel layer in one launch.
#pragma once
#include "nl_linattn.h"

namespace nl {

constexpr int WA_Q = 64;                  // queries per workgroup
constexpr int WA_MAX_DIM = 256;
constexpr int WA_SPLIT_KEYS = 2048;       // keys one split of the decode launch can hold

// queries [tok0, tok0 + nq) of the step, first one at position pos0; position p is in slot (key0 + p) % R
struct WinTile { int tok0, nq, pos0, stream, key0; };

struct WinParams {
    const float *proj;          // [token][ldp]
    int ldp, off_q, off_k, off_v, off_g;
    int heads, kv_heads, dk, dv;
    int nks, nvt;               // key tiles of 32, value tiles of 16
    const float *qnorm, *knorm; // [dk] or null
    float eps, scale, oscale;
    const float *slope, *sink;  // [heads] or null
    int head_gate;              // the gate is one value per head
    int window, R;              // window 0: everything
    void *K, *V;                // this layer run, stream 0
    long long kstride, vstride; // elements per stream
    void *q;                    // [token][heads][nks * 32]
    void *y;
    int y_nks, y_k0;
    const WinTile *tiles;
    // token arrays (prompts: of the step, decode: of the batch)
    const int *pos, *stream;
    // decode
    int nsplit;
    float *part;                // [token][heads][nsplit][dv + 2]
    unsigned *arrived;          // [token][heads], zero between launches
};

template <typename T> __device__ __forceinline__ T *ring_k(const WinParams &P, int stream, int g) {
    return reinterpret_cast<T *>(P.K) + stream * P.kstride + (long long)g * P.R * P.nks * 32;
}
template <typename T> __device__ __forceinline__ T *ring_v(const WinParams &P, int stream, int g) {
    return reinterpret_cast<T *>(P.V) + stream * P.vstride + (long long)g * P.R * P.nvt * 16;
}
__device__ __forceinline__ long long ring_k_at(int slot, int d, int nks) { return op_index(slot, d, nks); }
__device__ __forceinline__ long long ring_v_at(int slot, int d, int nvt) {
    return (((long long)(slot >> 5) * nvt + (d >> 4)) * 64 + ((slot & 15) >> 2) * 16 + (d & 15)) * 8 + ((slot & 31) >> 4) * 4 + (slot & 3);
}

// one wavefront per (token, head of q | k | v)
template <typename T>
__global__ void __launch_bounds__(256) win_prep_kernel(WinParams P) {
    const int n = blockIdx.x, u = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (u >= P.heads + 2 * P.kv_heads) return;
    const float *pr = P.proj + (long long)n * P.ldp;
    if (u >= P.heads + P.kv_heads) {
        const int g = u - P.heads - P.kv_heads, slot = P.pos[n] % P.R;
        T *V = ring_v<T>(P, P.stream[n], g);
        for (int d = lane; d < P.dv; d += 64) put(V + ring_v_at(slot, d, P.nvt), pr[P.off_v + g * P.dv + d]);
        return;
    }
    const bool isq = u < P.heads;
    const float *src = pr + (isq ? P.off_q + u * P.dk : P.off_k + (u - P.heads) * P.dk), *nw = isq ? P.qnorm : P.knorm;
    float v[WA_MAX_DIM / 64], ss = 0.f;
#pragma unroll
    for (int i = 0; i < WA_MAX_DIM / 64; i++) {
        v[i] = lane + 64 * i < P.dk ? src[lane + 64 * i] : 0.f;
        ss += v[i] * v[i];
    }
    const float inv = nw ? rsqrt_f32(wave_sum(ss) / (float)P.dk + P.eps) : 1.f;
    T *q = reinterpret_cast<T *>(P.q) + ((long long)n * P.heads + u) * P.nks * 32;
    T *K = isq ? nullptr : ring_k<T>(P, P.stream[n], u - P.heads);
    const int slot = isq ? 0 : P.pos[n] % P.R;
#pragma unroll
    for (int i = 0; i < WA_MAX_DIM / 64; i++) {
        const int d = lane + 64 * i;
        if (d >= P.nks * 32) break;
        const float o = d < P.dk ? v[i] * inv * (nw ? nw[d] : 1.f) : 0.f;
        if (isq) put(q + d, o);
        else put(K + ring_k_at(slot, d, P.nks), o);
    }
}

// scores live in units of log 2: 2^x is one instruction
__device__ __forceinline__ float exp2_f32(float x) { return __builtin_amdgcn_exp2f(x); }
constexpr float LOG2E = 1.4426950408889634f;

// keys per stage, 1 KiB pieces a wavefront fetches per stage, stages in the LDS ring, for at most NK key tiles and NV value tiles
template <typename T, int NK, int NV> struct WinGeom {
    static constexpr int KT = sizeof(T) == 2 ? 64 : 32, PW = ((KT / 16 * NK + KT / 32 * NV) * (int)sizeof(T) / 2 + 3) / 4, NST = PW <= 4 ? 4 : PW <= 8 ? 3 : 2;
};

// tiles x heads workgroups.  FULL: nks and nvt are NK and NV, else bounded by them.  Workgroups b, b + 8, ... run on one XCD: every XCD
// takes a contiguous range of (head, tile), so that a head's keys stay in one L2, long tiles (late ones) beside short ones.
template <typename T, int NK, int NV, bool FULL>
__global__ void __launch_bounds__(256) win_attn_kernel(WinParams P, int ntiles) {
    using G = WinGeom<T, NK, NV>;
    constexpr int KT = G::KT, UNIT = OPT * sizeof(T), NST = G::NST, PW = G::PW;
    extern __shared__ __align__(16) char lds[];
    const int total = ntiles * P.heads, per = (total + 7) / 8, id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || id >= total) return;
    const int h = id / ntiles, ti = id - h * ntiles;
    const WinTile tl = P.tiles[ti & 1 ? ti >> 1 : ntiles - 1 - (ti >> 1)];
    const int gk = h / (P.heads / P.kv_heads), tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15;
    const int nks = FULL ? NK : P.nks, nvt = FULL ? NV : P.nvt, qi = w * 16 + c, tok = tl.tok0 + min(qi, tl.nq - 1), qpos = tl.pos0 + min(qi, tl.nq - 1);
    const int win = P.window > 0 ? P.window : 0x7fffffff;
    Frag<T> qf[NK];
    {
        const T *q = reinterpret_cast<const T *>(P.q) + ((long long)tok * P.heads + h) * nks * 32 + g * 8;
#pragma unroll
        for (int k = 0; k < NK; k++)
            if (FULL || k < nks) qf[k] = *reinterpret_cast<const Frag<T> *>(q + k * 32);
    }
    const char *K = reinterpret_cast<const char *>(ring_k<T>(P, tl.stream, gk)), *V = reinterpret_cast<const char *>(ring_v<T>(P, tl.stream, gk));
    const int kpieces = KT / 16 * nks * (UNIT / 1024), vpieces = KT / 32 * nvt * (UNIT / 1024), stage = (kpieces + vpieces) * 1024;
    const int jhi = tl.pos0 + tl.nq - 1, jlo = max(0, tl.pos0 - win + 1), j0 = jlo / KT * KT;
    // queries of this wavefront: none of them sees keys outside [wlo, whi]
    const int wq = min(w * 16, tl.nq - 1), whi = tl.pos0 + min(w * 16 + 15, tl.nq - 1), wq0 = tl.pos0 + wq, wlo = max(0, wq0 - win + 1);
    auto issue = [&](int j, int st) {
        const int slot = (tl.key0 + j) % P.R;            // R is a multiple of KT: a tile of keys is one contiguous run
        const char *ks = K + (long long)(slot >> 4) * nks * UNIT + lane * 16, *vs = V + (long long)(slot >> 5) * nvt * UNIT + lane * 16;
#pragma unroll
        for (int i = 0; i < PW; i++) {                   // (the same number for every wavefront: pieces past the end repeat the last one)
            const int u = FULL && PW * 4 == (KT / 16 * NK + KT / 32 * NV) * (UNIT / 1024) ? i * 4 + w : min(i * 4 + w, kpieces + vpieces - 1);
            lds_dma16(u < kpieces ? ks + u * 1024 : vs + (u - kpieces) * 1024, lds + st * stage + u * 1024);
        }
    };
    f32x4 o[NV] = {};
    float m = -INFINITY, l = 0.f;
    const float scale = P.scale * LOG2E, slope = P.slope ? P.slope[h] * LOG2E : 0.f;
    float off[KT / 16][4];                               // slope * (key's place in the tile)
#pragma unroll
    for (int a = 0; a < KT / 16; a++)
#pragma unroll
        for (int i = 0; i < 4; i++) off[a][i] = slope * (float)(a * 16 + 4 * g + i);
#pragma unroll
    for (int i = 0; i < NST - 1; i++)
        if (j0 + i * KT <= jhi) issue(j0 + i * KT, i);
    int st = NST - 1;
    for (int j = j0; j <= jhi; j += KT) {
        if (jhi - j >= (NST - 2) * KT) vm_wait<PW *(NST - 2)>();
        else vm_wait<0>();
        lds_barrier();
        if (j + (NST - 1) * KT <= jhi) issue(j + (NST - 1) * KT, st);
        st = st + 1 == NST ? 0 : st + 1;                 // (now the current tile's stage)
        if (j > whi || j + KT - 1 < wlo) continue;       // (every wavefront meets the barrier of every tile)
        const char *kb = lds + st * stage, *vb = kb + kpieces * 1024;
        f32x4 s[KT / 16] = {};
#pragma unroll
        for (int k = 0; k < NK; k++)
            if (FULL || k < nks) {
#pragma unroll
                for (int a = 0; a < KT / 16; a++)
                    s[a] = mma(*reinterpret_cast<const Frag<T> *>(kb + (a * nks + k) * UNIT + lane * sizeof(Frag<T>)), qf[k], s[a]);
            }
        const float away = slope * (float)(qpos - j);
        float mx = m;
        if (j + KT - 1 <= wq0 && j >= whi - win + 1) {   // every query of the wavefront sees every key of the tile
#pragma unroll
            for (int a = 0; a < KT / 16; a++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    s[a][i] = fmaf(s[a][i], scale, off[a][i] - away);
                    mx = fmaxf(mx, s[a][i]);
                }
        } else {
#pragma unroll
            for (int a = 0; a < KT / 16; a++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int dist = qpos - (j + a * 16 + 4 * g + i);
                    s[a][i] = dist >= 0 && dist < win ? fmaf(s[a][i], scale, off[a][i] - away) : -INFINITY;
                    mx = fmaxf(mx, s[a][i]);
                }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float base = mx == -INFINITY ? 0.f : mx, corr = exp2_f32(m - base);
        m = mx;
        float add = 0.f;
        Frag<T> p[KT / 32];
#pragma unroll
        for (int a = 0; a < KT / 16; a++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float e = exp2_f32(s[a][i] - base);
                add += e;
                frag_set(p[a >> 1], (a & 1) * 4 + i, e);
            }
        l = l * corr + add;
#pragma unroll
        for (int t = 0; t < NV; t++)
            if (FULL || t < nvt) {
                o[t] *= corr;
#pragma unroll
                for (int b = 0; b < KT / 32; b++)
                    o[t] = mma(*reinterpret_cast<const Frag<T> *>(vb + (b * nvt + t) * UNIT + lane * sizeof(Frag<T>)), p[b], o[t]);
            }
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (qi >= tl.nq) return;
    float inv = P.oscale / l;
    if (P.sink) {
        const float sk = P.sink[h] * LOG2E, mm = fmaxf(m, sk), f = exp2_f32(m - mm);
        inv = P.oscale * f / (l * f + exp2_f32(sk - mm));
    }
    T *y = reinterpret_cast<T *>(P.y);
    const float *gz = P.proj + (long long)tok * P.ldp + P.off_g + (P.head_gate ? h : h * P.dv);
    const int gs = P.head_gate ? 0 : 1;
#pragma unroll
    for (int t = 0; t < NV; t++)
        if (FULL || t < nvt) {
            const int d = t * 16 + 4 * g, k = P.y_k0 + h * P.dv + d;
            if (d + 3 < P.dv && (k & 3) == 0) {
                f32x4 r;
#pragma unroll
                for (int i = 0; i < 4; i++) r[i] = o[t][i] * inv * (P.off_g < 0 ? 1.f : sigmoid_f32(gz[(d + i) * gs]));
                put4(y + op_index(tok, k, P.y_nks), r);
            } else
                for (int i = 0; i < 4; i++)
                    if (d + i < P.dv) put(y + op_index(tok, k + i, P.y_nks), o[t][i] * inv * (P.off_g < 0 ? 1.f : sigmoid_f32(gz[(d + i) * gs])));
        }
}

// --------------------------------------------------------------- decode ---

__host__ __device__ inline size_t win_decode_lds(int nks, int nvt) {
    return (size_t)(2 * nks * 32 + 2 * nvt * 16 + WA_SPLIT_KEYS + 64 + 16) * 4;
}

// one (head, key split, token of the batch) by a workgroup of 256; nks <= M.  The ring's first round of keys (TB tiles of 16 per
// wavefront) and values (VB blocks of 32) is requested before the norms: a split of 16 TB * 4 keys is one memory round trip.
template <typename T, int M>
__device__ __forceinline__ void win_decode_block(const WinParams &P, int h, int split, int n, int stream, int pos, char *lds) {
    constexpr int W = sizeof(T) == 2 ? 8 : 4, TB = W / M > 0 ? W / M : 1, VB = W;
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15, dk = P.dk, dv = P.dv, nks = P.nks, nvt = P.nvt;
    const int gq = P.heads / P.kv_heads, gk = h / gq;
    float *qn = reinterpret_cast<float *>(lds), *kn = qn + nks * 32, *vn = kn + nks * 32, *os = vn + nvt * 16, *sc = os + nvt * 16, *red = sc + WA_SPLIT_KEYS + 64;
    const float *pr = P.proj + (long long)n * P.ldp;
    const int win = P.window > 0 ? P.window : 0x7fffffff, lo = max(0, pos - win + 1);
    // the split's blocks of 32 keys, at most WA_SPLIT_KEYS / 32 + 2 of them; the last block holds the new position
    const int b0 = lo >> 5, nb = (pos >> 5) - b0 + 1, per = (nb + P.nsplit - 1) / P.nsplit, bf = b0 + split * per, bl = min(bf + per, b0 + nb);
    const bool newest = bf < bl && bl == b0 + nb;
    T *K = ring_k<T>(P, stream, gk), *V = ring_v<T>(P, stream, gk);
    const Frag<T> *Kf = reinterpret_cast<const Frag<T> *>(K) + lane, *Vf = reinterpret_cast<const Frag<T> *>(V) + lane;
    // wavefront 0 the query, wavefront 1 the new key, the others the new value
    float v[WA_MAX_DIM / 64], nv[WA_MAX_DIM / 64];
    const float *nw = w == 0 ? P.qnorm : P.knorm;
    if (w < 2) {
        const float *src = pr + (w == 0 ? P.off_q + h * dk : P.off_k + gk * dk);
#pragma unroll
        for (int i = 0; i < WA_MAX_DIM / 64; i++) {
            const bool in = lane + 64 * i < dk;
            v[i] = in ? src[lane + 64 * i] : 0.f;
            nv[i] = in && nw ? nw[lane + 64 * i] : 1.f;
        }
    } else {
#pragma unroll
        for (int i = 0; i < WA_MAX_DIM / 128; i++) v[i] = tid - 128 + 128 * i < dv ? pr[P.off_v + gk * dv + tid - 128 + 128 * i] : 0.f;
    }
    const float gate = P.off_g >= 0 && tid < dv ? pr[P.off_g + h * dv + tid] : 0.f;      // (dv <= 256)
    Frag<T> kf[TB][M], vf[VB];
    auto load_keys = [&](int t0) {                       // tiles t0, t0 + 4, ...
#pragma unroll
        for (int i = 0; i < TB; i++)
#pragma unroll
            for (int k = 0; k < M; k++)
                if (t0 + 4 * i < 2 * bl && k < nks) kf[i][k] = Kf[(long long)(((t0 + 4 * i) * 16 % P.R >> 4) * nks + k) * 64];
    };
    auto load_values = [&](int t, int bb) {
#pragma unroll
        for (int i = 0; i < VB; i++)
            if (bb + i < bl) vf[i] = Vf[(long long)(((bb + i) * 32 % P.R >> 5) * nvt + t) * 64];
    };
    const int kt0 = 2 * bf + w;
    load_keys(kt0);
    if (w < nvt) load_values(w, bf);
    if (w < 2) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < WA_MAX_DIM / 64; i++) ss += v[i] * v[i];
        const float inv = nw ? rsqrt_f32(wave_sum(ss) / (float)dk + P.eps) : 1.f;
#pragma unroll
        for (int i = 0; i < WA_MAX_DIM / 64; i++) {
            const int d = lane + 64 * i;
            if (d < nks * 32) (w == 0 ? qn : kn)[d] = d < dk ? v[i] * inv * nv[i] : 0.f;
        }
    } else {
#pragma unroll
        for (int i = 0; i < WA_MAX_DIM / 128; i++)
            if (tid - 128 + 128 * i < dv) vn[tid - 128 + 128 * i] = v[i];
    }
    lds_barrier();
    if (newest && h % gq == 0) {
        const int slot = pos % P.R;
        for (int d = tid; d < nks * 32; d += 256) put(K + ring_k_at(slot, d, nks), kn[d]);
        for (int d = tid; d < dv; d += 256) put(V + ring_v_at(slot, d, nvt), vn[d]);
    }
    const float slope = P.slope ? P.slope[h] : 0.f;
    float mx = -INFINITY;
    for (int t0 = kt0; t0 < 2 * bl; t0 += 4 * TB) {
        if (t0 != kt0) load_keys(t0);
        float dot[TB] = {};
#pragma unroll
        for (int k = 0; k < M; k++)
            if (k < nks) {
                const f32x4 q0 = *reinterpret_cast<const f32x4 *>(qn + k * 32 + g * 8), q1 = *reinterpret_cast<const f32x4 *>(qn + k * 32 + g * 8 + 4);
#pragma unroll
                for (int i = 0; i < TB; i++)
#pragma unroll
                    for (int x = 0; x < 4; x++) dot[i] = fmaf(frag_get(kf[i][k], 4 + x), q1[x], fmaf(frag_get(kf[i][k], x), q0[x], dot[i]));
            }
#pragma unroll
        for (int i = 0; i < TB; i++) {
            const int t = t0 + 4 * i, j = t * 16 + c;
            if (t >= 2 * bl) break;
            if (j == pos) {                              // the new key: from this step's projection, not from the ring
                dot[i] = 0.f;
                for (int x = g * 8; x < nks * 32; x += 32)
#pragma unroll
                    for (int y = 0; y < 8; y++) dot[i] = fmaf(kn[x + y], qn[x + y], dot[i]);
            }
            dot[i] += __shfl_xor(dot[i], 16);
            dot[i] += __shfl_xor(dot[i], 32);
            const float s = j >= lo && j <= pos ? dot[i] * P.scale - slope * (float)(pos - j) : -INFINITY;
            if (g == 0) sc[j - bf * 32] = s;
            mx = fmaxf(mx, s);
        }
    }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    if (lane == 0) red[w] = mx;
    lds_barrier();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float base = mx == -INFINITY ? 0.f : mx;
    float sum = 0.f;
    for (int i = tid; i < (bl - bf) * 32; i += 256) {
        const float e = sc[i] == -INFINITY ? 0.f : exp_f32(sc[i] - base);
        sc[i] = e;
        sum += e;
    }
    sum = wave_sum(sum);
    if (lane == 0) red[4 + w] = sum;
    lds_barrier();
    sum = red[4] + red[5] + red[6] + red[7];
    const float pnew = newest ? sc[pos - bf * 32] : 0.f;
    // values: a wavefront per tile of 16, lane (value c, key group g)
    for (int t = w; t < nvt; t += 4) {
        float a = 0.f;
        for (int bb = bf; bb < bl; bb += VB) {
            if (t != w || bb != bf) load_values(t, bb);
#pragma unroll
            for (int i = 0; i < VB; i++) {
                if (bb + i >= bl) break;
                const f32x4 p0 = *reinterpret_cast<const f32x4 *>(sc + (bb + i - bf) * 32 + g * 4), p1 = *reinterpret_cast<const f32x4 *>(sc + (bb + i - bf) * 32 + g * 4 + 16);
                const int jb = (bb + i) * 32 + g * 4;
#pragma unroll
                for (int x = 0; x < 4; x++) {
                    // keys outside the window weigh 0; the new key's value comes from this step's projection, not from the ring
                    const float v0 = jb + x == pos ? 0.f : frag_get(vf[i], x), v1 = jb + 16 + x == pos ? 0.f : frag_get(vf[i], 4 + x);
                    a = fmaf(p1[x], v1, fmaf(p0[x], v0, a));
                }
            }
        }
        a += __shfl_xor(a, 16);
        a += __shfl_xor(a, 32);
        if (g == 0) os[t * 16 + c] = t * 16 + c < dv ? a + (newest ? pnew * vn[t * 16 + c] : 0.f) : 0.f;
    }
    lds_barrier();
    T *y = reinterpret_cast<T *>(P.y);
    auto finish = [&](float val) {                       // value column tid
        put(y + op_index(n, P.y_k0 + h * dv + tid, P.y_nks), val * (P.off_g < 0 ? 1.f : sigmoid_f32(gate)) * P.oscale);
    };
    if (P.nsplit == 1) {
        if (tid < dv) finish(os[tid] / sum);
        return;
    }
    // Several splits: every one leaves (max, sum, unnormalised values); the last to arrive merges, nobody waits.  Everything that
    // crosses workgroups goes by agent-scope accesses (past the XCD's own L2), so "stored" is the wavefront's own counter at zero:
    // no cache is written back.
    float *mine = P.part + (((long long)n * P.heads + h) * P.nsplit + split) * (dv + 2);
    if (tid < dv) __hip_atomic_store(mine + 2 + tid, os[tid], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (tid == 0) {
        __hip_atomic_store(mine, mx, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(mine + 1, sum, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    vm_wait<0>();
    lds_barrier();
    unsigned *arr = P.arrived + n * P.heads + h;
    unsigned *last = reinterpret_cast<unsigned *>(red + 8);
    if (tid == 0) *last = __hip_atomic_fetch_add(arr, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    lds_barrier();
    if (*last + 1 != (unsigned)P.nsplit) return;
    const float *all = P.part + ((long long)n * P.heads + h) * P.nsplit * (dv + 2);
    auto rd = [&](int s, int i) { return __hip_atomic_load(all + (long long)s * (dv + 2) + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); };
    // every wavefront: the splits' weights, a lane per split (sc: weights; a workgroup's splits fit it)
    float gm = -INFINITY;
    for (int s = lane; s < P.nsplit; s += 64) gm = fmaxf(gm, rd(s, 0));
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) gm = fmaxf(gm, __shfl_xor(gm, o));
    float den = 0.f;
    for (int s = lane; s < P.nsplit; s += 64) {
        const float m = rd(s, 0), f = m == -INFINITY ? 0.f : exp_f32(m - gm);
        den += f * rd(s, 1);
        if (w == 0) sc[s] = f;
    }
    den = wave_sum(den);
    lds_barrier();
    if (tid < dv) {
        float a = 0.f;
        for (int s0 = 0; s0 < P.nsplit; s0 += 8) {
            float x[8];
#pragma unroll
            for (int i = 0; i < 8; i++) x[i] = rd(min(s0 + i, P.nsplit - 1), 2 + tid);
#pragma unroll
            for (int i = 0; i < 8; i++)
                if (s0 + i < P.nsplit) a = fmaf(sc[s0 + i], x[i], a);
        }
        finish(a / den);
    }
    if (tid == 0) __hip_atomic_store(arr, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}

// a decode batch's mixers: grid (attention heads x splits + linear-attention heads, tokens)
template <typename T, int M>
__global__ void __launch_bounds__(256) mix_decode_kernel(WinParams A, GlaParams L) {
    extern __shared__ __align__(16) char lds[];
    const int n = blockIdx.y, pos = A.pos[n], stream = A.stream[n], na = M ? A.heads * A.nsplit : 0;
    if constexpr (M > 0) {
        if ((int)blockIdx.x < na) {
            win_decode_block<T, M>(A, blockIdx.x / A.nsplit, blockIdx.x % A.nsplit, n, stream, pos, lds);
            return;
        }
    }
    gla_decode_block<T>(L, blockIdx.x - na, n, stream, pos, lds);
}

template <typename T>
hipError_t launch_mix_decode(const WinParams &A, const GlaParams &L, int n, hipStream_t st) {
    size_t lds = 0;
    if (A.heads) lds = win_decode_lds(A.nks, A.nvt);
    if (L.heads) lds = std::max(lds, gla_decode_lds(L.dkp, L.dvp, L.rank));
    auto go = [&](auto kfn) {
        hipLaunchKernelGGL(kfn, dim3(A.heads * A.nsplit + L.heads, n), dim3(256), lds, st, A, L);
        return hipGetLastError();
    };
    if (!A.heads) return go(mix_decode_kernel<T, 0>);
    if (A.nks <= 2) return go(mix_decode_kernel<T, 2>);
    if (A.nks <= 4) return go(mix_decode_kernel<T, 4>);
    return go(mix_decode_kernel<T, 8>);
}

template <typename T>
hipError_t launch_win_prep(const WinParams &P, int n_tokens, hipStream_t st) {
    hipLaunchKernelGGL(win_prep_kernel<T>, dim3(n_tokens, (P.heads + 2 * P.kv_heads + 3) / 4), dim3(256), 0, st, P);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_win_attn(const WinParams &P, int ntiles, hipStream_t st) {
    const size_t stage = (size_t)((sizeof(T) == 2 ? 4 : 2) * P.nks + (sizeof(T) == 2 ? 2 : 1) * P.nvt) * OPT * sizeof(T);
    auto go = [&](auto kfn, int stages) {
        const size_t lds = stages * stage;
        // (more than 64 KB of LDS needs the attribute; cheap enough to set at every such launch)
        if (lds > 65536)
            if (hipError_t s = hipFuncSetAttribute(reinterpret_cast<const void *>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)) return s;
        hipLaunchKernelGGL(kfn, dim3((ntiles * P.heads + 7) / 8 * 8), dim3(256), lds, st, P, ntiles);
        return hipGetLastError();
    };
    const int k = P.nks, v = P.nvt;
#define NL_WIN(NK, NV, FULL) return go(win_attn_kernel<T, NK, NV, FULL>, WinGeom<T, NK, NV>::NST)
    // sizes of their own: 64 / 64, 64 + 32 / 64, 128 / 128, 128 + 64 / 128
    if (k == 2 && v == 4) NL_WIN(2, 4, true);
    if (k == 3 && v == 4) NL_WIN(3, 4, true);
    if (k == 4 && v == 8) NL_WIN(4, 8, true);
    if (k == 6 && v == 8) NL_WIN(6, 8, true);
    if (k <= 1 && v <= 2) NL_WIN(1, 2, false);
    if (k <= 2 && v <= 4) NL_WIN(2, 4, false);
    if (k <= 4 && v <= 8) NL_WIN(4, 8, false);
    NL_WIN(8, 16, false);
#undef NL_WIN
}

}  // namespace nl
