// nl_linattn.h -- gated linear attention (a decay per key channel), 32-bit throughout:
//
//   S_t = diag(alpha_t) S_{t-1} + k_t v_t^T        o_t = S_t^T q_t        alpha = sigmoid(a2 (a1 h) + bias)^(1 / tau)
//
// per head, S [dk][dv] float32, carried from token to token in the stream's state slot.  Behind the recurrence: RMS norm of o
// over dv, a plain weight, silu(gate), a branch scale; the result leaves as the output product's operand (nl_mfma.h).
//
// PROMPTS.  A run of tokens of one stream is cut into sub-chunks of 16 tokens and segments of LA_SEG tokens.  With
// l_t = sum of log alpha from the sub-chunk's first token to t (gla_decay_kernel, one pass over all tokens) a sub-chunk is
//
//   o_t = (q_t e^{l_t})^T S  +  sum_{s <= t} A_ts v_s        A_ts = sum_d q_td k_sd e^{l_td - l_sd}
//   S  <- diag(e^{l_16}) S   +  sum_s (k_s e^{l_16 - l_s}) v_s^T
//
// all of it on v_mfma_f32_16x16x4_f32.  A wavefront owns 16 value columns of S in its accumulators: the accumulator layout
// D[row = 4 g + i][col] is, taken as step i, a B operand whose k slot g is row 4 g + i, so S feeds the first product without
// moving.  A_ts = (q e^l)(k e^{-l}) while no channel of the sub-chunk decays by more than e^-LA_FACTOR_MAX (the products stay in
// range and only relative roundings are added); a sub-chunk beyond that takes the exponent of the difference per pair.
// Segments of a long prompt run in parallel: gla_seg_kernel<.., false> (state increments from zero), gla_scan_kernel (a scan over
// the segments: every segment's starting state), gla_seg_kernel<.., true> (outputs).  A run that fits one segment starts with the
// last of them and the stored state.
//
// DECODE.  One workgroup per (head, stream): the state is read, decayed, updated, multiplied and written back in one pass
// (gla_decode_block, called from the fused mixer launch of nl_winattn.h).
#pragma once
#include "nl_mfma.h"

namespace nl {

constexpr int LA_SUB = 16;               // tokens per sub-chunk
constexpr int LA_SEG = 64;               // tokens per segment
constexpr float LA_FACTOR_MAX = 40.f;
constexpr int LA_MAX_DIM = 256;          // key / value size per head (padded)

struct GlaSub { int tok0, len; };                                 // sub-chunk: tokens [tok0, tok0 + len) of the step
struct GlaSeg { int tok0, len, sub0, stream, pos0, nseg, index; };  // segment `index` of the `nseg` of its run; pos0: the run's first position

struct GlaParams {
    const float *proj;         // projections of the step [token][ldp]: q, k, v, g, a1 at the offsets below
    int ldp, off_q, off_k, off_v, off_g, off_a1;
    int heads, dk, dv, rank;
    int dkp, dvp;              // dk, dv rounded up to 16: the state's leading dimensions
    const float *a2, *a2b, *norm;   // [rank][heads * dk], [heads * dk], [dv]
    float tau, eps, qscale, oscale;
    float *state;              // this layer run, stream 0: [heads][dkp][dvp]
    long long state_stride;    // floats per stream
    void *y;                   // output operand, this branch's columns from y_k0
    int y_nks, y_k0;
    // prompts
    const GlaSub *subs;
    const GlaSeg *segs;
    float *ldec;               // [token][heads * dk] cumulated log decays
    float *inc;                // [segment][heads][dkp][dvp] state increments, then starting states
    float *totlog;             // [segment][heads][dkp]
    const int *runs;           // gla_scan_kernel: first segment of every run with more than one segment
};

// log sigmoid(z) / tau = (min(z, 0) - log1p(e)) / tau, e = exp(-|z|) in (0, 1]: log1p by the area-tangent series
// log(1 + e) = 2 (s + s^3 / 3 + s^5 / 5 + ...), s = e / (2 + e) <= 1 / 3, cut behind s^17 (relative error below 2e-9)
__device__ __forceinline__ float gla_log_alpha(float z, float inv_tau) {
    const float e = exp_f32(-fminf(fabsf(z), 1e4f)), s = e * rcp_f32(2.f + e), w = s * s;
    float p = 1.f / 17.f;
    p = fmaf(p, w, 1.f / 15.f);
    p = fmaf(p, w, 1.f / 13.f);
    p = fmaf(p, w, 1.f / 11.f);
    p = fmaf(p, w, 1.f / 9.f);
    p = fmaf(p, w, 1.f / 7.f);
    p = fmaf(p, w, 1.f / 5.f);
    p = fmaf(p, w, 1.f / 3.f);
    return (fminf(z, 0.f) - 2.f * fmaf(s * w, p, s)) * inv_tau;
}

// grid (sub-chunks, channels / 256)
__global__ void __launch_bounds__(256) gla_decay_kernel(GlaParams P) {
    extern __shared__ __align__(16) char lds[];
    float *a1 = reinterpret_cast<float *>(lds);                  // [rank][16]
    const GlaSub sc = P.subs[blockIdx.x];
    for (int i = threadIdx.x; i < LA_SUB * P.rank; i += 256) {
        const int t = i / P.rank, r = i - t * P.rank;
        a1[r * LA_SUB + t] = t < sc.len ? P.proj[(long long)(sc.tok0 + t) * P.ldp + P.off_a1 + r] : 0.f;
    }
    const int C = P.heads * P.dk, c = min((int)(blockIdx.y * 256 + threadIdx.x), C - 1);
    const float b = P.a2b[c];
    f32x4 z[LA_SUB / 4];
#pragma unroll
    for (int q = 0; q < LA_SUB / 4; q++) z[q] = f32x4{b, b, b, b};
    __syncthreads();
#pragma unroll 8
    for (int r = 0; r < P.rank; r++) {
        const float wr = P.a2[(long long)r * C + c];
#pragma unroll
        for (int q = 0; q < LA_SUB / 4; q++) {
            const f32x4 x = *reinterpret_cast<const f32x4 *>(a1 + r * LA_SUB + q * 4);
#pragma unroll
            for (int i = 0; i < 4; i++) z[q][i] = fmaf(wr, x[i], z[q][i]);
        }
    }
    const float it = 1.f / P.tau;
    float l = 0.f;
#pragma unroll
    for (int t = 0; t < LA_SUB; t++) {
        l += gla_log_alpha(z[t >> 2][t & 3], it);
        if (t < sc.len && (int)(blockIdx.y * 256 + threadIdx.x) < C) P.ldec[(long long)(sc.tok0 + t) * C + c] = l;
    }
}

// grid (segments, heads), max(dvp, dkp) / 16 wavefronts; wavefront w < dvp / 16 owns value columns 16 w .. 16 w + 15, all of them load.
// The next sub-chunk's operands are requested before the current one is multiplied.
// NE: operand elements per thread, at least 16 dkp / threads (at most 4); WV: most wavefronts of a launch
template <typename T, int DKT, int NE, int WV, bool OUT>
__global__ void __launch_bounds__(WV * 64) gla_seg_kernel(GlaParams P) {
    extern __shared__ __align__(16) char lds[];
    const GlaSeg sg = P.segs[blockIdx.x];
    if (!OUT && (sg.nseg == 1 || sg.index + 1 == sg.nseg)) return;     // nobody starts from the state behind the last segment
    const int h = blockIdx.y, tid = threadIdx.x, nthr = blockDim.x, lane = tid & 63, w = tid >> 6, nw = nthr >> 6, g = lane >> 4, c = lane & 15;
    const int dk = P.dk, dkp = P.dkp, nkt = dkp >> 4, ld = dkp + 4, C = P.heads * dk, dvc = w * 16 + c;
    const int nv = P.dvp >> 4;
    const bool owner = w < nv, value = dvc < P.dv;
    float *qd = reinterpret_cast<float *>(lds);          // [16][ld]  q e^l
    float *ki = qd + 16 * ld;                            // [16][ld]  k e^-l
    float *ke = ki + 16 * ld;                            // [16][ld]  k e^{l_end - l}
    float *etot = ke + 16 * ld;                          // [dkp]     e^{l_end}
    float *A = etot + dkp;                                // [16][20]
    float *ssq = A + 16 * 20;                            // [nw][16] sums of squares
    int *flag = reinterpret_cast<int *>(ssq + nw * 16);  // [16] wavefront saw a decay beyond the factored range
    float *part = ssq + nw * 16 + 16;                    // [nw][256] partial A
    f32x4 S[DKT];
    const long long shead = (long long)dkp * P.dvp;
    float *stream_state = P.state + sg.stream * P.state_stride + h * shead;
    float *seg_state = P.inc + ((long long)blockIdx.x * P.heads + h) * shead;
    const int nsub = (sg.len + LA_SUB - 1) / LA_SUB;
    float rq[NE], rk[NE], rl[NE], re[NE], rv[4], rg[4];
    int et[NE], ed[NE];                                  // this thread's elements: token of the sub-chunk (16: none), channel
#pragma unroll
    for (int e = 0; e < NE; e++) {
        const int i = tid + e * nthr;
        et[e] = min(i / dkp, LA_SUB);
        ed[e] = i - i / dkp * dkp;
    }
    const char *proj = reinterpret_cast<const char *>(P.proj + (long long)sg.tok0 * P.ldp), *ldec = reinterpret_cast<const char *>(P.ldec + (long long)sg.tok0 * C + h * dk);
    auto fetch = [&](int sub) {
        const int u0 = sub * LA_SUB, len = min(LA_SUB, sg.len - u0);
#pragma unroll
        for (int e = 0; e < NE; e++) {
            rq[e] = rk[e] = rl[e] = re[e] = 0.f;
            if (et[e] < LA_SUB && ed[e] < dk) {
                re[e] = ld_off<float>(ldec, (unsigned)((u0 + len - 1) * C + ed[e]) * 4u);
                if (et[e] < len) {
                    const unsigned at = (unsigned)((u0 + et[e]) * P.ldp + h * dk + ed[e]);
                    rk[e] = ld_off<float>(proj, (at + P.off_k) * 4u);
                    rl[e] = ld_off<float>(ldec, (unsigned)((u0 + et[e]) * C + ed[e]) * 4u);
                    if (OUT) rq[e] = ld_off<float>(proj, (at + P.off_q) * 4u);
                }
            }
        }
        // value columns in B-operand order: step s holds token 4 s + g; the gates in accumulator order: token 4 g + i
#pragma unroll
        for (int s = 0; s < 4; s++) {
            rv[s] = owner && value && 4 * s + g < len ? ld_off<float>(proj, (unsigned)((u0 + 4 * s + g) * P.ldp + P.off_v + h * P.dv + dvc) * 4u) : 0.f;
            if (OUT) rg[s] = owner && value && 4 * g + s < len ? ld_off<float>(proj, (unsigned)((u0 + 4 * g + s) * P.ldp + P.off_g + h * P.dv + dvc) * 4u) : 0.f;
        }
    };
    fetch(0);
    {
        const float *from = !OUT || !owner ? nullptr : sg.nseg > 1 ? seg_state : sg.pos0 == 0 ? nullptr : stream_state;
#pragma unroll
        for (int dt = 0; dt < DKT; dt++) {
            S[dt] = f32x4{};
            if (from && dt < nkt)
#pragma unroll
                for (int i = 0; i < 4; i++) S[dt][i] = from[(long long)(dt * 16 + 4 * g + i) * P.dvp + dvc];
        }
    }
    const float inv_dv = 1.f / (float)P.dv;
    const int ycol = (int)op_index(0, P.y_k0 + h * P.dv + dvc, P.y_nks);
    const float nrm = OUT && value ? P.norm[dvc] * P.oscale : 0.f;
    for (int sub = 0; sub < nsub; sub++) {
        const int t0 = sg.tok0 + sub * LA_SUB, len = min(LA_SUB, sg.len - sub * LA_SUB);
        // operands of the sub-chunk; tokens beyond its length and channels beyond dk are zero
        bool strong = false;
#pragma unroll
        for (int e = 0; e < NE; e++) {
            const int t = et[e], d = ed[e];
            if (t < LA_SUB) {
                ke[t * ld + d] = rk[e] * exp_f32(re[e] - rl[e]);
                if (OUT) {
                    strong |= re[e] < -LA_FACTOR_MAX;
                    qd[t * ld + d] = rq[e] * P.qscale * exp_f32(rl[e]);
                    ki[t * ld + d] = rk[e] * exp_f32(fminf(-rl[e], LA_FACTOR_MAX));
                }
                if (t == 0) etot[d] = exp_f32(re[e]);
            }
        }
        float v[4], gz[4];
#pragma unroll
        for (int s = 0; s < 4; s++) { v[s] = rv[s]; gz[s] = rg[s]; }
        if (OUT) {
            const bool any = __any(strong);
            if (lane == 0) flag[w] = any;
        }
        lds_barrier();
        if (sub + 1 < nsub) fetch(sub + 1);
        bool slow = false;
        if (OUT)
            for (int q = 0; q < nw; q++) slow |= flag[q] != 0;
        f32x4 o = {};
        if (OUT) {
            if (!slow) {
                f32x4 a = {};
                for (int ks = w; ks < dkp / 4; ks += nw)
                    a = __builtin_amdgcn_mfma_f32_16x16x4f32(qd[c * ld + 4 * ks + g], ki[c * ld + 4 * ks + g], a, 0, 0, 0);
#pragma unroll
                for (int i = 0; i < 4; i++) part[w * 256 + (4 * g + i) * 16 + c] = a[i];
            }
            if (owner) {
#pragma unroll
                for (int dt = 0; dt < DKT; dt++)
                    if (dt < nkt) {
                        const f32x4 qv = *reinterpret_cast<const f32x4 *>(qd + c * ld + dt * 16 + 4 * g);
#pragma unroll
                        for (int i = 0; i < 4; i++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[i], S[dt][i], o, 0, 0, 0);
                    }
            }
        }
        if (owner) {
#pragma unroll
            for (int dt = 0; dt < DKT; dt++)
                if (dt < nkt) {
                    const f32x4 tl = *reinterpret_cast<const f32x4 *>(etot + dt * 16 + 4 * g);
#pragma unroll
                    for (int i = 0; i < 4; i++) S[dt][i] *= tl[i];
#pragma unroll
                    for (int s = 0; s < 4; s++) S[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ke[(4 * s + g) * ld + dt * 16 + c], v[s], S[dt], 0, 0, 0);
                }
        }
        lds_barrier();
        if (OUT) {
            for (int i = tid; i < 256; i += nthr) {
                const int t = i >> 4, s = i & 15;
                float a = 0.f;
                if (s <= t && t < len) {
                    if (!slow) {
                        const int np = min(nw, dkp / 4);
                        for (int q0 = 0; q0 < np; q0 += 8) {
                            float x[8];
#pragma unroll
                            for (int q = 0; q < 8; q++) x[q] = part[min(q0 + q, np - 1) * 256 + i];
#pragma unroll
                            for (int q = 0; q < 8; q++) a += q0 + q < np ? x[q] : 0.f;
                        }
                    } else {
                        const float *qp = P.proj + (long long)(t0 + t) * P.ldp + P.off_q + h * dk, *kp = P.proj + (long long)(t0 + s) * P.ldp + P.off_k + h * dk;
                        const float *lt = P.ldec + (long long)(t0 + t) * C + h * dk, *ls = P.ldec + (long long)(t0 + s) * C + h * dk;
#pragma unroll 1
                        for (int d = 0; d < dk; d++) a += qp[d] * P.qscale * kp[d] * exp_f32(lt[d] - ls[d]);
                    }
                }
                A[t * 20 + s] = a;
            }
            lds_barrier();
#pragma unroll
            for (int s = 0; s < 4; s++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(A[c * 20 + 4 * s + g], v[s], o, 0, 0, 0);
            // norm over the head's value columns: sums of squares over 16 lanes, then over the wavefronts
#pragma unroll
            for (int i = 0; i < 4; i++) {
                float ss = o[i] * o[i];
#pragma unroll
                for (int m = 1; m < 16; m <<= 1) ss += __shfl_xor(ss, m);
                if (c == 0) ssq[w * 16 + 4 * g + i] = ss;
            }
            lds_barrier();
            T *y = reinterpret_cast<T *>(P.y);
            f32x4 s2 = {};
            for (int q0 = 0; q0 < nv; q0 += 4) {
                f32x4 x[4];
#pragma unroll
                for (int q = 0; q < 4; q++) x[q] = *reinterpret_cast<const f32x4 *>(ssq + min(q0 + q, nv - 1) * 16 + 4 * g);
#pragma unroll
                for (int q = 0; q < 4; q++)
                    if (q0 + q < nv) s2 += x[q];
            }
            if (owner && value)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int t = 4 * g + i;
                    if (t < len) {
                        put(y + (unsigned)(((t0 + t) >> 4) * P.y_nks * OPT + ((t0 + t) & 15) * 8 + ycol), o[i] * rsqrt_f32(s2[i] * inv_dv + P.eps) * nrm * (gz[i] * sigmoid_f32(gz[i])));
                    }
                }
        }
    }
    if (!OUT) {
        // the segment's total log decay (every channel by one thread, from the sub-chunks' ends)
        for (int d = tid; d < dkp; d += nthr) {
            float a = 0.f;
            if (d < dk)
                for (int sub = 0; sub < nsub; sub++) a += P.ldec[(long long)(sg.tok0 + min(sub * LA_SUB + LA_SUB, sg.len) - 1) * C + h * dk + d];
            P.totlog[((long long)blockIdx.x * P.heads + h) * dkp + d] = a;
        }
    }
    if (owner && (!OUT || sg.index + 1 == sg.nseg)) {
        float *to = OUT ? stream_state : seg_state;
#pragma unroll
        for (int dt = 0; dt < DKT; dt++)
            if (dt < nkt)
#pragma unroll
                for (int i = 0; i < 4; i++) to[(long long)(dt * 16 + 4 * g + i) * P.dvp + dvc] = S[dt][i];
    }
}

// grid (state elements / 4 / 256, heads, runs): every segment's increment becomes its starting state
__global__ void __launch_bounds__(256) gla_scan_kernel(GlaParams P) {
    const int s0 = P.runs[blockIdx.z], h = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x, per = P.dkp * P.dvp / 4;
    if (e >= per) return;
    const GlaSeg sg = P.segs[s0];
    const int d = e * 4 / P.dvp;
    f32x4 S = {};
    if (sg.pos0 > 0) S = *reinterpret_cast<const f32x4 *>(P.state + sg.stream * P.state_stride + (long long)h * P.dkp * P.dvp + e * 4);
    f32x4 *at = reinterpret_cast<f32x4 *>(P.inc) + ((long long)s0 * P.heads + h) * per + e;
    const float *tl = P.totlog + ((long long)s0 * P.heads + h) * P.dkp + d;
    const long long astep = (long long)P.heads * per, tstep = (long long)P.heads * P.dkp;
    constexpr int U = 8;
    for (int i0 = 0; i0 < sg.nseg; i0 += U) {
        f32x4 inc[U];
        float dec[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int i = min(i0 + u, sg.nseg - 1);
            inc[u] = at[i * astep];
            dec[u] = tl[i * tstep];
        }
#pragma unroll
        for (int u = 0; u < U; u++)
            if (i0 + u < sg.nseg) {
                at[(i0 + u) * astep] = S;
                S = S * exp_f32(dec[u]) + inc[u];           // (the last segment's increment was not computed and is not used)
            }
    }
}

// one (head, token of a decode batch) by a workgroup of 256; lds: see gla_decode_lds
__host__ __device__ inline size_t gla_decode_lds(int dkp, int dvp, int rank) { return (size_t)(3 * dkp + dvp + 1024 + 8 + rank) * 4; }

template <typename T>
__device__ __forceinline__ void gla_decode_block(const GlaParams &P, int h, int n, int stream, int pos, char *lds) {
    constexpr int U = 8, RU = 16;
    const int tid = threadIdx.x, dk = P.dk, dv = P.dv, C = P.heads * dk;
    float *q = reinterpret_cast<float *>(lds), *k = q + P.dkp, *al = k + P.dkp, *v = al + P.dkp, *part = v + P.dvp, *red = part + 1024, *a1 = red + 8;
    const float *pr = P.proj + (long long)n * P.ldp;
    const int nc = P.dvp >> 2, rp = 256 / nc, c4 = tid % nc, r0 = tid / nc;
    f32x4 *S = reinterpret_cast<f32x4 *>(P.state + stream * P.state_stride + (long long)h * P.dkp * P.dvp) + c4;
    // everything that does not depend on this step's arithmetic is requested up front (head sizes are at most 256: one element per
    // thread), what is needed first in front: loads return in order
    const bool kc = tid < dk, vc = tid < dv;
    const float rq = kc ? pr[P.off_q + h * dk + tid] : 0.f, rk = kc ? pr[P.off_k + h * dk + tid] : 0.f, rv = vc ? pr[P.off_v + h * dv + tid] : 0.f;
    const float ra = tid < P.rank ? pr[P.off_a1 + tid] : 0.f;
    const float *w2 = P.a2 + h * dk + min(tid, dk - 1);
    float w[RU];
#pragma unroll
    for (int r = 0; r < RU; r++) w[r] = w2[(long long)min(r, P.rank - 1) * C];
    const float bias = kc ? P.a2b[h * dk + tid] : 0.f, gz = vc ? pr[P.off_g + h * dv + tid] : 0.f, nrm = vc ? P.norm[tid] * P.oscale : 0.f;
    f32x4 s[U];
    auto load = [&](int d0) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            s[u] = f32x4{};
            if (pos > 0 && r0 < rp && d0 + u * rp < dk) s[u] = S[(long long)(d0 + u * rp) * nc];
        }
    };
    load(r0);
    if (tid < P.rank) a1[tid] = ra;
    for (int i = tid + 256; i < P.rank; i += 256) a1[i] = pr[P.off_a1 + i];
    if (kc) { q[tid] = rq * P.qscale; k[tid] = rk; }
    if (tid < P.dvp) v[tid] = rv;
    lds_barrier();
    if (kc) {
        float z = bias;
#pragma unroll
        for (int r = 0; r < RU; r++)
            if (r < P.rank) z = fmaf(w[r], a1[r], z);
        for (int r = RU; r < P.rank; r++) z = fmaf(w2[(long long)r * C], a1[r], z);
        al[tid] = exp_f32(gla_log_alpha(z, 1.f / P.tau));
    }
    lds_barrier();
    f32x4 o = {};
    if (r0 < rp) {
        const f32x4 vv = *reinterpret_cast<const f32x4 *>(v + c4 * 4);
        for (int d0 = r0; d0 < dk; d0 += U * rp) {
            if (d0 != r0) load(d0);
#pragma unroll
            for (int u = 0; u < U; u++) {
                const int d = d0 + u * rp;
                if (d < dk) {
                    const f32x4 x = s[u] * al[d] + vv * k[d];
                    S[(long long)d * nc] = x;
                    o += x * q[d];
                }
            }
        }
        *reinterpret_cast<f32x4 *>(part + r0 * P.dvp + c4 * 4) = o;
    }
    lds_barrier();
    float val = 0.f;                                     // dvp <= 256: one value column per thread
    if (vc)
        for (int r = 0; r < rp; r++) val += part[r * P.dvp + tid];
    const float ss = wave_sum(val * val);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    lds_barrier();
    if (vc) {
        const float inv = rsqrt_f32((red[0] + red[1] + red[2] + red[3]) / (float)dv + P.eps);
        put(reinterpret_cast<T *>(P.y) + op_index(n, P.y_k0 + h * dv + tid, P.y_nks), val * inv * nrm * (gz * sigmoid_f32(gz)));
    }
}

template <typename T, bool OUT>
hipError_t launch_gla_seg(const GlaParams &P, int nsegs, hipStream_t st) {
    const int nw = std::max(P.dvp, P.dkp) / 16;
    const size_t lds = (size_t)(3 * 16 * (P.dkp + 4) + P.dkp + 16 * 20 + nw * 16 + 16 + nw * 256) * 4;
    auto go = [&](auto kfn) {
        if (lds > 65536)
            if (hipError_t s = hipFuncSetAttribute(reinterpret_cast<const void *>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)) return s;
        hipLaunchKernelGGL(kfn, dim3(nsegs, P.heads), dim3(nw * 64), lds, st, P);
        return hipGetLastError();
    };
    if (nw <= 8) {
        const bool two = 16 * P.dkp <= 2 * nw * 64;
        if (P.dkp <= 64) return two ? go(gla_seg_kernel<T, 4, 2, 8, OUT>) : go(gla_seg_kernel<T, 4, 4, 8, OUT>);
        return go(gla_seg_kernel<T, 8, 4, 8, OUT>);        // nw <= 8: dkp <= 128
    }
    if (P.dkp <= 128) return go(gla_seg_kernel<T, 8, 4, 16, OUT>);
    return go(gla_seg_kernel<T, 16, 4, 16, OUT>);
}

// the recurrence of a ragged step: runs = streams' token runs with more than one segment (their first segments in P.runs)
template <typename T>
hipError_t launch_gla(const GlaParams &P, int nsubs, int nsegs, int nruns, hipStream_t st) {
    hipLaunchKernelGGL(gla_decay_kernel, dim3(nsubs, (P.heads * P.dk + 255) / 256), dim3(256), (size_t)LA_SUB * P.rank * 4, st, P);
    if (nruns > 0) {
        if (hipError_t s = launch_gla_seg<T, false>(P, nsegs, st)) return s;
        hipLaunchKernelGGL(gla_scan_kernel, dim3((P.dkp * P.dvp / 4 + 255) / 256, P.heads, nruns), dim3(256), 0, st, P);
    }
    return launch_gla_seg<T, true>(P, nsegs, st);
}

}  // namespace nl
