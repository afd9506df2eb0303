// nl_stack.hip -- host side of libnanollama_stack.so: models described layer by layer (include/nanollama_stack.h).
//
// Weights go to MFMA operand order at upload (nl_mfma.h): the projections of a layer's mixers are ONE matrix (attention q | k | v | g,
// linear attention q | k | v | g | a1, every block padded to 16 rows), the output matrices of both branches are one matrix over the
// concatenated branch outputs (the branch scales enter in the branches' epilogues), gate and up alternate tile by tile.  A step is
//
//     lookup -> per layer run { [norm +] projections -> mixers -> output matrix + residual -> [norm +] gate | up -> down + residual }
//            -> [norm +] logits
//
// with the norm inside the product's launch for a handful of tokens and in a launch of its own otherwise.  A latent-attention mixer is
// two more products (nl_latent.h).  Where a model has norms behind its sublayers a product leaves its plain result, and the next launch
// that norms the residual stream adds it on the way, from one stream buffer to the other.  Layers of a loop are run
// several times with the same weights; every RUN has its own key / value ring and recurrent state per stream.  Decode steps are
// hipGraphs cached by (tokens, key splits, kind of chaining); prompts are ragged: any number of streams' token runs in one launch
// sequence, cut into the work lists of nl_linattn.h / nl_winattn.h on the host.
#include "../../include/nanollama_stack.h"
#include "nl_sample.h"
#include "nl_latent.h"

#include <algorithm>
#include <cmath>
#include <cstdarg>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <map>
#include <set>
#include <string>
#include <tuple>
#include <vector>

using namespace nl;

namespace {

thread_local std::string g_create_error;

inline int up(int n, int m) { return (n + m - 1) / m * m; }

struct Mat {                     // a product's weights in operand order
    void *w = nullptr;
    int rows = 0, k = 0, nrt = 0, nks = 0;
};

struct Layer {
    nl_layer_desc d{};
    Mat proj, out, gateup, down;
    Mat uq, uk, ukt, uv;         // latent attention: queries; keys and values from the latent; its transpose, a group of rows per head
    float *norm1p = nullptr, *norm2p = nullptr, *dqnorm = nullptr, *kvnorm = nullptr, *sink = nullptr, *rope = nullptr;
    float *gateb = nullptr, *upb = nullptr, *downb = nullptr;
    int tdq = 0, tdkv = 0, tg = -1, dimp = 0, rotp = 0, vdp = 0, kvt = 0;   // latent: projection rows, padded sizes, cache tiles of c (nks: all)
    float *norm1 = nullptr, *norm2 = nullptr, *qnorm = nullptr, *knorm = nullptr, *a2 = nullptr, *a2b = nullptr, *lnorm = nullptr, *slope = nullptr;
    int aq = 0, ak = 0, av = 0, ag = -1, lq = 0, lk = 0, lv = 0, lg = 0, la1 = 0;   // rows of the projection matrix
    int y_lin = 0;               // first column of the linear-attention branch in the output matrix
    int nks = 0, nvt = 0, R = 0, dkp = 0, dvp = 0;
    int xq_nks() const { return d.latent.heads * dimp / 32; }     // k tiles of the unrotated queries, head behind head
};

struct Run {                     // one execution of a layer
    int layer = 0;
    int kv_run = 0;              // latent attention: the run whose cache it reads
    bool add_embed = false;      // the embedding output is added behind this run (a pass of the loop ends here and another follows)
    char *K = nullptr, *V = nullptr;
    float *state = nullptr;
    long long kstride = 0, vstride = 0, sstride = 0;
};

}  // namespace

struct nl_engine {
    nl_stack_config c{};
    nl_config cfg{};             // what nl_get_config reports
    std::string err;
    std::vector<Layer> layers;
    std::vector<Run> runs;
    std::set<std::string> have;
    bool finalized = false, use_graph = true, trace = false;
    hipStream_t stream = nullptr;
    hipEvent_t ev0 = nullptr, ev1 = nullptr;
    std::vector<void *> allocs;
    size_t bytes_weights = 0, bytes_kv = 0, bytes_state = 0;
    void *stage = nullptr;
    size_t stage_cap = 0;

    Mat embed, head;             // rows = vocab: lookup table and output matrix (head.w == embed.w when they are one)
    float *final_norm = nullptr;
    int nksd = 0, ld = 0;        // k tiles of the width; leading dimension of the projections
    int cap = 0;                 // tokens of one launch sequence
    float *x = nullptr, *x0 = nullptr, *proj = nullptr, *logits = nullptr, *tracebuf = nullptr;
    int trace_tokens = 0;
    // norms behind the sublayers: a second stream buffer and the last sublayer's result, which the next norm of the stream takes in
    float *x2 = nullptr, *delta = nullptr, *xcur = nullptr;
    const float *pend = nullptr; // the norm's factor, null: nothing pending
    // latent attention: operand of the absorbed product, split results, expanded keys and values of kv_slots positions
    void *xq = nullptr, *ek = nullptr, *ev = nullptr;
    float *lpart = nullptr, *lml = nullptr;
    int kv_slots = 0;
    bool latent = false;
    void *h = nullptr, *y = nullptr, *act = nullptr, *q = nullptr;
    float *ldec = nullptr, *inc = nullptr, *totlog = nullptr, *part = nullptr;
    unsigned *arrived = nullptr;
    float *amax_val = nullptr;   // one token's logits: the largest of every 16 rows (the argmax reads these)
    int *amax_idx = nullptr;
    int lm_cap = 0;              // rows of `logits`
    int seg_cap = 0;
    // step metadata: pinned image and device copy of [tok | pos | stream | rows | subs | segs | tiles | runs | key tiles]
    int *h_meta = nullptr, *d_meta = nullptr;
    int m_pos = 0, m_stream = 0, m_rows = 0, m_subs = 0, m_segs = 0, m_tiles = 0, m_runs = 0, m_keys = 0, m_words = 0;
    int *ctl = nullptr, *ids = nullptr, *result = nullptr, *h_ctl = nullptr, *h_ids = nullptr;
    int ids_cap = 1024;
    float *h_logits = nullptr;
    std::vector<int> next_pos;   // per stream: the position its next token must have (or 0)
    struct Graph { hipGraph_t g; hipGraphExec_t x; };
    std::map<std::tuple<int, int, int>, Graph> graphs;
    SampScratch sp;
    int sp_cap = 0;

    int fail(int code, const char *fmt, ...) {
        char buf[512];
        va_list ap;
        va_start(ap, fmt);
        vsnprintf(buf, sizeof buf, fmt, ap);
        va_end(ap);
        err = buf;
        return code;
    }
    bool f32() const { return c.dtype == NL_DTYPE_F32; }
    size_t esize() const { return f32() ? 4 : 2; }
};

#define HIPCK(e, expr)                                                                               \
    do {                                                                                             \
        hipError_t _s = (expr);                                                                      \
        if (_s != hipSuccess) return (e)->fail(NL_ERR_HIP, "%s: %s", #expr, hipGetErrorString(_s)); \
    } while (0)

namespace {

// zero-filled device memory owned by the handle
template <typename P>
int dev_alloc(nl_engine *e, P *&p, size_t bytes, size_t &acct) {
    void *v = nullptr;
    const size_t n = std::max<size_t>(bytes, 256);
    HIPCK(e, hipMalloc(&v, n));
    e->allocs.push_back(v);
    HIPCK(e, hipMemsetAsync(v, 0, n, e->stream));
    acct += n;
    p = reinterpret_cast<P *>(v);
    return NL_OK;
}

int mat_alloc(nl_engine *e, Mat &m, int rows, int k) {
    m.rows = rows; m.k = k; m.nrt = (rows + 15) / 16; m.nks = (k + 31) / 32;
    return dev_alloc(e, m.w, (size_t)m.nrt * m.nks * OPT * e->esize(), e->bytes_weights);
}

// ---------------------------------------------------------------- weights ---

struct Dest {                    // where a tensor goes
    long long rows = 0, cols = 0;
    Mat *mat = nullptr;          // operand order ...
    int row0 = 0, k0 = 0, tstride = 1, toff = 0;
    float *vec = nullptr;        // ... or plain float, plus `add`, transposed if asked for
    bool transpose = false;
    float add = 0.f;
    // a place per source row instead (pack_mapped_kernel), in one or two matrices
    std::vector<int> rbase[2], kbase[2];
    Mat *mapped[2] = {nullptr, nullptr};
    bool tr[2] = {false, false};
};

bool find_dest(nl_engine *e, const char *name, Dest &d) {
    const int D = e->c.dim;
    if (!strcmp(name, "embed")) { d.rows = e->c.vocab; d.cols = D; d.mat = &e->embed; return true; }
    const float unit = e->c.plain_norm ? 0.f : 1.f;
    if (!strcmp(name, "head") && e->c.untied) { d.rows = e->c.vocab; d.cols = D; d.mat = &e->head; return true; }
    if (!strcmp(name, "final_norm")) { d.rows = 1; d.cols = D; d.vec = e->final_norm; d.add = unit; return true; }
    int n = -1, used = 0;
    if (sscanf(name, "layers.%d.%n", &n, &used) != 1 || used == 0 || n < 0 || n >= (int)e->layers.size()) return false;
    Layer &L = e->layers[n];
    const nl_attn_desc &A = L.d.attn;
    const nl_linattn_desc &G = L.d.lin;
    const std::string f = name + used;
    auto vec = [&](float *p, long long rows, long long cols, float add) { d.vec = p; d.rows = rows; d.cols = cols; d.add = add; return true; };
    auto in = [&](int row0, int rows) { d.mat = &L.proj; d.row0 = row0; d.rows = rows; d.cols = D; return true; };
    if (f == "norm1") return vec(L.norm1, 1, D, unit);
    if (f == "norm1_post" && e->c.post_norm) return vec(L.norm1p, 1, D, unit);
    const nl_latent_desc &N = L.d.latent;
    if (N.heads) {
        // adjacent places for the two of a rotated pair, in queries and keys alike
        auto pair = [&](int r) { return N.rot_adjacent || r >= N.rot_dims ? r : r < N.rot_dims / 2 ? 2 * r : 2 * (r - N.rot_dims / 2) + 1; };
        auto map = [&](int i, Mat &m, bool tr) { d.mapped[i] = &m; d.tr[i] = tr; d.rbase[i].resize(d.rows); d.kbase[i].assign(d.rows, 0); };
        auto size = [&](long long rows, long long cols) { d.rows = rows; d.cols = cols; };
        if (f == "latent.dq") return in(L.tdq, N.q_rank);
        if (f == "latent.g" && N.gate) return in(L.tg, N.heads);
        if (f == "latent.q_norm") return vec(L.dqnorm, 1, N.q_rank, 0.f);
        if (f == "latent.sink" && N.sink) return vec(L.sink, 1, N.heads, 0.f);
        if (N.kv_from < 0) {
            if (f == "latent.kv_norm") return vec(L.kvnorm, 1, N.kv_rank, 0.f);
            if (f == "latent.dkv") {
                size(N.kv_rank + N.rot_dim, D);
                map(0, L.proj, false);
                for (int r = 0; r < d.rows; r++) d.rbase[0][r] = L.tdkv + (r < N.kv_rank ? r : N.kv_rank + pair(r - N.kv_rank));
                return true;
            }
        }
        if (f == "latent.uq") {
            const int per = N.dim + N.rot_dim;
            size((long long)N.heads * per, N.q_rank);
            map(0, L.uq, false);
            for (int r = 0; r < d.rows; r++) {
                const int h = r / per, k = r - h * per;
                d.rbase[0][r] = k < N.dim ? h * L.dimp + k : N.heads * L.dimp + h * L.rotp + pair(k - N.dim);
            }
            return true;
        }
        if (f == "latent.uk") {
            size((long long)N.heads * N.dim, N.kv_rank);
            map(0, L.uk, false);
            map(1, L.ukt, true);
            for (int r = 0; r < d.rows; r++) {
                d.rbase[0][r] = r / N.dim * L.dimp + r % N.dim;
                d.rbase[1][r] = r / N.dim * L.kvt * 32;
                d.kbase[1][r] = r % N.dim;
            }
            return true;
        }
        if (f == "latent.uv") {
            size((long long)N.heads * N.vdim, N.kv_rank);
            map(0, L.uv, false);
            for (int r = 0; r < d.rows; r++) d.rbase[0][r] = r / N.vdim * L.vdp + r % N.vdim;
            return true;
        }
        if (f == "latent.o") { d.mat = &L.out; d.rows = D; d.cols = (long long)N.heads * N.vdim; return true; }
    }
    if (A.heads) {
        if (f == "attn.q") return in(L.aq, A.heads * A.dim);
        if (f == "attn.k") return in(L.ak, A.kv_heads * A.dim);
        if (f == "attn.v") return in(L.av, A.kv_heads * A.vdim);
        if (f == "attn.g" && A.gate) return in(L.ag, A.heads * A.vdim);
        if (f == "attn.q_norm" && A.qk_norm) return vec(L.qnorm, 1, A.dim, 0.f);
        if (f == "attn.k_norm" && A.qk_norm) return vec(L.knorm, 1, A.dim, 0.f);
        if (f == "attn.o") { d.mat = &L.out; d.rows = D; d.cols = A.heads * A.vdim; return true; }
    }
    if (G.heads) {
        if (f == "lin.q") return in(L.lq, G.heads * G.dim);
        if (f == "lin.k") return in(L.lk, G.heads * G.dim);
        if (f == "lin.v") return in(L.lv, G.heads * G.vdim);
        if (f == "lin.g") return in(L.lg, G.heads * G.vdim);
        if (f == "lin.a1") return in(L.la1, G.rank);
        if (f == "lin.a2") { d.transpose = true; return vec(L.a2, G.heads * G.dim, G.rank, 0.f); }
        if (f == "lin.a2_bias") return vec(L.a2b, 1, G.heads * G.dim, 0.f);
        if (f == "lin.norm") return vec(L.lnorm, 1, G.vdim, 0.f);
        if (f == "lin.o") { d.mat = &L.out; d.k0 = L.y_lin; d.rows = D; d.cols = G.heads * G.vdim; return true; }
    }
    if (L.d.ff) {
        if (f == "norm2") return vec(L.norm2, 1, D, unit);
        if (f == "norm2_post" && e->c.post_norm) return vec(L.norm2p, 1, D, unit);
        if (L.d.ff_bias) {
            if (f == "ff.gate_bias") return vec(L.gateb, 1, L.d.ff, 0.f);
            if (f == "ff.up_bias") return vec(L.upb, 1, L.d.ff, 0.f);
            if (f == "ff.down_bias") return vec(L.downb, 1, D, 0.f);
        }
        if (f == "ff.gate" || f == "ff.up") { d.mat = &L.gateup; d.tstride = 2; d.toff = f == "ff.up"; d.rows = L.d.ff; d.cols = D; return true; }
        if (f == "ff.down") { d.mat = &L.down; d.rows = D; d.cols = L.d.ff; return true; }
    }
    return false;
}

std::vector<std::string> wanted_tensors(const nl_engine *e) {
    std::vector<std::string> w = {"embed", "final_norm"};
    if (e->c.untied) w.push_back("head");
    for (size_t i = 0; i < e->layers.size(); i++) {
        const nl_layer_desc &d = e->layers[i].d;
        const std::string p = "layers." + std::to_string(i) + ".";
        auto add = [&](std::initializer_list<const char *> names) { for (const char *n : names) w.push_back(p + n); };
        add({"norm1"});
        if (e->c.post_norm) add({"norm1_post"});
        if (d.latent.heads) {
            add({"latent.dq", "latent.q_norm", "latent.uq", "latent.uk", "latent.uv", "latent.o"});
            if (d.latent.kv_from < 0) add({"latent.dkv", "latent.kv_norm"});
            if (d.latent.sink) add({"latent.sink"});
            if (d.latent.gate) add({"latent.g"});
        }
        if (d.attn.heads) {
            add({"attn.q", "attn.k", "attn.v", "attn.o"});
            if (d.attn.gate) add({"attn.g"});
            if (d.attn.qk_norm) add({"attn.q_norm", "attn.k_norm"});
        }
        if (d.lin.heads) add({"lin.q", "lin.k", "lin.v", "lin.g", "lin.a1", "lin.a2", "lin.a2_bias", "lin.norm", "lin.o"});
        if (d.ff) {
            add({"norm2", "ff.gate", "ff.up", "ff.down"});
            if (e->c.post_norm) add({"norm2_post"});
            if (d.ff_bias) add({"ff.gate_bias", "ff.up_bias", "ff.down_bias"});
        }
    }
    return w;
}

// cos and sin of every position and pair of a rotary layer, computed in double; YaRN: pairs that turn less than `slow` times over
// `original` positions are interpolated by `factor`, those that turn more than `fast` times stay, a ramp between them
std::vector<float> rope_table(const nl_latent_desc &N, int positions) {
    const int pairs = N.rot_dims / 2;
    const double n = N.rot_dims, pi = 3.14159265358979323846;
    std::vector<double> f(pairs);
    double mul = 1.0;
    for (int i = 0; i < pairs; i++) f[i] = std::pow(N.rope_base, -2.0 * i / n);
    if (N.yarn_factor != 0.0) {
        auto dim = [&](double turns) { return n * std::log(N.yarn_original / (2.0 * pi * turns)) / (2.0 * std::log(N.rope_base)); };
        const double lo = std::max(std::floor(dim(N.yarn_fast)), 0.0), hi = std::min(std::ceil(dim(N.yarn_slow)), n - 1.0);
        for (int i = 0; i < pairs; i++) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / N.yarn_factor * ramp + f[i] * (1.0 - ramp);
        }
        mul = 0.1 * std::log(N.yarn_factor) + 1.0;
    }
    std::vector<float> t((size_t)positions * pairs * 2);
    for (int p = 0; p < positions; p++)
        for (int i = 0; i < pairs; i++) {
            t[((size_t)p * pairs + i) * 2] = (float)(mul * std::cos(p * f[i]));
            t[((size_t)p * pairs + i) * 2 + 1] = (float)(mul * std::sin(p * f[i]));
        }
    return t;
}

// ------------------------------------------------------------------- step ---

// pieces of a prompt sequence whose expanded keys and values are in scratch together
struct KeyGroup { int tile0, ntiles, key0, nkeys; };     // query tiles and key tiles (of 16 positions) of the step's lists

struct StepIn {                  // one launch sequence
    int n = 0;                   // tokens
    const int *tok, *pos, *stream;   // device
    int nsplit = 1;              // decode
    bool decode = true;
    int nsubs = 0, nsegs = 0, nruns = 0, ntiles = 0;
    std::vector<KeyGroup> groups;
    int n_out = 0;               // rows of logits: of tokens rows[0 .. n_out) (device), or of every token when rows is null
    const int *rows = nullptr;
    float *logits = nullptr;
};

MatParams product_params(nl_engine *e, const Mat &m, const void *X, int n) {
    MatParams P{};
    P.W = m.w; P.X = X; P.nks = m.nks; P.nrt = m.nrt; P.n_tokens = n; P.rows = m.rows; P.neps = e->c.eps;
    return P;
}

// the product of norm(stream) with m, epilogue fields of P set by the caller: the norm runs inside the product's launch or leaves an operand of
// its own; what is pending behind the last sublayer is added on the way.  rows: only these tokens, and the stream stays as it is.
template <typename T, int EPI>
hipError_t normed_product(nl_engine *e, MatParams P, const float *nw, const int *rows = nullptr, bool last = false) {
    float *keep = last ? nullptr : e->xcur == e->x ? e->x2 : e->x;
    const int norm = e->pend ? 2 : 1;
    hipError_t s;
    if (!rows && few_norm_ok(P.n_tokens, P.nks, e->c.dim, e->c.dim)) {
        P.nx = e->xcur; P.nw = nw; P.nd = e->delta; P.ndw = e->pend; P.nxo = keep; P.ndim = e->c.dim;
        s = launch_product<T, EPI>(P, e->stream, norm);
    } else {
        NormParams N{};
        N.x = e->xcur; N.w = nw; N.rows = rows; N.out = e->h; N.dim = e->c.dim; N.nks = e->nksd; N.n_tokens = P.n_tokens; N.eps = e->c.eps;
        if (e->pend) { N.d = e->delta; N.dw = e->pend; N.x_out = keep; }
        if ((s = launch_norm_operand<T>(N, e->stream))) return s;
        P.X = e->h;
        s = launch_product<T, EPI>(P, e->stream);
    }
    if (e->pend && !last) { e->xcur = keep; e->pend = nullptr; }
    return s;
}

// a sublayer's last product: into the stream, or kept for the norm behind it
template <typename T>
hipError_t residual_product(nl_engine *e, const Mat &m, const void *X, int n, const float *bias, const float *post, const float *behind) {
    MatParams P = product_params(e, m, X, n);
    P.ldo = e->c.dim;
    if (!post) {
        P.out = e->xcur; P.add2 = behind;
        return launch_product<T, ST_RESID>(P, e->stream);
    }
    P.out = e->delta; P.bias = bias;
    e->pend = post;
    return launch_product<T, ST_F32>(P, e->stream);
}

template <typename T>
hipError_t logits_launch(nl_engine *e, const int *rows, int n, float *out) {
    MatParams P = product_params(e, e->head, nullptr, n);
    P.out = out; P.ldo = e->c.vocab;
    if (n == 1) { P.amax_val = e->amax_val; P.amax_idx = e->amax_idx; }
    return normed_product<T, ST_F32>(e, P, e->final_norm, rows, true);
}

// behind the projections: everything up to the output matrix's operand
template <typename T>
hipError_t latent_mixer(nl_engine *e, const StepIn &s, const Run &R, const Layer &L) {
    const hipStream_t st = e->stream;
    const nl_latent_desc &N = L.d.latent;
    hipError_t rc;
    LatentParams A{};
    A.proj = e->proj; A.ldp = L.proj.rows; A.off_c = L.tdkv; A.off_r = L.tdkv + N.kv_rank; A.off_g = L.tg;
    A.kv_rank = N.kv_rank; A.rot_dim = N.rot_dim; A.pairs = N.rot_dims / 2; A.kvt = L.kvt; A.nks = L.nks; A.norm = L.kvnorm; A.eps = e->c.eps; A.rope = L.rope;
    A.pos = s.pos; A.stream = s.stream; A.cache = e->runs[R.kv_run].K; A.stride = e->runs[R.kv_run].kstride; A.heads = N.heads; A.dv = N.vdim; A.scale = N.scale;
    A.q = e->q; A.nsplit = s.nsplit; A.part = e->lpart; A.ml = e->lml; A.W = L.uv.w; A.tph = L.vdp / 16; A.sink = L.sink; A.y = e->y; A.y_nks = L.out.nks;
    const LatentStore<T> store{N.kv_from < 0 ? s.n : 0, A};
    const int qt = (L.dimp + L.rotp) / 32;               // k tiles of an expanded key
    // queries: norm of their latent, product, rotation
    MatParams P = product_params(e, L.uq, nullptr, s.n);
    HeadRows &H = P.hd;
    H.q = e->q; H.heads = N.heads; H.split = N.heads * L.dimp; H.hrows[0] = L.dimp; H.hrows[1] = L.rotp; H.pairs = A.pairs; H.rope = L.rope; H.pos = s.pos;
    H.ld = (s.decode ? L.nks : qt) * 32;
    H.col[1] = s.decode ? L.kvt * 32 : L.dimp;
    if (s.decode) { H.xq = e->xq; H.xq_nks = L.xq_nks(); }
    if (few_norm_ok(s.n, L.uq.nks, N.q_rank, L.proj.rows)) {
        P.nx = e->proj + L.tdq; P.nw = L.dqnorm; P.ndim = N.q_rank; P.nld = L.proj.rows;
        rc = store.units ? launch_product<T, ST_HEADS>(P, st, 1, store) : launch_product<T, ST_HEADS>(P, st, 1);
    } else {
        NormParams Q{};
        Q.x = e->proj + L.tdq; Q.ld = L.proj.rows; Q.w = L.dqnorm; Q.out = e->h; Q.dim = N.q_rank; Q.nks = L.uq.nks; Q.n_tokens = s.n; Q.eps = e->c.eps;
        if ((rc = store.units ? launch_norm_operand<T>(Q, st, store) : launch_norm_operand<T>(Q, st))) return rc;
        P.X = e->h;
        rc = launch_product<T, ST_HEADS>(P, st);
    }
    if (rc) return rc;
    if (s.decode) {
        MatParams B = product_params(e, L.ukt, e->xq, s.n);
        B.x_nks = L.xq_nks(); B.group = L.kvt * 2;
        B.hd.q = e->q; B.hd.heads = N.heads; B.hd.ld = L.nks * 32; B.hd.split = L.ukt.rows; B.hd.hrows[0] = L.kvt * 32;
        if ((rc = launch_product<T, ST_HEADS>(B, st)) || (rc = launch_latent_decode<T>(A, s.n, st))) return rc;
        return launch_latent_out<T>(A, s.n, st);
    }
    WinParams W{};
    W.pos = s.pos; W.stream = s.stream; W.nsplit = 1; W.y = e->y; W.y_nks = L.out.nks; W.proj = e->proj; W.ldp = L.proj.rows;
    W.off_g = L.tg; W.head_gate = 1; W.heads = W.kv_heads = N.heads; W.dk = qt * 32; W.dv = N.vdim; W.nks = qt; W.nvt = L.vdp / 16;
    W.eps = e->c.eps; W.scale = N.scale; W.oscale = 1.f; W.sink = L.sink; W.R = e->kv_slots; W.K = e->ek; W.V = e->ev; W.q = e->q;
    for (const KeyGroup &g : s.groups) {
        const int *list = e->d_meta + e->m_keys + g.key0;
        MatParams K = product_params(e, L.uk, A.cache, g.nkeys * 16);
        K.x_nks = L.nks; K.x_tile = list;
        K.kr.dst = e->ek; K.kr.hrows = L.dimp; K.kr.nt = qt; K.kr.slots = e->kv_slots;
        RotatedKeys<T> rk{g.nkeys * (L.nks - L.kvt), A.cache, list, L.nks, L.kvt, N.heads, e->kv_slots, L.dimp / 32, qt, e->ek};
        MatParams V = product_params(e, L.uv, A.cache, g.nkeys * 16);
        V.x_nks = L.nks; V.x_tile = list;
        V.kr.dst = e->ev; V.kr.hrows = L.vdp; V.kr.nt = W.nvt; V.kr.slots = e->kv_slots;
        W.tiles = reinterpret_cast<const WinTile *>(e->d_meta + e->m_tiles) + g.tile0;
        if ((rc = launch_many<T, ST_KEYS>(K, st, rk)) || (rc = launch_many<T, ST_VALUES>(V, st)) || (rc = launch_win_attn<T>(W, g.ntiles, st))) return rc;
    }
    return hipSuccess;
}

template <typename T>
hipError_t launch_sequence(nl_engine *e, const StepIn &s) {
    const hipStream_t st = e->stream;
    const int D = e->c.dim;
    hipError_t rc;
    LookupParams E{};
    e->xcur = e->x;
    e->pend = nullptr;
    E.table = e->embed.w; E.tok = s.tok; E.nks = e->nksd; E.dim = D; E.scale = e->c.embed_scale; E.x = e->x; E.x0 = e->x0;
    hipLaunchKernelGGL(lookup_kernel<T>, dim3(s.n), dim3(256), 0, st, E);
    for (size_t r = 0; r < e->runs.size(); r++) {
        const Run &R = e->runs[r];
        const Layer &L = e->layers[R.layer];
        const nl_attn_desc &A = L.d.attn;
        const nl_linattn_desc &G = L.d.lin;
        const float *behind = R.add_embed ? e->x0 : nullptr;
        MatParams J = product_params(e, L.proj, nullptr, s.n);
        J.out = e->proj; J.ldo = L.proj.rows;
        if ((rc = normed_product<T, ST_F32>(e, J, L.norm1))) return rc;
        WinParams W{};
        W.pos = s.pos; W.stream = s.stream; W.nsplit = 1; W.y = e->y; W.y_nks = L.out.nks; W.proj = e->proj; W.ldp = L.proj.rows;
        if (A.heads) {
            W.off_q = L.aq; W.off_k = L.ak; W.off_v = L.av; W.off_g = L.ag; W.heads = A.heads; W.kv_heads = A.kv_heads; W.dk = A.dim; W.dv = A.vdim;
            W.nks = L.nks; W.nvt = L.nvt; W.qnorm = L.qnorm; W.knorm = L.knorm; W.eps = e->c.eps; W.scale = A.scale; W.oscale = A.mix_scale;
            W.slope = L.slope; W.window = A.window; W.R = L.R; W.K = R.K; W.V = R.V; W.kstride = R.kstride; W.vstride = R.vstride;
            W.q = e->q; W.nsplit = s.decode ? s.nsplit : 1; W.part = e->part; W.arrived = e->arrived;
            W.tiles = reinterpret_cast<const WinTile *>(e->d_meta + e->m_tiles);
        }
        GlaParams N{};
        if (G.heads) {
            N.proj = e->proj; N.ldp = L.proj.rows; N.off_q = L.lq; N.off_k = L.lk; N.off_v = L.lv; N.off_g = L.lg; N.off_a1 = L.la1;
            N.heads = G.heads; N.dk = G.dim; N.dv = G.vdim; N.rank = G.rank; N.dkp = L.dkp; N.dvp = L.dvp; N.a2 = L.a2; N.a2b = L.a2b; N.norm = L.lnorm;
            N.tau = G.tau; N.eps = e->c.eps; N.qscale = (float)(1.0 / std::sqrt((double)G.dim)); N.oscale = G.mix_scale;
            N.state = R.state; N.state_stride = R.sstride; N.y = e->y; N.y_nks = L.out.nks; N.y_k0 = L.y_lin;
            N.subs = reinterpret_cast<const GlaSub *>(e->d_meta + e->m_subs); N.segs = reinterpret_cast<const GlaSeg *>(e->d_meta + e->m_segs);
            N.runs = e->d_meta + e->m_runs; N.ldec = e->ldec; N.inc = e->inc; N.totlog = e->totlog;
        }
        if (L.d.latent.heads) {
            if ((rc = latent_mixer<T>(e, s, R, L))) return rc;
        } else if (s.decode) {
            if ((rc = launch_mix_decode<T>(W, N, s.n, st))) return rc;
        } else {
            if (A.heads && ((rc = launch_win_prep<T>(W, s.n, st)) || (rc = launch_win_attn<T>(W, s.ntiles, st)))) return rc;
            if (G.heads && (rc = launch_gla<T>(N, s.nsubs, s.nsegs, s.nruns, st))) return rc;
        }
        if ((rc = residual_product<T>(e, L.out, e->y, s.n, nullptr, L.norm1p, L.d.ff ? nullptr : behind))) return rc;
        if (L.d.ff) {
            MatParams F = product_params(e, L.gateup, nullptr, s.n);
            F.act = e->act; F.act_nks = L.down.nks; F.act_silu = L.d.ff_act == NL_ACT_SILU; F.bias = L.gateb; F.bias2 = L.upb;
            if ((rc = normed_product<T, ST_GATED>(e, F, L.norm2))) return rc;
            if ((rc = residual_product<T>(e, L.down, e->act, s.n, L.downb, L.norm2p, behind))) return rc;
        }
        if (e->trace) {
            float *to = e->tracebuf + r * (size_t)s.n * D;
            if (e->pend) {       // (the stream as the next norm will make it)
                NormParams Q{};
                Q.x = e->xcur; Q.w = L.norm1; Q.out = e->h; Q.dim = D; Q.nks = e->nksd; Q.n_tokens = s.n; Q.eps = e->c.eps; Q.d = e->delta; Q.dw = e->pend; Q.x_out = to;
                if ((rc = launch_norm_operand<T>(Q, st))) return rc;
            } else if ((rc = hipMemcpyAsync(to, e->xcur, (size_t)s.n * D * 4, hipMemcpyDeviceToDevice, st))) return rc;
            if (behind)      // (the run's last product has added it already: taken off again when the trace is read)
                if ((rc = hipMemcpyAsync(e->tracebuf + (e->runs.size() + r) * (size_t)s.n * D, e->x0, (size_t)s.n * D * 4, hipMemcpyDeviceToDevice, st))) return rc;
        }
    }
    return s.n_out > 0 ? logits_launch<T>(e, s.rows, s.n_out, s.logits) : hipGetLastError();
}

int run_sequence(nl_engine *e, const StepIn &s) {
    if (e->trace) e->trace_tokens = s.n;
    const hipError_t rc = e->f32() ? launch_sequence<float>(e, s) : launch_sequence<bf16>(e, s);
    if (rc != hipSuccess) return e->fail(NL_ERR_HIP, "step launch: %s", hipGetErrorString(rc));
    return NL_OK;
}

// key-range splits of a decode step: enough workgroups for the chip, at least 128 keys each, never more keys than one split holds
int splits_for(const nl_engine *e, int n, int max_pos) {
    int out = 1;
    for (const Layer &L : e->layers) {
        if (L.d.latent.heads) {
            const int nb = max_pos / LT_KEYS + 1, want = std::min({256 / std::max(1, n * ((L.d.latent.heads + 15) / 16)), nb, LT_MAX_SPLITS});
            int p = 1;
            while (p * 2 <= want) p *= 2;
            out = std::max(out, p);
        }
        if (!L.d.attn.heads) continue;
        const int seen = L.d.attn.window > 0 ? std::min(L.d.attn.window, max_pos + 1) : max_pos + 1, nb = seen / 32 + 2;
        const int need = (nb * 32 + WA_SPLIT_KEYS - 1) / WA_SPLIT_KEYS, want = std::min(512 / std::max(1, n * L.d.attn.heads), nb / 4);
        int p = 1;
        while (p < need || (p * 2 <= want && p < 64)) p *= 2;
        out = std::max(out, p);
    }
    return out;
}

enum { CH_BATCH = 0, CH_CALL = 1, CH_CHAIN = 2, CH_SAMPLE = 3 };
constexpr int CHAIN_STEPS = 16;

// queue one decode step (kind CH_CHAIN: `steps` of them): from the batch arrays (CH_BATCH) or the control block
int queue_decode(nl_engine *e, int kind, int n, int max_pos, int steps = 1) {
    const int nsplit = splits_for(e, n, max_pos);
    StepIn s;
    s.n = n; s.nsplit = nsplit; s.n_out = n; s.logits = e->logits;
    if (kind == CH_BATCH) { s.tok = e->d_meta; s.pos = e->d_meta + e->m_pos; s.stream = e->d_meta + e->m_stream; }
    else { s.tok = e->ctl + CTL_TOKEN; s.pos = e->ctl + CTL_POS; s.stream = e->ctl + CTL_STREAM; }
    auto body = [&]() -> int {
        for (int i = 0; i < steps; i++) {
            if (int rc = run_sequence(e, s)) return rc;
            if (kind == CH_BATCH) hipLaunchKernelGGL(bargmax_kernel, dim3(n), dim3(1024), 0, e->stream, e->logits, e->c.vocab, e->ids);
            else if (kind != CH_SAMPLE) {
                ArgmaxParams A{};
                A.logits = e->logits; A.n = e->c.vocab; A.part_val = e->amax_val; A.part_idx = e->amax_idx; A.npart = e->head.nrt; A.ctl = e->ctl; A.ids = e->ids; A.result = e->result;
                hipLaunchKernelGGL(argmax_kernel, dim3(1), dim3(1024), 0, e->stream, A);
            }
        }
        const hipError_t s2 = hipGetLastError();
        return s2 == hipSuccess ? NL_OK : e->fail(NL_ERR_HIP, "argmax launch: %s", hipGetErrorString(s2));
    };
    if (!e->use_graph || e->trace) return body();
    const auto key = std::make_tuple(n, nsplit, kind * 64 + steps);
    auto it = e->graphs.find(key);
    if (it == e->graphs.end()) {
        nl_engine::Graph G{nullptr, nullptr};
        HIPCK(e, hipStreamBeginCapture(e->stream, hipStreamCaptureModeThreadLocal));
        const int rc = body();
        const hipError_t ce = hipStreamEndCapture(e->stream, &G.g);
        if (rc) { if (G.g) (void)hipGraphDestroy(G.g); return rc; }
        if (ce != hipSuccess || !G.g) return e->fail(NL_ERR_HIP, "graph capture: %s", hipGetErrorString(ce));
        HIPCK(e, hipGraphInstantiate(&G.x, G.g, nullptr, nullptr, 0));
        it = e->graphs.emplace(key, G).first;
    }
    HIPCK(e, hipGraphLaunch(it->second.x, e->stream));
    return NL_OK;
}

// ------------------------------------------------------------- positions ---

int check_tokens(nl_engine *e, int stream, const int *tokens, int n, int pos0) {
    if (!e->finalized) return e->fail(NL_ERR_STATE, "step before nl_finalize");
    if (stream < 0 || stream >= e->c.max_streams) return e->fail(NL_ERR_INVALID, "stream %d out of range", stream);
    if (n <= 0 || pos0 < 0 || pos0 > e->c.seq_len - n) return e->fail(NL_ERR_INVALID, "%d tokens at position %d: outside [0, %d)", n, pos0, e->c.seq_len);
    for (int i = 0; i < n; i++)
        if (tokens[i] < 0 || tokens[i] >= e->c.vocab) return e->fail(NL_ERR_INVALID, "token %d out of range [0,%d)", tokens[i], e->c.vocab);
    if (pos0 != 0 && pos0 != e->next_pos[stream])
        return e->fail(NL_ERR_STATE, "stream %d goes on at position %d (or starts again at 0), not at %d", stream, e->next_pos[stream], pos0);
    return NL_OK;
}

int set_ctl(nl_engine *e, int token, int pos, int chain, int stream) {
    HIPCK(e, hipStreamSynchronize(e->stream));       // the pinned block is reused
    memset(e->h_ctl, 0, CTL_WORDS * sizeof(int));
    e->h_ctl[CTL_TOKEN] = token; e->h_ctl[CTL_POS] = pos; e->h_ctl[CTL_CHAIN] = chain; e->h_ctl[CTL_STREAM] = stream;
    HIPCK(e, hipMemcpyAsync(e->ctl, e->h_ctl, CTL_WORDS * sizeof(int), hipMemcpyHostToDevice, e->stream));
    return NL_OK;
}

// ------------------------------------------------------------ ragged steps ---

struct Piece { int stream, tok0, n, pos0; };     // tokens [tok0, tok0 + n) of the caller's array

// One launch sequence of prompt pieces (distinct streams, at most cap tokens); want: caller-array indices that fall into it, in order.
// Logits rows go to out (host, row stride vocab) in groups of lm_cap; the last group's stay in e->logits.
int run_pieces(nl_engine *e, const std::vector<Piece> &ps, const int *tokens, const std::vector<int> &want, float *out, int *argmax_out) {
    HIPCK(e, hipStreamSynchronize(e->stream));       // the pinned metadata is reused
    int *m = e->h_meta;
    StepIn s;
    s.decode = false;
    int n = 0, nsubs = 0, nsegs = 0, ntiles = 0, nruns = 0, nkeys = 0;
    std::vector<int> rows;
    size_t w = 0;
    for (const Piece &p : ps) {
        GlaSub *subs = reinterpret_cast<GlaSub *>(m + e->m_subs);
        GlaSeg *segs = reinterpret_cast<GlaSeg *>(m + e->m_segs);
        WinTile *tiles = reinterpret_cast<WinTile *>(m + e->m_tiles);
        for (int i = 0; i < p.n; i++) { m[n + i] = tokens[p.tok0 + i]; m[e->m_pos + n + i] = p.pos0 + i; m[e->m_stream + n + i] = p.stream; }
        const int nseg = (p.n + LA_SEG - 1) / LA_SEG;
        if (nseg > 1) m[e->m_runs + nruns++] = nsegs;
        for (int i = 0; i < nseg; i++) segs[nsegs++] = GlaSeg{n + i * LA_SEG, std::min(LA_SEG, p.n - i * LA_SEG), nsubs + i * (LA_SEG / LA_SUB), p.stream, p.pos0, nseg, i};
        for (int t = 0; t < p.n; t += LA_SUB) subs[nsubs++] = GlaSub{n + t, std::min(LA_SUB, p.n - t)};
        int key0 = 0;
        if (e->latent) {             // every position so far is expanded: groups of pieces that fit the scratch
            const int slots = up(p.pos0 + p.n, 64), per = up(e->c.seq_len, 64) / 16;
            if (s.groups.empty() || s.groups.back().nkeys * 16 + slots > e->kv_slots) s.groups.push_back({ntiles, 0, nkeys, 0});
            KeyGroup &g = s.groups.back();
            key0 = g.nkeys * 16;
            for (int i = 0; i < slots / 16; i++) m[e->m_keys + nkeys++] = p.stream * per + i;
            g.nkeys += slots / 16;
            g.ntiles += (p.n + WA_Q - 1) / WA_Q;
        }
        for (int t = 0; t < p.n; t += WA_Q) tiles[ntiles++] = WinTile{n + t, std::min(WA_Q, p.n - t), p.pos0 + t, p.stream, key0};
        for (; w < want.size() && want[w] < p.tok0 + p.n; w++) rows.push_back(n + want[w] - p.tok0);
        n += p.n;
    }
    s.n = n; s.nsubs = nsubs; s.nsegs = nsegs; s.nruns = nruns; s.ntiles = ntiles;
    for (size_t i = 0; i < rows.size(); i++) m[e->m_rows + i] = rows[i];
    HIPCK(e, hipMemcpyAsync(e->d_meta, m, (size_t)(e->m_keys + nkeys) * sizeof(int), hipMemcpyHostToDevice, e->stream));
    s.tok = e->d_meta; s.pos = e->d_meta + e->m_pos; s.stream = e->d_meta + e->m_stream;
    s.logits = e->logits;
    int rc;
    for (size_t r0 = 0; r0 == 0 || r0 < rows.size(); r0 += e->lm_cap) {
        const int nr = (int)std::min(rows.size() - r0, (size_t)e->lm_cap);
        if (r0 == 0) {
            s.n_out = nr; s.rows = e->d_meta + e->m_rows;
            if ((rc = run_sequence(e, s))) return rc;
        } else {
            const int *rp = e->d_meta + e->m_rows + r0;
            const hipError_t hr = e->f32() ? logits_launch<float>(e, rp, nr, e->logits) : logits_launch<bf16>(e, rp, nr, e->logits);
            if (hr != hipSuccess) return e->fail(NL_ERR_HIP, "logits launch: %s", hipGetErrorString(hr));
        }
        if (nr == 0) break;
        if (argmax_out) {
            hipLaunchKernelGGL(bargmax_kernel, dim3(nr), dim3(1024), 0, e->stream, e->logits, e->c.vocab, e->ids);
            HIPCK(e, hipMemcpyAsync(e->h_ids, e->ids, (size_t)nr * 4, hipMemcpyDeviceToHost, e->stream));
        }
        if (out) {
            if (nr == 1) {
                HIPCK(e, hipMemcpyAsync(e->h_logits, e->logits, (size_t)e->c.vocab * 4, hipMemcpyDeviceToHost, e->stream));
                HIPCK(e, hipStreamSynchronize(e->stream));
                if (out != e->h_logits) memcpy(out, e->h_logits, (size_t)e->c.vocab * 4);
            } else HIPCK(e, hipMemcpyAsync(out + r0 * e->c.vocab, e->logits, (size_t)nr * e->c.vocab * 4, hipMemcpyDeviceToHost, e->stream));
        }
        HIPCK(e, hipStreamSynchronize(e->stream));
        if (argmax_out) memcpy(argmax_out + r0, e->h_ids, (size_t)nr * 4);
    }
    for (const Piece &p : ps) e->next_pos[p.stream] = p.pos0 + p.n;
    return NL_OK;
}

// a decode batch of at most FEW_MAX_TOKENS streams
int run_decode(nl_engine *e, const int *streams, const int *tokens, const int *pos, int n, float *logits_out, int *next_ids) {
    HIPCK(e, hipStreamSynchronize(e->stream));
    int mp = 0;
    for (int i = 0; i < n; i++) {
        e->h_meta[i] = tokens[i]; e->h_meta[e->m_pos + i] = pos[i]; e->h_meta[e->m_stream + i] = streams[i];
        mp = std::max(mp, pos[i]);
    }
    HIPCK(e, hipMemcpyAsync(e->d_meta, e->h_meta, (size_t)e->m_rows * sizeof(int), hipMemcpyHostToDevice, e->stream));
    if (int rc = queue_decode(e, CH_BATCH, n, mp)) return rc;
    if (next_ids) HIPCK(e, hipMemcpyAsync(e->h_ids, e->ids, (size_t)n * 4, hipMemcpyDeviceToHost, e->stream));
    if (logits_out) HIPCK(e, hipMemcpyAsync(logits_out, e->logits, (size_t)n * e->c.vocab * 4, hipMemcpyDeviceToHost, e->stream));
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (next_ids) memcpy(next_ids, e->h_ids, (size_t)n * 4);
    for (int i = 0; i < n; i++) e->next_pos[streams[i]] = pos[i] + 1;
    return NL_OK;
}

}  // namespace

// ================================================================== C ABI ===

extern "C" {

int nl_abi_version(void) { return 2; }
#ifndef NL_SRC_SHA
#define NL_SRC_SHA "unknown"
#endif
#ifndef NL_GIT_HEAD
#define NL_GIT_HEAD "unknown"
#endif
const char *nl_build_info(void) { return "src=" NL_SRC_SHA " git=" NL_GIT_HEAD; }
int nl_device_count(void) {
    int n = 0;
    return hipGetDeviceCount(&n) == hipSuccess ? n : 0;
}
const char *nl_last_error(nl_handle h) { return h ? h->err.c_str() : g_create_error.c_str(); }

int nl_create_stack(const nl_stack_config *cfg, const nl_layer_desc *ld, nl_handle *out) {
    if (!cfg || !ld || !out) { g_create_error = "null argument"; return NL_ERR_INVALID; }
    *out = nullptr;
    nl_stack_config c = *cfg;
    if (c.max_streams <= 0) c.max_streams = 1;
    if (c.max_step_tokens <= 0) c.max_step_tokens = 2048;
    auto bad = [&](const std::string &m) { g_create_error = m; return (int)NL_ERR_INVALID; };
    auto no = [&](const std::string &m) { g_create_error = m; return (int)NL_ERR_UNSUPPORTED; };
    if (c.vocab <= 0 || c.dim <= 0 || c.n_layers <= 0 || c.seq_len <= 0) return bad("config: non-positive dimension");
    if (c.dtype != NL_DTYPE_BF16 && c.dtype != NL_DTYPE_F32) return bad("config: dtype");
    if (c.loop_times > 1 && c.post_norm) return no("config: a loop in a model with norms behind its sublayers");
    if (c.loop_times > 1 && (c.loop_start < 0 || c.loop_stop <= c.loop_start || c.loop_stop > c.n_layers)) return bad("config: loop range");
    for (int i = 0; i < c.n_layers; i++) {
        const nl_attn_desc &A = ld[i].attn;
        const nl_linattn_desc &G = ld[i].lin;
        const std::string at = "layer " + std::to_string(i) + ": ";
        const nl_latent_desc &N = ld[i].latent;
        if (!A.heads && !G.heads && !N.heads) return bad(at + "no mixer");
        if (N.heads) {
            if (A.heads || G.heads) return no(at + "latent attention beside another mixer");
            if (N.heads < 0 || N.dim <= 0 || N.rot_dim <= 0 || N.vdim <= 0 || N.q_rank <= 0 || N.kv_rank <= 0 || N.rot_dims < 0 || N.rot_dims % 2 || N.rot_dims > N.rot_dim ||
                !(N.rope_base > 0.0)) return bad(at + "latent attention sizes");
            if (N.yarn_factor != 0.0 && (!(N.yarn_factor > 0.0) || !(N.yarn_original > 0.0) || !(N.yarn_fast > 0.0) || !(N.yarn_slow > 0.0) || N.rope_base == 1.0))
                return bad(at + "rotary scaling");
            if (up(N.dim, 32) + up(N.rot_dim, 32) > WA_MAX_DIM || N.vdim > WA_MAX_DIM) return no(at + "latent attention head sizes up to 256");
            if (up(N.kv_rank, 32) + up(N.rot_dim, 32) > LT_MAX_TILES * 32) return no(at + "latent and rotated key sizes up to 768 together");
            if (N.kv_from >= 0) {
                const nl_latent_desc &S = ld[std::min(N.kv_from, i)].latent;
                if (N.kv_from >= i || !S.heads || S.kv_from >= 0 || S.kv_rank != N.kv_rank || S.rot_dim != N.rot_dim || S.rot_dims != N.rot_dims || S.rot_adjacent != N.rot_adjacent)
                    return bad(at + "kv_from must name an earlier latent attention layer with keys of its own and equal key sizes");
            }
        }
        if (A.heads) {
            if (A.heads < 0 || A.kv_heads <= 0 || A.heads % A.kv_heads || A.dim <= 0 || A.vdim <= 0 || A.window < 0) return bad(at + "attention sizes");
            if (A.dim > WA_MAX_DIM || A.vdim > WA_MAX_DIM) return no(at + "attention head sizes up to 256");
        }
        if (G.heads) {
            if (G.heads < 0 || G.dim <= 0 || G.vdim <= 0 || G.rank <= 0 || !(G.tau > 0.f)) return bad(at + "linear attention sizes");
            if (G.dim > LA_MAX_DIM || G.vdim > LA_MAX_DIM || G.rank > 1024) return no(at + "linear attention head sizes up to 256, rank up to 1024");
        }
        if (ld[i].ff < 0 || (ld[i].ff_act != NL_ACT_GELU_TANH && ld[i].ff_act != NL_ACT_SILU)) return bad(at + "feed-forward");
        if (ld[i].ff && ld[i].ff_bias && !c.post_norm) return no(at + "feed-forward biases without norms behind the sublayers");
    }
    int ndev = 0;
    hipError_t s = hipGetDeviceCount(&ndev);
    if (s != hipSuccess || ndev == 0) { g_create_error = std::string("no HIP device: ") + hipGetErrorString(s); return NL_ERR_HIP; }
    if (c.device < 0 || c.device >= ndev) return bad("config: device ordinal out of range");
    nl_engine *e = new nl_engine();
    e->c = c;
    e->use_graph = !(c.flags & NL_FLAG_NO_GRAPH) && !getenv("NL_NO_GRAPH");
    auto fail = [&](int rc) { g_create_error = e->err; nl_destroy(e); return rc; };
    if ((s = hipSetDevice(c.device)) != hipSuccess || (s = hipStreamCreateWithFlags(&e->stream, hipStreamNonBlocking)) != hipSuccess ||
        (s = hipEventCreate(&e->ev0)) != hipSuccess || (s = hipEventCreate(&e->ev1)) != hipSuccess) {
        e->err = std::string("device init: ") + hipGetErrorString(s);
        return fail(NL_ERR_HIP);
    }
    const int D = c.dim;
    size_t &bw = e->bytes_weights;
    int rc;
    e->nksd = (D + 31) / 32;
    if ((rc = mat_alloc(e, e->embed, c.vocab, D)) || (rc = dev_alloc(e, e->final_norm, (size_t)D * 4, bw))) return fail(rc);
    e->head = e->embed;
    if (c.untied && (rc = mat_alloc(e, e->head, c.vocab, D))) return fail(rc);
    e->layers.resize(c.n_layers);
    for (int i = 0; i < c.n_layers; i++) {
        Layer &L = e->layers[i];
        L.d = ld[i];
        const nl_attn_desc &A = L.d.attn;
        const nl_linattn_desc &G = L.d.lin;
        int rows = 0;
        auto block = [&](int n) { const int at = rows; rows += up(n, 16); return at; };
        if (A.heads) {
            L.aq = block(A.heads * A.dim); L.ak = block(A.kv_heads * A.dim); L.av = block(A.kv_heads * A.vdim);
            if (A.gate) L.ag = block(A.heads * A.vdim);
            L.nks = (A.dim + 31) / 32; L.nvt = (A.vdim + 15) / 16;
            L.y_lin = up(A.heads * A.vdim, 32);
        }
        if (G.heads) {
            L.lq = block(G.heads * G.dim); L.lk = block(G.heads * G.dim); L.lv = block(G.heads * G.vdim); L.lg = block(G.heads * G.vdim); L.la1 = block(G.rank);
            L.dkp = up(G.dim, 16); L.dvp = up(G.vdim, 16);
        }
        const nl_latent_desc &N = L.d.latent;
        if (N.heads) {
            e->latent = true;
            L.tdq = block(N.q_rank);
            if (N.kv_from < 0) L.tdkv = block(N.kv_rank + N.rot_dim);
            if (N.gate) L.tg = block(N.heads);
            L.dimp = up(N.dim, 32); L.rotp = up(N.rot_dim, 32); L.vdp = up(N.vdim, 16); L.kvt = up(N.kv_rank, 32) / 32; L.nks = L.kvt + L.rotp / 32;
            L.y_lin = N.heads * N.vdim;
            if ((rc = mat_alloc(e, L.uq, N.heads * (L.dimp + L.rotp), N.q_rank)) || (rc = mat_alloc(e, L.uk, N.heads * L.dimp, N.kv_rank)) ||
                (rc = mat_alloc(e, L.ukt, N.heads * L.kvt * 32, L.dimp)) || (rc = mat_alloc(e, L.uv, N.heads * L.vdp, N.kv_rank)) ||
                (rc = dev_alloc(e, L.dqnorm, (size_t)N.q_rank * 4, bw)) || (rc = dev_alloc(e, L.kvnorm, (size_t)N.kv_rank * 4, bw)) ||
                (N.sink && (rc = dev_alloc(e, L.sink, (size_t)N.heads * 4, bw)))) return fail(rc);
        }
        if (c.post_norm && ((rc = dev_alloc(e, L.norm1p, (size_t)D * 4, bw)) || (rc = dev_alloc(e, L.norm2p, (size_t)D * 4, bw)))) return fail(rc);
        if (L.d.ff && L.d.ff_bias && ((rc = dev_alloc(e, L.gateb, (size_t)up(L.d.ff, 16) * 4, bw)) || (rc = dev_alloc(e, L.upb, (size_t)up(L.d.ff, 16) * 4, bw)) ||
                                      (rc = dev_alloc(e, L.downb, (size_t)up(D, 16) * 4, bw)))) return fail(rc);
        if ((rc = mat_alloc(e, L.proj, rows, D)) || (rc = mat_alloc(e, L.out, D, L.y_lin + G.heads * G.vdim)) || (rc = dev_alloc(e, L.norm1, (size_t)D * 4, bw))) return fail(rc);
        if (A.heads && A.qk_norm && ((rc = dev_alloc(e, L.qnorm, (size_t)A.dim * 4, bw)) || (rc = dev_alloc(e, L.knorm, (size_t)A.dim * 4, bw)))) return fail(rc);
        if (A.heads && A.distance_bias) {
            std::vector<float> sl(A.heads);
            for (int h = 0; h < A.heads; h++) sl[h] = (float)std::exp2(-8.0 * (h + 1) / A.heads);
            if ((rc = dev_alloc(e, L.slope, (size_t)A.heads * 4, bw))) return fail(rc);
            if ((s = hipStreamSynchronize(e->stream)) != hipSuccess || (s = hipMemcpy(L.slope, sl.data(), (size_t)A.heads * 4, hipMemcpyHostToDevice)) != hipSuccess) {
                e->err = hipGetErrorString(s);
                return fail(NL_ERR_HIP);
            }
        }
        if (G.heads && ((rc = dev_alloc(e, L.a2, (size_t)G.heads * G.dim * G.rank * 4, bw)) || (rc = dev_alloc(e, L.a2b, (size_t)G.heads * G.dim * 4, bw)) ||
                        (rc = dev_alloc(e, L.lnorm, (size_t)G.vdim * 4, bw)))) return fail(rc);
        if (L.d.ff && ((rc = mat_alloc(e, L.gateup, 2 * up(L.d.ff, 16), D)) || (rc = mat_alloc(e, L.down, D, L.d.ff)) || (rc = dev_alloc(e, L.norm2, (size_t)D * 4, bw)))) return fail(rc);
    }
    // the order of execution
    const int lt = std::max(1, c.loop_times);
    auto add = [&](int a, int b) { for (int i = a; i < b; i++) { Run r; r.layer = i; e->runs.push_back(r); } };
    if (lt == 1) add(0, c.n_layers);
    else {
        add(0, c.loop_start);
        for (int p = 0; p < lt; p++) {
            add(c.loop_start, c.loop_stop);
            if (p + 1 < lt) e->runs.back().add_embed = true;
        }
        add(c.loop_stop, c.n_layers);
    }
    for (size_t r = 0; r < e->runs.size(); r++) {
        const nl_latent_desc &N = e->layers[e->runs[r].layer].d.latent;
        e->runs[r].kv_run = (int)r;
        if (N.heads && N.kv_from >= 0)
            for (size_t q = 0; q < r; q++)
                if (e->runs[q].layer == N.kv_from) e->runs[r].kv_run = (int)q;
    }
    nl_config &g = e->cfg;
    g.n_layers = c.n_layers; g.dim = D; g.vocab = c.vocab; g.seq_len = c.seq_len; g.rms_eps = c.eps; g.max_streams = c.max_streams; g.device = c.device;
    g.tp_size = 1; g.flags = c.flags;
    *out = e;
    return NL_OK;
}

int nl_get_config(nl_handle h, nl_config *out) {
    if (!h || !out) return NL_ERR_INVALID;
    *out = h->cfg;
    return NL_OK;
}

int nl_upload_tensor(nl_handle e, const char *name, uint32_t type, const void *data, uint64_t nbytes, uint64_t rows, uint64_t cols) {
    if (!e || !name || !data) return NL_ERR_INVALID;
    if (e->finalized) return e->fail(NL_ERR_STATE, "upload after nl_finalize");
    if (type != NL_GGML_F32 && type != NL_GGML_BF16) return e->fail(NL_ERR_UNSUPPORTED, "%s: tensor type %u (float32 and bfloat16 are taken)", name, type);
    Dest d;
    if (!find_dest(e, name, d)) return e->fail(NL_ERR_INVALID, "unknown tensor %s", name);
    if ((long long)rows != d.rows || (long long)cols != d.cols)
        return e->fail(NL_ERR_INVALID, "%s is [%llu, %llu], expected [%lld, %lld]", name, (unsigned long long)rows, (unsigned long long)cols, d.rows, d.cols);
    const size_t need = (size_t)d.rows * d.cols * (type == NL_GGML_F32 ? 4 : 2);
    if (nbytes != need) return e->fail(NL_ERR_INVALID, "%s: %llu bytes, expected %zu", name, (unsigned long long)nbytes, need);
    HIPCK(e, hipSetDevice(e->c.device));
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (e->stage_cap < need) {
        if (e->stage) HIPCK(e, hipFree(e->stage));
        e->stage = nullptr;
        e->stage_cap = 0;
        HIPCK(e, hipMalloc(&e->stage, need));
        e->stage_cap = need;
    }
    HIPCK(e, hipMemcpy(e->stage, data, need, hipMemcpyHostToDevice));
    const long long n = d.rows * d.cols;
    const int f32 = type == NL_GGML_F32, grid = (int)std::min<long long>((n + 255) / 256, 8192);
    if (d.mapped[0]) {
        int *maps = nullptr;
        HIPCK(e, hipMalloc((void **)&maps, (size_t)d.rows * 2 * sizeof(int)));
        hipError_t s = hipSuccess;
        for (int i = 0; i < 2 && d.mapped[i] && s == hipSuccess; i++) {
            Mat &m = *d.mapped[i];
            if ((s = hipMemcpy(maps, d.rbase[i].data(), (size_t)d.rows * sizeof(int), hipMemcpyHostToDevice)) != hipSuccess ||
                (s = hipMemcpy(maps + d.rows, d.kbase[i].data(), (size_t)d.rows * sizeof(int), hipMemcpyHostToDevice)) != hipSuccess) break;
            if (e->f32()) hipLaunchKernelGGL(pack_mapped_kernel<float>, dim3(grid), dim3(256), 0, e->stream, e->stage, f32, d.rows, d.cols, reinterpret_cast<float *>(m.w), m.nks, maps, maps + d.rows, (int)d.tr[i]);
            else hipLaunchKernelGGL(pack_mapped_kernel<bf16>, dim3(grid), dim3(256), 0, e->stream, e->stage, f32, d.rows, d.cols, reinterpret_cast<bf16 *>(m.w), m.nks, maps, maps + d.rows, (int)d.tr[i]);
            s = hipStreamSynchronize(e->stream);     // (the maps are reused)
        }
        (void)hipFree(maps);
        HIPCK(e, s);
    } else if (d.vec) hipLaunchKernelGGL(widen_kernel, dim3(grid), dim3(256), 0, e->stream, e->stage, f32, n, d.add, d.vec, d.transpose ? (int)d.cols : 1);
    else if (e->f32()) hipLaunchKernelGGL(pack_operand_kernel<float>, dim3(grid), dim3(256), 0, e->stream, e->stage, f32, d.rows, d.cols, reinterpret_cast<float *>(d.mat->w), d.mat->nks, d.row0, d.k0, d.tstride, d.toff);
    else hipLaunchKernelGGL(pack_operand_kernel<bf16>, dim3(grid), dim3(256), 0, e->stream, e->stage, f32, d.rows, d.cols, reinterpret_cast<bf16 *>(d.mat->w), d.mat->nks, d.row0, d.k0, d.tstride, d.toff);
    HIPCK(e, hipGetLastError());
    HIPCK(e, hipStreamSynchronize(e->stream));       // the staging buffer is reused
    e->have.insert(name);
    return NL_OK;
}

int nl_finalize(nl_handle e) {
    if (!e) return NL_ERR_INVALID;
    if (e->finalized) return e->fail(NL_ERR_STATE, "nl_finalize called twice");
    for (const std::string &w : wanted_tensors(e))
        if (!e->have.count(w)) return e->fail(NL_ERR_MISSING, "tensor %s was not uploaded", w.c_str());
    HIPCK(e, hipSetDevice(e->c.device));
    if (e->stage) { HIPCK(e, hipFree(e->stage)); e->stage = nullptr; e->stage_cap = 0; }
    const int D = e->c.dim, S = e->c.max_streams;
    const size_t es = e->esize();
    e->cap = std::min(up(e->c.max_step_tokens, 64), up(std::max(e->c.seq_len, std::min(S, FEW_MAX_TOKENS)), 64));
    const int cap = e->cap, few = std::min(std::max(S, 1), FEW_MAX_TOKENS);
    e->lm_cap = std::max(FEW_MAX_TOKENS, std::min(cap, 256));
    int ldmax = 0, yk = 0, ak = 0, hk = e->nksd;
    size_t xq = 0, ek = 0, ev = 0, lpart = 0, lml = 0;
    std::map<std::tuple<int, double, double, double, double, double>, float *> ropes;
    // scratch for expanded keys: the longest sequence, or whole prompts that fill a launch sequence
    e->kv_slots = std::max(up(e->c.seq_len, 64), 2 * cap);
    size_t qrow = 0, qfew = 0, ldec = 0, inc = 0, tot = 0, part = 0, arr = 0;
    const int segs = cap / LA_SEG + std::min(cap, S) + 1, subs = cap / LA_SUB + std::min(cap, S) + 1, tiles = cap / WA_Q + std::min(cap, S) + 1;
    for (Layer &L : e->layers) {
        const nl_attn_desc &A = L.d.attn;
        const nl_linattn_desc &G = L.d.lin;
        ldmax = std::max(ldmax, L.proj.rows); yk = std::max(yk, L.out.nks); ak = std::max(ak, L.d.ff ? L.down.nks : 0);
        if (A.heads) {
            // the ring: every position while they fit, else what the window needs beside the tokens one launch sequence adds
            const long long whole = up(e->c.seq_len, 64), ring = A.window > 0 ? (long long)up(A.window - 1 + cap, 64) : whole;
            L.R = (int)std::min(whole, ring);
            qrow = std::max(qrow, (size_t)A.heads * L.nks * 32);
            for (int n = 1; n <= few; n++) {
                const size_t sp = splits_for(e, n, e->c.seq_len - 1);
                part = std::max(part, (size_t)n * A.heads * sp * (A.vdim + 2));
            }
            arr = std::max(arr, (size_t)few * A.heads);
        }
        const nl_latent_desc &N = L.d.latent;
        if (N.heads) {
            L.R = up(e->c.seq_len, 64);
            hk = std::max(hk, L.uq.nks);
            qrow = std::max(qrow, (size_t)N.heads * (L.dimp + L.rotp));
            ek = std::max(ek, (size_t)N.heads * e->kv_slots * (L.dimp + L.rotp));
            ev = std::max(ev, (size_t)N.heads * e->kv_slots * L.vdp);
            xq = std::max(xq, (size_t)up(few, 16) * N.heads * L.dimp);
            qfew = std::max(qfew, (size_t)few * N.heads * L.nks * 32);
            for (int n = 1; n <= few; n++) {
                const size_t sp = splits_for(e, n, e->c.seq_len - 1);
                lpart = std::max(lpart, (size_t)n * N.heads * sp * L.kvt * 32);
                lml = std::max(lml, (size_t)n * N.heads * sp * 2);
            }
            float *&rope = ropes[std::make_tuple(N.rot_dims, N.rope_base, N.yarn_factor, N.yarn_original, N.yarn_fast, N.yarn_slow)];
            if (!rope && N.rot_dims) {
                const std::vector<float> t = rope_table(N, e->c.seq_len);
                if (int rc = dev_alloc(e, rope, t.size() * 4, e->bytes_weights)) return rc;
                HIPCK(e, hipStreamSynchronize(e->stream));
                HIPCK(e, hipMemcpy(rope, t.data(), t.size() * 4, hipMemcpyHostToDevice));
            }
            L.rope = rope;
        }
        if (G.heads) {
            ldec = std::max(ldec, (size_t)cap * G.heads * G.dim);
            inc = std::max(inc, (size_t)segs * G.heads * L.dkp * L.dvp);
            tot = std::max(tot, (size_t)segs * G.heads * L.dkp);
        }
    }
    size_t &bs = e->bytes_state, &bk = e->bytes_kv;
    const size_t tt = (size_t)up(cap, 128) / 16;         // token tiles (whole token blocks)
    int rc;
    bool loop = false;
    for (const Run &r : e->runs) loop |= r.add_embed;
    if ((rc = dev_alloc(e, e->x, (size_t)cap * D * 4, bs)) || (loop && (rc = dev_alloc(e, e->x0, (size_t)cap * D * 4, bs))) ||
        (rc = dev_alloc(e, e->proj, (size_t)cap * ldmax * 4, bs)) || (rc = dev_alloc(e, e->logits, (size_t)e->lm_cap * e->c.vocab * 4, bs)) ||
        (rc = dev_alloc(e, e->h, std::max(tt, (size_t)up(e->lm_cap, 128) / 16) * hk * OPT * es, bs)) || (rc = dev_alloc(e, e->y, tt * yk * OPT * es, bs)) ||
        (ak && (rc = dev_alloc(e, e->act, tt * ak * OPT * es, bs))) || (qrow && (rc = dev_alloc(e, e->q, std::max((size_t)cap * qrow, qfew) * es, bs))) ||
        (e->c.post_norm && ((rc = dev_alloc(e, e->x2, (size_t)cap * D * 4, bs)) || (rc = dev_alloc(e, e->delta, (size_t)cap * D * 4, bs)))) ||
        (e->latent && ((rc = dev_alloc(e, e->xq, xq * es, bs)) || (rc = dev_alloc(e, e->ek, ek * es, bs)) || (rc = dev_alloc(e, e->ev, ev * es, bs)) ||
                       (rc = dev_alloc(e, e->lpart, lpart * 4, bs)) || (rc = dev_alloc(e, e->lml, lml * 4, bs)))) ||
        (ldec && ((rc = dev_alloc(e, e->ldec, ldec * 4, bs)) || (rc = dev_alloc(e, e->inc, inc * 4, bs)) || (rc = dev_alloc(e, e->totlog, tot * 4, bs)))) ||
        (arr && ((rc = dev_alloc(e, e->part, part * 4, bs)) || (rc = dev_alloc(e, e->arrived, arr * 4, bs)))))
        return rc;
    e->seg_cap = segs;
    for (Run &r : e->runs) {
        const Layer &L = e->layers[r.layer];
        if (L.d.attn.heads) {
            r.kstride = (long long)L.d.attn.kv_heads * L.R * L.nks * 32;
            r.vstride = (long long)L.d.attn.kv_heads * L.R * L.nvt * 16;
            if ((rc = dev_alloc(e, r.K, (size_t)S * r.kstride * es, bk)) || (rc = dev_alloc(e, r.V, (size_t)S * r.vstride * es, bk))) return rc;
        }
        if (L.d.latent.heads && L.d.latent.kv_from < 0) {
            r.kstride = (long long)L.R * L.nks * 32;
            if ((rc = dev_alloc(e, r.K, (size_t)S * r.kstride * es, bk))) return rc;
        }
        if (L.d.lin.heads) {
            r.sstride = (long long)L.d.lin.heads * L.dkp * L.dvp;
            if ((rc = dev_alloc(e, r.state, (size_t)S * r.sstride * 4, bk))) return rc;
        }
    }
    const int tk = std::max(cap, FEW_MAX_TOKENS);
    e->m_pos = tk; e->m_stream = 2 * tk; e->m_rows = 3 * tk;
    e->m_subs = 4 * tk;
    e->m_segs = e->m_subs + subs * (int)(sizeof(GlaSub) / 4);
    e->m_tiles = e->m_segs + segs * (int)(sizeof(GlaSeg) / 4);
    e->m_runs = e->m_tiles + tiles * (int)(sizeof(WinTile) / 4);
    e->m_keys = e->m_runs + segs;
    e->m_words = e->m_keys + (e->latent ? std::min(cap, S) * (up(e->c.seq_len, 64) / 16) : 0);
    if ((rc = dev_alloc(e, e->d_meta, (size_t)e->m_words * 4, bs)) || (rc = dev_alloc(e, e->ctl, CTL_WORDS * 4, bs)) ||
        (rc = dev_alloc(e, e->ids, (size_t)std::max(e->ids_cap, e->lm_cap) * 4, bs)) || (rc = dev_alloc(e, e->result, 4, bs)) ||
        (rc = dev_alloc(e, e->amax_val, (size_t)e->head.nrt * 4, bs)) || (rc = dev_alloc(e, e->amax_idx, (size_t)e->head.nrt * 4, bs))) return rc;
    HIPCK(e, hipHostMalloc((void **)&e->h_meta, (size_t)e->m_words * 4, hipHostMallocDefault));
    HIPCK(e, hipHostMalloc((void **)&e->h_ctl, 64, hipHostMallocDefault));
    HIPCK(e, hipHostMalloc((void **)&e->h_ids, (size_t)std::max(e->ids_cap, e->lm_cap) * 4, hipHostMallocDefault));
    HIPCK(e, hipHostMalloc((void **)&e->h_logits, (size_t)e->c.vocab * 4, hipHostMallocDefault));
    memset(e->h_meta, 0, (size_t)e->m_words * 4);
    e->next_pos.assign(S, 0);
    HIPCK(e, hipStreamSynchronize(e->stream));
    e->finalized = true;
    return NL_OK;
}

int nl_destroy(nl_handle e) {
    if (!e) return NL_OK;
    (void)hipSetDevice(e->c.device);
    if (e->stream) (void)hipStreamSynchronize(e->stream);
    for (auto &g : e->graphs) { (void)hipGraphExecDestroy(g.second.x); (void)hipGraphDestroy(g.second.g); }
    samp_free(e->sp);
    for (void *p : e->allocs) (void)hipFree(p);
    if (e->stage) (void)hipFree(e->stage);
    if (e->tracebuf) (void)hipFree(e->tracebuf);
    void *pinned[] = {e->h_meta, e->h_ctl, e->h_ids, e->h_logits};
    for (void *p : pinned) if (p) (void)hipHostFree(p);
    if (e->ev0) (void)hipEventDestroy(e->ev0);
    if (e->ev1) (void)hipEventDestroy(e->ev1);
    if (e->stream) (void)hipStreamDestroy(e->stream);
    delete e;
    return NL_OK;
}

// O(1): keys of other requests are never visible (masked by position) and a stream's step at position 0 starts from a zero state
int nl_reset(nl_handle e, int stream) {
    if (!e) return NL_ERR_INVALID;
    if (!e->finalized) return e->fail(NL_ERR_STATE, "reset before nl_finalize");
    if (stream < 0 || stream >= e->c.max_streams) return e->fail(NL_ERR_INVALID, "stream %d out of range", stream);
    e->next_pos[stream] = 0;
    return NL_OK;
}

float *nl_host_logits(nl_handle e) { return e && e->finalized ? e->h_logits : nullptr; }

static int one_token(nl_handle e, int stream, int token, int pos, float *logits_out, int *next_id) {
    if (!e) return NL_ERR_INVALID;
    int rc = check_tokens(e, stream, &token, 1, pos);
    if (rc) return rc;
    HIPCK(e, hipSetDevice(e->c.device));
    if ((rc = set_ctl(e, token, pos, 0, stream)) || (rc = queue_decode(e, CH_CALL, 1, pos))) return rc;
    if (logits_out) HIPCK(e, hipMemcpyAsync(e->h_logits, e->logits, (size_t)e->c.vocab * 4, hipMemcpyDeviceToHost, e->stream));
    if (next_id) HIPCK(e, hipMemcpyAsync(e->h_ids, e->result, 4, hipMemcpyDeviceToHost, e->stream));
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (logits_out && logits_out != e->h_logits) memcpy(logits_out, e->h_logits, (size_t)e->c.vocab * 4);
    if (next_id) *next_id = e->h_ids[0];
    e->next_pos[stream] = pos + 1;
    return NL_OK;
}
int nl_forward(nl_handle e, int stream, int token, int pos, float *logits_out) { return one_token(e, stream, token, pos, logits_out, nullptr); }
int nl_forward_argmax(nl_handle e, int stream, int token, int pos, int *next_id) {
    return next_id ? one_token(e, stream, token, pos, nullptr, next_id) : (int)NL_ERR_INVALID;
}

int nl_decode_greedy(nl_handle e, int stream, int token, int pos, int n_steps, int *ids_out, int *n_done) {
    if (!e || !ids_out || n_steps < 0) return NL_ERR_INVALID;
    int rc = check_tokens(e, stream, &token, 1, pos);
    if (rc) return rc;
    HIPCK(e, hipSetDevice(e->c.device));
    const int n = std::min({n_steps, e->c.seq_len - pos, e->ids_cap});
    if ((rc = set_ctl(e, token, pos, 1, stream))) return rc;
    for (int i = 0; i < n;) {
        const int k = n - i >= CHAIN_STEPS ? CHAIN_STEPS : 1;
        if ((rc = queue_decode(e, CH_CHAIN, 1, pos + i + k - 1, k))) return rc;
        i += k;
    }
    if (n > 0) HIPCK(e, hipMemcpyAsync(e->h_ids, e->ids, (size_t)n * 4, hipMemcpyDeviceToHost, e->stream));
    HIPCK(e, hipStreamSynchronize(e->stream));
    memcpy(ids_out, e->h_ids, (size_t)n * 4);
    if (n > 0) e->next_pos[stream] = pos + n;
    if (n_done) *n_done = n;
    return NL_OK;
}

int nl_sample_decode(nl_handle e, int stream, int pos, int n_steps, const nl_sample_params *p, const float *uniforms, int *recent,
                     int *n_recent, int *ids_out, int *n_done) {
    if (!e || !ids_out || !uniforms || !recent || !n_recent || n_steps < 0) return NL_ERR_INVALID;
    if (const char *m = sample_params_error(p)) return e->fail(NL_ERR_INVALID, "%s", m);
    if (!e->finalized) return e->fail(NL_ERR_STATE, "sample before nl_finalize");
    if (stream < 0 || stream >= e->c.max_streams) return e->fail(NL_ERR_INVALID, "stream %d out of range", stream);
    if (pos < 1 || pos > e->c.seq_len) return e->fail(NL_ERR_INVALID, "pos %d out of range [1,%d]", pos, e->c.seq_len);
    if (pos != e->next_pos[stream]) return e->fail(NL_ERR_STATE, "stream %d goes on at position %d, not at %d", stream, e->next_pos[stream], pos);
    if (*n_recent < 0 || *n_recent > p->rep_window) return e->fail(NL_ERR_INVALID, "n_recent %d exceeds rep_window %d", *n_recent, p->rep_window);
    HIPCK(e, hipSetDevice(e->c.device));
    const int n = std::min({n_steps, e->c.seq_len - pos, e->ids_cap});
    if (n_done) *n_done = std::max(n, 0);
    if (n <= 0) return NL_OK;
    int rc;
    if (e->sp_cap < n) {
        HIPCK(e, hipStreamSynchronize(e->stream));
        samp_free(e->sp);
        e->sp_cap = 0;
        HIPCK(e, samp_alloc(e->sp, e->c.vocab, e->ids_cap));
        HIPCK(e, hipDeviceSynchronize());            // (its clears ran on another stream)
        e->sp_cap = e->ids_cap;
    }
    // the sampler stores its pick as the next token and moves the position on: it starts one below
    if ((rc = set_ctl(e, 0, pos - 1, 0, stream))) return rc;
    HIPCK(e, hipMemcpyAsync(e->sp.uniforms, uniforms, (size_t)n * 4, hipMemcpyHostToDevice, e->stream));
    if (*n_recent > 0) HIPCK(e, hipMemcpyAsync(e->sp.recent, recent, (size_t)*n_recent * 4, hipMemcpyHostToDevice, e->stream));
    HIPCK(e, hipMemcpyAsync(e->sp.recent_n, n_recent, 4, hipMemcpyHostToDevice, e->stream));
    for (int i = 0; i < n; i++) {
        HIPCK(e, launch_sample(e->sp, e->logits, e->c.vocab, *p, e->ctl, e->ids, e->stream));
        if ((rc = queue_decode(e, CH_SAMPLE, 1, pos + i))) return rc;
    }
    HIPCK(e, hipMemcpyAsync(ids_out, e->ids, (size_t)n * 4, hipMemcpyDeviceToHost, e->stream));
    HIPCK(e, hipMemcpyAsync(n_recent, e->sp.recent_n, 4, hipMemcpyDeviceToHost, e->stream));
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (*n_recent > 0) HIPCK(e, hipMemcpy(recent, e->sp.recent, (size_t)*n_recent * 4, hipMemcpyDeviceToHost));
    e->next_pos[stream] = pos + n;
    return NL_OK;
}

// checked entries, all decode launches (one token each) or all prompt launches
static int step_entries(nl_handle e, int n_entries, const int *streams, const int *n_tokens, const int *pos0, const int *tokens, int n_want,
                        const int *want, float *logits_out, int *next_ids) {
    const int V = e->c.vocab;
    int rc;
    if (std::all_of(n_tokens, n_tokens + n_entries, [](int k) { return k == 1; })) {
        std::vector<float> all;
        for (int i0 = 0, w = 0; i0 < n_entries; i0 += FEW_MAX_TOKENS) {
            const int m = std::min(FEW_MAX_TOKENS, n_entries - i0);
            int w1 = w;
            while (w1 < n_want && want[w1] < i0 + m) w1++;
            const bool direct = w1 - w == m;             // every entry's row is wanted: no detour
            if (w1 > w && !direct) all.resize((size_t)m * V);
            if ((rc = run_decode(e, streams + i0, tokens + i0, pos0 + i0, m, w1 == w ? nullptr : direct ? logits_out + (size_t)w * V : all.data(),
                                 next_ids ? next_ids + i0 : nullptr))) return rc;
            if (!direct)
                for (int k = w; k < w1; k++) memcpy(logits_out + (size_t)k * V, all.data() + (size_t)(want[k] - i0) * V, (size_t)V * 4);
            w = w1;
        }
        return NL_OK;
    }
    // prompts: entries are cut so that a launch sequence holds at most cap tokens; an entry's cuts follow one another
    std::vector<Piece> ps;
    int room = e->cap, at = 0, w = 0;
    std::vector<int> last_of;                            // per piece: the entry whose last token it holds, or -1
    auto flush = [&]() -> int {
        if (ps.empty()) return NL_OK;
        std::vector<int> wl;                             // rows to compute: wanted ones and, for next_ids, the entries' last tokens
        std::vector<int> src;                            // ... index into want or -1
        std::vector<std::pair<int, int>> ends;           // (row, entry)
        int k = w;
        for (size_t i = 0; i < ps.size(); i++) {
            const int hi = ps[i].tok0 + ps[i].n;
            bool got = false;
            for (; k < n_want && want[k] < hi; k++) { wl.push_back(want[k]); src.push_back(k); got = want[k] == hi - 1; }
            if (next_ids && last_of[i] >= 0) {
                if (!got) { wl.push_back(hi - 1); src.push_back(-1); }
                ends.push_back({(int)wl.size() - 1, last_of[i]});
            }
        }
        const int nw = k - w;
        std::vector<int> am(next_ids ? wl.size() : 0);
        int r;
        if (nw == (int)wl.size()) r = run_pieces(e, ps, tokens, wl, nw ? logits_out + (size_t)w * V : nullptr, next_ids && !wl.empty() ? am.data() : nullptr);
        else {
            std::vector<float> all(nw ? wl.size() * (size_t)V : 0);
            r = run_pieces(e, ps, tokens, wl, nw ? all.data() : nullptr, am.data());
            if (!r && nw)
                for (size_t i = 0; i < wl.size(); i++)
                    if (src[i] >= 0) memcpy(logits_out + (size_t)src[i] * V, all.data() + i * V, (size_t)V * 4);
        }
        if (r) return r;
        for (auto &en : ends) next_ids[en.second] = am[en.first];
        w = k;
        ps.clear();
        last_of.clear();
        room = e->cap;
        return NL_OK;
    };
    for (int i = 0; i < n_entries; i++) {
        for (int t = 0; t < n_tokens[i];) {
            if (room == 0 && (rc = flush())) return rc;
            const int m = std::min(room, n_tokens[i] - t);
            ps.push_back({streams[i], at + t, m, pos0[i] + t});
            t += m;
            room -= m;
            last_of.push_back(t == n_tokens[i] ? i : -1);
        }
        at += n_tokens[i];
    }
    return flush();
}

int nl_step(nl_handle e, int n_entries, const int *streams, const int *n_tokens, const int *pos0, const int *tokens, int n_want,
            const int *want, float *logits_out, int *next_ids) {
    if (!e || n_entries < 0 || n_want < 0) return NL_ERR_INVALID;
    if (n_entries == 0) return NL_OK;
    if (!streams || !n_tokens || !pos0 || !tokens || (n_want && (!want || !logits_out))) return e->fail(NL_ERR_INVALID, "null argument");
    int rc, total = 0;
    bool decode = true;
    std::set<int> seen;
    for (int i = 0; i < n_entries; i++) {
        if ((rc = check_tokens(e, streams[i], tokens + total, n_tokens[i], pos0[i]))) return rc;
        if (!seen.insert(streams[i]).second) return e->fail(NL_ERR_INVALID, "stream %d appears twice in one step", streams[i]);
        decode &= n_tokens[i] == 1;
        total += n_tokens[i];
    }
    for (int i = 0; i < n_want; i++)
        if (want[i] < 0 || want[i] >= total || (i && want[i] <= want[i - 1])) return e->fail(NL_ERR_INVALID, "want must be ascending indices of this step's tokens");
    HIPCK(e, hipSetDevice(e->c.device));
    if (e->latent && !decode && n_entries > 1) {
        // one-token entries attend the latents themselves: a decode batch of their own, the others' positions are expanded
        for (int part = 0; part < 2; part++) {
            std::vector<int> st, nt, p0, tk, wt, src, ent;
            for (int i = 0, at = 0, w = 0; i < n_entries; at += n_tokens[i++]) {
                const bool mine = (n_tokens[i] == 1) == (part == 0);
                for (; w < n_want && want[w] < at + n_tokens[i]; w++)
                    if (mine) { wt.push_back((int)tk.size() + want[w] - at); src.push_back(w); }
                if (!mine) continue;
                st.push_back(streams[i]); nt.push_back(n_tokens[i]); p0.push_back(pos0[i]); ent.push_back(i);
                tk.insert(tk.end(), tokens + at, tokens + at + n_tokens[i]);
            }
            if (st.empty()) continue;
            if ((int)st.size() == n_entries) break;      // (no entry of one token: the whole step below)
            std::vector<float> lg(wt.size() * (size_t)e->c.vocab);
            std::vector<int> ids(st.size());
            if ((rc = step_entries(e, (int)st.size(), st.data(), nt.data(), p0.data(), tk.data(), (int)wt.size(), wt.data(), lg.data(), next_ids ? ids.data() : nullptr))) return rc;
            for (size_t k = 0; k < src.size(); k++) memcpy(logits_out + (size_t)src[k] * e->c.vocab, lg.data() + k * e->c.vocab, (size_t)e->c.vocab * 4);
            if (next_ids)
                for (size_t k = 0; k < ent.size(); k++) next_ids[ent[k]] = ids[k];
            if (part == 1) return NL_OK;
        }
    }
    return step_entries(e, n_entries, streams, n_tokens, pos0, tokens, n_want, want, logits_out, next_ids);
}

int nl_prefill(nl_handle e, int stream, const int *tokens, int n, int pos0, float *last_logits_out) {
    if (!e || !tokens || n < 0) return NL_ERR_INVALID;
    if (n == 0) return NL_OK;
    int rc = check_tokens(e, stream, tokens, n, pos0);
    if (rc) return rc;
    HIPCK(e, hipSetDevice(e->c.device));
    for (int t = 0; t < n; t += e->cap) {
        const int m = std::min(e->cap, n - t);
        // the last token's logits stay on the device: the sampler and nl_decode_greedy's caller start from them
        const std::vector<int> want = t + m == n ? std::vector<int>{n - 1} : std::vector<int>{};
        if ((rc = run_pieces(e, {{stream, t, m, pos0 + t}}, tokens, want, t + m == n ? last_logits_out : nullptr, nullptr))) return rc;
    }
    return NL_OK;
}

int nl_forward_batch(nl_handle e, const int *streams, const int *tokens, const int *pos, int n, float *logits_out, int *next_ids) {
    if (!e || !streams || !tokens || !pos || n < 0) return NL_ERR_INVALID;
    if (n > e->c.max_streams) return e->fail(NL_ERR_INVALID, "batch of %d exceeds max_streams %d", n, e->c.max_streams);
    std::vector<int> one(std::max(n, 1), 1), want(std::max(n, 1));
    for (int i = 0; i < n; i++) want[i] = i;
    return nl_step(e, n, streams, one.data(), pos, tokens, logits_out ? n : 0, want.data(), logits_out, next_ids);
}

int nl_synchronize(nl_handle e) {
    if (!e) return NL_ERR_INVALID;
    HIPCK(e, hipStreamSynchronize(e->stream));
    return NL_OK;
}
int nl_timer_start(nl_handle e) {
    if (!e) return NL_ERR_INVALID;
    HIPCK(e, hipEventRecord(e->ev0, e->stream));
    return NL_OK;
}
int nl_timer_stop(nl_handle e, float *ms) {
    if (!e || !ms) return NL_ERR_INVALID;
    HIPCK(e, hipEventRecord(e->ev1, e->stream));
    HIPCK(e, hipEventSynchronize(e->ev1));
    HIPCK(e, hipEventElapsedTime(ms, e->ev0, e->ev1));
    return NL_OK;
}
int nl_memory_usage(nl_handle e, uint64_t *w, uint64_t *kv, uint64_t *st) {
    if (!e) return NL_ERR_INVALID;
    if (w) *w = e->bytes_weights;
    if (kv) *kv = e->bytes_kv;
    if (st) *st = e->bytes_state;
    return NL_OK;
}

int nl_trace_layers(nl_handle e, int on) {
    if (!e) return NL_ERR_INVALID;
    if (!e->finalized) return e->fail(NL_ERR_STATE, "trace before nl_finalize");
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (on && !e->tracebuf) HIPCK(e, hipMalloc((void **)&e->tracebuf, 2 * e->runs.size() * (size_t)e->cap * e->c.dim * 4));
    e->trace = on != 0;
    e->trace_tokens = 0;
    return NL_OK;
}

int64_t nl_debug_read(nl_handle e, const char *which, int stream, float *out, int64_t max_floats) {
    if (!e || !which || !out) return NL_ERR_INVALID;
    if (!e->finalized) return e->fail(NL_ERR_STATE, "read before nl_finalize");
    HIPCK(e, hipStreamSynchronize(e->stream));
    if (!strcmp(which, "layers")) {
        if (!e->trace) return e->fail(NL_ERR_STATE, "nl_trace_layers is off");
        const size_t per = (size_t)e->trace_tokens * e->c.dim, R = e->runs.size();
        if ((int64_t)(R * per) > max_floats) return e->fail(NL_ERR_INVALID, "buffer too small");
        HIPCK(e, hipMemcpy(out, e->tracebuf, R * per * 4, hipMemcpyDeviceToHost));
        std::vector<float> x0(per);
        for (size_t r = 0; r < R; r++)
            if (e->runs[r].add_embed) {
                HIPCK(e, hipMemcpy(x0.data(), e->tracebuf + (R + r) * per, per * 4, hipMemcpyDeviceToHost));
                for (size_t i = 0; i < per; i++) out[r * per + i] -= x0[i];
            }
        return (int64_t)(R * per);
    }
    const float *src = nullptr;
    int64_t n = 0;
    if (!strcmp(which, "x")) { src = e->xcur ? e->xcur : e->x; n = e->c.dim; }
    else if (!strcmp(which, "logits")) { src = e->logits; n = e->c.vocab; }
    else if (!strncmp(which, "state", 5)) {              // "state<run>": the recurrent state of a layer run
        const int r = atoi(which + 5);
        if (r < 0 || r >= (int)e->runs.size() || !e->runs[r].state || stream < 0 || stream >= e->c.max_streams) return e->fail(NL_ERR_INVALID, "no such state");
        src = e->runs[r].state + stream * e->runs[r].sstride;
        n = e->runs[r].sstride;
    } else return e->fail(NL_ERR_INVALID, "unknown buffer %s", which);
    n = std::min(n, max_floats);
    HIPCK(e, hipMemcpy(out, src, (size_t)n * 4, hipMemcpyDeviceToHost));
    return n;
}

}  // extern "C"
