// The layered hybrid decoder: a stack of layers whose sequence mixers differ (sliding-window attention, WKV time
// mixing, channel-wise gated delta rule, generalised delta rule, attention and a matrix memory side by side), each with an
// optional feed-forward (PolyNorm, GELU or a mixture of experts); a range of layers may run several times over, every pass
// with a state of its own.
//
// Like the Llama model, everything a step touches is allocated once, a decode step is a fixed sequence of launches
// that reads the token and the position from device memory and is replayed as one HIP graph, and prompts run on the
// GEMMs.  Decode, launches per layer: input norm + projections (one product; for WKV the five token-shift products
// side by side), the mixer, output projection + residual, norm + up, PolyNorm + down + residual.  The gates of a gated
// residual are further rows of the products that read the same normalised vector: the mixer's of the input projections,
// the feed-forward's (and a router's) of the up product.
//
// Layouts: weights [out, in] with both sizes rounded up to a multiple of 8 (zeros), the input projections of a mixer
// one after the other in one matrix; activations f32, rows of the rounded size.  A norm of the rounded row is taken
// over K' instead of K elements: with eps' = eps K / K' and gains times sqrt(K / K') it is the norm of the row itself.
#include "mixers.h"
#include "model_common.h"
#include "seq_state.h"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <functional>
#include <memory>
#include <string>

static int pad8(int n) { return (n + 7) & ~7; }

namespace {

struct Param {  // where a named tensor goes
    std::string name;
    std::vector<int64_t> shape;
    void *dst = nullptr;
    bool f32 = false;      // f32 on the device whatever the weight dtype
    size_t rows = 0, cols = 0, ld = 0;
    float add = 0.f, mul = 1.f;  // stored value = (v + add) * mul
    std::function<std::vector<float>(const std::vector<float> &)> expand;  // ... or what this makes of the whole tensor, [n] f32
    void *dst2 = nullptr;  // columns from col_split on go to a second matrix
    size_t col_split = 0;
};

struct Layer {
    lumen_hybrid_layer c = {};
    // rows of the projection matrix and where its blocks start
    int n_proj = 0, off_q = 0, off_k = 0, off_v = 0, off_g = 0, off_b = 0, off_lo = 0, off_hi = 0;
    int off_a = 0, off_rg = 0;           // general delta: removal rates; gated residual: gate of the mixer
    int off_mq = 0, off_mk = 0, off_mv = 0, off_mg = 0, off_mi = 0, off_mf = 0;  // parallel: the matrix memory's
    int od2 = 0;                         // parallel: channels of the matrix memory's output (rounded)
    int n_up = 0, up_at = 0;             // rows of the up product; where the feed-forward's (the router's) start
    int bias_n = 0;                      // distances of the attention's bias table
    int seg = 0, seg_last = 0;           // WKV: rows of a token-shift product
    int od = 0;                          // channels of the mixer's output (rounded)
    void *w_proj = nullptr, *w_o = nullptr, *w_lo = nullptr, *w_hi = nullptr, *w_up = nullptr, *w_down = nullptr;
    float *norm1 = nullptr, *norm2 = nullptr, *act = nullptr;
    float *norm1_b = nullptr, *norm1_a = nullptr, *norm2_b = nullptr, *norm2_a = nullptr;  // Dynamic Tanh: shift, alpha
    float *rg1_b = nullptr, *rg2_b = nullptr, *a_bias = nullptr;
    void *w_o2 = nullptr, *w_eup = nullptr, *w_edown = nullptr;
    float *temp = nullptr, *bias_tab = nullptr, *sink = nullptr, *i_bias = nullptr, *f_bias = nullptr, *out1 = nullptr, *out2 = nullptr;
    float *q_norm = nullptr, *k_norm = nullptr, *r1 = nullptr, *r2 = nullptr;            // attention
    float *mu = nullptr, *bias = nullptr, *u = nullptr, *a_log = nullptr, *taps = nullptr, *gain = nullptr;
    int lo_rank = 0, hi_rank = 0;        // rounded
    int window = 0, cap = 0, slices = 1;
    bool fold = false;                   // the output projection folds the slices of a decode step
    int channels() const { return 2 * c.kv_heads * c.dim + c.heads * c.vdim; }
};

struct Run {  // one pass through one layer
    int layer = 0, pass = -1;  // pass >= 0: the loop's input step comes first
    int st_matrix = -1, st_aux = -1, st_k = -1, st_v = -1;  // (parallel: st_aux is the matrix memory's running maximum)
};

}  // namespace

struct lumen_hybrid {
    lumen_ctx *ctx = nullptr;
    lumen_hybrid_config cfg = {};
    bool bf16 = false;
    size_t esz = 4;
    int W = 0;  // width, rounded
    float eps_w = 0.f;  // eps of the norms over rounded rows
    std::vector<Layer> layers;
    std::vector<Run> runs;
    std::vector<Param> params;
    float *embed = nullptr, *final_norm = nullptr, *final_b = nullptr, *final_a = nullptr, *loop_step = nullptr, *positions = nullptr;
    void *head = nullptr, *loop_x = nullptr, *loop_x0 = nullptr;
    std::unique_ptr<SeqState> state;
    int len = 0;
    unsigned step = 0;  // forward passes since the reset: which slot of a two-slot state block is current (mirror of *d_step)
    int max_proj = 0, max_od = 0, max_ff = 0, max_lo = 0, max_hi = 0, max_heads = 0, max_od2 = 0, max_top = 0, max_act = 0, max_experts = 0;
    size_t max_raw = 0;  // floats per token of the matrix memory's raw output
    // decode
    float *x0 = nullptr, *xa = nullptr, *xb = nullptr, *proj = nullptr, *mixed = nullptr, *ff = nullptr, *logits = nullptr,
          *steps = nullptr, *c0 = nullptr, *part = nullptr, *mixed2 = nullptr, *pair = nullptr, *act = nullptr;
    int *d_sel = nullptr;
    int *d_tok = nullptr, *d_pos = nullptr, *tok_hist = nullptr, *d_err = nullptr;
    unsigned *d_step = nullptr, *amax_epoch = nullptr;
    unsigned long long *amax_word = nullptr;
    int decode_mode = LUMEN_DECODE_GRAPH;
    hipGraph_t graph = nullptr;
    hipGraphExec_t graph_exec = nullptr;
    // prompt
    int pf_cap = 0, pf_logit_cap = 0;
    std::vector<void *> pf_allocs;
    float *p_x0 = nullptr, *p_xa = nullptr, *p_xb = nullptr, *p_n = nullptr, *p_proj = nullptr, *p_mixes = nullptr, *p_mixed = nullptr,
          *p_ff = nullptr, *p_steps = nullptr, *p_q = nullptr, *p_k = nullptr, *p_v = nullptr, *p_lo = nullptr, *p_hi = nullptr,
          *p_z = nullptr, *p_gate = nullptr, *p_logits = nullptr, *p_rows = nullptr, *p_raw = nullptr, *p_scan = nullptr, *p_mixed2 = nullptr,
          *p_y = nullptr, *p_y2 = nullptr, *p_rg = nullptr, *p_route = nullptr, *p_selw = nullptr, *p_act = nullptr, *p_eout = nullptr;
    int *p_ids = nullptr, *p_idx = nullptr, *p_plan = nullptr;
    std::vector<void *> allocs;
    // per-class event times of a profiled step
    struct Probe *probe = nullptr;
};

// ------------------------------------------------------------------ creation
static int alloc_zero(lumen_hybrid *m, void **p, size_t bytes, std::vector<void *> *list = nullptr) {
    bytes = bytes ? bytes : 16;
    HIP_TRY(hipMalloc(p, bytes));
    (list ? *list : m->allocs).push_back(*p);
    HIP_TRY(hipMemsetAsync(*p, 0, bytes, m->ctx->stream));
    return LUMEN_OK;
}
template <typename T>
static int alloc_t(lumen_hybrid *m, T **p, size_t n, std::vector<void *> *list = nullptr) {
    return alloc_zero(m, (void **)p, n * sizeof(T), list);
}

extern "C" int lumen_hybrid_destroy(lumen_hybrid *m) {
    if (!m) return LUMEN_OK;
    hipStreamSynchronize(m->ctx->stream);
    if (m->graph_exec) hipGraphExecDestroy(m->graph_exec);
    if (m->graph) hipGraphDestroy(m->graph);
    for (void *p : m->allocs) hipFree(p);
    for (void *p : m->pf_allocs) hipFree(p);
    hipFree(m->p_logits);
    delete m;
    return LUMEN_OK;
}

static void add_param(lumen_hybrid *m, const std::string &name, std::vector<int64_t> shape, void *dst, bool f32, size_t rows,
                      size_t cols, size_t ld, float add = 0.f, float mul = 1.f) {
    Param p;
    p.name = name; p.shape = std::move(shape); p.dst = dst; p.f32 = f32; p.rows = rows; p.cols = cols; p.ld = ld; p.add = add; p.mul = mul;
    m->params.push_back(p);
}

// rows [row0, row0 + rows) of a weight matrix with rows of `cols` values
static void add_matrix(lumen_hybrid *m, const std::string &name, void *base, int row0, int rows, int cols) {
    add_param(m, name, {rows, cols}, (char *)base + (size_t)row0 * pad8(cols) * m->esz, false, rows, cols, pad8(cols));
}
static void add_vector(lumen_hybrid *m, const std::string &name, float *dst, int n) {
    add_param(m, name, {n}, dst, true, 1, n, n);
}
// A norm of the residual stream: gains, and for Dynamic Tanh the shift and alpha stored beside them.
static int create_norm(lumen_hybrid *m, const std::string &name, float **w, float **b, float **alpha) {
    const int n = m->cfg.width;
    LUMEN_TRY(alloc_t(m, w, m->W));
    if (m->cfg.norm_kind == LUMEN_NORM_RMS) {
        add_param(m, name, {n}, *w, true, 1, n, n, m->cfg.norm_offset, sqrtf((float)n / (float)m->W));
        return LUMEN_OK;
    }
    LUMEN_TRY(alloc_t(m, b, m->W));
    LUMEN_TRY(alloc_t(m, alpha, 4));
    add_vector(m, name, *w, n);
    add_vector(m, name + ".b", *b, n);
    add_param(m, name + ".alpha", {}, *alpha, true, 1, 1, 1);
    return LUMEN_OK;
}

// Row of a distance bias of `rows` rows for distance n: one row per distance in the lower half, a logarithmic scale up
// to `most` above.  (Distances at which the scale meets a whole number belong to the row that starts there: the small
// addend keeps the quotient of two logarithms from falling short of it.)
static int bias_row(int n, int rows, int most) {
    const int half = rows / 2;
    if (n < half) return n;
    if (n >= most || half < 1 || most <= half) return rows - 1;
    return std::min(rows - 1, half + (int)std::floor(std::log((double)n / half) / std::log((double)most / half) * (rows - half) + 1e-9));
}

static int check_layer(const lumen_hybrid_layer &c, int i) {
    if (c.heads <= 0 || c.kv_heads <= 0 || c.dim <= 0 || c.vdim <= 0 || c.ff < 0)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: non-positive size", i);
    if (c.heads % c.kv_heads) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: %d heads over %d key/value heads", i, c.heads, c.kv_heads);
    if (c.dim > MIX_MAX_DIM || c.vdim > MIX_MAX_DIM)
        LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: heads wider than %d", i, MIX_MAX_DIM);
    switch (c.mixer) {
        case LUMEN_MIXER_WINDOW_ATTENTION:
            if (c.window < 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: window %d", i, c.window);
            break;
        case LUMEN_MIXER_WKV:
            if (c.kv_heads != c.heads || c.vdim != c.dim) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: WKV heads are square and unshared", i);
            if (c.rank_lo <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: decay rank %d", i, c.rank_lo);
            break;
        case LUMEN_MIXER_GENERAL_DELTA:
            if (c.kv_heads != c.heads || c.vdim != c.dim) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: general delta heads are square and unshared", i);
            if (c.rank_lo <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: decay rank %d", i, c.rank_lo);
            break;
        case LUMEN_MIXER_PARALLEL:
            if (c.mem_heads <= 0 || c.mem_dim <= 0 || c.mem_vdim <= 0 || c.bias_rows < 2 || c.bias_max <= 0 || !(c.gate_cap > 0.f))
                LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: matrix memory %d x %d x %d, gate cap %g, %d bias rows up to %d", i, c.mem_heads,
                           c.mem_dim, c.mem_vdim, c.gate_cap, c.bias_rows, c.bias_max);
            if (c.mem_dim > MIX_MAX_DIM || c.mem_vdim > MIX_MAX_DIM)
                LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: heads wider than %d", i, MIX_MAX_DIM);
            if (c.mem_heads * c.mem_vdim > 16384) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: inner sizes above 16384", i);
            break;
            break;
        case LUMEN_MIXER_CHANNEL_DELTA:
            if (c.rank_lo <= 0 || c.rank_hi <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: ranks %d, %d", i, c.rank_lo, c.rank_hi);
            if (c.conv < 1 || c.conv > MIX_MAX_TAPS) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: %d convolution taps", i, c.conv);
            break;
        default: LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: layer %d: unknown mixer %d", i, c.mixer);
    }
    if (c.rank_lo > MIX_MAX_RANK || c.rank_hi > MIX_MAX_RANK)
        LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: ranks above %d", i, MIX_MAX_RANK);
    if (c.ff > 16384 || c.heads * c.vdim > 16384 || c.heads * c.dim > 16384)
        LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: inner sizes above 16384 do not fit the GEMV's LDS stage", i);
    if (c.ff > 0 && c.ff_kind == LUMEN_FF_EXPERTS) {
        if (c.experts <= 0 || c.groups <= 0 || c.experts % c.groups || c.keep <= 0 || c.keep > c.groups || c.top <= 0 ||
            c.top > c.keep * (c.experts / c.groups))
            LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: layer %d: %d of %d experts, %d of %d groups", i, c.top, c.experts, c.keep, c.groups);
        if (c.experts > EXPERTS_MAX || c.top > EXPERTS_MAX_TOP || c.top * pad8(c.ff) > 16384)
            LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: %d experts, %d at a time of %d", i, c.experts, c.top, c.ff);
    } else if (c.ff > 0 && c.ff_kind != LUMEN_FF_POLYNORM && c.ff_kind != LUMEN_FF_GELU) {
        LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: layer %d: unknown feed-forward %d", i, c.ff_kind);
    }
    return LUMEN_OK;
}

// A design's layers fit together where its norm and residual have the products that take them.
static int check_design(const lumen_hybrid_config &c, const lumen_hybrid_layer &y, int i) {
    const bool dyt = c.norm_kind == LUMEN_NORM_DYT;
    const bool later = y.mixer == LUMEN_MIXER_GENERAL_DELTA || y.mixer == LUMEN_MIXER_PARALLEL;
    if (later != dyt || (y.ff > 0 && (y.ff_kind != LUMEN_FF_POLYNORM) != dyt) || (c.residual_gate != 0) != dyt)
        LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: layer %d: Dynamic Tanh goes with gated residuals, general delta or parallel mixers and GELU or "
                   "expert feed-forwards", i);
    return LUMEN_OK;
}

static int create_layer(lumen_hybrid *m, Layer &L, int i) {
    const lumen_hybrid_layer &c = L.c;
    const int W = m->cfg.width, H = c.heads, G = c.kv_heads, D = c.dim, Dv = c.vdim;
    const std::string p = "l" + std::to_string(i) + ".", mp = p + "mix.";
    auto weight = [&](void **w, int rows, int cols) { return alloc_zero(m, w, (size_t)pad8(rows) * pad8(cols) * m->esz); };
    L.od = pad8(H * Dv);
    L.lo_rank = pad8(c.rank_lo);
    L.hi_rank = pad8(c.rank_hi);
    LUMEN_TRY(create_norm(m, p + "norm1", &L.norm1, &L.norm1_b, &L.norm1_a));
    LUMEN_TRY(weight(&L.w_o, W, H * Dv));
    auto block = [&](int n) {  // the next block of the projection matrix
        const int off = L.n_proj;
        L.n_proj += pad8(n);
        return off;
    };
    if (c.mixer == LUMEN_MIXER_WINDOW_ATTENTION) {
        L.off_q = block(H * D); L.off_k = block(G * D); L.off_v = block(G * Dv); L.off_g = block(H * Dv);
        LUMEN_TRY(weight(&L.w_proj, L.n_proj, W));
        add_matrix(m, mp + "q", L.w_proj, L.off_q, H * D, W);
        add_matrix(m, mp + "k", L.w_proj, L.off_k, G * D, W);
        add_matrix(m, mp + "v", L.w_proj, L.off_v, G * Dv, W);
        add_matrix(m, mp + "g", L.w_proj, L.off_g, H * Dv, W);
        LUMEN_TRY(alloc_t(m, &L.q_norm, H * D));
        LUMEN_TRY(alloc_t(m, &L.k_norm, G * D));
        LUMEN_TRY(alloc_t(m, &L.r1, H));
        LUMEN_TRY(alloc_t(m, &L.r2, H));
        add_vector(m, mp + "q.norm", L.q_norm, H * D);
        add_vector(m, mp + "k.norm", L.k_norm, G * D);
        add_vector(m, mp + "r1", L.r1, H);
        add_vector(m, mp + "r2", L.r2, H);
        const int max_seq = m->cfg.max_seq_len;
        L.window = c.window > 0 ? std::min(c.window, max_seq) : max_seq;
        L.cap = std::min(max_seq, L.window - 1 + m->cfg.max_chunk);
        L.slices = window_attn_slices(L.window);
        // (every workgroup of the output projection then reads every slice's state: it pays while that stays tens of MB)
        const size_t fold_bytes = (size_t)gemv_grid(m->ctx, m->W, L.od, m->bf16, EPI_RESIDUAL, nullptr) * L.od * GEMV_FOLD_MAX_SLICES * sizeof(float);
        L.fold = L.slices > 1 && L.slices <= GEMV_FOLD_MAX_SLICES && Dv % 4 == 0 && L.od == H * Dv && m->W < 8192 &&
                 fold_bytes <= ((size_t)64 << 20);
    } else if (c.mixer == LUMEN_MIXER_WKV) {
        L.seg = pad8(H * D);
        L.seg_last = L.lo_rank;
        L.off_q = block(H * D); L.off_k = block(H * D); L.off_v = block(H * D); L.off_g = block(H * D); L.off_lo = block(c.rank_lo);
        LUMEN_TRY(weight(&L.w_proj, L.n_proj, W));
        LUMEN_TRY(alloc_t(m, &L.mu, (size_t)5 * m->W));
        const char *names[5] = {"r", "k", "v", "g", "w"};
        for (int s = 0; s < 5; ++s) {
            add_vector(m, mp + "mu." + names[s], L.mu + (size_t)s * m->W, W);
            if (s < 4) add_matrix(m, mp + names[s], L.w_proj, s * L.seg, H * D, W);
        }
        add_matrix(m, mp + "w1", L.w_proj, L.off_lo, c.rank_lo, W);
        LUMEN_TRY(weight(&L.w_lo, H * D, c.rank_lo));
        add_matrix(m, mp + "w2", L.w_lo, 0, H * D, c.rank_lo);
        LUMEN_TRY(alloc_t(m, &L.bias, H * D));
        LUMEN_TRY(alloc_t(m, &L.u, H * D));
        LUMEN_TRY(alloc_t(m, &L.gain, H * D));
        add_vector(m, mp + "w0", L.bias, H * D);
        add_param(m, mp + "u", {H, D}, L.u, true, 1, (size_t)H * D, (size_t)H * D);
        add_vector(m, mp + "norm", L.gain, H * D);
    } else if (c.mixer == LUMEN_MIXER_GENERAL_DELTA) {
        L.off_q = block(H * D); L.off_k = block(H * D); L.off_v = block(H * D); L.off_g = block(H * D); L.off_a = block(H * D);
        L.off_lo = block(c.rank_lo); L.off_rg = block(W);
        LUMEN_TRY(weight(&L.w_proj, L.n_proj, W));
        add_matrix(m, mp + "r", L.w_proj, L.off_q, H * D, W);
        add_matrix(m, mp + "k", L.w_proj, L.off_k, H * D, W);
        add_matrix(m, mp + "v", L.w_proj, L.off_v, H * D, W);
        add_matrix(m, mp + "g", L.w_proj, L.off_g, H * D, W);
        add_matrix(m, mp + "a", L.w_proj, L.off_a, H * D, W);
        add_matrix(m, mp + "w1", L.w_proj, L.off_lo, c.rank_lo, W);
        LUMEN_TRY(weight(&L.w_lo, H * D, c.rank_lo));
        add_matrix(m, mp + "w2", L.w_lo, 0, H * D, c.rank_lo);
        LUMEN_TRY(alloc_t(m, &L.bias, H * D));
        LUMEN_TRY(alloc_t(m, &L.a_bias, H * D));
        LUMEN_TRY(alloc_t(m, &L.gain, H * D));
        add_vector(m, mp + "w0", L.bias, H * D);
        add_vector(m, mp + "a.b", L.a_bias, H * D);
        add_vector(m, mp + "norm", L.gain, H * D);
    } else if (c.mixer == LUMEN_MIXER_PARALLEL) {
        const int Hm = c.mem_heads, Dm = c.mem_dim, Vm = c.mem_vdim;
        const std::string lp = mp + "left.", rp = mp + "right.";
        L.off_q = block(H * D); L.off_k = block(G * D); L.off_v = block(G * Dv); L.off_g = block(H);
        L.off_mq = block(Hm * Dm); L.off_mk = block(Hm * Dm); L.off_mv = block(Hm * Vm); L.off_mg = block(Hm * Vm);
        L.off_mi = block(Hm); L.off_mf = block(Hm); L.off_rg = block(W);
        LUMEN_TRY(weight(&L.w_proj, L.n_proj, W));
        add_matrix(m, lp + "q", L.w_proj, L.off_q, H * D, W);
        add_matrix(m, lp + "k", L.w_proj, L.off_k, G * D, W);
        add_matrix(m, lp + "v", L.w_proj, L.off_v, G * Dv, W);
        add_matrix(m, lp + "g", L.w_proj, L.off_g, H, W);
        add_matrix(m, rp + "q", L.w_proj, L.off_mq, Hm * Dm, W);
        add_matrix(m, rp + "k", L.w_proj, L.off_mk, Hm * Dm, W);
        add_matrix(m, rp + "v", L.w_proj, L.off_mv, Hm * Vm, W);
        add_matrix(m, rp + "g", L.w_proj, L.off_mg, Hm * Vm, W);
        add_matrix(m, rp + "i", L.w_proj, L.off_mi, Hm, W);
        add_matrix(m, rp + "f", L.w_proj, L.off_mf, Hm, W);
        // attention
        const int B = c.bias_rows, most = c.bias_max;
        L.bias_n = 1;  // distances up to the first whose row is the last one, and to all further ones
        while (bias_row(L.bias_n - 1, B, most) < B - 1 && L.bias_n < m->cfg.max_seq_len) ++L.bias_n;
        LUMEN_TRY(alloc_t(m, &L.bias_tab, (size_t)H * L.bias_n));
        LUMEN_TRY(alloc_t(m, &L.temp, H));
        LUMEN_TRY(alloc_t(m, &L.sink, H));
        const int n = L.bias_n;
        add_param(m, lp + "rel", {B, H}, L.bias_tab, true, 1, (size_t)B * H, (size_t)B * H);
        m->params.back().expand = [B, H, n, most](const std::vector<float> &rel) {
            std::vector<float> tab((size_t)H * n);
            for (int h = 0; h < H; ++h)
                for (int d = 0; d < n; ++d) tab[(size_t)h * n + d] = rel[(size_t)bias_row(d, B, most) * H + h] * 1.44269504088896341f;
            return tab;
        };
        add_vector(m, lp + "temp", L.temp, H);
        add_vector(m, lp + "sink", L.sink, H);
        L.window = L.cap = m->cfg.max_seq_len;
        L.slices = window_attn_slices(L.window);
        // matrix memory
        L.od2 = pad8(Hm * Vm);
        LUMEN_TRY(weight(&L.w_o2, W, Hm * Vm));
        add_matrix(m, rp + "o", L.w_o2, 0, W, Hm * Vm);
        LUMEN_TRY(alloc_t(m, &L.i_bias, Hm));
        LUMEN_TRY(alloc_t(m, &L.f_bias, Hm));
        LUMEN_TRY(alloc_t(m, &L.gain, Hm * Vm));
        add_vector(m, rp + "i.b", L.i_bias, Hm);
        add_vector(m, rp + "f.b", L.f_bias, Hm);
        add_vector(m, rp + "norm", L.gain, Hm * Vm);
        LUMEN_TRY(alloc_t(m, &L.out1, m->W));
        LUMEN_TRY(alloc_t(m, &L.out2, m->W));
        add_vector(m, lp + "out", L.out1, W);
        add_vector(m, rp + "out", L.out2, W);
        m->max_od2 = std::max(m->max_od2, L.od2);
        m->max_raw = std::max(m->max_raw, (size_t)Hm * (Vm + 1));
        m->max_heads = std::max(m->max_heads, Hm * std::max(Dm, Vm));
    } else {
        L.off_q = block(G * D); L.off_k = block(G * D); L.off_v = block(H * Dv); L.off_b = block(H);
        L.off_lo = block(c.rank_lo); L.off_hi = block(c.rank_hi);
        LUMEN_TRY(weight(&L.w_proj, L.n_proj, W));
        add_matrix(m, mp + "q", L.w_proj, L.off_q, G * D, W);
        add_matrix(m, mp + "k", L.w_proj, L.off_k, G * D, W);
        add_matrix(m, mp + "v", L.w_proj, L.off_v, H * Dv, W);
        add_matrix(m, mp + "b", L.w_proj, L.off_b, H, W);
        add_matrix(m, mp + "a1", L.w_proj, L.off_lo, c.rank_lo, W);
        add_matrix(m, mp + "g1", L.w_proj, L.off_hi, c.rank_hi, W);
        LUMEN_TRY(weight(&L.w_lo, H * D, c.rank_lo));
        LUMEN_TRY(weight(&L.w_hi, H * Dv, c.rank_hi));
        add_matrix(m, mp + "a2", L.w_lo, 0, H * D, c.rank_lo);
        add_matrix(m, mp + "g2", L.w_hi, 0, H * Dv, c.rank_hi);
        LUMEN_TRY(alloc_t(m, &L.taps, (size_t)L.channels() * c.conv));
        const int rows[3] = {G * D, G * D, H * Dv};
        const char *names[3] = {"q.conv", "k.conv", "v.conv"};
        size_t at = 0;
        for (int s = 0; s < 3; ++s) {
            add_param(m, mp + names[s], {rows[s], c.conv}, L.taps + at * c.conv, true, rows[s], c.conv, c.conv);
            at += rows[s];
        }
        LUMEN_TRY(alloc_t(m, &L.bias, H * D));
        LUMEN_TRY(alloc_t(m, &L.a_log, H));
        LUMEN_TRY(alloc_t(m, &L.gain, Dv));
        add_vector(m, mp + "dt_bias", L.bias, H * D);
        add_vector(m, mp + "A_log", L.a_log, H);
        add_vector(m, mp + "norm", L.gain, Dv);
    }
    add_matrix(m, mp + (c.mixer == LUMEN_MIXER_PARALLEL ? "left.o" : "o"), L.w_o, 0, W, H * Dv);
    if (m->cfg.residual_gate) {
        LUMEN_TRY(alloc_t(m, &L.rg1_b, m->W));
        add_matrix(m, p + "rg1", L.w_proj, L.off_rg, W, W);
        add_vector(m, p + "rg1.b", L.rg1_b, W);
    }
    if (c.ff > 0) {
        const bool experts = c.ff_kind == LUMEN_FF_EXPERTS;
        LUMEN_TRY(create_norm(m, p + "norm2", &L.norm2, &L.norm2_b, &L.norm2_a));
        // the up product: the feed-forward's gate, then the up matrix or the router
        L.up_at = m->cfg.residual_gate ? m->W : 0;
        L.n_up = L.up_at + pad8(experts ? c.experts : c.ff);
        LUMEN_TRY(weight(&L.w_up, L.n_up, W));
        if (m->cfg.residual_gate) {
            LUMEN_TRY(alloc_t(m, &L.rg2_b, m->W));
            add_matrix(m, p + "rg2", L.w_up, 0, W, W);
            add_vector(m, p + "rg2.b", L.rg2_b, W);
        }
        if (experts) {
            const size_t F = pad8(c.ff), K = m->W, E = c.experts;
            add_matrix(m, p + "mlp.router", L.w_up, L.up_at, c.experts, W);
            LUMEN_TRY(alloc_zero(m, &L.w_eup, E * 2 * F * K * m->esz));
            LUMEN_TRY(alloc_zero(m, &L.w_edown, E * K * F * m->esz));
            for (size_t e = 0; e < E; ++e) {  // gate and up rows in turn
                const std::string ep = p + "mlp.e" + std::to_string(e) + ".";
                char *up = (char *)L.w_eup + e * 2 * F * K * m->esz;
                add_param(m, ep + "gate", {c.ff, W}, up, false, c.ff, W, 2 * K);
                add_param(m, ep + "up", {c.ff, W}, up + K * m->esz, false, c.ff, W, 2 * K);
                add_param(m, ep + "down", {W, c.ff}, (char *)L.w_edown + e * K * F * m->esz, false, W, c.ff, F);
            }
            m->max_top = std::max(m->max_top, c.top);
            m->max_act = std::max(m->max_act, c.top * (int)F);
            m->max_experts = std::max(m->max_experts, pad8(c.experts));
        } else {
            LUMEN_TRY(weight(&L.w_down, W, c.ff));
            add_matrix(m, p + "mlp.up", L.w_up, L.up_at, c.ff, W);
            add_matrix(m, p + "mlp.down", L.w_down, 0, W, c.ff);
            if (c.ff_kind == LUMEN_FF_POLYNORM) {
                LUMEN_TRY(alloc_t(m, &L.act, 4));
                add_vector(m, p + "mlp.act", L.act, 4);
            }
        }
    }
    m->max_proj = std::max(m->max_proj, L.n_proj);
    m->max_od = std::max(m->max_od, L.od);
    m->max_ff = std::max(m->max_ff, L.n_up);
    m->max_lo = std::max(m->max_lo, L.lo_rank);
    m->max_hi = std::max(m->max_hi, L.hi_rank);
    m->max_heads = std::max(m->max_heads, std::max(H * D, H * Dv));
    return LUMEN_OK;
}

static int create_impl(lumen_hybrid *m, const lumen_hybrid_layer *layers) {
    const lumen_hybrid_config &c = m->cfg;
    lumen_ctx *ctx = m->ctx;
    const int W = m->W, V = c.vocab_size;
    m->layers.resize(c.num_layers);
    LUMEN_TRY(alloc_t(m, &m->embed, (size_t)V * W));
    add_param(m, "embed", {V, c.width}, m->embed, true, V, c.width, W, 0.f, c.embed_scale);
    if (c.max_positions > 0) {
        LUMEN_TRY(alloc_t(m, &m->positions, (size_t)c.max_positions * W));
        add_param(m, "pos", {c.max_positions, c.width}, m->positions, true, c.max_positions, c.width, W);
    }
    if (c.loop_times > 0) {
        LUMEN_TRY(alloc_t(m, &m->loop_step, (size_t)c.loop_times * W));
        if (c.loop_kind == LUMEN_LOOP_MIX) {
            LUMEN_TRY(alloc_zero(m, &m->loop_x, (size_t)W * W * m->esz));
            LUMEN_TRY(alloc_zero(m, &m->loop_x0, (size_t)W * W * m->esz));
            Param p;
            p.name = "loop.in"; p.shape = {c.width, 2 * c.width}; p.dst = m->loop_x; p.dst2 = m->loop_x0; p.col_split = c.width;
            p.rows = c.width; p.cols = 2 * (size_t)c.width; p.ld = W;
            m->params.push_back(p);
        }
        add_param(m, "loop.step", {c.loop_times, c.width}, m->loop_step, true, c.loop_times, c.width, W);
    }
    for (int i = 0; i < c.num_layers; ++i) {
        m->layers[i].c = layers[i];
        LUMEN_TRY(create_layer(m, m->layers[i], i));
    }
    LUMEN_TRY(create_norm(m, "final.norm", &m->final_norm, &m->final_b, &m->final_a));
    LUMEN_TRY(alloc_zero(m, &m->head, (size_t)V * W * m->esz));
    add_matrix(m, "head", m->head, 0, V, c.width);

    auto add_run = [&](int layer, int pass) {
        Run r;
        const Layer &L = m->layers[layer];
        r.layer = layer;
        r.pass = pass;
        if (L.c.mixer == LUMEN_MIXER_WINDOW_ATTENTION || L.c.mixer == LUMEN_MIXER_PARALLEL) {
            r.st_k = m->state->reserve(SeqState::ROLLING, (size_t)L.c.kv_heads * L.cap * ((L.c.dim + 3) & ~3));
            r.st_v = m->state->reserve(SeqState::ROLLING, (size_t)L.c.kv_heads * L.cap * ((L.c.vdim + 3) & ~3));
            if (L.c.mixer == LUMEN_MIXER_PARALLEL) {
                r.st_matrix = m->state->reserve(SeqState::ZEROED, (size_t)L.c.mem_heads * recurrence_columns(REC_MEMORY, L.c.mem_vdim) *
                                                                      recurrence_rows(L.c.mem_dim));
                r.st_aux = m->state->reserve(SeqState::ZEROED, L.c.mem_heads);
            }
        } else if (L.c.mixer == LUMEN_MIXER_GENERAL_DELTA) {
            r.st_matrix = m->state->reserve(SeqState::ZEROED, (size_t)L.c.heads * L.c.vdim * recurrence_rows(L.c.dim));
        } else {
            r.st_matrix = m->state->reserve(SeqState::ZEROED, (size_t)L.c.heads * L.c.vdim * recurrence_rows(L.c.dim));
            r.st_aux = m->state->reserve(SeqState::ZEROED, L.c.mixer == LUMEN_MIXER_WKV ? (size_t)2 * W
                                                                                        : (size_t)2 * (L.c.conv - 1) * L.channels());
        }
        m->runs.push_back(r);
    };
    m->state.reset(new SeqState());
    const int start = c.loop_times > 0 ? c.loop_start : 0, stop = c.loop_times > 0 ? c.loop_stop : 0;
    for (int i = 0; i < start; ++i) add_run(i, -1);
    for (int t = 0; t < (c.loop_times > 0 ? c.loop_times : 0); ++t)
        for (int i = start; i < stop; ++i) add_run(i, i == start ? t : -1);
    for (int i = stop; i < c.num_layers; ++i) add_run(i, -1);
    LUMEN_TRY(m->state->commit(ctx));

    LUMEN_TRY(alloc_t(m, &m->x0, W));
    LUMEN_TRY(alloc_t(m, &m->xa, W));
    LUMEN_TRY(alloc_t(m, &m->xb, W));
    LUMEN_TRY(alloc_t(m, &m->c0, W));
    LUMEN_TRY(alloc_t(m, &m->steps, (size_t)std::max(c.loop_times, 1) * W));
    LUMEN_TRY(alloc_t(m, &m->proj, m->max_proj));
    LUMEN_TRY(alloc_t(m, &m->mixed, m->max_od));
    LUMEN_TRY(alloc_t(m, &m->ff, m->max_ff));
    LUMEN_TRY(alloc_t(m, &m->mixed2, m->max_od2));
    LUMEN_TRY(alloc_t(m, &m->pair, (size_t)2 * W));
    LUMEN_TRY(alloc_t(m, &m->act, m->max_act));
    LUMEN_TRY(alloc_t(m, &m->d_sel, m->max_top));
    LUMEN_TRY(alloc_t(m, &m->logits, V));
    size_t part = 4;
    for (const Layer &L : m->layers)
        if (L.slices > 1) part = std::max(part, (size_t)L.c.heads * L.slices * (L.c.vdim + 2));
    LUMEN_TRY(alloc_t(m, &m->part, part));
    LUMEN_TRY(alloc_t(m, &m->d_tok, 4));
    LUMEN_TRY(alloc_t(m, &m->d_pos, 4));
    LUMEN_TRY(alloc_t(m, &m->d_err, 4));
    LUMEN_TRY(alloc_t(m, &m->d_step, 4));
    LUMEN_TRY(alloc_t(m, &m->amax_epoch, 4));
    LUMEN_TRY(alloc_t(m, &m->amax_word, std::max(gemv_max_blocks(ctx), ctx->num_cus)));
    LUMEN_TRY(alloc_t(m, &m->tok_hist, (size_t)c.max_seq_len + 1));
    HIP_TRY(hipStreamSynchronize(ctx->stream));
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_create(lumen_ctx *ctx, const lumen_hybrid_config *cfg, const lumen_hybrid_layer *layers, lumen_hybrid **out) {
    if (!ctx || !cfg || !layers || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: null argument");
    *out = nullptr;
    if (cfg->vocab_size <= 0 || cfg->width <= 0 || cfg->num_layers <= 0 || cfg->max_seq_len <= 0)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: non-positive size");
    if (cfg->weight_dtype != LUMEN_DTYPE_F32 && cfg->weight_dtype != LUMEN_DTYPE_BF16)
        LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: weight_dtype %d", cfg->weight_dtype);
    if (cfg->loop_times < 0 || (cfg->loop_times > 0 && (cfg->loop_start < 0 || cfg->loop_stop <= cfg->loop_start || cfg->loop_stop > cfg->num_layers)))
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: loop [%d, %d) x %d over %d layers", cfg->loop_start, cfg->loop_stop, cfg->loop_times,
                   cfg->num_layers);
    if (cfg->width > 16384) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: width above 16384 does not fit the GEMV's LDS stage");
    if (cfg->vocab_size >= (1 << 24)) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_create: vocabulary of %d", cfg->vocab_size);
    if (cfg->norm_kind != LUMEN_NORM_RMS && cfg->norm_kind != LUMEN_NORM_DYT) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: norm_kind %d", cfg->norm_kind);
    if (cfg->loop_kind != LUMEN_LOOP_MIX && cfg->loop_kind != LUMEN_LOOP_ADD) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_create: loop_kind %d", cfg->loop_kind);
    if (cfg->max_positions > 0 && cfg->max_seq_len > cfg->max_positions)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_create: sequences of %d with %d positions", cfg->max_seq_len, cfg->max_positions);
    for (int i = 0; i < cfg->num_layers; ++i) {
        LUMEN_TRY(check_layer(layers[i], i));
        LUMEN_TRY(check_design(*cfg, layers[i], i));
    }
    HIP_TRY(hipSetDevice(ctx->device));
    lumen_hybrid *m = new lumen_hybrid();
    m->ctx = ctx;
    m->cfg = *cfg;
    if (m->cfg.max_chunk <= 0) m->cfg.max_chunk = 2048;
    m->cfg.max_chunk = std::min(m->cfg.max_chunk, cfg->max_seq_len);
    m->bf16 = cfg->weight_dtype == LUMEN_DTYPE_BF16;
    m->esz = m->bf16 ? 2 : 4;
    m->W = pad8(cfg->width);
    m->eps_w = cfg->norm_eps * (float)cfg->width / (float)m->W;
    const int rc = create_impl(m, layers);
    if (rc != LUMEN_OK) {
        lumen_hybrid_destroy(m);
        return rc;
    }
    *out = m;
    return LUMEN_OK;
}

// ------------------------------------------------------------------ parameters
extern "C" int lumen_hybrid_num_params(const lumen_hybrid *m, int *n_out) {
    if (!m || !n_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_num_params: null argument");
    *n_out = (int)m->params.size();
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_param_info(const lumen_hybrid *m, int index, char *name, int name_len, int64_t *shape, int *ndim) {
    if (!m || !name || name_len <= 0 || !shape || !ndim) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_param_info: null argument");
    if (index < 0 || index >= (int)m->params.size()) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_param_info: index %d", index);
    const Param &p = m->params[index];
    snprintf(name, (size_t)name_len, "%s", p.name.c_str());
    *ndim = (int)p.shape.size();
    for (size_t i = 0; i < p.shape.size() && i < 2; ++i) shape[i] = p.shape[i];
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_set_param(lumen_hybrid *m, const char *name, const void *data, int dtype, const int64_t *shape, int ndim) {
    if (!m || !name || !data || ndim < 0 || (!shape && ndim > 0)) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_set_param: null argument");
    if (dtype != LUMEN_DTYPE_F32 && dtype != LUMEN_DTYPE_BF16) LUMEN_FAIL(LUMEN_ERR_INVALID, "Unsupported dtype: %d for %s", dtype, name);
    for (const Param &p : m->params) {
        if (p.name != name) continue;
        if (std::vector<int64_t>(shape, shape + ndim) != p.shape) LUMEN_FAIL(LUMEN_ERR_SHAPE, "Shape mismatch for %s", name);
        HIP_TRY(hipSetDevice(m->ctx->device));
        const bool to_f32 = p.f32 || !m->bf16;
        const size_t esz = to_f32 ? 4 : 2, src_esz = dtype == LUMEN_DTYPE_BF16 ? 2 : 4;
        if (p.expand) {
            std::vector<float> in(p.rows * p.cols);
            if (dtype == LUMEN_DTYPE_BF16) bf16_to_f32_host((const uint16_t *)data, in.data(), in.size());
            else memcpy(in.data(), data, in.size() * 4);
            const std::vector<float> out = p.expand(in);
            HIP_TRY(hipMemcpyAsync(p.dst, out.data(), out.size() * 4, hipMemcpyHostToDevice, m->ctx->stream));
            HIP_TRY(hipStreamSynchronize(m->ctx->stream));
            return LUMEN_OK;
        }
        const bool convert = p.add != 0.f || p.mul != 1.f || to_f32 != (dtype == LUMEN_DTYPE_F32);
        const size_t chunk = std::max<size_t>(1, ((size_t)16 << 20) / p.cols);
        std::vector<float> wide;
        std::vector<uint16_t> narrow;
        for (size_t r0 = 0; r0 < p.rows; r0 += chunk) {
            const size_t nr = std::min(chunk, p.rows - r0), n = nr * p.cols;
            const char *src = (const char *)data + r0 * p.cols * src_esz;
            if (convert) {
                wide.resize(n);
                if (dtype == LUMEN_DTYPE_BF16) bf16_to_f32_host((const uint16_t *)src, wide.data(), n);
                else memcpy(wide.data(), src, n * 4);
                if (p.add != 0.f || p.mul != 1.f)
                    for (float &v : wide) v = (v + p.add) * p.mul;
                src = (const char *)wide.data();
                if (!to_f32) {
                    narrow.resize(n);
                    f32_to_bf16_host(wide.data(), narrow.data(), n);
                    src = (const char *)narrow.data();
                }
            }
            const size_t first = p.dst2 ? p.col_split : p.cols;
            HIP_TRY(hipMemcpy2DAsync((char *)p.dst + r0 * p.ld * esz, p.ld * esz, src, p.cols * esz, first * esz, nr, hipMemcpyHostToDevice,
                                     m->ctx->stream));
            if (p.dst2)
                HIP_TRY(hipMemcpy2DAsync((char *)p.dst2 + r0 * p.ld * esz, p.ld * esz, src + first * esz, p.cols * esz,
                                         (p.cols - first) * esz, nr, hipMemcpyHostToDevice, m->ctx->stream));
            HIP_TRY(hipStreamSynchronize(m->ctx->stream));
        }
        return LUMEN_OK;
    }
    LUMEN_FAIL(LUMEN_ERR_INVALID, "Parameter %s not found in model", name);
}

extern "C" int lumen_hybrid_load_safetensors(lumen_hybrid *m, const char *path, int *n_loaded_out, int *n_missing_out) {
    if (n_loaded_out) *n_loaded_out = 0;
    if (n_missing_out) *n_missing_out = 0;
    if (!m || !path) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_load_safetensors: null argument");
    std::vector<std::string> names;
    std::vector<std::vector<int64_t>> shapes;
    for (const Param &p : m->params) {
        names.push_back(p.name);
        shapes.push_back(p.shape);
    }
    return load_safetensors_into(path, names, shapes,
                                 [m](const char *n, const void *d, int t, const int64_t *sh, int nd) {
                                     return lumen_hybrid_set_param(m, n, d, t, sh, nd);
                                 },
                                 n_loaded_out, n_missing_out);
}

// ------------------------------------------------------------------ decode
// Launch classes of a decode step, for per-kernel timing.
enum { HC_EMBED = 0, HC_LOOP, HC_PROJ_ATTN, HC_ATTN, HC_PROJ_WKV, HC_WKV, HC_PROJ_DELTA, HC_DELTA, HC_OUT, HC_UP, HC_DOWN, HC_HEAD,
       HC_PROJ_GENERAL, HC_GENERAL, HC_PROJ_PARALLEL, HC_MEMORY, HC_PAIR, HC_EXPERT_UP, HC_EXPERT_DOWN, HC_COUNT };

struct Probe {
    std::vector<hipEvent_t> ev;
    std::vector<int> cls;
    std::string names[HC_COUNT];
};

static int timed(lumen_hybrid *m, int cls, int rc_launch(lumen_hybrid *, const void *), const void *arg) {
    Probe *p = m->probe;
    if (!p) return rc_launch(m, arg);
    hipEvent_t e0, e1;
    HIP_TRY(hipEventCreate(&e0));
    HIP_TRY(hipEventCreate(&e1));
    p->ev.push_back(e0);
    p->ev.push_back(e1);
    p->cls.push_back(cls);
    HIP_TRY(hipEventRecord(e0, m->ctx->stream));
    LUMEN_TRY(rc_launch(m, arg));
    HIP_TRY(hipEventRecord(e1, m->ctx->stream));
    p->names[cls] = m->ctx->last_kernel;
    return LUMEN_OK;
}
static int do_gemv(lumen_hybrid *m, const void *a) { return launch_gemv(m->ctx, *(const GemvArgs *)a); }
static int do_attn(lumen_hybrid *m, const void *a) { return launch_window_attn_decode(m->ctx, *(const WindowAttnArgs *)a); }
static int do_pair(lumen_hybrid *m, const void *a) { return launch_gated_residual(m->ctx, *(const GatedResidualArgs *)a); }
static int do_experts_up(lumen_hybrid *m, const void *a) { return launch_experts_up(m->ctx, *(const ExpertsArgs *)a); }
static int do_experts_down(lumen_hybrid *m, const void *a) { return launch_experts_down(m->ctx, *(const ExpertsArgs *)a); }
static int do_rec(lumen_hybrid *m, const void *a) { return launch_recurrence_decode(m->ctx, *(const RecurrenceDecodeArgs *)a); }

static GemvArgs gemv_args(const lumen_hybrid *m, const void *w, int N, int K, const float *x, float *y) {
    GemvArgs g = {};
    g.W = w; g.N = N; g.K = K; g.x = x; g.y = y; g.w_bf16 = m->bf16; g.pro = PRO_NONE; g.epi = EPI_STORE;
    return g;
}
static void gemv_norm(const lumen_hybrid *m, GemvArgs &g, const float *gains, const float *shift, const float *alpha) {
    g.pro = m->cfg.norm_kind == LUMEN_NORM_DYT ? PRO_DYT : PRO_RMSNORM;
    g.norm_w = gains; g.norm_b = shift; g.norm_alpha = alpha; g.eps = m->eps_w;
}
static void gemv_residual(GemvArgs &g, const float *residual, float alpha) {
    g.epi = EPI_RESIDUAL; g.residual = residual; g.alpha = alpha;
}

static WindowAttnArgs attn_args(const lumen_hybrid *m, const Layer &L, const Run &r, const float *proj, int stride) {
    WindowAttnArgs a = {};
    a.q = proj + L.off_q; a.k = proj + L.off_k; a.v = proj + L.off_v; a.gate = proj + L.off_g; a.stride = stride;
    a.q_norm_w = L.q_norm; a.k_norm_w = L.k_norm; a.norm_eps = m->cfg.norm_eps;
    a.k_ring = m->state->ptr(r.st_k); a.v_ring = m->state->ptr(r.st_v);
    a.cap = L.cap; a.dpad = (L.c.dim + 3) & ~3; a.vpad = (L.c.vdim + 3) & ~3;
    a.heads = L.c.heads; a.kv_heads = L.c.kv_heads; a.dim = L.c.dim; a.vdim = L.c.vdim; a.window = L.window; a.gate_act = GATE_SIGMOID;
    a.scale = L.c.scale; a.softcap = L.c.softcap; a.r1 = L.r1; a.r2 = L.r2; a.slices = L.slices;
    a.temp = L.temp; a.bias_tab = L.bias_tab; a.bias_n = L.bias_n; a.sink = L.sink; a.gate_heads = L.c.mixer == LUMEN_MIXER_PARALLEL;
    return a;
}

#define MEMORY_DEN_EPS 1e-6f
static const float GENERAL_DECAY = 0.60653065971263342f;  // e^{-1/2}

// What the decode kernels of the general delta rule and of the matrix memory are told.
static RecurrenceDecodeArgs later_decode_args(lumen_hybrid *m, const Layer &L, const Run &r) {
    const lumen_hybrid_config &c = m->cfg;
    RecurrenceDecodeArgs a = {};
    a.w_bf16 = m->bf16; a.proj = m->proj; a.unit_eps = c.unit_eps; a.norm_eps = c.norm_eps; a.gain = L.gain; a.state = m->state->ptr(r.st_matrix);
    if (L.c.mixer == LUMEN_MIXER_GENERAL_DELTA) {
        a.kind = REC_GENERAL; a.heads = a.kv_heads = L.c.heads; a.dim = a.vdim = L.c.dim;
        a.off_q = L.off_q; a.off_k = L.off_k; a.off_v = L.off_v; a.off_gate = L.off_g; a.off_a = L.off_a; a.off_lo = L.off_lo;
        a.w_lo = L.w_lo; a.r_lo = L.lo_rank; a.bias = L.bias; a.a_bias = L.a_bias; a.z_scale = GENERAL_DECAY; a.out = m->mixed;
    } else {
        a.kind = REC_MEMORY; a.heads = a.kv_heads = L.c.mem_heads; a.dim = L.c.mem_dim; a.vdim = L.c.mem_vdim;
        a.off_q = L.off_mq; a.off_k = L.off_mk; a.off_v = L.off_mv; a.off_gate = L.off_mg; a.off_i = L.off_mi; a.off_f = L.off_mf;
        a.i_bias = L.i_bias; a.f_bias = L.f_bias; a.cap = L.c.gate_cap; a.den_eps = MEMORY_DEN_EPS; a.q_scale = 1.0f / sqrtf((float)L.c.mem_dim);
        a.m = m->state->ptr(r.st_aux); a.out = m->mixed2;
    }
    return a;
}

static ExpertsArgs experts_args(const lumen_hybrid *m, const Layer &L) {
    ExpertsArgs a = {};
    a.r = RouterShape{L.c.experts, L.c.groups, L.c.keep, L.c.top, L.c.router_scale};
    a.w_up = L.w_eup; a.w_down = L.w_edown; a.w_bf16 = m->bf16; a.dim = m->W; a.ff = pad8(L.c.ff); a.limit = L.c.limit;
    return a;
}

// The residual stream after every layer run, for a caller that asks: rows of `width` floats, [runs][total][width].
struct Tap {
    float *host = nullptr;
    size_t total = 0, at = 0;
};
static int tap_rows(lumen_hybrid *m, const Tap *tap, size_t run, const float *x, int rows) {
    if (!tap || !tap->host) return LUMEN_OK;
    const size_t w = (size_t)m->cfg.width * sizeof(float);
    HIP_TRY(hipMemcpy2DAsync(tap->host + (run * tap->total + tap->at) * m->cfg.width, w, x, (size_t)m->W * sizeof(float), w, rows,
                             hipMemcpyDeviceToHost, m->ctx->stream));
    HIP_TRY(hipStreamSynchronize(m->ctx->stream));
    return LUMEN_OK;
}

static int embed_rows(lumen_hybrid *m, const int *ids, int n, const int *pos_dev, int pos, float *out) {
    const lumen_hybrid_config &c = m->cfg;
    if (!m->positions) return launch_embedding(m->ctx, m->embed, ids, n, m->W, c.vocab_size, out);
    return launch_embedding_pos(m->ctx, m->embed, ids, m->positions, pos_dev, pos, n, m->W, c.vocab_size, c.max_positions, out);
}

static int enqueue_decode_step(lumen_hybrid *m, const Tap *tap = nullptr) {
    const lumen_hybrid_config &c = m->cfg;
    lumen_ctx *ctx = m->ctx;
    const int W = m->W;
    LUMEN_TRY(embed_rows(m, m->d_tok, 1, m->d_pos, 0, m->x0));
    const bool mix = c.loop_times > 0 && c.loop_kind == LUMEN_LOOP_MIX;
    if (mix) {
        GemvArgs g = gemv_args(m, m->loop_x0, W, W, m->x0, m->c0);
        LUMEN_TRY(timed(m, HC_LOOP, do_gemv, &g));
        LUMEN_TRY(launch_add_steps(ctx, m->c0, m->loop_step, m->steps, c.loop_times, 1, W));
    }
    const float *cur = m->x0;  // the residual stream; written in place once it has left x0
    auto out = [&]() { return cur == m->x0 ? m->xa : const_cast<float *>(cur); };
    for (size_t ri = 0; ri < m->runs.size(); ++ri) {
        const Run &r = m->runs[ri];
        const Layer &L = m->layers[r.layer];
        if (r.pass >= 0) {
            float *y = cur == m->xa ? m->xb : m->xa;
            if (mix) {
                GemvArgs g = gemv_args(m, m->loop_x, W, W, cur, y);
                gemv_residual(g, m->steps + (size_t)r.pass * W, 1.0f);
                LUMEN_TRY(timed(m, HC_LOOP, do_gemv, &g));
            } else {
                LUMEN_TRY(launch_add_steps(ctx, cur, m->loop_step + (size_t)r.pass * W, y, 1, 1, W));
            }
            cur = y;
        }
        if (L.c.mixer == LUMEN_MIXER_WKV) {
            GemvArgs g = gemv_args(m, L.w_proj, L.seg, W, cur, m->proj);
            gemv_norm(m, g, L.norm1, nullptr, nullptr);
            g.pro = PRO_SHIFT; g.shift_mu = L.mu; g.shift_state = m->state->ptr(r.st_aux); g.shift_step = m->d_step;
            g.shift_segs = 5; g.shift_rows = L.seg; g.shift_last_rows = L.seg_last;
            LUMEN_TRY(timed(m, HC_PROJ_WKV, do_gemv, &g));
        } else {
            GemvArgs g = gemv_args(m, L.w_proj, L.n_proj, W, cur, m->proj);
            gemv_norm(m, g, L.norm1, L.norm1_b, L.norm1_a);
            const int cls = L.c.mixer == LUMEN_MIXER_WINDOW_ATTENTION ? HC_PROJ_ATTN
                            : L.c.mixer == LUMEN_MIXER_CHANNEL_DELTA  ? HC_PROJ_DELTA
                            : L.c.mixer == LUMEN_MIXER_GENERAL_DELTA  ? HC_PROJ_GENERAL
                                                                      : HC_PROJ_PARALLEL;
            LUMEN_TRY(timed(m, cls, do_gemv, &g));
        }
        if (L.c.mixer == LUMEN_MIXER_WINDOW_ATTENTION || L.c.mixer == LUMEN_MIXER_PARALLEL) {
            WindowAttnArgs a = attn_args(m, L, r, m->proj, L.n_proj);
            a.out = m->mixed; a.pos_dev = m->d_pos; a.part = m->part; a.leave_slices = L.fold;
            LUMEN_TRY(timed(m, HC_ATTN, do_attn, &a));
            if (L.c.mixer == LUMEN_MIXER_PARALLEL) {
                const RecurrenceDecodeArgs rm = later_decode_args(m, L, r);
                LUMEN_TRY(timed(m, HC_MEMORY, do_rec, &rm));
            }
        } else if (L.c.mixer == LUMEN_MIXER_GENERAL_DELTA) {
            const RecurrenceDecodeArgs a = later_decode_args(m, L, r);
            LUMEN_TRY(timed(m, HC_GENERAL, do_rec, &a));
        } else {
            const bool wkv = L.c.mixer == LUMEN_MIXER_WKV;
            RecurrenceDecodeArgs a = {};
            a.kind = wkv ? REC_WKV : REC_DELTA;
            a.heads = L.c.heads; a.kv_heads = L.c.kv_heads; a.dim = L.c.dim; a.vdim = L.c.vdim; a.w_bf16 = m->bf16;
            a.proj = m->proj;
            a.off_q = L.off_q; a.off_k = L.off_k; a.off_v = L.off_v; a.off_b = L.off_b; a.off_lo = L.off_lo; a.off_hi = L.off_hi; a.off_gate = L.off_g;
            a.w_lo = L.w_lo; a.w_hi = L.w_hi; a.r_lo = L.lo_rank; a.r_hi = L.hi_rank;
            a.bias = L.bias; a.a_log = L.a_log; a.u = L.u; a.taps_w = L.taps; a.conv = wkv ? nullptr : m->state->ptr(r.st_aux);
            a.taps = L.c.conv; a.unit_eps = c.unit_eps; a.q_scale = 1.0f / sqrtf((float)L.c.dim);
            a.step = m->d_step; a.gain = L.gain; a.gain_shared = !wkv; a.norm_eps = c.norm_eps;
            a.state = m->state->ptr(r.st_matrix); a.out = m->mixed;
            LUMEN_TRY(timed(m, wkv ? HC_WKV : HC_DELTA, do_rec, &a));
        }
        if (L.c.mixer == LUMEN_MIXER_PARALLEL) {
            // both output projections in one launch, the one of more columns first
            GemvArgs g = gemv_args(m, L.w_o, W, L.od, m->mixed, m->pair);
            g.pro = PRO_PAIR; g.W2 = L.w_o2; g.x2 = m->mixed2; g.y2 = m->pair + W; g.K2 = L.od2;
            if (L.od2 > L.od) { std::swap(g.W, g.W2); std::swap(g.x, g.x2); std::swap(g.y, g.y2); std::swap(g.K, g.K2); }
            LUMEN_TRY(timed(m, HC_OUT, do_gemv, &g));
            GatedResidualArgs p = {};
            p.x = cur; p.y = m->pair; p.y2 = m->pair + W; p.w1 = L.out1; p.w2 = L.out2; p.pair_scale = 0.5f; p.eps = c.norm_eps;
            p.gate = m->proj + L.off_rg; p.gate_b = L.rg1_b; p.out = out(); p.rows = 1; p.dim = W; p.width = c.width;
            LUMEN_TRY(timed(m, HC_PAIR, do_pair, &p));
            cur = p.out;
        } else {
            GemvArgs g = gemv_args(m, L.w_o, W, L.od, m->mixed, out());
            gemv_residual(g, cur, c.residual_mult);
            if (c.residual_gate) { g.res_gate = m->proj + L.off_rg; g.res_gate_b = L.rg1_b; }
            if (L.fold) {
                g.pro = PRO_ATTN_FOLD; g.attn_part = m->part; g.attn_pos = m->d_pos; g.attn_nslices = L.slices; g.attn_d = L.c.vdim;
                g.attn_trip = WINDOW_SLICE_KEYS; g.attn_short_rows = 0; g.attn_window = L.window; g.attn_gate = m->proj + L.off_g;
            }
            LUMEN_TRY(timed(m, HC_OUT, do_gemv, &g));
            cur = g.y;
        }
        if (L.c.ff > 0) {
            GemvArgs g = gemv_args(m, L.w_up, L.n_up, W, cur, m->ff);
            gemv_norm(m, g, L.norm2, L.norm2_b, L.norm2_a);
            if (L.c.ff_kind == LUMEN_FF_GELU) g.gelu_from = L.up_at;
            LUMEN_TRY(timed(m, HC_UP, do_gemv, &g));
            if (L.c.ff_kind == LUMEN_FF_EXPERTS) {
                ExpertsArgs e = experts_args(m, L);
                e.z = m->ff + L.up_at; e.x = cur; e.norm_alpha = L.norm2_a; e.norm_w = L.norm2; e.norm_b = L.norm2_b; e.gate = m->ff; e.gate_b = L.rg2_b;
                e.act = m->act; e.sel = m->d_sel; e.y = out();
                LUMEN_TRY(timed(m, HC_EXPERT_UP, do_experts_up, &e));
                LUMEN_TRY(timed(m, HC_EXPERT_DOWN, do_experts_down, &e));
                cur = e.y;
            } else {
                g = gemv_args(m, L.w_down, W, pad8(L.c.ff), m->ff + L.up_at, out());
                gemv_residual(g, cur, c.residual_mult);
                if (c.residual_gate) { g.res_gate = m->ff; g.res_gate_b = L.rg2_b; }
                if (L.c.ff_kind == LUMEN_FF_POLYNORM) { g.pro = PRO_POLYNORM; g.norm_w = L.act; g.eps = c.norm_eps; g.norm_dim = L.c.ff; }
                LUMEN_TRY(timed(m, HC_DOWN, do_gemv, &g));
                cur = g.y;
            }
        }
        LUMEN_TRY(tap_rows(m, tap, ri, cur, 1));
    }
    GemvArgs g = gemv_args(m, m->head, c.vocab_size, W, cur, m->logits);
    gemv_norm(m, g, m->final_norm, m->final_b, m->final_a);
    g.softcap = c.logit_softcap;
    g.epi = EPI_ARGMAX; g.amax_word = m->amax_word; g.amax_epoch = m->amax_epoch; g.err_dev = m->d_err; g.spin_limit = HANDOVER_MAX_SPINS;
    g.tok_out = m->d_tok; g.pos_inc = m->d_pos; g.tok_hist = m->tok_hist; g.step_inc = m->d_step;
    return timed(m, HC_HEAD, do_gemv, &g);
}

static int launch_step(lumen_hybrid *m) {
    if (m->decode_mode != LUMEN_DECODE_GRAPH) return enqueue_decode_step(m);
    if (!m->graph_exec) LUMEN_TRY(record_graph(m->ctx->stream, [&]() { return enqueue_decode_step(m); }, &m->graph, &m->graph_exec));
    HIP_TRY(hipGraphLaunch(m->graph_exec, m->ctx->stream));
    return LUMEN_OK;
}

// after a synchronisation: did the arg-max tail's wait run into its limit?
static int check_handover(lumen_hybrid *m) {
    int err = 0;
    HIP_TRY(hipMemcpy(&err, m->d_err, sizeof(int), hipMemcpyDeviceToHost));
    if (!err) return LUMEN_OK;
    HIP_TRY(hipMemset(m->d_err, 0, sizeof(int)));
    LUMEN_FAIL(LUMEN_ERR_HIP, "decode: a workgroup gave up waiting for a value handed over inside a launch; the results of this call are invalid");
}

__global__ void set_counters_kernel(int *pos, unsigned *step, int p, unsigned s) {
    *pos = p;
    *step = s;
}
static int sync_counters(lumen_hybrid *m) {
    hipLaunchKernelGGL(set_counters_kernel, dim3(1), dim3(1), 0, m->ctx->stream, m->d_pos, m->d_step, m->len, m->step);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

static int check_ids(const lumen_hybrid *m, const int32_t *ids, int s) {
    for (int t = 0; t < s; ++t)
        if (ids[t] < 0 || ids[t] >= m->cfg.vocab_size)
            LUMEN_FAIL(LUMEN_ERR_EMBED_OOB, "Embedding index out of bounds: %d >= %d", ids[t], m->cfg.vocab_size);
    return LUMEN_OK;
}
static int check_room(const lumen_hybrid *m, int add) {
    if (add > m->cfg.max_seq_len - m->len)
        LUMEN_FAIL(LUMEN_ERR_KV_OVERFLOW, "sequence too long: new_len=%d > max_seq=%d", m->len + add, m->cfg.max_seq_len);
    return LUMEN_OK;
}

// ------------------------------------------------------------------ prompt
static int ensure_prompt_buffers(lumen_hybrid *m, int s) {
    if (s <= m->pf_cap) return LUMEN_OK;
    HIP_TRY(hipStreamSynchronize(m->ctx->stream));
    for (void *p : m->pf_allocs) hipFree(p);
    m->pf_allocs.clear();
    m->pf_cap = 0;
    const size_t S = (size_t)s, W = m->W;
    auto get = [&](float **p, size_t n) { return alloc_t(m, p, n, &m->pf_allocs); };
    bool wkv = false;
    for (const Layer &L : m->layers) wkv |= L.c.mixer == LUMEN_MIXER_WKV;
    LUMEN_TRY(get(&m->p_x0, S * W));
    LUMEN_TRY(get(&m->p_xa, S * W));
    LUMEN_TRY(get(&m->p_xb, S * W));
    LUMEN_TRY(get(&m->p_n, S * W));
    LUMEN_TRY(get(&m->p_rows, S * W));
    LUMEN_TRY(get(&m->p_proj, S * m->max_proj));
    if (wkv) LUMEN_TRY(get(&m->p_mixes, 5 * S * W));
    LUMEN_TRY(get(&m->p_mixed, S * m->max_od));
    LUMEN_TRY(get(&m->p_ff, S * m->max_ff));
    LUMEN_TRY(get(&m->p_steps, S * W * std::max(m->cfg.loop_times, 1)));
    LUMEN_TRY(get(&m->p_q, S * m->max_heads));
    LUMEN_TRY(get(&m->p_k, S * m->max_heads));
    LUMEN_TRY(get(&m->p_v, S * m->max_heads));
    LUMEN_TRY(get(&m->p_lo, S * m->max_lo));
    LUMEN_TRY(get(&m->p_hi, S * m->max_hi));
    LUMEN_TRY(get(&m->p_z, S * pad8(m->max_heads)));
    LUMEN_TRY(get(&m->p_gate, S * pad8(m->max_heads)));
    if (m->cfg.residual_gate) {
        LUMEN_TRY(get(&m->p_y, S * W));
        LUMEN_TRY(get(&m->p_rg, S * W));
    }
    if (m->max_od2) {
        LUMEN_TRY(get(&m->p_y2, S * W));
        LUMEN_TRY(get(&m->p_raw, S * m->max_raw));
        LUMEN_TRY(get(&m->p_mixed2, S * m->max_od2));
        size_t scan = 0;
        for (const Layer &L : m->layers) scan = std::max(scan, memory_scan_floats(s, L.c.mem_heads));
        LUMEN_TRY(get(&m->p_scan, scan));
    }
    if (m->max_top) {
        size_t plan = 0;
        for (const Layer &L : m->layers)
            if (L.c.ff > 0 && L.c.ff_kind == LUMEN_FF_EXPERTS) plan = std::max(plan, experts_plan_ints(s, experts_args(m, L).r));
        LUMEN_TRY(get(&m->p_route, S * m->max_experts));
        LUMEN_TRY(get(&m->p_selw, S * m->max_top));
        LUMEN_TRY(get(&m->p_act, S * m->max_act));
        LUMEN_TRY(get(&m->p_eout, S * m->max_top * W));
        LUMEN_TRY(alloc_t(m, &m->p_plan, plan, &m->pf_allocs));
    }
    LUMEN_TRY(alloc_t(m, &m->p_ids, S, &m->pf_allocs));
    LUMEN_TRY(alloc_t(m, &m->p_idx, S, &m->pf_allocs));
    m->pf_cap = s;
    return LUMEN_OK;
}

static GemmArgs gemm_args(const lumen_hybrid *m, const float *A, const void *w, float *C, int M, int N, int K) {
    GemmArgs g = {};
    g.A = A; g.W = w; g.C = C; g.M = M; g.N = N; g.K = K; g.w_bf16 = m->bf16; g.epi = EPI_STORE;
    return g;
}

static int prompt_attention(lumen_hybrid *m, const Layer &L, const Run &r, int s) {
    WindowAttnArgs a = attn_args(m, L, r, m->p_proj, L.n_proj);
    LUMEN_TRY(launch_gemm(m->ctx, gemm_args(m, m->p_n, L.w_proj, m->p_proj, s, L.n_proj, m->W)));
    a.out = m->p_mixed; a.out_stride = L.od; a.pos = m->len; a.s = s; a.qn = m->p_q;
    return launch_window_attn_prefill(m->ctx, a);
}

static int prompt_wkv(lumen_hybrid *m, const Layer &L, const Run &r, int s) {
    lumen_ctx *ctx = m->ctx;
    const int W = m->W, H = L.c.heads, D = L.c.dim;
    float *shift = m->state->ptr(r.st_aux);
    const unsigned slot = m->step & 1u;
    LUMEN_TRY(launch_token_shift(ctx, m->p_n, L.mu, shift + (size_t)slot * W, shift + (size_t)(slot ^ 1u) * W, m->p_mixes, 5, s, W));
    // r, k, v, gate and the decay's inner vector: a matrix each, one after the other
    float *part[5];
    for (int i = 0; i < 5; ++i) {
        part[i] = m->p_proj + (size_t)i * s * L.seg;
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_mixes + (size_t)i * s * W, (const char *)L.w_proj + (size_t)i * L.seg * W * m->esz, part[i],
                                             s, i < 4 ? L.seg : L.seg_last, W)));
    }
    LUMEN_TRY(launch_tanh(ctx, part[4], m->p_lo, (size_t)s * L.seg_last));
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_lo, L.w_lo, m->p_z, s, L.seg, L.lo_rank)));
    RecurrenceArgs a = {};
    a.kind = REC_WKV; a.heads = H; a.rep = 1; a.dim = D; a.vdim = D; a.s = s;
    a.q = part[0]; a.k = part[1]; a.v = part[2]; a.z = m->p_z;
    a.q_stride = a.k_stride = a.v_stride = a.z_stride = L.seg;
    a.bias = L.bias; a.u = L.u; a.state = m->state->ptr(r.st_matrix); a.out = m->p_mixed; a.out_stride = L.od;
    LUMEN_TRY(launch_recurrence(ctx, a));
    return launch_head_norm_gate(ctx, m->p_mixed, L.od, L.gain, 0, part[3], L.seg, GATE_SILU, s, H, D, m->cfg.norm_eps);
}

static int prompt_delta(lumen_hybrid *m, const Layer &L, const Run &r, int s) {
    lumen_ctx *ctx = m->ctx;
    const int H = L.c.heads, G = L.c.kv_heads, D = L.c.dim, Dv = L.c.vdim, keep = L.c.conv - 1;
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, L.w_proj, m->p_proj, s, L.n_proj, m->W)));
    float *conv = m->state->ptr(r.st_aux);
    const unsigned slot = m->step & 1u;
    DeltaPrepArgs p = {};
    p.in = m->p_proj; p.stride = L.n_proj; p.off_q = L.off_q; p.off_k = L.off_k; p.off_v = L.off_v; p.off_a1 = L.off_lo; p.off_g1 = L.off_hi;
    p.ra = L.lo_rank; p.rg = L.hi_rank; p.taps_w = L.taps;
    p.conv_prev = conv + (size_t)slot * keep * L.channels();
    p.conv_next = conv + (size_t)(slot ^ 1u) * keep * L.channels();
    p.q = m->p_q; p.k = m->p_k; p.v = m->p_v; p.a1 = m->p_lo; p.g1 = m->p_hi;
    p.taps = L.c.conv; p.heads = H; p.kv_heads = G; p.dim = D; p.vdim = Dv; p.s = s;
    p.unit_eps = m->cfg.unit_eps; p.q_scale = 1.0f / sqrtf((float)D);
    LUMEN_TRY(launch_delta_prep(ctx, p));
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_lo, L.w_lo, m->p_z, s, pad8(H * D), L.lo_rank)));
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_hi, L.w_hi, m->p_gate, s, pad8(H * Dv), L.hi_rank)));
    RecurrenceArgs a = {};
    a.kind = REC_DELTA; a.heads = H; a.rep = H / G; a.dim = D; a.vdim = Dv; a.s = s;
    a.q = m->p_q; a.k = m->p_k; a.v = m->p_v; a.z = m->p_z; a.b = m->p_proj + L.off_b;
    a.q_stride = a.k_stride = G * D; a.v_stride = H * Dv; a.z_stride = pad8(H * D); a.b_stride = L.n_proj;
    a.bias = L.bias; a.a_log = L.a_log; a.state = m->state->ptr(r.st_matrix); a.out = m->p_mixed; a.out_stride = L.od;
    LUMEN_TRY(launch_recurrence(ctx, a));
    return launch_head_norm_gate(ctx, m->p_mixed, L.od, L.gain, 1, m->p_gate, pad8(H * Dv), GATE_SIGMOID, s, H, Dv, m->cfg.norm_eps);
}

static int prompt_general(lumen_hybrid *m, const Layer &L, const Run &r, int s) {
    lumen_ctx *ctx = m->ctx;
    const int H = L.c.heads, D = L.c.dim, n = L.n_proj;
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, L.w_proj, m->p_proj, s, n, m->W)));
    LUMEN_TRY(launch_tanh_rows(ctx, m->p_proj + L.off_lo, n, m->p_lo, s, L.lo_rank));
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_lo, L.w_lo, m->p_z, s, pad8(H * D), L.lo_rank)));
    RecurrenceArgs a = {};
    a.kind = REC_GENERAL; a.heads = H; a.rep = 1; a.dim = a.vdim = D; a.s = s;
    a.q = m->p_proj + L.off_q; a.k = m->p_proj + L.off_k; a.v = m->p_proj + L.off_v; a.b = m->p_proj + L.off_a; a.z = m->p_z;
    a.q_stride = a.k_stride = a.v_stride = a.b_stride = n; a.z_stride = pad8(H * D);
    a.bias = L.bias; a.b_bias = L.a_bias; a.unit_eps = m->cfg.unit_eps; a.z_scale = GENERAL_DECAY;
    a.state = m->state->ptr(r.st_matrix); a.out = m->p_mixed; a.out_stride = L.od;
    LUMEN_TRY(launch_recurrence(ctx, a));
    return launch_head_norm_gate(ctx, m->p_mixed, L.od, L.gain, 0, m->p_proj + L.off_g, n, GATE_SIGMOID, s, H, D, m->cfg.norm_eps);
}

static int prompt_memory(lumen_hybrid *m, const Layer &L, const Run &r, int s) {
    const int H = L.c.mem_heads, D = L.c.mem_dim, V = L.c.mem_vdim, n = L.n_proj;
    RecurrenceArgs a = {};
    a.kind = REC_MEMORY; a.heads = H; a.rep = 1; a.dim = D; a.vdim = V; a.s = s;
    a.q = m->p_proj + L.off_mq; a.k = m->p_proj + L.off_mk; a.v = m->p_proj + L.off_mv; a.gi = m->p_proj + L.off_mi; a.gf = m->p_proj + L.off_mf;
    a.q_stride = a.k_stride = a.v_stride = a.g_stride = n;
    a.gi_bias = L.i_bias; a.gf_bias = L.f_bias; a.cap = L.c.gate_cap; a.q_scale = 1.0f / sqrtf((float)D);
    a.m = m->state->ptr(r.st_aux); a.m_out = m->p_scan; a.state = m->state->ptr(r.st_matrix); a.out = m->p_raw; a.out_stride = H * (V + 1);
    LUMEN_TRY(launch_recurrence(m->ctx, a));
    return launch_memory_read(m->ctx, m->p_raw, m->p_scan, m->p_mixed2, L.od2, L.gain, m->p_proj + L.off_mg, n, GATE_SIGMOID, s, H, V, m->cfg.norm_eps,
                              MEMORY_DEN_EPS);
}

// Mixer and feed-forward of a layer whose residuals are gated, p_n holding norm1 of cur; the sums go to x.  next: the norm that
// p_n is to hold afterwards (null gains: none).
struct NormRef {
    const float *w, *b, *alpha;
};
static int prompt_gated_layer(lumen_hybrid *m, const Layer &L, const Run &r, int s, const float *cur, float *x, NormRef next) {
    lumen_ctx *ctx = m->ctx;
    const lumen_hybrid_config &c = m->cfg;
    const int W = m->W;
    GatedResidualArgs p = {};
    p.eps = c.norm_eps; p.rows = s; p.dim = W; p.width = c.width;
    auto sum = [&](const float *from, const float *gate, int stride, const float *gate_b, NormRef n) {
        p.x = from; p.gate = gate; p.gate_stride = stride; p.gate_b = gate_b; p.out = x;
        p.norm_w = n.w; p.norm_b = n.b; p.norm_alpha = n.alpha; p.norm_out = n.w ? m->p_n : nullptr;
        return launch_gated_residual(ctx, p);
    };
    const NormRef norm2 = {L.norm2, L.norm2_b, L.norm2_a};
    if (L.c.mixer == LUMEN_MIXER_PARALLEL) {
        LUMEN_TRY(prompt_attention(m, L, r, s));
        LUMEN_TRY(prompt_memory(m, L, r, s));
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_mixed2, L.w_o2, m->p_y2, s, W, L.od2)));
        p.y2 = m->p_y2; p.w1 = L.out1; p.w2 = L.out2; p.pair_scale = 0.5f;
    } else {
        LUMEN_TRY(prompt_general(m, L, r, s));
    }
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_mixed, L.w_o, m->p_y, s, W, L.od)));
    p.y = m->p_y;
    LUMEN_TRY(sum(cur, m->p_proj + L.off_rg, L.n_proj, L.rg1_b, L.c.ff > 0 ? norm2 : next));
    if (L.c.ff <= 0) return LUMEN_OK;
    LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, L.w_up, m->p_rg, s, W, W)));
    const void *up = (const char *)L.w_up + (size_t)L.up_at * W * m->esz;
    p.y2 = nullptr;
    if (L.c.ff_kind == LUMEN_FF_EXPERTS) {
        const int E = pad8(L.c.experts);
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, up, m->p_route, s, E, W)));
        ExpertsArgs e = experts_args(m, L);
        e.z = m->p_route; e.z_stride = E; e.rows = m->p_n; e.sel_w = m->p_selw; e.p_act = m->p_act; e.out = m->p_eout; e.plan = m->p_plan; e.s = s;
        LUMEN_TRY(launch_experts_prefill(ctx, e));
        p.y = m->p_eout; p.top = L.c.top; p.sel_w = m->p_selw;
    } else {
        const int F = pad8(L.c.ff);
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, up, m->p_ff, s, F, W)));
        LUMEN_TRY(launch_gelu(ctx, m->p_ff, m->p_ff, (size_t)s * F));
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_ff, L.w_down, m->p_y, s, W, F)));
    }
    return sum(x, m->p_rg, W, L.rg2_b, next);
}

// s tokens (two or more) from the live state on; logits of the rows `want` [n_want] to logits_host.
static int run_prompt(lumen_hybrid *m, const int32_t *ids, int s, const int *want, int n_want, float *logits_host, const Tap *tap) {
    const lumen_hybrid_config &c = m->cfg;
    lumen_ctx *ctx = m->ctx;
    const int W = m->W, V = c.vocab_size;
    LUMEN_TRY(ensure_prompt_buffers(m, s));
    HIP_TRY(hipMemcpyAsync(m->p_ids, ids, sizeof(int) * (size_t)s, hipMemcpyHostToDevice, ctx->stream));
    LUMEN_TRY(embed_rows(m, m->p_ids, s, nullptr, m->len, m->p_x0));
    const bool mix = c.loop_times > 0 && c.loop_kind == LUMEN_LOOP_MIX, dyt = c.norm_kind == LUMEN_NORM_DYT;
    if (mix) {
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_x0, m->loop_x0, m->p_n, s, W, W)));
        LUMEN_TRY(launch_add_steps(ctx, m->p_n, m->loop_step, m->p_steps, c.loop_times, s, W));
    }
    const float *cur = m->p_x0;
    bool normed = false;  // p_n holds norm1 of the next layer: it came with the product that finished cur
    auto out = [&]() { return cur == m->p_x0 ? m->p_xa : const_cast<float *>(cur); };
    auto residual_gemm = [&](GemmArgs g, const float *residual, float alpha, const float *norm) {
        g.epi = EPI_RESIDUAL; g.residual = residual; g.alpha = alpha;
        if (norm) { g.norm_w = norm; g.norm_out = m->p_n; g.norm_eps = m->eps_w; }
        normed = norm != nullptr;
        cur = g.C;
        return launch_gemm(ctx, g);
    };
    for (size_t ri = 0; ri < m->runs.size(); ++ri) {
        const Run &r = m->runs[ri];
        const Layer &L = m->layers[r.layer];
        const Run *next = ri + 1 < m->runs.size() ? &m->runs[ri + 1] : nullptr;
        const Layer *next_layer = next && next->pass < 0 ? &m->layers[next->layer] : nullptr;
        const float *next_norm = next_layer ? next_layer->norm1 : nullptr;
        if (r.pass >= 0 && !mix) {
            float *y = cur == m->p_xa ? m->p_xb : m->p_xa;
            LUMEN_TRY(launch_add_steps(ctx, cur, m->loop_step + (size_t)r.pass * W, y, 1, s, W));
            cur = y;
            normed = false;
        } else if (r.pass >= 0)
            LUMEN_TRY(residual_gemm(gemm_args(m, cur, m->loop_x, cur == m->p_xa ? m->p_xb : m->p_xa, s, W, W),
                                    m->p_steps + (size_t)r.pass * s * W, 1.0f, L.norm1));
        if (!normed && dyt) LUMEN_TRY(launch_dyt(ctx, cur, L.norm1_a, L.norm1, L.norm1_b, m->p_n, s, W));
        else if (!normed) LUMEN_TRY(launch_rmsnorm(ctx, cur, L.norm1, m->p_n, s, W, m->eps_w));
        if (c.residual_gate) {
            float *x = out();
            LUMEN_TRY(prompt_gated_layer(m, L, r, s, cur, x, next_layer ? NormRef{next_layer->norm1, next_layer->norm1_b, next_layer->norm1_a} : NormRef{}));
            cur = x;
            normed = next_layer != nullptr;
            LUMEN_TRY(tap_rows(m, tap, ri, cur, s));
            continue;
        }
        if (L.c.mixer == LUMEN_MIXER_WINDOW_ATTENTION) LUMEN_TRY(prompt_attention(m, L, r, s));
        else if (L.c.mixer == LUMEN_MIXER_WKV) LUMEN_TRY(prompt_wkv(m, L, r, s));
        else LUMEN_TRY(prompt_delta(m, L, r, s));
        LUMEN_TRY(residual_gemm(gemm_args(m, m->p_mixed, L.w_o, out(), s, W, L.od), cur, c.residual_mult, L.c.ff > 0 ? L.norm2 : next_norm));
        if (L.c.ff > 0) {
            const int F = pad8(L.c.ff);
            LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, L.w_up, m->p_ff, s, F, W)));
            LUMEN_TRY(launch_polynorm(ctx, m->p_ff, L.act, m->p_ff, s, L.c.ff, F, c.norm_eps));
            LUMEN_TRY(residual_gemm(gemm_args(m, m->p_ff, L.w_down, out(), s, W, F), cur, c.residual_mult, next_norm));
        }
        LUMEN_TRY(tap_rows(m, tap, ri, cur, s));
    }
    m->len += s;
    m->step += 1;
    LUMEN_TRY(sync_counters(m));
    if (n_want == 1) {
        GemvArgs g = gemv_args(m, m->head, V, W, cur + (size_t)want[0] * W, m->logits);
        gemv_norm(m, g, m->final_norm, m->final_b, m->final_a);
        g.softcap = c.logit_softcap;
        LUMEN_TRY(launch_gemv(ctx, g));
        return lumen_download(ctx, logits_host, m->logits, sizeof(float) * (size_t)V);
    }
    if (n_want > 1) {
        if (n_want > m->pf_logit_cap) {
            HIP_TRY(hipStreamSynchronize(ctx->stream));
            hipFree(m->p_logits);
            m->p_logits = nullptr;
            m->pf_logit_cap = 0;
            HIP_TRY(hipMalloc((void **)&m->p_logits, (size_t)n_want * V * sizeof(float)));
            m->pf_logit_cap = n_want;
        }
        HIP_TRY(hipMemcpyAsync(m->p_idx, want, sizeof(int) * (size_t)n_want, hipMemcpyHostToDevice, ctx->stream));
        LUMEN_TRY(launch_gather_rows(ctx, cur, m->p_idx, m->p_rows, n_want, W));
        if (dyt) LUMEN_TRY(launch_dyt(ctx, m->p_rows, m->final_a, m->final_norm, m->final_b, m->p_n, n_want, W));
        else LUMEN_TRY(launch_rmsnorm(ctx, m->p_rows, m->final_norm, m->p_n, n_want, W, m->eps_w));
        LUMEN_TRY(launch_gemm(ctx, gemm_args(m, m->p_n, m->head, m->p_logits, n_want, V, W)));
        if (c.logit_softcap > 0.f) LUMEN_TRY(launch_softcap(ctx, m->p_logits, c.logit_softcap, (size_t)n_want * V));
        return lumen_download(ctx, logits_host, m->p_logits, sizeof(float) * (size_t)n_want * V);
    }
    // (nothing to bring back: the ids' upload must still be done before the caller's array goes)
    HIP_TRY(hipStreamSynchronize(ctx->stream));
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_forward(lumen_hybrid *m, const int32_t *ids, int s, const int32_t *want, int n_want, float *logits_host,
                                    float *residual_host) {
    if (!m || !ids || (n_want > 0 && (!want || !logits_host))) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_forward: null argument");
    if (s <= 0 || n_want < 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_forward: empty input");
    for (int i = 0; i < n_want; ++i)
        if (want[i] < 0 || want[i] >= s || (i && want[i] <= want[i - 1]))
            LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_forward: rows of logits must ascend within the %d tokens", s);
    HIP_TRY(hipSetDevice(m->ctx->device));
    LUMEN_TRY(check_ids(m, ids, s));
    LUMEN_TRY(check_room(m, s));
    Tap tap;
    tap.host = residual_host;
    tap.total = (size_t)s;
    const int V = m->cfg.vocab_size;
    int w = 0;
    for (int t = 0; t < s;) {
        const int n = std::min(m->cfg.max_chunk, s - t);
        tap.at = (size_t)t;
        int nw = 0;
        std::vector<int> rows;
        for (; w + nw < n_want && want[w + nw] < t + n; ++nw) rows.push_back(want[w + nw] - t);
        float *lg = logits_host ? logits_host + (size_t)w * V : nullptr;
        if (n > 1) {
            LUMEN_TRY(run_prompt(m, ids + t, n, rows.data(), nw, lg, &tap));
        } else {
            hipStream_t st = m->ctx->stream;
            HIP_TRY(hipMemcpyAsync(m->d_tok, ids + t, sizeof(int), hipMemcpyHostToDevice, st));
            HIP_TRY(hipStreamSynchronize(st));
            if (residual_host) LUMEN_TRY(enqueue_decode_step(m, &tap));
            else LUMEN_TRY(launch_step(m));
            m->len += 1;
            m->step += 1;
            if (nw) {
                LUMEN_TRY(lumen_download(m->ctx, lg, m->logits, sizeof(float) * (size_t)V));
                LUMEN_TRY(check_handover(m));
            }
        }
        w += nw;
        t += n;
    }
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_decode_greedy(lumen_hybrid *m, int first_id, int n, int32_t *ids_out, float *logits_out) {
    if (!m) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_decode_greedy: null model");
    if (n < 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "hybrid_decode_greedy: n=%d", n);
    const int32_t first = first_id;
    LUMEN_TRY(check_ids(m, &first, 1));
    if (n == 0) return LUMEN_OK;
    HIP_TRY(hipSetDevice(m->ctx->device));
    LUMEN_TRY(check_room(m, n));
    hipStream_t st = m->ctx->stream;
    const size_t V = (size_t)m->cfg.vocab_size;
    HIP_TRY(hipMemcpyAsync(m->d_tok, &first, sizeof(int), hipMemcpyHostToDevice, st));
    HIP_TRY(hipStreamSynchronize(st));
    const int len0 = m->len;
    for (int t = 0; t < n; ++t) {
        LUMEN_TRY(launch_step(m));
        m->len += 1;
        m->step += 1;
        if (logits_out) HIP_TRY(hipMemcpyAsync(logits_out + (size_t)t * V, m->logits, sizeof(float) * V, hipMemcpyDeviceToHost, st));
    }
    HIP_TRY(hipStreamSynchronize(st));
    // the arg-max tail leaves every pick at the index of the position it is the token of
    if (ids_out) HIP_TRY(hipMemcpy(ids_out, m->tok_hist + len0 + 1, sizeof(int) * (size_t)n, hipMemcpyDeviceToHost));
    return check_handover(m);
}

extern "C" int lumen_hybrid_decode_profile(lumen_hybrid *m, int first_id, int n, double *ms_sum_out, int *count_out, int n_classes) {
    if (!m || !ms_sum_out || !count_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_decode_profile: null argument");
    if (n_classes < HC_COUNT) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_decode_profile: need %d classes", (int)HC_COUNT);
    const int32_t first = first_id;
    LUMEN_TRY(check_ids(m, &first, 1));
    for (int i = 0; i < n_classes; ++i) { ms_sum_out[i] = 0.0; count_out[i] = 0; }
    HIP_TRY(hipSetDevice(m->ctx->device));
    LUMEN_TRY(check_room(m, n));
    hipStream_t st = m->ctx->stream;
    HIP_TRY(hipMemcpyAsync(m->d_tok, &first, sizeof(int), hipMemcpyHostToDevice, st));
    HIP_TRY(hipStreamSynchronize(st));
    int rc = LUMEN_OK;
    for (int t = 0; t < n && rc == LUMEN_OK; ++t) {
        Probe probe;
        m->probe = &probe;
        m->ctx->note_kernels = true;
        rc = enqueue_decode_step(m);
        m->ctx->note_kernels = false;
        m->probe = nullptr;
        const hipError_t e = hipStreamSynchronize(st);
        if (rc == LUMEN_OK && e == hipSuccess) {
            m->len += 1;
            m->step += 1;
            for (size_t i = 0; i < probe.cls.size(); ++i) {
                float ms = 0.f;
                if (hipEventElapsedTime(&ms, probe.ev[2 * i], probe.ev[2 * i + 1]) == hipSuccess) {
                    ms_sum_out[probe.cls[i]] += ms;
                    count_out[probe.cls[i]] += 1;
                }
            }
        }
        for (hipEvent_t ev : probe.ev) hipEventDestroy(ev);
        if (rc == LUMEN_OK && e != hipSuccess) {
            lumen_set_error("hybrid_decode_profile step %d: %s", t, hipGetErrorString(e));
            rc = LUMEN_ERR_HIP;
        }
        if (rc == LUMEN_OK) rc = check_handover(m);
    }
    return rc;
}

extern "C" int lumen_hybrid_generate_turn(lumen_hybrid *m, const int32_t *new_tokens, int n_new, const int32_t *history, int n_history,
                                          const lumen_sampling *sp, const int32_t *stop_ids, int n_stop, int32_t *out_ids, int out_cap,
                                          int *n_out) {
    if (n_out) *n_out = 0;
    if (!m) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_generate_turn: null argument");
    TurnModel t;
    t.vocab = m->cfg.vocab_size;
    t.max_len = m->cfg.max_seq_len;
    t.forward = [m](const int32_t *ids, int n, float *logits) {
        const int32_t last = n - 1;
        return lumen_hybrid_forward(m, ids, n, &last, 1, logits, nullptr);
    };
    t.len = [m](int *n) { return lumen_hybrid_len(m, n); };
    return generate_turn(t, new_tokens, n_new, history, n_history, sp, stop_ids, n_stop, out_ids, out_cap, n_out);
}

extern "C" int lumen_hybrid_reset(lumen_hybrid *m) {
    if (!m) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_reset: null model");
    HIP_TRY(hipSetDevice(m->ctx->device));
    m->len = 0;
    m->step = 0;
    LUMEN_TRY(m->state->reset());
    return sync_counters(m);
}

extern "C" int lumen_hybrid_len(const lumen_hybrid *m, int *len_out) {
    if (!m || !len_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_len: null argument");
    *len_out = m->len;
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_num_runs(const lumen_hybrid *m, int *n_out) {
    if (!m || !n_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_num_runs: null argument");
    *n_out = (int)m->runs.size();
    return LUMEN_OK;
}

extern "C" int lumen_hybrid_set_decode_mode(lumen_hybrid *m, int mode) {
    if (!m) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_set_decode_mode: null model");
    if (mode != LUMEN_DECODE_EAGER && mode != LUMEN_DECODE_GRAPH) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "hybrid_set_decode_mode: mode %d", mode);
    m->decode_mode = mode;
    return LUMEN_OK;
}

// weights once per layer run (a looped layer's are read again), recurrent state read and written, the window's rows
extern "C" int lumen_hybrid_decode_bytes(const lumen_hybrid *m, int len, double *bytes_out) {
    if (!m || !bytes_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "hybrid_decode_bytes: null argument");
    const double W = m->W, e = (double)m->esz;
    double b = (double)m->cfg.vocab_size * W * e;
    if (m->loop_x) b += W * W * e * (1.0 + m->cfg.loop_times);
    for (const Run &r : m->runs) {
        const Layer &L = m->layers[r.layer];
        b += e * (W * L.n_proj + W * L.od + W * L.od2 + W * L.n_up);
        if (L.c.ff_kind == LUMEN_FF_EXPERTS && L.c.ff > 0) b += e * 3.0 * W * pad8(L.c.ff) * L.c.top;
        else b += e * W * pad8(L.c.ff);
        if (L.c.mixer == LUMEN_MIXER_WINDOW_ATTENTION || L.c.mixer == LUMEN_MIXER_PARALLEL) {
            b += 4.0 * std::min(len, L.window) * L.c.kv_heads * (double)(L.c.dim + L.c.vdim);
            if (r.st_matrix >= 0) b += 2.0 * 4.0 * (double)m->state->floats(r.st_matrix);
        } else {
            b += e * ((double)L.c.heads * L.c.dim * L.lo_rank + (double)L.c.heads * L.c.vdim * L.hi_rank);
            b += 2.0 * 4.0 * (double)m->state->floats(r.st_matrix);
        }
    }
    *bytes_out = b;
    return LUMEN_OK;
}

// ------------------------------------------------------------------ the mechanisms as operators
extern "C" int lumen_polynorm_f32(lumen_ctx *ctx, const float *z, const float *coef, float *out, int rows, int dim, float eps) {
    if (!ctx || !z || !coef || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "polynorm: null argument");
    if (rows < 0 || dim <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "polynorm: rows=%d dim=%d", rows, dim);
    return launch_polynorm(ctx, z, coef, out, rows, dim, dim, eps);
}

extern "C" int lumen_token_shift_f32(lumen_ctx *ctx, const float *h, const float *mu, const float *prev, float *next, float *mixes, int n,
                                     int s, int dim) {
    if (!ctx || !h || !mu || !prev || !next || !mixes) LUMEN_FAIL(LUMEN_ERR_INVALID, "token_shift: null argument");
    if (n <= 0 || s <= 0 || dim <= 0 || prev == next) LUMEN_FAIL(LUMEN_ERR_SHAPE, "token_shift: n=%d s=%d dim=%d", n, s, dim);
    return launch_token_shift(ctx, h, mu, prev, next, mixes, n, s, dim);
}

extern "C" int lumen_recurrence_state_rows(int dim, int *rows_out) {
    if (!rows_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "recurrence_state_rows: null argument");
    if (dim <= 0 || dim > MIX_MAX_DIM) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "recurrence: heads of %d (at most %d)", dim, MIX_MAX_DIM);
    *rows_out = recurrence_rows(dim);
    return LUMEN_OK;
}

extern "C" int lumen_wkv_f32(lumen_ctx *ctx, const float *r, const float *k, const float *v, const float *z, const float *bias, const float *u,
                             float *state, float *out, int s, int heads, int dim) {
    if (!ctx || !r || !k || !v || !z || !bias || !u || !state || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "wkv: null argument");
    if (s < 0 || heads <= 0 || dim <= 0 || dim > MIX_MAX_DIM) LUMEN_FAIL(LUMEN_ERR_SHAPE, "wkv: s=%d heads=%d dim=%d", s, heads, dim);
    RecurrenceArgs a = {};
    a.kind = REC_WKV; a.heads = heads; a.rep = 1; a.dim = a.vdim = dim; a.s = s;
    a.q = r; a.k = k; a.v = v; a.z = z; a.bias = bias; a.u = u; a.state = state; a.out = out;
    a.q_stride = a.k_stride = a.v_stride = a.z_stride = a.out_stride = heads * dim;
    return launch_recurrence(ctx, a);
}

extern "C" int lumen_channel_delta_f32(lumen_ctx *ctx, const float *q, const float *k, const float *v, const float *z, const float *b,
                                       const float *bias, const float *a_log, float *state, float *out, int s, int heads, int kv_heads,
                                       int dim, int vdim) {
    if (!ctx || !q || !k || !v || !z || !b || !bias || !a_log || !state || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "channel_delta: null argument");
    if (s < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0 || vdim <= 0 || dim > MIX_MAX_DIM || vdim > MIX_MAX_DIM)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "channel_delta: s=%d heads=%d/%d dim=%d vdim=%d", s, heads, kv_heads, dim, vdim);
    RecurrenceArgs a = {};
    a.kind = REC_DELTA; a.heads = heads; a.rep = heads / kv_heads; a.dim = dim; a.vdim = vdim; a.s = s;
    a.q = q; a.k = k; a.v = v; a.z = z; a.b = b; a.bias = bias; a.a_log = a_log; a.state = state; a.out = out;
    a.q_stride = a.k_stride = kv_heads * dim; a.v_stride = a.out_stride = heads * vdim; a.z_stride = heads * dim; a.b_stride = heads;
    return launch_recurrence(ctx, a);
}

extern "C" int lumen_conv_unit_f32(lumen_ctx *ctx, const float *qkv, const float *taps_w, const float *prev, float *next, float *q, float *k,
                                   float *v, int s, int taps, int heads, int kv_heads, int dim, int vdim, float unit_eps, float q_scale) {
    if (!ctx || !qkv || !taps_w || !prev || !next || !q || !k || !v) LUMEN_FAIL(LUMEN_ERR_INVALID, "conv_unit: null argument");
    if (s < 0 || taps < 1 || taps > MIX_MAX_TAPS || heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || prev == next)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "conv_unit: s=%d taps=%d", s, taps);
    DeltaPrepArgs p = {};
    p.in = qkv; p.stride = 2 * kv_heads * dim + heads * vdim; p.off_k = kv_heads * dim; p.off_v = 2 * kv_heads * dim;
    p.taps_w = taps_w; p.conv_prev = prev; p.conv_next = next; p.q = q; p.k = k; p.v = v;
    p.taps = taps; p.heads = heads; p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim; p.s = s; p.unit_eps = unit_eps; p.q_scale = q_scale;
    return launch_delta_prep(ctx, p);
}

extern "C" int lumen_head_norm_gate_f32(lumen_ctx *ctx, float *o, const float *gain, int gain_shared, const float *gate, int gate_act, int rows,
                                        int heads, int vdim, float eps) {
    if (!ctx || !o || !gain) LUMEN_FAIL(LUMEN_ERR_INVALID, "head_norm_gate: null argument");
    if (rows < 0 || heads <= 0 || vdim <= 0 || gate_act < GATE_NONE || gate_act > GATE_SILU) LUMEN_FAIL(LUMEN_ERR_SHAPE, "head_norm_gate: rows=%d", rows);
    return launch_head_norm_gate(ctx, o, heads * vdim, gain, gain_shared, gate, heads * vdim, gate_act, rows, heads, vdim, eps);
}

extern "C" int lumen_dynamic_tanh_f32(lumen_ctx *ctx, const float *x, const float *alpha, const float *w, const float *b, float *out, int rows, int dim) {
    if (!ctx || !x || !alpha || !w || !b || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "dynamic_tanh: null argument");
    if (rows < 0 || dim <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "dynamic_tanh: rows=%d dim=%d", rows, dim);
    return launch_dyt(ctx, x, alpha, w, b, out, rows, dim);
}

extern "C" int lumen_gated_residual_f32(lumen_ctx *ctx, const float *x, const float *y, const float *y2, const float *w1, const float *w2,
                                        const float *gate, const float *gate_b, float *out, int rows, int dim, int width, float pair_scale, float eps) {
    if (!ctx || !x || !y || !gate || !gate_b || !out || (y2 && (!w1 || !w2))) LUMEN_FAIL(LUMEN_ERR_INVALID, "gated_residual: null argument");
    if (rows < 0 || dim <= 0 || dim % 4 || width <= 0 || width > dim) LUMEN_FAIL(LUMEN_ERR_SHAPE, "gated_residual: rows=%d dim=%d width=%d", rows, dim, width);
    GatedResidualArgs a = {};
    a.x = x; a.y = y; a.y2 = y2; a.w1 = w1; a.w2 = w2; a.gate = gate; a.gate_stride = dim; a.gate_b = gate_b; a.out = out;
    a.rows = rows; a.dim = dim; a.width = width; a.pair_scale = pair_scale; a.eps = eps;
    return launch_gated_residual(ctx, a);
}

extern "C" int lumen_general_delta_f32(lumen_ctx *ctx, const float *r, const float *k, const float *v, const float *z, const float *a_raw,
                                       const float *z_bias, const float *a_bias, float *state, float *out, int s, int heads, int dim, int vdim,
                                       float unit_eps) {
    if (!ctx || !r || !k || !v || !z || !a_raw || !z_bias || !a_bias || !state || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "general_delta: null argument");
    if (s < 0 || heads <= 0 || dim <= 0 || vdim <= 0 || dim > MIX_MAX_DIM || vdim > MIX_MAX_DIM)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "general_delta: s=%d heads=%d dim=%d vdim=%d", s, heads, dim, vdim);
    RecurrenceArgs a = {};
    a.kind = REC_GENERAL; a.heads = heads; a.rep = 1; a.dim = dim; a.vdim = vdim; a.s = s;
    a.q = r; a.k = k; a.v = v; a.z = z; a.b = a_raw; a.bias = z_bias; a.b_bias = a_bias; a.unit_eps = unit_eps; a.z_scale = GENERAL_DECAY;
    a.q_stride = a.k_stride = a.z_stride = a.b_stride = heads * dim; a.v_stride = a.out_stride = heads * vdim;
    a.state = state; a.out = out;
    return launch_recurrence(ctx, a);
}

extern "C" int lumen_matrix_memory_f32(lumen_ctx *ctx, const float *q, const float *k, const float *v, const float *gi, const float *gf,
                                       const float *i_bias, const float *f_bias, const float *gain, float *state, float *m, float *out, int s, int heads,
                                       int dim, int vdim, float cap, float eps) {
    if (!ctx || !q || !k || !v || !gi || !gf || !i_bias || !f_bias || !gain || !state || !m || !out)
        LUMEN_FAIL(LUMEN_ERR_INVALID, "matrix_memory: null argument");
    if (s <= 0 || heads <= 0 || dim <= 0 || vdim <= 0 || dim > MIX_MAX_DIM || vdim > MIX_MAX_DIM || !(cap > 0.f))
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "matrix_memory: s=%d heads=%d dim=%d vdim=%d cap=%g", s, heads, dim, vdim, cap);
    float *raw = nullptr, *scan = nullptr;
    auto run = [&]() {
        HIP_TRY(hipMalloc((void **)&raw, sizeof(float) * (size_t)s * heads * (vdim + 1)));
        HIP_TRY(hipMalloc((void **)&scan, sizeof(float) * memory_scan_floats(s, heads)));
        RecurrenceArgs a = {};
        a.kind = REC_MEMORY; a.heads = heads; a.rep = 1; a.dim = dim; a.vdim = vdim; a.s = s;
        a.q = q; a.k = k; a.v = v; a.gi = gi; a.gf = gf; a.gi_bias = i_bias; a.gf_bias = f_bias; a.g_stride = heads; a.cap = cap;
        a.q_stride = a.k_stride = heads * dim; a.v_stride = heads * vdim; a.q_scale = 1.0f / sqrtf((float)dim);
        a.m = m; a.m_out = scan; a.state = state; a.out = raw; a.out_stride = heads * (vdim + 1);
        LUMEN_TRY(launch_recurrence(ctx, a));
        return launch_memory_read(ctx, raw, scan, out, heads * vdim, gain, nullptr, 0, GATE_NONE, s, heads, vdim, eps, MEMORY_DEN_EPS);
    };
    const int rc = run();
    hipStreamSynchronize(ctx->stream);
    hipFree(raw);
    hipFree(scan);
    return rc;
}

static int check_router(const char *what, int rows, int experts, int groups, int keep, int top) {
    if (rows < 0 || experts <= 0 || groups <= 0 || experts % groups || keep <= 0 || keep > groups || top <= 0 || top > keep * (experts / groups))
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "%s: %d rows, %d of %d experts, %d of %d groups", what, rows, top, experts, keep, groups);
    if (experts > EXPERTS_MAX || top > EXPERTS_MAX_TOP) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "%s: %d experts, %d at a time", what, experts, top);
    return LUMEN_OK;
}

extern "C" int lumen_route_f32(lumen_ctx *ctx, const float *z, int *sel, float *w, int rows, int experts, int groups, int keep, int top, float scale) {
    if (!ctx || !z || !sel || !w) LUMEN_FAIL(LUMEN_ERR_INVALID, "route: null argument");
    LUMEN_TRY(check_router("route", rows, experts, groups, keep, top));
    return launch_route(ctx, RouterShape{experts, groups, keep, top, scale}, z, experts, rows, sel, w);
}

extern "C" int lumen_experts_f32(lumen_ctx *ctx, const float *h, const float *z, const void *w_up, const void *w_down, int w_bf16, float *out, float *w,
                                 int s, int dim, int ff, int experts, int groups, int keep, int top, float scale, float limit) {
    if (!ctx || !h || !z || !w_up || !w_down || !out || !w) LUMEN_FAIL(LUMEN_ERR_INVALID, "experts: null argument");
    LUMEN_TRY(check_router("experts", s, experts, groups, keep, top));
    if (dim <= 0 || ff <= 0 || dim % 8 || ff % 8) LUMEN_FAIL(LUMEN_ERR_SHAPE, "experts: dim=%d ff=%d", dim, ff);
    float *act = nullptr;
    int *plan = nullptr;
    ExpertsArgs e = {};
    e.r = RouterShape{experts, groups, keep, top, scale};
    auto run = [&]() {
        HIP_TRY(hipMalloc((void **)&act, sizeof(float) * (size_t)s * top * ff + 16));
        HIP_TRY(hipMalloc((void **)&plan, sizeof(int) * experts_plan_ints(s, e.r) + 16));
        e.w_up = w_up; e.w_down = w_down; e.w_bf16 = w_bf16; e.dim = dim; e.ff = ff; e.limit = limit; e.z = z; e.z_stride = experts;
        e.rows = h; e.sel_w = w; e.p_act = act; e.out = out; e.plan = plan; e.s = s;
        return launch_experts_prefill(ctx, e);
    };
    const int rc = run();
    hipStreamSynchronize(ctx->stream);
    hipFree(act);
    hipFree(plan);
    return rc;
}

// One operator call of the window attention; `shape` holds what differs from caller to caller.
static int window_attn_operator(lumen_ctx *ctx, const float *q, const float *k, const float *v, const float *gate, float *k_ring, float *v_ring, int cap,
                                float *out, int s, int pos, int heads, int kv_heads, int dim, int vdim, int window, const WindowAttnArgs &shape) {
    if (!ctx || !q || !k || !v || !k_ring || !v_ring || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "window_attn: null argument");
    if (s <= 0 || pos < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0 || vdim <= 0 || window <= 0)
        LUMEN_FAIL(LUMEN_ERR_SHAPE, "window_attn: s=%d pos=%d heads=%d/%d dim=%d vdim=%d window=%d", s, pos, heads, kv_heads, dim, vdim, window);
    if (dim > MIX_MAX_DIM || vdim > MIX_MAX_DIM) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "window_attn: heads wider than %d", MIX_MAX_DIM);
    if (cap < window - 1 + s) LUMEN_FAIL(LUMEN_ERR_KV_OVERFLOW, "window_attn: ring of %d positions for a window of %d and %d tokens", cap, window, s);
    // the projections as the model lays them out: one row of q | k | v | gate blocks per token
    const int nq = heads * dim, nk = kv_heads * dim, nv = kv_heads * vdim, ng = shape.gate_heads ? heads : heads * vdim, stride = nq + nk + nv + (gate ? ng : 0);
    float *rows = nullptr, *qn = nullptr, *part = nullptr;
    int *d_pos = nullptr;
    const int slices = window_attn_slices(window);
    auto run = [&]() {
        HIP_TRY(hipMalloc((void **)&rows, sizeof(float) * (size_t)s * stride));
        HIP_TRY(hipMalloc((void **)&qn, sizeof(float) * (size_t)s * nq));
        HIP_TRY(hipMalloc((void **)&part, sizeof(float) * (size_t)heads * slices * (vdim + 2)));
        HIP_TRY(hipMalloc((void **)&d_pos, sizeof(int)));
        const float *src[4] = {q, k, v, gate};
        const int n[4] = {nq, nk, nv, ng};
        size_t off[4] = {0, 0, 0, 0}, at = 0;
        for (int i = 0; i < (gate ? 4 : 3); ++i) {
            off[i] = at;
            HIP_TRY(hipMemcpy2DAsync(rows + at, (size_t)stride * 4, src[i], (size_t)n[i] * 4, (size_t)n[i] * 4, s, hipMemcpyDeviceToDevice, ctx->stream));
            at += n[i];
        }
        HIP_TRY(hipMemcpyAsync(d_pos, &pos, sizeof(int), hipMemcpyHostToDevice, ctx->stream));
        WindowAttnArgs a = shape;
        a.q = rows; a.k = rows + off[1]; a.v = rows + off[2]; a.gate = gate ? rows + off[3] : nullptr; a.stride = stride;
        a.out = out; a.out_stride = heads * vdim;
        a.k_ring = k_ring; a.v_ring = v_ring; a.cap = cap; a.dpad = (dim + 3) & ~3; a.vpad = (vdim + 3) & ~3;
        a.heads = heads; a.kv_heads = kv_heads; a.dim = dim; a.vdim = vdim; a.window = window; a.gate_act = gate ? GATE_SIGMOID : GATE_NONE;
        a.pos_dev = d_pos; a.pos = pos; a.s = s; a.qn = qn; a.part = part; a.slices = slices;
        return s == 1 ? launch_window_attn_decode(ctx, a) : launch_window_attn_prefill(ctx, a);
    };
    const int rc = run();
    hipStreamSynchronize(ctx->stream);
    hipFree(rows);
    hipFree(qn);
    hipFree(part);
    hipFree(d_pos);
    return rc;
}

extern "C" int lumen_window_attn_f32(lumen_ctx *ctx, const float *q, const float *k, const float *v, const float *gate, const float *q_norm,
                                     const float *k_norm, const float *r1, const float *r2, float *k_ring, float *v_ring, int cap, float *out,
                                     int s, int pos, int heads, int kv_heads, int dim, int vdim, int window, float scale, float softcap,
                                     float norm_eps) {
    if ((r1 == nullptr) != (r2 == nullptr)) LUMEN_FAIL(LUMEN_ERR_INVALID, "window_attn: one of the two bias vectors");
    WindowAttnArgs a = {};
    a.q_norm_w = q_norm; a.k_norm_w = k_norm; a.norm_eps = norm_eps; a.scale = scale; a.softcap = softcap; a.r1 = r1; a.r2 = r2;
    return window_attn_operator(ctx, q, k, v, gate, k_ring, v_ring, cap, out, s, pos, heads, kv_heads, dim, vdim, window, a);
}

extern "C" int lumen_biased_attn_f32(lumen_ctx *ctx, const float *q, const float *k, const float *v, const float *gate, const float *temp,
                                     const float *bias_tab, int bias_n, const float *sink, float *k_ring, float *v_ring, int cap, float *out, int s, int pos,
                                     int heads, int kv_heads, int dim, int vdim, int window, float scale) {
    if (bias_tab && bias_n < 1) LUMEN_FAIL(LUMEN_ERR_SHAPE, "biased_attn: a bias table of %d", bias_n);
    WindowAttnArgs a = {};
    a.scale = scale; a.temp = temp; a.bias_tab = bias_tab; a.bias_n = bias_n; a.sink = sink; a.gate_heads = 1;
    return window_attn_operator(ctx, q, k, v, gate, k_ring, v_ring, cap, out, s, pos, heads, kv_heads, dim, vdim, window, a);
}
