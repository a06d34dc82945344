// Launchers of the sequence mixers beside the Llama attention: sliding-window attention with score shaping over a
// rolling key / value store, the WKV recurrence and the channel-wise gated delta rule, and the row operations they
// need.  Every launcher validates nothing: callers check shapes first.
#pragma once
#include "internal.h"

enum GateAct { GATE_NONE = 0, GATE_SIGMOID = 1, GATE_SILU = 2 };

#define MIX_MAX_DIM 256   // head sizes the mixer kernels are built for
#define MIX_MAX_TAPS 16   // longest causal convolution
#define MIX_MAX_RANK 1024 // longest inner size of a low-rank product taken inside a decode kernel

// ------------------------------------------------------------- row operations (elementwise.hip)
// out = a N(z) + b N(z^2) + c N(z^3) + e over the first dim of each row's `stride` elements (out may be z);
// coef = {a, b, c, e}
int launch_polynorm(lumen_ctx *ctx, const float *z, const float *coef, float *out, int rows, int dim, int stride, float eps);
// mixes [n][s][dim]: h_t + (h_{t-1} - h_t) mu_i; h_{-1} is prev [dim], the last h goes to next [dim] (not prev)
int launch_token_shift(lumen_ctx *ctx, const float *h, const float *mu, const float *prev, float *next, float *mixes, int n,
                       int s, int dim);
// out [times][rows][dim] = base [rows][dim] + step [times][dim]
int launch_add_steps(lumen_ctx *ctx, const float *base, const float *step, float *out, int times, int rows, int dim);
// out row i = x row idx[i]
int launch_gather_rows(lumen_ctx *ctx, const float *x, const int *idx, float *out, int n, int dim);
int launch_tanh(lumen_ctx *ctx, const float *x, float *out, size_t n);
int launch_tanh_rows(lumen_ctx *ctx, const float *x, int stride, float *out, int rows, int n);  // tanh of a block of columns, into a matrix of its own
int launch_gelu(lumen_ctx *ctx, const float *x, float *out, size_t n);                           // z Phi(z)
int launch_softcap(lumen_ctx *ctx, float *x, float cap, size_t n);                               // in place: cap tanh(x / cap)
// row t = W[ids[t]] + P[pos0 + t]; pos_dev (or null): pos0 in device memory
int launch_embedding_pos(lumen_ctx *ctx, const float *W, const int *ids_dev, const float *P, const int *pos_dev, int pos0, int n, int dim, int vocab,
                         int positions, float *out);
// Dynamic Tanh: tanh(*alpha x) w + b
int launch_dyt(lumen_ctx *ctx, const float *x, const float *alpha, const float *w, const float *b, float *out, int rows, int dim);
// out = x + sigmoid(gate + gate_b) v per element, rows of `dim` floats (a multiple of 4).  v is y; or, with y2, pair_scale (N(y) w1 +
// N(y2) w2), N dividing by the root mean square over `width` elements; or, with top > 0, the sum of the rows [row * top, (row + 1) top)
// of y weighted by sel_w.  norm_out (or null) receives the Dynamic Tanh of the result.
struct GatedResidualArgs {
    const float *x, *y, *y2, *w1, *w2;
    float pair_scale, eps;
    int top;
    const float *sel_w;
    const float *gate, *gate_b;
    int gate_stride;
    float *out;
    const float *norm_alpha, *norm_w, *norm_b;
    float *norm_out;
    int rows, dim, width;
};
int launch_gated_residual(lumen_ctx *ctx, const GatedResidualArgs &a);

// ------------------------------------------------------------- sliding-window attention (window_attention.hip)
// One sequence.  Keys and values of the last `cap` positions live in a ring: position p in slot p % cap, k_ring
// [kv_heads][cap][dpad], v_ring [kv_heads][cap][vpad] (rows padded with zeros to a multiple of 4).  Position i sees
// 0 <= i - j < window.  score = (q . k) scale, then softcap tanh(score / softcap) when softcap > 0, then less
// r1[h] ln(1 + r2[h] (i - j)) when r1 is given, then plus bias_tab[h][min(i - j, bias_n - 1)] when that is; softmax, whose
// denominator also holds exp(sink[h]) when sink is given; the output is multiplied by the activation of `gate`.
struct WindowAttnArgs {
    const float *q, *k, *v, *gate;   // rows of one projection buffer (row stride in floats), heads one after the other
    int stride;
    float *out;                      // [s][out_stride]
    int out_stride;
    const float *q_norm_w, *k_norm_w;  // gains of the RMSNorm over ALL of q's (k's) heads together, or null
    float norm_eps;
    float *k_ring, *v_ring;
    int cap, dpad, vpad;
    int heads, kv_heads, dim, vdim, window, gate_act;
    float scale, softcap;
    const float *r1, *r2;            // [heads] or null
    const float *temp;               // [heads] or null: scale is scale * temp[h]
    const float *bias_tab;           // [heads][bias_n] or null, times log2 e; distances past the end take the last entry
    int bias_n;
    const float *sink;               // [heads] or null
    int gate_heads;                  // gate holds one value per head (else one per channel)
    const int *pos_dev;              // decode: device int, position of the token
    int pos;                         // prompt: position of the first of s tokens
    int s;
    float *qn;                       // prompt: normalised queries [s][heads * dim], may be q's own rows when stride fits
    float *part;                     // decode over more than one slice: states [heads][slices][vdim + 2] (ctx, max in log2 units, sum)
    int slices;
    int leave_slices;                // ... for the output projection to fold (PRO_ATTN_FOLD), gate included: out is not written
};
#define WINDOW_SLICE_KEYS 256
int window_attn_slices(int window);                       // slices of a decode step over that window
int launch_window_attn_decode(lumen_ctx *ctx, const WindowAttnArgs &a);   // one token: norm, append, attend, gate
int launch_window_attn_prefill(lumen_ctx *ctx, const WindowAttnArgs &a);  // s tokens; cap >= window - 1 + s

// ------------------------------------------------------------- recurrences (recurrence.hip)
enum RecurrenceKind { REC_WKV = 0, REC_DELTA = 1, REC_GENERAL = 2, REC_MEMORY = 3 };
int recurrence_rows(int dim);  // key rows of a stored state column: dim rounded up to 64, 128 or 256
// s tokens of all heads.  state [heads][vdim][recurrence_rows(dim)], read and written.
//   WKV:   w = exp(-exp(z + bias));            o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T
//   delta: g = exp(-exp(a_log) softplus(z + bias));  S <- diag(g) S;  S <- S + k (sigmoid(b) (v - S^T k))^T;  o = S^T q
//   general delta: w = exp(-z_scale sigmoid(z + bias)), a = sigmoid(b + b_bias) per key channel, u = k / sqrt(sum k^2 + unit_eps);
//          S <- diag(w) S - (a u) (u^T S) + k v^T (both terms read the old state);  o = S^T q
//   memory: per head log gates i = cap tanh((gi + gi_bias) / cap), f = log sigmoid(cap tanh((gf + gf_bias) / cap)), m' = max(f + m, i);
//          S <- exp(f + m - m') S + exp(i - m') k v^T, and n likewise with k alone, kept as value column vdim (state
//          [heads][vdim + 1][rows], out rows [heads][vdim + 1], raw: S^T (q_scale q) and n . (q_scale q)); the running
//          maxima go to m_out [heads][s + 1] (m_out[.][0]: before the first token), the last one back to m
struct RecurrenceArgs {
    int kind, heads, rep, dim, vdim, s;  // head h reads q / k head h / rep
    const float *q, *k, *v, *z, *b;      // token rows, strides in floats (WKV: q is r)
    int q_stride, k_stride, v_stride, z_stride, b_stride;
    const float *bias;                   // [heads * dim]
    const float *a_log;                  // delta [heads]
    const float *u;                      // WKV [heads * dim]
    const float *b_bias;                 // general delta [heads * dim] (b: rows of heads * dim)
    float unit_eps, z_scale;             // general delta
    const float *gi, *gf, *gi_bias, *gf_bias;  // memory: token rows of stride g_stride, [heads]
    int g_stride;
    float cap, q_scale;
    float *m, *m_out;                    // memory
    float *state, *out;
    int out_stride;                      // out [s][out_stride], heads one after the other
};
int recurrence_columns(int kind, int vdim);  // value columns of the stored state
size_t memory_scan_floats(int s, int heads);  // floats of m_out (maxima, then log gates)
int launch_recurrence(lumen_ctx *ctx, const RecurrenceArgs &a);
// o [rows][stride] of heads x vdim, in place: o / rms(o) per head, times gain (one per channel, or one [vdim] for all heads), times act(gate)
int launch_head_norm_gate(lumen_ctx *ctx, float *o, int stride, const float *gain, int gain_shared, const float *gate,
                          int gate_stride, int gate_act, int rows, int heads, int vdim, float eps);
// reads the matrix memory's raw output rows [rows][heads][vdim + 1]: o = S^T q / (max(|n . q|, exp(-m)) + den_eps), then norm, gain
// [heads * vdim] and gate as above, into out [rows][out_stride]
int launch_memory_read(lumen_ctx *ctx, const float *raw, const float *m_scan, float *out, int out_stride, const float *gain, const float *gate,
                       int gate_stride, int gate_act, int rows, int heads, int vdim, float eps, float den_eps);
// Prompt front end of the delta rule: causal convolution + SiLU of q, k, v (channel c of the three one after the
// other reads taps_w[c][taps]), unit vectors of q and k per kv head, q times q_scale.  in: projection rows with the
// three blocks at off_q, off_k, off_v; conv_prev / conv_next [taps - 1][channels]: inputs before the first / after the
// last token, oldest first (distinct buffers).  Copies blocks a1 and g1 (ra, rg wide) out as matrices of their own.
struct DeltaPrepArgs {
    const float *in;
    int stride, off_q, off_k, off_v, off_a1, off_g1, ra, rg;
    const float *taps_w, *conv_prev;
    float *conv_next, *q, *k, *v, *a1, *g1;
    int taps, heads, kv_heads, dim, vdim, s;
    float unit_eps, q_scale;
};
int launch_delta_prep(lumen_ctx *ctx, const DeltaPrepArgs &a);

// One token, one launch: everything between the input projections and the output projection.  proj is the token's
// projection vector with its blocks at the given offsets; w_lo / w_hi are the second factors of the low-rank
// products (decay rows [heads * dim][r_lo], gate rows [heads * vdim][r_hi]), f32 or bf16.
struct RecurrenceDecodeArgs {
    int kind, heads, kv_heads, dim, vdim, w_bf16;
    const float *proj;
    int off_q, off_k, off_v, off_b, off_lo, off_hi, off_gate;
    const void *w_lo, *w_hi;
    int r_lo, r_hi;               // row lengths (a multiple of 8)
    const float *bias, *a_log, *u;
    const float *taps_w;          // delta: [channels][taps]
    float *conv;                  // delta: [2][taps - 1][channels], slot (*step & 1) read, the other written
    int taps;
    float unit_eps, q_scale;
    const unsigned *step;
    const float *gain;
    int gain_shared;
    float norm_eps;
    int off_a;                    // general delta: removal rates
    const float *a_bias;
    float z_scale;
    int off_i, off_f;             // memory: gates
    const float *i_bias, *f_bias;
    float cap, den_eps, *m;
    float *state, *out;           // out [heads * vdim]
};
int launch_recurrence_decode(lumen_ctx *ctx, const RecurrenceDecodeArgs &a);

// ------------------------------------------------------------- mixture of experts (experts.hip)
// Scores sigmoid(z); experts form `groups` groups of neighbours, a group's score is the sum of its two largest, only the best
// `keep` groups' experts can be chosen; the `top` best are, with weights s / (their sum + 1e-20) * scale.  Ties go to the lower index.
struct RouterShape {
    int experts, groups, keep, top;
    float scale;
};
#define EXPERTS_MAX 1024   // experts of a layer
#define EXPERTS_MAX_TOP 64 // experts of a token
// An expert is down (act(gate x, up x)), act(g, u) = min(g, limit) sigmoid(1.702 min(g, limit)) (clamp(u, -limit, limit) + 1).
// w_up [experts][2 ff][dim], gate and up rows in turn; w_down [experts][dim][ff]; ff and dim multiples of 8.
struct ExpertsArgs {
    RouterShape r;
    const void *w_up, *w_down;
    int w_bf16, dim, ff;
    float limit;
    const float *z;                 // router logits, rows of z_stride
    int z_stride;
    // decode: x is normalised (Dynamic Tanh) on the way in; the result is y = x + sigmoid(gate + gate_b) (weighted sum)
    const float *x, *norm_alpha, *norm_w, *norm_b, *gate, *gate_b;
    float *act, *y;                 // [top][ff]; [dim]
    int *sel;                       // [top]
    // prompt: rows normalised already; sel_w [s][top] and out [s][top][dim] (not weighted yet)
    const float *rows;
    float *sel_w, *p_act, *out;     // p_act [s * top][ff]
    int *plan;                      // experts_plan_ints(s, r) ints
    int s;
};
int launch_experts_up(lumen_ctx *ctx, const ExpertsArgs &a);    // one token: route, gate|up of the chosen experts
int launch_experts_down(lumen_ctx *ctx, const ExpertsArgs &a);  // ... down, weighted sum, gated residual
size_t experts_plan_ints(int s, const RouterShape &r);
int launch_experts_prefill(lumen_ctx *ctx, const ExpertsArgs &a);
int launch_route(lumen_ctx *ctx, const RouterShape &r, const float *z, int z_stride, int rows, int *sel, float *sel_w);

void lumen_warm_experts(hipStream_t s);
void lumen_warm_window_attention(hipStream_t s);
void lumen_warm_recurrence(hipStream_t s);
