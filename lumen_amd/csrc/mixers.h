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

// ------------------------------------------------------------- sliding-window attention (window_attention.hip)
// One sequence.  Keys and values of the last `cap` positions live in a ring: position p in slot p % cap, k_ring
// [kv_heads][cap][dpad], v_ring [kv_heads][cap][vpad] (rows padded with zeros to a multiple of 4).  Position i sees
// 0 <= i - j < window.  score = (q . k) scale, then softcap tanh(score / softcap) when softcap > 0, then less
// r1[h] ln(1 + r2[h] (i - j)) when r1 is given; softmax; the output is multiplied by the activation of `gate`.
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
enum RecurrenceKind { REC_WKV = 0, REC_DELTA = 1 };
int recurrence_rows(int dim);  // key rows of a stored state column: dim rounded up to 64, 128 or 256
// s tokens of all heads.  state [heads][vdim][recurrence_rows(dim)], read and written.
//   WKV:   w = exp(-exp(z + bias));            o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T
//   delta: g = exp(-exp(a_log) softplus(z + bias));  S <- diag(g) S;  S <- S + k (sigmoid(b) (v - S^T k))^T;  o = S^T q
struct RecurrenceArgs {
    int kind, heads, rep, dim, vdim, s;  // head h reads q / k head h / rep
    const float *q, *k, *v, *z, *b;      // token rows, strides in floats (WKV: q is r)
    int q_stride, k_stride, v_stride, z_stride, b_stride;
    const float *bias;                   // [heads * dim]
    const float *a_log;                  // delta [heads]
    const float *u;                      // WKV [heads * dim]
    float *state, *out;
    int out_stride;                      // out [s][out_stride], heads one after the other
};
int launch_recurrence(lumen_ctx *ctx, const RecurrenceArgs &a);
// o [rows][stride] of heads x vdim, in place: o / rms(o) per head, times gain (one per channel, or one [vdim] for all heads), times act(gate)
int launch_head_norm_gate(lumen_ctx *ctx, float *o, int stride, const float *gain, int gain_shared, const float *gate,
                          int gate_stride, int gate_act, int rows, int heads, int vdim, float eps);
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
    float *state, *out;           // out [heads * vdim]
};
int launch_recurrence_decode(lumen_ctx *ctx, const RecurrenceDecodeArgs &a);

void lumen_warm_window_attention(hipStream_t s);
void lumen_warm_recurrence(hipStream_t s);
