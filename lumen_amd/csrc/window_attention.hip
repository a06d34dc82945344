// Causal attention over a sliding window with shaped scores (soft cap, logarithmic distance bias), RMSNorm of the whole
// query and key projections in front and an element-wise output gate behind.  Keys and values live in a ring of `cap`
// positions (slot = position mod cap): what a window can still see is never overwritten, and memory does not grow
// with the sequence.  All arithmetic is f32.
#include "mixers.h"
#include "wave_reduce.h"

typedef float v4f __attribute__((ext_vector_type(4)));

// tanh by the continued fraction x / (1 + x^2 / (3 + x^2 / (5 + x^2 / (7 + x^2 / 9)))) up to 0.9 (truncation below
// 2.4e-8 there), by 1 - 2 / (e^{2 |x|} + 1) beyond: the absolute error stays small against x, which a soft cap multiplies.
__device__ __forceinline__ float tanh_near(float x) {
    const float y = x * x;
    return x * fmaf(y, y + 105.0f, 945.0f) * __builtin_amdgcn_rcpf(fmaf(y, fmaf(y, 15.0f, 420.0f), 945.0f));
}
__device__ __forceinline__ float tanh_w(float x) {
    const float y = x * x, near = tanh_near(x);
    const float far = 1.0f - 2.0f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(2.88539008177792681f * fabsf(x)) + 1.0f);
    return y <= 0.81f ? near : copysignf(far, x);
}

// Scores are kept in log2 units (times log2 e), so that a weight is one base-2 exponential and the distance bias
// r1 ln(1 + r2 d) is r1 log2(1 + r2 d).
#define LOG2E 1.44269504088896341f
struct ScoreShape {
    float in, out, r1, r2;  // score = out tanh(in dot), or in dot when out is 0
    bool log_bias;
    __device__ ScoreShape(float scale, float softcap, float r1_, float r2_, bool log_bias_) : r1(r1_), r2(r2_), log_bias(log_bias_) {
        const float log2e = LOG2E;
        in = softcap > 0.f ? scale / softcap : scale * log2e;
        out = softcap > 0.f ? softcap * log2e : 0.f;
    }
    __device__ float operator()(float dot, int dist) const {
        float s = in * dot;
        if (out > 0.f) s = out * tanh_w(s);
        return log_bias ? less_bias(s, dist) : s;
    }
    // the same in steps, for a wavefront that looks at its scores together
    __device__ float capped_near(float x) const { return out * tanh_near(x); }
    __device__ float less_bias(float s, int dist) const { return fmaf(-r1, __builtin_amdgcn_logf(fmaf(r2, (float)dist, 1.0f)), s); }
};

__device__ __forceinline__ float gate_w(float z, int act) {
    const float sig = 1.0f / (1.0f + expf(-z));
    return act == GATE_SIGMOID ? sig : act == GATE_SILU ? z * sig : 1.0f;
}

// ------------------------------------------------------------------ decode
#define WD_THREADS 512
#define WD_WAVES (WD_THREADS / 64)

int window_attn_slices(int window) { return (window + WINDOW_SLICE_KEYS - 1) / WINDOW_SLICE_KEYS; }

// One workgroup per (query head, slice of up to 512 keys).  Scores: a key belongs to a row of 16 lanes, 16-byte loads;
// thread k then shapes score k; the value rows are walked by groups of 16, 32 or 64 lanes whose sums meet in LDS.
// DB: 64-float blocks of a key row, LV: lanes per value row.
template <int DB, int LV>
__global__ __launch_bounds__(WD_THREADS) void window_decode_kernel(WindowAttnArgs a) {
    constexpr int GROUPS = WD_THREADS / LV;
    constexpr int KEYS = WINDOW_SLICE_KEYS / (WD_WAVES * 4);  // keys of a row of 16 lanes
    constexpr int U = DB == 1 ? 8 : DB == 2 ? 4 : 2;          // key rows in flight
    constexpr int VA = WINDOW_SLICE_KEYS / GROUPS < 8 ? WINDOW_SLICE_KEYS / GROUPS : 8;  // value rows requested ahead
    __shared__ __align__(16) float qs[DB * 64], kn[DB * 64], vn[LV * 4];
    __shared__ float sc[WINDOW_SLICE_KEYS];
    __shared__ __align__(16) float ctx[GROUPS][LV * 4];
    __shared__ float red[2][WD_WAVES], red_m[WD_WAVES], red_l[WD_WAVES];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15;
    const int h = blockIdx.x, slice = blockIdx.y, rep = a.heads / a.kv_heads, hk = h / rep, D = a.dim, Dv = a.vdim;
    const int pos = *a.pos_dev;
    const int lo = max(0, pos - a.window + 1) + slice * WINDOW_SLICE_KEYS;  // first key of the slice
    const int n = min(WINDOW_SLICE_KEYS, pos + 1 - lo);
    if (n <= 0) return;
    const bool has_new = lo + n - 1 == pos;
    const float *kr = a.k_ring + (size_t)hk * a.cap * a.dpad, *vr = a.v_ring + (size_t)hk * a.cap * a.vpad;
    const int slot_lo = lo % a.cap;
    auto slot_of = [&](int key) {  // (a slice never wraps twice: it is no longer than the ring)
        const int x = slot_lo + key;
        return (size_t)(x >= a.cap ? x - a.cap : x);
    };

    // Every load is issued unconditionally, positions clamped: keys past the slice get no weight, channels past a row meet
    // zero queries or no output.  (A load behind a condition would be waited for before the next one goes out.)
    const int row0 = wave * 4 + (lane >> 4);  // this row's keys: row0, row0 + 32, ...
    v4f kb[U][DB];
    auto fetch = [&](int i0) {
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int key = min(row0 + (i0 + i) * (WD_WAVES * 4), n - 1);
            const float *p = kr + slot_of(key) * a.dpad;
#pragma unroll
            for (int b = 0; b < DB; ++b) kb[i][b] = *(const v4f *)(p + min(b * 64 + i16 * 4, a.dpad - 4));
        }
    };
    fetch(0);
    const int grp = tid / LV, d4 = (tid % LV) * 4;
    auto value_row = [&](int key) { return *(const v4f *)(vr + slot_of(min(key, n - 1)) * a.vpad + min(d4, a.vpad - 4)); };
    v4f vb[VA];
#pragma unroll
    for (int i = 0; i < VA; ++i) vb[i] = value_row(grp + i * GROUPS);

    // queries and the new key, normalised over all heads together; what each thread turns into the head's q, k and v is
    // requested along with the values the sums are taken over
    const int dq = min(tid, D - 1), dv = min(tid, Dv - 1);
    const float own_q = a.q[h * D + dq], own_k = a.k[hk * D + dq], own_v = a.v[hk * Dv + dv];
    const float gain_q = a.q_norm_w ? a.q_norm_w[h * D + dq] : 1.f, gain_k = a.k_norm_w ? a.k_norm_w[hk * D + dq] : 1.f;
    const float gate = a.gate && a.slices == 1 ? a.gate[a.gate_heads ? h : h * Dv + dv] : 0.f;
    const float temp = a.temp ? a.temp[h] : 1.f, sink = a.sink ? a.sink[h] * LOG2E : -INFINITY;
    const float tab = a.bias_tab ? a.bias_tab[(size_t)h * a.bias_n + min(max(pos - lo - tid, 0), a.bias_n - 1)] : 0.f;  // of key tid
    const float r1 = a.r1 ? a.r1[h] : 0.f, r2 = a.r1 ? a.r2[h] : 0.f;
    float sq = 0.f, sk = 0.f;
    if (a.q_norm_w) {
        const int nq = a.heads * D;
#pragma unroll 4
        for (int i = tid; i < nq; i += WD_THREADS) sq = fmaf(a.q[i], a.q[i], sq);
    }
    if (a.k_norm_w && has_new) {
        const int nk = a.kv_heads * D;
#pragma unroll 4
        for (int i = tid; i < nk; i += WD_THREADS) sk = fmaf(a.k[i], a.k[i], sk);
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if (lane == 0) {
        red[0][wave] = sq;
        red[1][wave] = sk;
    }
    __syncthreads();
    sq = sk = 0.f;
#pragma unroll
    for (int w = 0; w < WD_WAVES; ++w) {
        sq += red[0][w];
        sk += red[1][w];
    }
    const float iq = a.q_norm_w ? 1.0f / sqrtf(sq / (float)(a.heads * D) + a.norm_eps) : 1.f;
    const float ik = a.k_norm_w ? 1.0f / sqrtf(sk / (float)(a.kv_heads * D) + a.norm_eps) : 1.f;
    const bool writer = has_new && h % rep == 0;
    const size_t slot = (size_t)(pos % a.cap);
    static_assert(DB * 64 <= WD_THREADS && LV * 4 <= WD_THREADS, "one thread per channel");
    if (tid < DB * 64) {
        const float k = has_new && tid < D ? own_k * ik * gain_k : 0.f;
        qs[tid] = tid < D ? own_q * iq * gain_q : 0.f;
        kn[tid] = k;
        if (writer && tid < a.dpad) a.k_ring[((size_t)hk * a.cap + slot) * a.dpad + tid] = k;
    }
    if (tid < LV * 4) {
        const float v = has_new && tid < Dv ? own_v : 0.f;
        vn[tid] = v;
        if (writer && tid < a.vpad) a.v_ring[((size_t)hk * a.cap + slot) * a.vpad + tid] = v;
    }
    __syncthreads();

    v4f q4[DB];
#pragma unroll
    for (int b = 0; b < DB; ++b) q4[b] = *(const v4f *)(qs + b * 64 + i16 * 4);
    for (int i0 = 0; i0 < KEYS; i0 += U) {
        if (i0 * (WD_WAVES * 4) >= n) break;  // (uniform)
        if (i0) fetch(i0);
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int key = row0 + (i0 + i) * (WD_WAVES * 4);
            const bool is_new = lo + key == pos;
            float s = 0.f;
#pragma unroll
            for (int b = 0; b < DB; ++b) {
                v4f k4 = kb[i][b];
                if (is_new) k4 = *(const v4f *)(kn + b * 64 + i16 * 4);
                s = fmaf(q4[b].x, k4.x, s);
                s = fmaf(q4[b].y, k4.y, s);
                s = fmaf(q4[b].z, k4.z, s);
                s = fmaf(q4[b].w, k4.w, s);
            }
            s = row16_sum(s);
            if (i16 == 0 && key < n) sc[key] = s;
        }
    }
    __syncthreads();
    const ScoreShape shape(a.scale * temp, a.softcap, r1, r2, a.r1 != nullptr);
    float s = -INFINITY;
    if (tid < n) s = shape(sc[tid], pos - lo - tid) + tab;
    float m = wave_max(s);
    if (lane == 0) red_m[wave] = m;
    __syncthreads();
    m = red_m[0];
#pragma unroll
    for (int w = 1; w < WD_WAVES; ++w) m = fmaxf(m, red_m[w]);
    if (slice == 0) m = fmaxf(m, sink);
    const float p = tid < n ? __builtin_amdgcn_exp2f(s - m) : 0.f;
    if (tid < WINDOW_SLICE_KEYS) sc[tid] = p;
    float l = wave_sum(p);
    if (lane == 0) red_l[wave] = l;
    __syncthreads();
    l = 0.f;
#pragma unroll
    for (int w = 0; w < WD_WAVES; ++w) l += red_l[w];
    if (slice == 0 && a.sink) l += __builtin_amdgcn_exp2f(sink - m);  // (once, whatever the number of slices)

    v4f acc = {0.f, 0.f, 0.f, 0.f};
    auto add = [&](int key, v4f v4) {
        if (lo + key == pos) v4 = *(const v4f *)(vn + d4);
        const float w = key < n ? sc[key] : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = fmaf(w, v4[e], acc[e]);
    };
#pragma unroll
    for (int i = 0; i < VA; ++i) add(grp + i * GROUPS, vb[i]);
#pragma unroll 4
    for (int key = grp + VA * GROUPS; key < n; key += GROUPS) add(key, value_row(key));
    *(v4f *)(&ctx[grp][d4]) = acc;
    __syncthreads();
    if (tid < Dv) {
        float o = 0.f;
#pragma unroll 8
        for (int g = 0; g < GROUPS; ++g) o += ctx[g][tid];
        if (a.slices > 1) a.part[((size_t)h * a.slices + slice) * (Dv + 2) + tid] = o;
        else a.out[h * Dv + tid] = o / l * (a.gate ? gate_w(gate, a.gate_act) : 1.0f);
    }
    if (a.slices > 1 && tid == 0) {
        float *pp = a.part + ((size_t)h * a.slices + slice) * (Dv + 2) + Dv;
        pp[0] = m;
        pp[1] = l;
    }
}

// Adds the slices of a head in slice order: one workgroup per head, a thread per channel.  The slices' maxima and sums
// are looked at by one wavefront, 64 at a time; a channel's values are requested WM_AHEAD slices at a time, the first of them
// before the weights are known.
#define WM_AHEAD 16
#define WM_SLICES 1024
__global__ __launch_bounds__(256) void window_merge_kernel(WindowAttnArgs a) {
    __shared__ float ws[WM_SLICES];
    __shared__ float total;
    const int h = blockIdx.x, tid = threadIdx.x, Dv = a.vdim, d = min(tid, Dv - 1);
    const float *part = a.part + (size_t)h * a.slices * (Dv + 2);
    const float gate = a.gate ? a.gate[a.gate_heads ? h : h * Dv + d] : 0.f;
    const int used = min(a.slices, (min(a.window, *a.pos_dev + 1) + WINDOW_SLICE_KEYS - 1) / WINDOW_SLICE_KEYS);
    float v[WM_AHEAD];
    auto fetch = [&](int s0) {
#pragma unroll
        for (int i = 0; i < WM_AHEAD; ++i) v[i] = part[(size_t)min(s0 + i, used - 1) * (Dv + 2) + d];
    };
    fetch(0);
    if (tid < 64) {
        const int mine = min(tid, used - 1);
        const float m0 = part[(size_t)mine * (Dv + 2) + Dv], l0 = part[(size_t)mine * (Dv + 2) + Dv + 1];
        float m = m0;
        for (int s = tid + 64; s < used; s += 64) m = fmaxf(m, part[(size_t)s * (Dv + 2) + Dv]);
        m = wave_max(m);
        float l = 0.f;
        for (int s = tid; s < used; s += 64) {
            const float w = __builtin_amdgcn_exp2f((s == tid ? m0 : part[(size_t)s * (Dv + 2) + Dv]) - m);
            ws[s] = w;
            l = fmaf(s == tid ? l0 : part[(size_t)s * (Dv + 2) + Dv + 1], w, l);
        }
        l = wave_sum(l);
        if (tid == 0) total = l;
    }
    __syncthreads();
    float o = 0.f;
    for (int s0 = 0; s0 < used; s0 += WM_AHEAD) {
        if (s0) fetch(s0);
#pragma unroll
        for (int i = 0; i < WM_AHEAD; ++i) o = s0 + i < used ? fmaf(v[i], ws[s0 + i], o) : o;
    }
    if (tid < Dv) a.out[h * Dv + tid] = o / total * (a.gate ? gate_w(gate, a.gate_act) : 1.0f);
}

int launch_window_attn_decode(lumen_ctx *ctx, const WindowAttnArgs &a) {
    const dim3 grid(a.heads, a.slices), block(WD_THREADS);
    const int db = a.dim <= 64 ? 1 : a.dim <= 128 ? 2 : 4, lv = a.vdim <= 64 ? 16 : a.vdim <= 128 ? 32 : 64;
    note_kernel(ctx, "window_decode_kernel<%d, %d>", db, lv);
#define WD_LAUNCH(DB)                                                                                              \
    do {                                                                                                           \
        if (lv == 16) hipLaunchKernelGGL((window_decode_kernel<DB, 16>), grid, block, 0, ctx->stream, a);          \
        else if (lv == 32) hipLaunchKernelGGL((window_decode_kernel<DB, 32>), grid, block, 0, ctx->stream, a);     \
        else hipLaunchKernelGGL((window_decode_kernel<DB, 64>), grid, block, 0, ctx->stream, a);                   \
    } while (0)
    if (db == 1) WD_LAUNCH(1);
    else if (db == 2) WD_LAUNCH(2);
    else WD_LAUNCH(4);
#undef WD_LAUNCH
    if (a.slices > WM_SLICES) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "window attention: %d slices of a decode step (at most %d)", a.slices, WM_SLICES);
    if (a.slices > 1 && !a.leave_slices) hipLaunchKernelGGL(window_merge_kernel, dim3(a.heads), dim3(256), 0, ctx->stream, a);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ------------------------------------------------------------------ prompt
// One workgroup per token: norms over all heads, queries out, key and value into the ring.
__global__ __launch_bounds__(256) void window_append_kernel(WindowAttnArgs a) {
    __shared__ float red[2][4];
    const int t = blockIdx.x, tid = threadIdx.x;
    const float *q = a.q + (size_t)t * a.stride, *k = a.k + (size_t)t * a.stride, *v = a.v + (size_t)t * a.stride;
    const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim;
    float sq = 0.f, sk = 0.f;
    for (int i = tid; i < nq; i += 256) sq = fmaf(q[i], q[i], sq);
    for (int i = tid; i < nk; i += 256) sk = fmaf(k[i], k[i], sk);
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) {
        red[0][tid >> 6] = sq;
        red[1][tid >> 6] = sk;
    }
    __syncthreads();
    sq = (red[0][0] + red[0][1]) + (red[0][2] + red[0][3]);
    sk = (red[1][0] + red[1][1]) + (red[1][2] + red[1][3]);
    const float iq = 1.0f / sqrtf(sq / (float)nq + a.norm_eps), ik = 1.0f / sqrtf(sk / (float)nk + a.norm_eps);
    for (int i = tid; i < nq; i += 256) a.qn[(size_t)t * nq + i] = a.q_norm_w ? q[i] * iq * a.q_norm_w[i] : q[i];
    const size_t slot = (size_t)((a.pos + t) % a.cap);
    for (int i = tid; i < a.kv_heads * a.dpad; i += 256) {
        const int g = i / a.dpad, d = i % a.dpad;
        float x = 0.f;
        if (d < a.dim) {
            x = k[g * a.dim + d];
            if (a.k_norm_w) x = x * ik * a.k_norm_w[g * a.dim + d];
        }
        a.k_ring[((size_t)g * a.cap + slot) * a.dpad + d] = x;
    }
    for (int i = tid; i < a.kv_heads * a.vpad; i += 256) {
        const int g = i / a.vpad, d = i % a.vpad;
        a.v_ring[((size_t)g * a.cap + slot) * a.vpad + d] = d < a.vdim ? v[g * a.vdim + d] : 0.f;
    }
}

// Online-softmax attention on the f32 matrix instruction.  A workgroup takes 64 queries of one head, a wavefront 16 of
// them; keys come in tiles of 32 through LDS.  Everything is transposed so that a lane owns one query: S^T = K Q^T (a
// lane (c, g) ends up with the scores of query c against keys 4 g + r), the weights of step r are then the B operand of
// O^T += V^T P^T as they stand, and the rescale factor is a scalar of the lane.  NB: 16-channel blocks the registers
// are laid out for.
#define WP_Q 64
#define WP_K 32
// Which head and which block of queries a workgroup takes.  Later queries see more keys, and workgroup n runs where
// workgroups n + 256, n + 512, ... run (round robin over 8 XCDs of 32 compute units): blocks are handed out from the last
// queries to the first, every other round of 256 in the opposite order, so that a compute unit's workgroups add up to
// about the same number of keys; neighbouring heads, which share keys, go to one XCD.
__device__ __forceinline__ void window_prefill_place(int n, int blocks, int heads, int &h, int &tb) {
    const int round = n >> 8;
    if ((round & 1) && (round + 1) * 256 <= blocks * heads) n = (round << 8) + ((31 - ((n & 255) >> 3)) << 3) + (n & 7);
    tb = blocks - 1 - n / heads;
    h = n % heads;
    if (heads % 8 == 0) h = (h & 7) * (heads >> 3) + (h >> 3);
}
template <int NB, bool FULL>
__global__ __launch_bounds__(256) void window_prefill_kernel(WindowAttnArgs a, int nd_, int nv_) {
    const int nd = FULL ? NB : nd_, nv = FULL ? NB : nv_;
    LUMEN_DYNAMIC_LDS(float, lds);
    const int kld = nd * 16 + 4, vld = nv * 16 + 4;
    float *ks = lds, *vs = lds + WP_K * kld;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    int h, tb;
    window_prefill_place((int)(blockIdx.y * gridDim.x + blockIdx.x), (int)gridDim.x, a.heads, h, tb);
    const int hk = h / (a.heads / a.kv_heads), D = a.dim, Dv = a.vdim;
    const int t0 = tb * WP_Q, tw = t0 + wave * 16, t = tw + c;  // first token of the workgroup / wavefront, own token
    const int last = min(t0 + WP_Q, a.s) - 1;
    const int i = a.pos + t;  // own position
    const ScoreShape shape(a.scale * (a.temp ? a.temp[h] : 1.f), a.softcap, a.r1 ? a.r1[h] : 0.f, a.r1 ? a.r2[h] : 0.f, a.r1 != nullptr);
    const float *tab = a.bias_tab ? a.bias_tab + (size_t)h * a.bias_n : nullptr;
    const float tab_far = tab ? tab[a.bias_n - 1] : 0.f;
    const float *kr = a.k_ring + (size_t)hk * a.cap * a.dpad, *vr = a.v_ring + (size_t)hk * a.cap * a.vpad;

    v4f qf[NB], acc[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) {
        qf[b] = v4f{0.f, 0.f, 0.f, 0.f};
        acc[b] = v4f{0.f, 0.f, 0.f, 0.f};
        if (b < nd && t < a.s) {
            const float *p = a.qn + ((size_t)t * a.heads + h) * D;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = b * 16 + g * 4 + e;
                if (d < D) qf[b][e] = p[d];
            }
        }
    }
    float m = -INFINITY, l = 0.f;
    if (a.sink) {  // (the sums of the four lane groups of a query are added at the end: the sink counts in one of them)
        m = a.sink[h] * LOG2E;
        l = g == 0 ? 1.f : 0.f;
    }
    const int j_first = max(0, a.pos + t0 - a.window + 1), j_last = a.pos + last;
    const int w_first = max(0, a.pos + tw - a.window + 1), w_last = a.pos + min(tw + 15, a.s - 1);  // of this wavefront
    // The tile in front travels in registers while this one is worked on.  Positions past the last key and channels past
    // the rows are clamped: the former get no weight, the latter meet zero queries or no output.
    constexpr int PER = (WP_K * NB * 4 + 255) / 256;  // 16-byte pieces of K and of V per thread
    v4f tk[PER], tv[PER];
    auto fetch = [&](int j0, int slot0) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = tid + i * 256;
            int row = e / (nd * 4), x = slot0 + min(min(row, WP_K - 1), j_last - j0);
            x = x >= a.cap ? x - a.cap : x;
            tk[i] = *(const v4f *)(kr + (size_t)x * a.dpad + min((e % (nd * 4)) * 4, a.dpad - 4));
            row = e / (nv * 4);
            x = slot0 + min(min(row, WP_K - 1), j_last - j0);
            x = x >= a.cap ? x - a.cap : x;
            tv[i] = *(const v4f *)(vr + (size_t)x * a.vpad + min((e % (nv * 4)) * 4, a.vpad - 4));
        }
    };
    int slot = j_first % a.cap;
    fetch(j_first, slot);
    for (int j0 = j_first; j0 <= j_last; j0 += WP_K) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = tid + i * 256;
            if (e < WP_K * nd * 4) *(v4f *)(ks + e / (nd * 4) * kld + e % (nd * 4) * 4) = tk[i];
            if (e < WP_K * nv * 4) *(v4f *)(vs + e / (nv * 4) * vld + e % (nv * 4) * 4) = tv[i];
        }
        __syncthreads();
        slot += WP_K;
        while (slot >= a.cap) slot -= a.cap;
        if (j0 + WP_K <= j_last) fetch(j0 + WP_K, slot);
        if (tw >= a.s || j0 > w_last || j0 + WP_K - 1 < w_first) continue;  // (uniform in the wavefront)
        v4f sc[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) sc[u] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int b = 0; b < NB; ++b)
            if (b < nd) {
                v4f kf[2];
#pragma unroll
                for (int u = 0; u < 2; ++u) kf[u] = *(const v4f *)(ks + (u * 16 + c) * kld + b * 16 + g * 4);
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int u = 0; u < 2; ++u) sc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[u][e], qf[b][e], sc[u], 0, 0, 0);
            }
        float mx = m;
        const int dist0 = i - j0 - g * 4;
        if (shape.out > 0.f) {
            // (most scores stay well below the cap: the far form of tanh is left out where the whole wavefront does)
            bool far = false;
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    sc[u][r] *= shape.in;
                    far |= fabsf(sc[u][r]) > 0.9f;
                }
            if (__any(far)) {
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sc[u][r] = shape.out * tanh_w(sc[u][r]);
            } else {
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sc[u][r] = shape.capped_near(sc[u][r]);
            }
        } else {
            sc[0] *= shape.in;
            sc[1] *= shape.in;
        }
        if (shape.log_bias) {
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) sc[u][r] = shape.less_bias(sc[u][r], dist0 - (u * 16 + r));
        }
        if (tab) {
            if (a.pos + tw - (j0 + WP_K - 1) >= a.bias_n - 1) {  // (uniform: every distance of the tile is past the table)
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sc[u][r] += tab_far;
            } else {
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sc[u][r] += tab[min(max(dist0 - (u * 16 + r), 0), a.bias_n - 1)];
            }
        }
        if (j0 + WP_K - 1 > a.pos + tw || j0 <= w_last - a.window) {  // (a tile every query of the wavefront sees whole needs no mask)
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int dist = dist0 - (u * 16 + r);
                    sc[u][r] = dist >= 0 && dist < a.window ? sc[u][r] : -INFINITY;
                }
        }
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) mx = fmaxf(mx, sc[u][r]);
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float base = mx > -INFINITY ? mx : 0.f;  // (a query that has seen nothing yet keeps zero weights)
        const float f = __builtin_amdgcn_exp2f(m - base);
        m = mx;
        l *= f;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                sc[u][r] = __builtin_amdgcn_exp2f(sc[u][r] - base);
                l += sc[u][r];
            }
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[b] *= f;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
                for (int b = 0; b < NB; ++b)  // (accumulators take turns: none waits for its own last product)
                    if (b < nv)
                        acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(vs[(u * 16 + g * 4 + r) * vld + b * 16 + c], sc[u][r], acc[b], 0, 0, 0);
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (t >= a.s) return;
    const float inv = 1.0f / l;
    float *o = a.out + (size_t)t * a.out_stride + (size_t)h * Dv;
    const float *gp = a.gate ? a.gate + (size_t)t * a.stride + (a.gate_heads ? (size_t)h : (size_t)h * Dv) : nullptr;
#pragma unroll
    for (int b = 0; b < NB; ++b)
        if (b < nv) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = b * 16 + g * 4 + r;
                if (d < Dv) o[d] = acc[b][r] * inv * (gp ? gate_w(gp[a.gate_heads ? 0 : d], a.gate_act) : 1.0f);
            }
        }
}

int launch_window_attn_prefill(lumen_ctx *ctx, const WindowAttnArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(window_append_kernel, dim3(a.s), dim3(256), 0, ctx->stream, a);
    LUMEN_CHECK_LAUNCH();
    const int nd = (a.dim + 15) / 16, nv = (a.vdim + 15) / 16;
    const size_t lds = (size_t)WP_K * ((nd + nv) * 16 + 8) * sizeof(float);
    const dim3 grid((a.s + WP_Q - 1) / WP_Q, a.heads);
    const int nb = nd > nv ? nd : nv;
#define WP_LAUNCH_F(NB, FULL)                                                                                                       \
    do {                                                                                                                            \
        if (lds > 64 * 1024)                                                                                                        \
            HIP_TRY(hipFuncSetAttribute((const void *)window_prefill_kernel<NB, FULL>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)); \
        hipLaunchKernelGGL((window_prefill_kernel<NB, FULL>), grid, dim3(256), lds, ctx->stream, a, nd, nv);                        \
    } while (0)
#define WP_LAUNCH(NB)                                    \
    do {                                                 \
        if (nd == NB && nv == NB) WP_LAUNCH_F(NB, true); \
        else WP_LAUNCH_F(NB, false);                     \
    } while (0)
    if (nb <= 4) WP_LAUNCH(4);
    else if (nb <= 8) WP_LAUNCH(8);
    else WP_LAUNCH(16);
#undef WP_LAUNCH
#undef WP_LAUNCH_F
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

LUMEN_DEFINE_WARM(window_attention)
