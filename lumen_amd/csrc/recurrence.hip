// Matrix-state recurrences: the WKV time mixing, the channel-wise gated delta rule, the generalised delta rule and the
// matrix memory with exponential gates.  All keep one f32 matrix
// S [dim, vdim] per head; its columns (value channels) never meet, so a workgroup owns a few columns of one head.
//
// Mapping: a column belongs to a row of 16 lanes, lane i of the row holding key channels [i KR, (i + 1) KR) of it in
// registers (KR = 4, 8, 16: heads up to 64, 128, 256 wide; channels beyond the head's width are zero and stay zero).
// A sum over key channels is KR multiply-adds in the lane and four DPP additions.  In memory a column is contiguous
// ([heads][vdim][16 KR]), so the state travels in 16-byte pieces, once per launch.
#include "mixers.h"
#include "wave_reduce.h"

typedef float v4f __attribute__((ext_vector_type(4)));
typedef unsigned int v4u __attribute__((ext_vector_type(4)));

int recurrence_columns(int kind, int vdim) { return kind == REC_MEMORY ? vdim + 1 : vdim; }
int recurrence_rows(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }

__device__ __forceinline__ float sigmoid_r(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_r(float z) { return z * sigmoid_r(z); }
__device__ __forceinline__ float softplus_r(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float gate_r(float z, int act) { return act == GATE_SILU ? silu_r(z) : act == GATE_SIGMOID ? sigmoid_r(z) : 1.0f; }

template <int KIND>
__device__ __forceinline__ float decay_r(float z, float bias, float a) {
    // WKV: exp(-exp(z + bias)); delta: exp(-a softplus(z + bias)) with a = exp(a_log); general delta: exp(-a sigmoid(z + bias))
    if (KIND == REC_GENERAL) return expf(-a * sigmoid_r(z + bias));
    return KIND == REC_WKV ? expf(-expf(z + bias)) : expf(-a * softplus_r(z + bias));
}

template <int KR>
__device__ __forceinline__ void load_kr(float (&d)[KR], const float *p) {
#pragma unroll
    for (int i = 0; i < KR; i += 4) {
        const v4f v = *(const v4f *)(p + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) d[i + e] = v[e];
    }
}
template <int KR>
__device__ __forceinline__ void store_kr(float *p, const float (&d)[KR]) {
#pragma unroll
    for (int i = 0; i < KR; i += 4) *(v4f *)(p + i) = v4f{d[i], d[i + 1], d[i + 2], d[i + 3]};
}

// One token of one column.  q, k, w (decay) and uk (WKV: u k) are the lane's channels; returns o (in all 16 lanes).
template <int KIND, int KR>
__device__ __forceinline__ float column_step(float (&S)[KR], const float (&q)[KR], const float (&k)[KR], const float (&w)[KR],
                                             const float (&u)[KR], float v, float beta) {
    float o = 0.f;
    if (KIND == REC_WKV) {
        float bonus = 0.f;
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            o = fmaf(q[i], S[i], o);
            bonus = fmaf(q[i], u[i] * k[i], bonus);
            S[i] = fmaf(w[i], S[i], k[i] * v);
        }
        return row16_sum(fmaf(bonus, v, o));
    }
    float p = 0.f;
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        S[i] *= w[i];
        p = fmaf(k[i], S[i], p);
    }
    const float d = beta * (v - row16_sum(p));
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        S[i] = fmaf(k[i], d, S[i]);
        o = fmaf(q[i], S[i], o);
    }
    return row16_sum(o);
}

// The same for the general delta rule: uk the unit key, ak the removal rates times it.
template <int KR>
__device__ __forceinline__ float column_step_general(float (&S)[KR], const float (&q)[KR], const float (&k)[KR], const float (&w)[KR],
                                                     const float (&uk)[KR], const float (&ak)[KR], float v) {
    float p = 0.f, o = 0.f;
#pragma unroll
    for (int i = 0; i < KR; ++i) p = fmaf(uk[i], S[i], p);
    p = row16_sum(p);
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        S[i] = fmaf(w[i], S[i], fmaf(-ak[i], p, k[i] * v));
        o = fmaf(q[i], S[i], o);
    }
    return row16_sum(o);
}

// ... and for the matrix memory: one decay for all channels, k times its weight.
template <int KR>
__device__ __forceinline__ float column_step_memory(float (&S)[KR], const float (&q)[KR], const float (&k)[KR], float keep, float v) {
    float o = 0.f;
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        S[i] = fmaf(keep, S[i], k[i] * v);
        o = fmaf(q[i], S[i], o);
    }
    return row16_sum(o);
}

__device__ __forceinline__ float memory_log_input(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float memory_log_forget(float z, float cap) {  // log sigmoid(x) = min(x, 0) - ln(1 + e^{-|x|})
    const float x = cap * tanhf(z / cap);
    return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

// ---------------------------------------------------------- prompt, token by token
#define REC_TOK 16  // tokens staged at a time
#define REC_COLS 16 // columns of a workgroup: 4 wavefronts x 4 rows of lanes

// Workgroup = 16 columns of one head; the tokens' q, k, decay rows and values pass through LDS 16 tokens at a time,
// the next 16 on their way from memory meanwhile.
template <int KIND, int KR>
__global__ __launch_bounds__(256) void recurrence_kernel(RecurrenceArgs a) {
    constexpr int DP = 16 * KR;
    constexpr int PER = REC_TOK * DP / 256;  // elements of a staged array per thread
    __shared__ __align__(16) float qs[REC_TOK][DP], ks[REC_TOK][DP], ws[REC_TOK][DP];
    __shared__ float vs[REC_TOK][REC_COLS], os[REC_TOK][REC_COLS], bs[REC_TOK];
    const int tid = threadIdx.x, lane = tid & 63, i16 = lane & 15;
    const int lc = (tid >> 6) * 4 + (lane >> 4);  // column within the workgroup
    const int h = blockIdx.y, hk = h / a.rep, col0 = blockIdx.x * REC_COLS, col = col0 + lc;
    const int D = a.dim, Dv = a.vdim, T = a.s;
    const bool live = col < Dv;
    const float decay_a = KIND == REC_DELTA ? expf(a.a_log[h]) : 0.f;
    float *Sg = a.state + ((size_t)h * Dv + (live ? col : 0)) * DP + i16 * KR;
    float S[KR], u[KR];
    load_kr<KR>(S, Sg);
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const int kc = i16 * KR + i;
        u[i] = KIND == REC_WKV && kc < D ? a.u[h * D + kc] : 0.f;
    }
    float rq[PER], rk[PER], rz[PER], rv, rb = 0.f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = tid + i * 256, t = e / DP, c = e % DP;
            const bool ok = t0 + t < T && c < D;
            rq[i] = ok ? a.q[(size_t)(t0 + t) * a.q_stride + hk * D + c] : 0.f;
            rk[i] = ok ? a.k[(size_t)(t0 + t) * a.k_stride + hk * D + c] : 0.f;
            rz[i] = ok ? a.z[(size_t)(t0 + t) * a.z_stride + h * D + c] : 0.f;
        }
        const int t = tid / REC_COLS, c = col0 + tid % REC_COLS;
        rv = t0 + t < T && c < Dv ? a.v[(size_t)(t0 + t) * a.v_stride + h * Dv + c] : 0.f;
        if (KIND == REC_DELTA && tid < REC_TOK) rb = t0 + tid < T ? a.b[(size_t)(t0 + tid) * a.b_stride + h] : 0.f;
    };
    fetch(0);
    for (int t0 = 0; t0 < T; t0 += REC_TOK) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = tid + i * 256, t = e / DP, c = e % DP;
            qs[t][c] = rq[i];
            ks[t][c] = rk[i];
            ws[t][c] = c < D ? decay_r<KIND>(rz[i], a.bias[h * D + c], decay_a) : 0.f;
        }
        vs[tid / REC_COLS][tid % REC_COLS] = rv;
        if (KIND == REC_DELTA && tid < REC_TOK) bs[tid] = sigmoid_r(rb);
        __syncthreads();
        if (t0 + REC_TOK < T) fetch(t0 + REC_TOK);
        const int n = min(REC_TOK, T - t0);
        for (int t = 0; t < n; ++t) {
            float q[KR], k[KR], w[KR];
            load_kr<KR>(q, &qs[t][i16 * KR]);
            load_kr<KR>(k, &ks[t][i16 * KR]);
            load_kr<KR>(w, &ws[t][i16 * KR]);
            const float o = column_step<KIND, KR>(S, q, k, w, u, vs[t][lc], KIND == REC_DELTA ? bs[t] : 0.f);
            if (i16 == 0) os[t][lc] = o;
        }
        __syncthreads();
        {
            const int t = tid / REC_COLS, c = col0 + tid % REC_COLS;
            if (t < n && c < Dv) a.out[(size_t)(t0 + t) * a.out_stride + h * Dv + c] = os[t][tid % REC_COLS];
        }
    }
    if (live) store_kr<KR>(Sg, S);
}

// ---------------------------------------------------------- prompt, 16 tokens at a time
// Over a chunk of 16 tokens both recurrences are matrix products with the state S the chunk starts from.  With G_t the
// product of the decays up to token t (WKV reads the state before its own token: up to t - 1), and G_t / G_s always
// the product of the decays in between -- formed by multiplying, never by dividing, so that strong decays stay exact --
//   delta: U = T (V - K~ S),  T = (I + diag(b) tril(A, -1))^-1 diag(b),  A_ts = sum_d k_t k_s G_t / G_s,  K~_t = G_t k_t
//   WKV:   U = V
//   O = Q~ S + B U,  B_ts = sum_d q_t k_s G_t / G_s  (WKV: s < t, and sum_d q u k on the diagonal),  Q~_t = G_t q_t
//   S <- diag(G_16) S + K^^T U,  K^_s = (G_16 / G_s) k_s.
// K~, Q~, K^, T, B and G_16 do not depend on S: recurrence_chunk_prep_kernel makes them for all chunks in parallel;
// recurrence_chunk_kernel then walks the chunks of a head with S in the accumulators of the f32 matrix instruction.
// The general delta rule removes what its unit key u reads, at rates of its own: with P_t = u_t^T S before token t,
//   P = T (U~ S + A V),  T = (I + tril(R, -1))^-1,  A_ts = sum_d u_t k_s G_{t-1} / G_s,  R_ts = sum_d u_t (a u)_s G_{t-1} / G_s
//   O = Q~ S + B V - C P,  C_ts = sum_d q_t (a u)_s G_t / G_s;   S <- diag(G_16) S + K^^T V - W^^T P,  W^_s = (G_16 / G_s) (a u)_s.
// The matrix memory is the WKV form with B's diagonal in place and one decay for all channels; its input weights ride on K^
// and B, the normaliser n is one more value column whose values are 1.
#define REC_CHUNK 16
static __host__ __device__ __forceinline__ size_t rec_ws_floats(int kind, int dp) { return kind == REC_GENERAL ? (size_t)65 * dp + 1024 : (size_t)49 * dp + 512; }
struct ChunkWs {  // one chunk of one head
    float *kt, *qt, *kh, *gc, *t, *b;  // [16][dp], [16][dp], [dp][16], [dp], [16][16], [16][16]
    float *ta, *c, *wh;                // general delta: T A, C, W^ [dp][16]
    __device__ ChunkWs(float *base, int dp)
        : kt(base), qt(base + 16 * dp), kh(base + 32 * dp), gc(base + 48 * dp), t(base + 49 * dp), b(base + 49 * dp + 256), ta(base + 49 * dp + 512),
          c(base + 49 * dp + 768), wh(base + 49 * dp + 1024) {}
};

template <int KIND, int KR>
__global__ __launch_bounds__(256) void recurrence_chunk_prep_kernel(RecurrenceArgs a, float *ws_base, int vec) {
    constexpr int DP = 16 * KR;
    __shared__ __align__(16) float qs[REC_CHUNK][DP], ks[REC_CHUNK][DP], gs[REC_CHUNK][DP];
    __shared__ float As[REC_CHUNK][REC_CHUNK + 1], bs[REC_CHUNK];
    const int tid = threadIdx.x, s = tid >> 4, i16 = tid & 15;
    const int h = blockIdx.y, hk = h / a.rep, D = a.dim, t0 = blockIdx.x * REC_CHUNK;
    const bool live = t0 + s < a.s;
    const float decay_a = KIND == REC_DELTA ? expf(a.a_log[h]) : 0.f;
    float q[KR], k[KR], g[KR], uk[KR];
    {   // (positions beyond the head or the sequence are clamped, so that all requests go out together)
        const size_t t = (size_t)min(t0 + s, a.s - 1);
        const float *pq = a.q + t * a.q_stride + hk * D, *pk = a.k + t * a.k_stride + hk * D, *pz = a.z + t * a.z_stride + h * D;
        const float *pb = a.bias + h * D, *pu = KIND == REC_WKV ? a.u + h * D : pb;
        float z[KR], bias[KR], u[KR];
        if (vec) {  // rows of whole 16-byte pieces
#pragma unroll
            for (int i = 0; i < KR; i += 4) {
                const int c = min(i16 * KR + i, D - 4);
                const v4f vq = *(const v4f *)(pq + c), vk = *(const v4f *)(pk + c), vz = *(const v4f *)(pz + c), vb = *(const v4f *)(pb + c),
                          vu = *(const v4f *)(pu + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    q[i + e] = vq[e];
                    k[i + e] = vk[e];
                    z[i + e] = vz[e];
                    bias[i + e] = vb[e];
                    u[i + e] = vu[e];
                }
            }
        } else {
#pragma unroll
            for (int i = 0; i < KR; ++i) {
                const int c = min(i16 * KR + i, D - 1);
                q[i] = pq[c];
                k[i] = pk[c];
                z[i] = pz[c];
                bias[i] = pb[c];
                u[i] = pu[c];
            }
        }
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            const bool ok = live && i16 * KR + i < D;
            q[i] = ok ? q[i] : 0.f;
            k[i] = ok ? k[i] : 0.f;
            g[i] = ok ? decay_r<KIND>(z[i], bias[i], decay_a) : 1.f;  // (a missing token changes nothing)
            uk[i] = u[i] * k[i];
        }
    }
    store_kr<KR>(&qs[s][i16 * KR], q);
    store_kr<KR>(&ks[s][i16 * KR], k);
    store_kr<KR>(&gs[s][i16 * KR], g);
    if (KIND == REC_DELTA && tid < REC_CHUNK) bs[tid] = t0 + tid < a.s ? sigmoid_r(a.b[(size_t)(t0 + tid) * a.b_stride + h]) : 0.f;
    __syncthreads();
    ChunkWs w(ws_base + ((size_t)h * gridDim.x + blockIdx.x) * rec_ws_floats(KIND, DP), DP);
    // decays up to this token, and the rows that meet the chunk's first state
    float G[KR], kr[KR];
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        G[i] = 1.f;
        kr[i] = k[i];
    }
    for (int t = 0; t < REC_CHUNK; ++t) {
        float gt[KR], qt[KR];
        load_kr<KR>(gt, &gs[t][i16 * KR]);
        load_kr<KR>(qt, &qs[t][i16 * KR]);
        const bool before = t < s, after = t > s;
        float da = 0.f, db = 0.f;
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            G[i] *= before ? gt[i] : 1.f;
            if (KIND == REC_DELTA) kr[i] *= after ? gt[i] : 1.f;
            db = fmaf(KIND == REC_WKV && !after ? uk[i] : kr[i], qt[i], db);
        }
        if (KIND == REC_DELTA) {
            float kt[KR];
            load_kr<KR>(kt, &ks[t][i16 * KR]);
#pragma unroll
            for (int i = 0; i < KR; ++i) da = fmaf(kr[i], kt[i], da);
            da = row16_sum(da);
        } else {
#pragma unroll
            for (int i = 0; i < KR; ++i) kr[i] *= after ? gt[i] : 1.f;
        }
        db = row16_sum(db);
        if (i16 == 0) {
            w.b[t * REC_CHUNK + s] = before ? 0.f : db;
            if (KIND == REC_DELTA) As[t][s] = after ? da : 0.f;
        }
    }
    float rq[KR], rk[KR];
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const float inc = G[i] * g[i];
        rq[i] = q[i] * (KIND == REC_DELTA ? inc : G[i]);
        rk[i] = k[i] * inc;
        G[i] = inc;
    }
    store_kr<KR>(w.qt + s * DP + i16 * KR, rq);
    if (KIND == REC_DELTA) store_kr<KR>(w.kt + s * DP + i16 * KR, rk);
    if (s == REC_CHUNK - 1) store_kr<KR>(w.gc + i16 * KR, G);
    __syncthreads();  // (everyone is done with qs; As is complete)
    store_kr<KR>(&qs[s][i16 * KR], kr);
    __syncthreads();
    for (int e = tid; e < DP * 4; e += 256) {  // K^ goes out transposed
        const int d = e >> 2, s4 = (e & 3) * 4;
        *(v4f *)(w.kh + d * REC_CHUNK + s4) = v4f{qs[s4][d], qs[s4 + 1][d], qs[s4 + 2][d], qs[s4 + 3][d]};
    }
    if (KIND == REC_DELTA) {
        if (tid < REC_CHUNK) {  // column tid of T by forward substitution
            float x[REC_CHUNK];
#pragma unroll
            for (int i = 0; i < REC_CHUNK; ++i) {
                float sum = 0.f;
#pragma unroll
                for (int l = 0; l < i; ++l) sum = fmaf(As[i][l], x[l], sum);
                x[i] = (i == tid ? 1.f : 0.f) - bs[i] * sum;
                w.t[i * REC_CHUNK + tid] = x[i] * bs[tid];
            }
        }
    }
}

// The general delta rule's operands: thread (s, i16) of 16 x 16 holds token s, channels [i16 KR, (i16 + 1) KR).
template <int KR>
__global__ __launch_bounds__(256) void general_chunk_prep_kernel(RecurrenceArgs a, float *ws_base) {
    constexpr int DP = 16 * KR;
    __shared__ __align__(16) float qs[REC_CHUNK][DP], us[REC_CHUNK][DP], gs[REC_CHUNK][DP];
    __shared__ float As[REC_CHUNK][REC_CHUNK + 1], Rs[REC_CHUNK][REC_CHUNK + 1], Ts[REC_CHUNK][REC_CHUNK + 1];
    const int tid = threadIdx.x, s = tid >> 4, i16 = tid & 15;
    const int h = blockIdx.y, D = a.dim, t0 = blockIdx.x * REC_CHUNK;
    const bool live = t0 + s < a.s;
    float q[KR], kr[KR], br[KR], g[KR], u[KR];
    {   // (positions beyond the head or the sequence are clamped, so that all requests go out together)
        const size_t t = (size_t)min(t0 + s, a.s - 1);
        const float *pq = a.q + t * a.q_stride + h * D, *pk = a.k + t * a.k_stride + h * D, *pz = a.z + t * a.z_stride + h * D;
        const float *pb = a.b + t * a.b_stride + h * D;
        float z[KR], b[KR], zb[KR], bb[KR], ss = 0.f;
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            const int c = min(i16 * KR + i, D - 1);
            q[i] = pq[c];
            kr[i] = pk[c];
            z[i] = pz[c];
            b[i] = pb[c];
            zb[i] = a.bias[h * D + c];
            bb[i] = a.b_bias[h * D + c];
        }
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            const bool ok = live && i16 * KR + i < D;
            q[i] = ok ? q[i] : 0.f;
            kr[i] = ok ? kr[i] : 0.f;
            g[i] = ok ? decay_r<REC_GENERAL>(z[i], zb[i], a.z_scale) : 1.f;  // (a missing token changes nothing)
            ss = fmaf(kr[i], kr[i], ss);
        }
        const float inv = 1.0f / sqrtf(row16_sum(ss) + a.unit_eps);
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            u[i] = kr[i] * inv;
            br[i] = sigmoid_r(b[i] + bb[i]) * u[i];
        }
    }
    store_kr<KR>(&qs[s][i16 * KR], q);
    store_kr<KR>(&us[s][i16 * KR], u);
    store_kr<KR>(&gs[s][i16 * KR], g);
    __syncthreads();
    ChunkWs w(ws_base + ((size_t)h * gridDim.x + blockIdx.x) * rec_ws_floats(REC_GENERAL, DP), DP);
    float G[KR];
#pragma unroll
    for (int i = 0; i < KR; ++i) G[i] = 1.f;
    for (int t = 0; t < REC_CHUNK; ++t) {
        float gt[KR], qt[KR], ut[KR];
        load_kr<KR>(gt, &gs[t][i16 * KR]);
        load_kr<KR>(qt, &qs[t][i16 * KR]);
        load_kr<KR>(ut, &us[t][i16 * KR]);
        const bool before = t < s, after = t > s;
        float ak = 0.f, ab = 0.f, ok = 0.f, ob = 0.f;
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            G[i] *= before ? gt[i] : 1.f;
            ak = fmaf(kr[i], ut[i], ak);  // what token t's unit key reads of token s, decayed up to t - 1
            ab = fmaf(br[i], ut[i], ab);
            kr[i] *= after ? gt[i] : 1.f;
            br[i] *= after ? gt[i] : 1.f;
            ok = fmaf(kr[i], qt[i], ok);
            ob = fmaf(br[i], qt[i], ob);
        }
        ak = row16_sum(ak);
        ab = row16_sum(ab);
        ok = row16_sum(ok);
        ob = row16_sum(ob);
        if (i16 == 0) {
            As[t][s] = after ? ak : 0.f;
            Rs[t][s] = after ? ab : 0.f;
            w.b[t * REC_CHUNK + s] = before ? 0.f : ok;
            w.c[t * REC_CHUNK + s] = before ? 0.f : -ob;
        }
    }
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        u[i] *= G[i];  // decays before the token
        G[i] *= g[i];
        q[i] *= G[i];
    }
    store_kr<KR>(w.kt + s * DP + i16 * KR, u);
    store_kr<KR>(w.qt + s * DP + i16 * KR, q);
    if (s == REC_CHUNK - 1) store_kr<KR>(w.gc + i16 * KR, G);
    __syncthreads();  // (everyone is done with qs and us; As and Rs are complete)
    store_kr<KR>(&qs[s][i16 * KR], kr);
    store_kr<KR>(&us[s][i16 * KR], br);
    if (tid < REC_CHUNK) {  // column tid of T by forward substitution
        float x[REC_CHUNK];
#pragma unroll
        for (int i = 0; i < REC_CHUNK; ++i) {
            float sum = 0.f;
#pragma unroll
            for (int l = 0; l < i; ++l) sum = fmaf(Rs[i][l], x[l], sum);
            x[i] = (i == tid ? 1.f : 0.f) - sum;
            Ts[i][tid] = x[i];
        }
    }
    __syncthreads();
    for (int e = tid; e < DP * 4; e += 256) {  // K^ and -W^ go out transposed
        const int d = e >> 2, s4 = (e & 3) * 4;
        *(v4f *)(w.kh + d * REC_CHUNK + s4) = v4f{qs[s4][d], qs[s4 + 1][d], qs[s4 + 2][d], qs[s4 + 3][d]};
        *(v4f *)(w.wh + d * REC_CHUNK + s4) = v4f{-us[s4][d], -us[s4 + 1][d], -us[s4 + 2][d], -us[s4 + 3][d]};
    }
    float ta = 0.f;
#pragma unroll
    for (int l = 0; l < REC_CHUNK; ++l) ta = fmaf(Ts[s][l], As[l][i16], ta);
    w.ta[s * REC_CHUNK + i16] = ta;
    w.t[s * REC_CHUNK + i16] = Ts[s][i16];
}

// The matrix memory's running maxima: m_t = max(f_t + m_{t-1}, i_t) is a chain of maps m -> max(F + m, M), which compose:
// a workgroup per head takes 256 tokens per trip, a token per thread.  out: maxima [heads][s + 1], then log gates
// [heads][s] input and forget.
size_t memory_scan_floats(int s, int heads) { return (size_t)heads * (3 * (size_t)s + 1); }
struct MemoryScan {
    float *m, *i, *f;
    __device__ MemoryScan(float *base, int h, int heads, int s)
        : m(base + (size_t)h * (s + 1)), i(base + (size_t)heads * (s + 1) + (size_t)h * s), f(base + (size_t)heads * (2 * (size_t)s + 1) + (size_t)h * s) {}
};
__global__ __launch_bounds__(256) void memory_scan_kernel(RecurrenceArgs a) {
    __shared__ float wf[4], wm[4];
    const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const MemoryScan o(a.m_out, h, a.heads, a.s);
    const float bi = a.gi_bias[h], bf = a.gf_bias[h];
    float m = a.m[h];
    __syncthreads();
    if (tid == 0) o.m[0] = m;
    for (int t0 = 0; t0 < a.s; t0 += 256) {
        const int t = t0 + tid;
        const size_t tc = (size_t)min(t, a.s - 1);
        const float i = memory_log_input(a.gi[tc * a.g_stride + h] + bi, a.cap), f = memory_log_forget(a.gf[tc * a.g_stride + h] + bf, a.cap);
        // inclusive scan of (F, M) over the wavefront; a missing token is the identity
        float F = t < a.s ? f : 0.f, M = t < a.s ? i : -INFINITY;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const float pf = __shfl_up(F, d, 64), pm = __shfl_up(M, d, 64);
            if (lane >= d) {
                M = fmaxf(F + pm, M);
                F += pf;
            }
        }
        if (lane == 63) {
            wf[wave] = F;
            wm[wave] = M;
        }
        __syncthreads();
        float start = m;  // the maximum before this wavefront's tokens
        for (int w = 0; w < wave; ++w) start = fmaxf(wf[w] + start, wm[w]);
        if (t < a.s) {
            o.m[t + 1] = fmaxf(F + start, M);
            o.i[t] = i;
            o.f[t] = f;
        }
#pragma unroll
        for (int w = 0; w < 4; ++w) m = fmaxf(wf[w] + m, wm[w]);
        __syncthreads();
    }
    if (tid == 0) a.m[h] = m;
}

// The matrix memory's operands, tokens and channels as above.
template <int KR>
__global__ __launch_bounds__(256) void memory_chunk_prep_kernel(RecurrenceArgs a, float *ws_base) {
    constexpr int DP = 16 * KR;
    __shared__ __align__(16) float qs[REC_CHUNK][DP];
    __shared__ float fs[REC_CHUNK], is[REC_CHUNK], ms[REC_CHUNK + 1];
    const int tid = threadIdx.x, s = tid >> 4, i16 = tid & 15;
    const int h = blockIdx.y, D = a.dim, t0 = blockIdx.x * REC_CHUNK;
    const bool live = t0 + s < a.s;
    const size_t tc = (size_t)min(t0 + s, a.s - 1);
    const float *pq = a.q + tc * a.q_stride + h * D, *pk = a.k + tc * a.k_stride + h * D;
    float q[KR], k[KR];
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const int c = min(i16 * KR + i, D - 1);
        q[i] = pq[c];
        k[i] = pk[c];
    }
    const MemoryScan scan(a.m_out, h, a.heads, a.s);
    if (tid < REC_CHUNK) {  // (a missing token keeps everything and adds nothing)
        fs[tid] = t0 + tid < a.s ? scan.f[t0 + tid] : 0.f;
        is[tid] = t0 + tid < a.s ? scan.i[t0 + tid] : -INFINITY;
    }
    if (tid < REC_CHUNK + 1) ms[tid] = scan.m[min(t0 + tid, a.s)];
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const bool ok = live && i16 * KR + i < D;
        q[i] = ok ? q[i] * a.q_scale : 0.f;
        k[i] = ok ? k[i] : 0.f;
    }
    store_kr<KR>(&qs[s][i16 * KR], q);
    __syncthreads();
    ChunkWs w(ws_base + ((size_t)h * gridDim.x + blockIdx.x) * rec_ws_floats(REC_MEMORY, DP), DP);
    float upto = 0.f, since = 0.f;  // log decays: of the chunk's first tokens up to this one, and from this one on
    for (int t = 0; t < REC_CHUNK; ++t) {
        if (t <= s) upto += fs[t];
        else since += fs[t];
        float qt[KR], d = 0.f;
        load_kr<KR>(qt, &qs[t][i16 * KR]);
#pragma unroll
        for (int i = 0; i < KR; ++i) d = fmaf(k[i], qt[i], d);
        d = row16_sum(d);
        if (i16 == 0) w.b[t * REC_CHUNK + s] = t < s ? 0.f : d * expf(since + is[s] - ms[t + 1]);
    }
    const float fq = expf(upto + ms[0] - ms[s + 1]), fk = expf(since + is[s] - ms[REC_CHUNK]);
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        q[i] *= fq;
        k[i] *= fk;
    }
    store_kr<KR>(w.qt + s * DP + i16 * KR, q);
    if (s == REC_CHUNK - 1) {
        float G[KR];
#pragma unroll
        for (int i = 0; i < KR; ++i) G[i] = fq;
        store_kr<KR>(w.gc + i16 * KR, G);
    }
    __syncthreads();  // (everyone is done with qs)
    store_kr<KR>(&qs[s][i16 * KR], k);
    __syncthreads();
    for (int e = tid; e < DP * 4; e += 256) {
        const int d = e >> 2, s4 = (e & 3) * 4;
        *(v4f *)(w.kh + d * REC_CHUNK + s4) = v4f{qs[s4][d], qs[s4 + 1][d], qs[s4 + 2][d], qs[s4 + 3][d]};
    }
}

template <int KIND, int RT>
struct ChunkFrag {
    v4f kt[RT], qt[RT], kh[RT], gc[RT], t, b;
    v4f wh[KIND == REC_GENERAL ? RT : 1], ta, c;
    float v[4];
};

// Workgroup = 16 columns of one head; its four wavefronts hold a quarter of the key rows each (RT tiles of 16).  Operands:
// lane (c, g) gives A[c][.] and B[.][c] for the four contraction indices 4 g + r of step r; accumulator r is row 4 g + r,
// column c -- so an accumulator tile is the B operand of the next product as it stands.  The wavefronts' partial K~ S meet
// in LDS once per chunk; their partial outputs (a quarter of Q~ S and of B U each) ride along with the NEXT chunk's
// meeting, and each wavefront then writes a quarter of the finished rows.
template <int KIND, int RT>
__global__ __launch_bounds__(256) void recurrence_chunk_kernel(RecurrenceArgs a, float *ws_base, int chunks) {
    constexpr int DP = RT * 64;
    __shared__ float red[2][2][4][4][64];  // [parity][K~ S, output][wavefront][r][lane]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    constexpr bool READS = KIND == REC_DELTA || KIND == REC_GENERAL;  // what a token writes depends on the state
    const int h = blockIdx.x, col = blockIdx.y * 16 + c, Dv = a.vdim, T = a.s;
    const int cols = KIND == REC_MEMORY ? Dv + 1 : Dv;
    const bool live = col < cols, ones = KIND == REC_MEMORY && col >= Dv;
    float *Sg = a.state + ((size_t)h * cols + (live ? col : 0)) * DP + wave * RT * 16 + g * 4;
    v4f S[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) S[i] = *(const v4f *)(Sg + i * 16);
    // lane offsets from a chunk's (uniform) base pointers
    const unsigned d0 = wave * RT * 16, off_q = c * DP + d0 + g * 4, off_kh = (d0 + c) * REC_CHUNK + g * 4, off_gc = d0 + g * 4, off_t = c * REC_CHUNK + g * 4;
    const unsigned colc = h * Dv + min(col, Dv - 1), vs = a.v_stride;
    unsigned off_v[4], off_v_last[4];  // ... of the last chunk, whose tokens may end early: clamped, not skipped (a load behind a
                             // branch would make the wavefront wait for all that are in flight)
    const int t_last = (chunks - 1) * REC_CHUNK;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        off_v[r] = (unsigned)(g * 4 + r) * vs + colc;
        off_v_last[r] = (unsigned)(min(t_last + g * 4 + r, T - 1) - t_last) * vs + colc;
    }
    const float *wsh = ws_base + (size_t)h * chunks * rec_ws_floats(KIND, DP);
    auto load = [&](ChunkFrag<KIND, RT> &f, int n) {
        const ChunkWs w(const_cast<float *>(wsh) + (size_t)n * rec_ws_floats(KIND, DP), DP);
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            f.qt[i] = *(const v4f *)(w.qt + (off_q + i * 16));
            if (READS) f.kt[i] = *(const v4f *)(w.kt + (off_q + i * 16));
            if (KIND == REC_GENERAL) f.wh[i] = *(const v4f *)(w.wh + (off_kh + i * 16 * REC_CHUNK));
            f.kh[i] = *(const v4f *)(w.kh + (off_kh + i * 16 * REC_CHUNK));
            f.gc[i] = *(const v4f *)(w.gc + (off_gc + i * 16));
        }
        if (READS) f.t = *(const v4f *)(w.t + off_t);
        if (KIND == REC_GENERAL) {
            f.ta = *(const v4f *)(w.ta + off_t);
            f.c = *(const v4f *)(w.c + off_t);
        }
        f.b = *(const v4f *)(w.b + off_t);
        const bool last = n == chunks - 1;
#pragma unroll
        for (int r = 0; r < 4; ++r) f.v[r] = *(a.v + (size_t)n * REC_CHUNK * vs + (last ? off_v_last[r] : off_v[r]));
    };
    v4f O = {0.f, 0.f, 0.f, 0.f};  // this wavefront's part of the chunk before
    auto put = [&](int what, int n, const v4f x) {
#pragma unroll
        for (int r = 0; r < 4; ++r) red[n & 1][what][wave][r][lane] = x[r];
    };
    auto sum = [&](int what, int n, int r) {
        return (red[n & 1][what][0][r][lane] + red[n & 1][what][1][r][lane]) + (red[n & 1][what][2][r][lane] + red[n & 1][what][3][r][lane]);
    };
    auto write_out = [&](int n, float o) {  // row `wave` of each group of four tokens of chunk n
        const int t = n * REC_CHUNK + g * 4 + wave;
        if (live && t < T) a.out[(size_t)t * a.out_stride + h * cols + col] = o;
    };
    auto work = [&](const ChunkFrag<KIND, RT> &f, int n) {
        v4f P = {0.f, 0.f, 0.f, 0.f}, Q = {0.f, 0.f, 0.f, 0.f};
        put(1, n, O);
#pragma unroll
        for (int i = 0; i < RT; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (READS) P = __builtin_amdgcn_mfma_f32_16x16x4f32(f.kt[i][r], S[i][r], P, 0, 0, 0);
                Q = __builtin_amdgcn_mfma_f32_16x16x4f32(f.qt[i][r], S[i][r], Q, 0, 0, 0);
            }
        if (READS) put(0, n, P);
        __syncthreads();  // (one per chunk: the other half of red is written before the next one)
        v4f U = {0.f, 0.f, 0.f, 0.f}, R, X = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            R[r] = n * REC_CHUNK + g * 4 + r < T ? (ones ? 1.f : f.v[r]) : 0.f;
            if (KIND == REC_DELTA) R[r] -= sum(0, n, r);
        }
        if (KIND == REC_GENERAL) {  // U: the values; X: what the unit keys read
            U = R;
#pragma unroll
            for (int r = 0; r < 4; ++r) X = __builtin_amdgcn_mfma_f32_16x16x4f32(f.ta[r], R[r], X, 0, 0, 0);
#pragma unroll
            for (int r = 0; r < 4; ++r) X = __builtin_amdgcn_mfma_f32_16x16x4f32(f.t[r], sum(0, n, r), X, 0, 0, 0);
        } else if (KIND == REC_DELTA) {
#pragma unroll
            for (int r = 0; r < 4; ++r) U = __builtin_amdgcn_mfma_f32_16x16x4f32(f.t[r], R[r], U, 0, 0, 0);
        } else {
            U = R;
        }
        const float o_before = sum(1, n, wave);
#pragma unroll
        for (int i = 0; i < RT; ++i) S[i] *= f.gc[i];
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int i = 0; i < RT; ++i) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.kh[i][r], U[r], S[i], 0, 0, 0);
        if (KIND == REC_GENERAL) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
                for (int i = 0; i < RT; ++i) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.wh[i][r], X[r], S[i], 0, 0, 0);
            const float cw = wave == 0 ? f.c[0] : wave == 1 ? f.c[1] : wave == 2 ? f.c[2] : f.c[3];
            const float xw = wave == 0 ? X[0] : wave == 1 ? X[1] : wave == 2 ? X[2] : X[3];
            Q = __builtin_amdgcn_mfma_f32_16x16x4f32(cw, xw, Q, 0, 0, 0);
        }
        // (the quarter of B U that this wavefront adds: contraction step `wave`)
        const float bw = wave == 0 ? f.b[0] : wave == 1 ? f.b[1] : wave == 2 ? f.b[2] : f.b[3];
        const float uw = wave == 0 ? U[0] : wave == 1 ? U[1] : wave == 2 ? U[2] : U[3];
        O = __builtin_amdgcn_mfma_f32_16x16x4f32(bw, uw, Q, 0, 0, 0);
        if (n > 0) write_out(n - 1, o_before);
    };
    // the operands of the next two chunks travel while one is worked on (they come from beyond L2: one chunk's work is
    // shorter than that trip); requests past the end repeat the last chunk
    ChunkFrag<KIND, RT> f0, f1, f2;
    load(f0, 0);
    load(f1, min(1, chunks - 1));
    for (int n = 0; n < chunks; n += 3) {
        load(f2, min(n + 2, chunks - 1));
        work(f0, n);
        if (n + 1 >= chunks) break;
        load(f0, min(n + 3, chunks - 1));
        work(f1, n + 1);
        if (n + 2 >= chunks) break;
        load(f1, min(n + 4, chunks - 1));
        work(f2, n + 2);
    }
    put(1, chunks, O);
    __syncthreads();
    write_out(chunks - 1, sum(1, chunks, wave));
    if (live)
#pragma unroll
        for (int i = 0; i < RT; ++i) *(v4f *)(Sg + i * 16) = S[i];
}

static int mixer_reserve_workspace(lumen_ctx *ctx, size_t bytes) {
    if (ctx->mixer_ws_bytes >= bytes) return LUMEN_OK;
    HIP_TRY(hipStreamSynchronize(ctx->stream));
    if (ctx->mixer_ws) hipFree(ctx->mixer_ws);
    ctx->mixer_ws = nullptr;
    ctx->mixer_ws_bytes = 0;
    HIP_TRY(hipMalloc((void **)&ctx->mixer_ws, bytes));
    ctx->mixer_ws_bytes = bytes;
    return LUMEN_OK;
}

size_t recurrence_workspace_bytes(int kind, int s, int heads, int dim) {
    return (size_t)((s + REC_CHUNK - 1) / REC_CHUNK) * heads * rec_ws_floats(kind, recurrence_rows(dim)) * sizeof(float);
}

// The general delta rule and the matrix memory: chunks whatever the number of tokens.
static int launch_recurrence_chunks(lumen_ctx *ctx, const RecurrenceArgs &a) {
    const int rows = recurrence_rows(a.dim), chunks = (a.s + REC_CHUNK - 1) / REC_CHUNK;
    LUMEN_TRY(mixer_reserve_workspace(ctx, recurrence_workspace_bytes(a.kind, a.s, a.heads, a.dim)));
    float *ws = ctx->mixer_ws;
    const dim3 pgrid(chunks, a.heads), grid(a.heads, (recurrence_columns(a.kind, a.vdim) + 15) / 16);
    if (a.kind == REC_MEMORY) hipLaunchKernelGGL(memory_scan_kernel, dim3(a.heads), dim3(256), 0, ctx->stream, a);
#define REC_LAUNCH(KR)                                                                                                       \
    do {                                                                                                                     \
        if (a.kind == REC_GENERAL) {                                                                                         \
            hipLaunchKernelGGL((general_chunk_prep_kernel<KR>), pgrid, dim3(256), 0, ctx->stream, a, ws);                    \
            hipLaunchKernelGGL((recurrence_chunk_kernel<REC_GENERAL, KR / 4>), grid, dim3(256), 0, ctx->stream, a, ws, chunks); \
        } else {                                                                                                             \
            hipLaunchKernelGGL((memory_chunk_prep_kernel<KR>), pgrid, dim3(256), 0, ctx->stream, a, ws);                     \
            hipLaunchKernelGGL((recurrence_chunk_kernel<REC_MEMORY, KR / 4>), grid, dim3(256), 0, ctx->stream, a, ws, chunks); \
        }                                                                                                                    \
    } while (0)
    if (rows == 64) REC_LAUNCH(4);
    else if (rows == 128) REC_LAUNCH(8);
    else REC_LAUNCH(16);
#undef REC_LAUNCH
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// below this many tokens they are taken one by one
#define REC_CHUNKED_MIN 8

int launch_recurrence(lumen_ctx *ctx, const RecurrenceArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    if (a.kind == REC_GENERAL || a.kind == REC_MEMORY) return launch_recurrence_chunks(ctx, a);
    const int rows = recurrence_rows(a.dim);
    if (a.s >= REC_CHUNKED_MIN) {
        LUMEN_TRY(mixer_reserve_workspace(ctx, recurrence_workspace_bytes(a.kind, a.s, a.heads, a.dim)));
        const int chunks = (a.s + REC_CHUNK - 1) / REC_CHUNK;
        // (heads along x: the column blocks of a head, which read the same operands, share an XCD's L2 when the heads
        // are a multiple of 8)
        const dim3 pgrid(chunks, a.heads), grid(a.heads, (a.vdim + 15) / 16);
        float *ws = ctx->mixer_ws;
        const int vec = a.dim % 4 == 0 && a.q_stride % 4 == 0 && a.k_stride % 4 == 0 && a.z_stride % 4 == 0 &&
                        (((uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.z | (uintptr_t)a.bias | (uintptr_t)a.u) & 15) == 0;
#define REC_LAUNCH(KR)                                                                                                            \
    do {                                                                                                                          \
        if (a.kind == REC_WKV) {                                                                                                  \
            hipLaunchKernelGGL((recurrence_chunk_prep_kernel<REC_WKV, KR>), pgrid, dim3(256), 0, ctx->stream, a, ws, vec);        \
            hipLaunchKernelGGL((recurrence_chunk_kernel<REC_WKV, KR / 4>), grid, dim3(256), 0, ctx->stream, a, ws, chunks);       \
        } else {                                                                                                                  \
            hipLaunchKernelGGL((recurrence_chunk_prep_kernel<REC_DELTA, KR>), pgrid, dim3(256), 0, ctx->stream, a, ws, vec);      \
            hipLaunchKernelGGL((recurrence_chunk_kernel<REC_DELTA, KR / 4>), grid, dim3(256), 0, ctx->stream, a, ws, chunks);     \
        }                                                                                                                         \
    } while (0)
        if (rows == 64) REC_LAUNCH(4);
        else if (rows == 128) REC_LAUNCH(8);
        else REC_LAUNCH(16);
#undef REC_LAUNCH
        LUMEN_CHECK_LAUNCH();
        return LUMEN_OK;
    }
    const dim3 grid((a.vdim + REC_COLS - 1) / REC_COLS, a.heads);
#define REC_LAUNCH(KR)                                                                                            \
    do {                                                                                                          \
        if (a.kind == REC_WKV) hipLaunchKernelGGL((recurrence_kernel<REC_WKV, KR>), grid, dim3(256), 0, ctx->stream, a); \
        else hipLaunchKernelGGL((recurrence_kernel<REC_DELTA, KR>), grid, dim3(256), 0, ctx->stream, a);           \
    } while (0)
    if (rows == 64) REC_LAUNCH(4);
    else if (rows == 128) REC_LAUNCH(8);
    else REC_LAUNCH(16);
#undef REC_LAUNCH
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// One wavefront per (row, head).
__global__ __launch_bounds__(256) void head_norm_gate_kernel(float *o, int stride, const float *__restrict__ gain, int gain_shared,
                                                             const float *__restrict__ gate, int gate_stride, int gate_act,
                                                             int rows, int heads, int vdim, float eps) {
    const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (unit >= (long)rows * heads) return;  // (a whole wavefront)
    const int row = (int)(unit / heads), h = (int)(unit % heads);
    float *p = o + (size_t)row * stride + (size_t)h * vdim;
    const float *gp = gate ? gate + (size_t)row * gate_stride + (size_t)h * vdim : nullptr;
    const float *w = gain + (gain_shared ? 0 : (size_t)h * vdim);
    float ss = 0.f;
    for (int c = lane; c < vdim; c += 64) ss = fmaf(p[c], p[c], ss);
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)vdim + eps);
    for (int c = lane; c < vdim; c += 64) p[c] = p[c] * inv * w[c] * (gp ? gate_r(gp[c], gate_act) : 1.0f);
}

int launch_head_norm_gate(lumen_ctx *ctx, float *o, int stride, const float *gain, int gain_shared, const float *gate,
                          int gate_stride, int gate_act, int rows, int heads, int vdim, float eps) {
    if (rows <= 0) return LUMEN_OK;
    const long units = (long)rows * heads;
    hipLaunchKernelGGL(head_norm_gate_kernel, dim3((unsigned)((units + 3) / 4)), dim3(256), 0, ctx->stream, o, stride, gain,
                       gain_shared, gate, gate_stride, gate_act, rows, heads, vdim, eps);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// One wavefront per (row, head): the matrix memory's output is read, normalised and gated.
__global__ __launch_bounds__(256) void memory_read_kernel(const float *__restrict__ raw, const float *__restrict__ m_scan, float *__restrict__ out,
                                                          int out_stride, const float *__restrict__ gain, const float *__restrict__ gate,
                                                          int gate_stride, int gate_act, int rows, int heads, int vdim, float eps, float den_eps) {
    const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (unit >= (long)rows * heads) return;  // (a whole wavefront)
    const int row = (int)(unit / heads), h = (int)(unit % heads);
    const float *p = raw + (size_t)unit * (vdim + 1);
    const float den = fmaxf(fabsf(p[vdim]), expf(-m_scan[(size_t)h * (rows + 1) + row + 1])) + den_eps;
    float ss = 0.f;
    for (int c = lane; c < vdim; c += 64) {
        const float o = p[c] / den;
        ss = fmaf(o, o, ss);
    }
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)vdim + eps);
    const float *gp = gate ? gate + (size_t)row * gate_stride + (size_t)h * vdim : nullptr;
    for (int c = lane; c < vdim; c += 64)
        out[(size_t)row * out_stride + (size_t)h * vdim + c] = p[c] / den * inv * gain[(size_t)h * vdim + c] * (gp ? gate_r(gp[c], gate_act) : 1.0f);
}

int launch_memory_read(lumen_ctx *ctx, const float *raw, const float *m_scan, float *out, int out_stride, const float *gain, const float *gate,
                       int gate_stride, int gate_act, int rows, int heads, int vdim, float eps, float den_eps) {
    if (rows <= 0) return LUMEN_OK;
    const long units = (long)rows * heads;
    hipLaunchKernelGGL(memory_read_kernel, dim3((unsigned)((units + 3) / 4)), dim3(256), 0, ctx->stream, raw, m_scan, out, out_stride, gain, gate,
                       gate_stride, gate_act, rows, heads, vdim, eps, den_eps);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// Causal convolution + SiLU of a head of q, of k or of v, the unit norm of the first two: one wavefront per head (unit) and
// 8 tokens, weights and the inputs' sliding window in registers.  TAPS: taps the registers are laid out for (missing
// ones have weight zero); CH: 64-channel blocks of a head.  The last unit copies the two low-rank blocks.
#define PREP_TOK 8
template <int TAPS, int CH>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a, int units) {
    const long id = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63, t0 = (int)(id / units) * PREP_TOK, u = (int)(id % units);
    if (t0 >= a.s) return;  // (a whole wavefront)
    const int G = a.kv_heads, nq = G * a.dim, nv = a.heads * a.vdim, channels = 2 * nq + nv, keep = a.taps - 1;
    const int nt = min(PREP_TOK, a.s - t0);
    if (u == units - 1) {
        for (int t = t0; t < t0 + nt; ++t) {
            const float *row = a.in + (size_t)t * a.stride;
            for (int i = lane; i < a.ra; i += 64) a.a1[(size_t)t * a.ra + i] = row[a.off_a1 + i];
            for (int i = lane; i < a.rg; i += 64) a.g1[(size_t)t * a.rg + i] = row[a.off_g1 + i];
        }
        return;
    }
    const int part = u < G ? 0 : u < 2 * G ? 1 : 2, head = u - part * G, n = part == 2 ? a.vdim : a.dim;
    const int ch0 = part * nq + head * n, off = (part == 0 ? a.off_q : part == 1 ? a.off_k : a.off_v) + head * n;
    float y[CH][PREP_TOK], ss[PREP_TOK];
#pragma unroll
    for (int t = 0; t < PREP_TOK; ++t) ss[t] = 0.f;
#pragma unroll
    for (int b = 0; b < CH; ++b) {
        const bool ok = b * 64 + lane < n;
        const int c = min(b * 64 + lane, n - 1);
        float w[TAPS], x[TAPS - 1 + PREP_TOK];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
            const int jj = j - (TAPS - a.taps);
            w[j] = a.taps_w[(size_t)(ch0 + c) * a.taps + max(jj, 0)];
            w[j] = jj >= 0 ? w[j] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < TAPS - 1 + PREP_TOK; ++i) {  // input of token t0 - (TAPS - 1) + i, or the state's
            const int src = min(t0 - (TAPS - 1) + i, a.s - 1);
            const float *p = src >= 0 || src < -keep ? a.in + (size_t)max(src, 0) * a.stride + off + c
                                                     : a.conv_prev + (size_t)(keep + src) * channels + ch0 + c;
            x[i] = *p;
        }
#pragma unroll
        for (int t = 0; t < PREP_TOK; ++t) {
            float acc = 0.f;
#pragma unroll
            for (int j = 0; j < TAPS; ++j) acc = fmaf(w[j], x[t + j], acc);
            y[b][t] = ok ? silu_r(acc) : 0.f;
            ss[t] = fmaf(y[b][t], y[b][t], ss[t]);
        }
        if (ok && t0 + nt == a.s) {  // the last taps - 1 inputs stay for the next portion
            for (int j = 0; j < keep; ++j) {
                const int src = a.s - keep + j;
                a.conv_next[(size_t)j * channels + ch0 + c] = src >= 0 ? a.in[(size_t)src * a.stride + off + c]
                                                                       : a.conv_prev[(size_t)(keep + src) * channels + ch0 + c];
            }
        }
    }
    float *dst = part == 0 ? a.q : part == 1 ? a.k : a.v;
    const int row = part == 2 ? nv : nq;
#pragma unroll
    for (int t = 0; t < PREP_TOK; ++t) {
        const float f = part == 2 ? 1.0f : (part == 0 ? a.q_scale : 1.0f) / sqrtf(wave_sum(ss[t]) + a.unit_eps);
        if (t < nt) {
#pragma unroll
            for (int b = 0; b < CH; ++b)
                if (b * 64 + lane < n) dst[(size_t)(t0 + t) * row + (size_t)head * n + b * 64 + lane] = y[b][t] * f;
        }
    }
}

int launch_delta_prep(lumen_ctx *ctx, const DeltaPrepArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    const int units = 2 * a.kv_heads + a.heads + 1, widest = a.dim > a.vdim ? a.dim : a.vdim;
    const long waves = (long)((a.s + PREP_TOK - 1) / PREP_TOK) * units;
    const dim3 grid((unsigned)((waves + 3) / 4));
#define PREP_LAUNCH(CH)                                                                                              \
    do {                                                                                                             \
        if (a.taps <= 4) hipLaunchKernelGGL((delta_prep_kernel<4, CH>), grid, dim3(256), 0, ctx->stream, a, units);  \
        else hipLaunchKernelGGL((delta_prep_kernel<MIX_MAX_TAPS, CH>), grid, dim3(256), 0, ctx->stream, a, units);   \
    } while (0)
    if (widest <= 64) PREP_LAUNCH(1);
    else if (widest <= 128) PREP_LAUNCH(2);
    else PREP_LAUNCH(4);
#undef PREP_LAUNCH
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ------------------------------------------------------------------ decode
#define RD_THREADS 1024
#define RD_WAVES (RD_THREADS / 64)
#define RD_COLS (RD_WAVES * 4)  // state columns per trip

// A quarter of the dot product of a weight row of n (a multiple of 8) values with a vector in LDS: lane p of four takes
// every fourth 8-value piece; pieces are requested RD_AHEAD at a time.
#define RD_AHEAD 4
template <bool BF16>
struct RowPart {
    v4u w[RD_AHEAD][BF16 ? 1 : 2];
    const char *row;
    int n, p;
    __device__ void fetch(int k0) {
#pragma unroll
        for (int i = 0; i < RD_AHEAD; ++i) {
            const int k = min(k0 + i * 32 + p * 8, n - 8);
#pragma unroll
            for (int e = 0; e < (BF16 ? 1 : 2); ++e) w[i][e] = *(const v4u *)(row + (size_t)k * (BF16 ? 2 : 4) + 16 * e);
        }
    }
    __device__ void start(const void *base, size_t r, int n_, int p_) {
        row = (const char *)base + r * n_ * (BF16 ? 2 : 4);
        n = n_;
        p = p_;
        fetch(0);
    }
    __device__ float dot(const float *xs) {
        float s = 0.f;
        for (int k0 = 0; k0 < n; k0 += RD_AHEAD * 32) {
            if (k0) fetch(k0);
#pragma unroll
            for (int i = 0; i < RD_AHEAD; ++i) {
                const int k = k0 + i * 32 + p * 8;
                if (k < n) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        if (BF16) {
                            s = fmaf(__uint_as_float(w[i][0][e] << 16), xs[k + 2 * e], s);
                            s = fmaf(__uint_as_float(w[i][0][e] & 0xffff0000u), xs[k + 2 * e + 1], s);
                        } else {
                            s = fmaf(__uint_as_float(w[i][0][e]), xs[k + e], s);
                            s = fmaf(__uint_as_float(w[i][BF16 ? 0 : 1][e]), xs[k + 4 + e], s);
                        }
                    }
                }
            }
        }
        s += __shfl_xor(s, 1, 64);
        s += __shfl_xor(s, 2, 64);
        return s;
    }
};

// One workgroup per head, 64 state columns per trip, NT trips.  The state and the low-rank rows are requested first
// (they depend on nothing), then the head's inputs are made: convolution and unit norms (delta), decay and gate rows.
template <int KIND, int KR, int NT, bool BF16>
__global__ __launch_bounds__(RD_THREADS) void recurrence_decode_kernel(RecurrenceDecodeArgs a) {
    constexpr int DP = 16 * KR;
    constexpr bool DECAYS = KIND != REC_MEMORY;  // a decay per channel, from a low-rank product
    __shared__ __align__(16) float qs[DP], ks[DP], ws[DP], as[KIND == REC_GENERAL ? DP : 4];
    __shared__ float vs[MIX_MAX_DIM + 1], os[MIX_MAX_DIM + 1], gs[MIX_MAX_DIM];
    __shared__ __align__(16) float lo[DECAYS ? MIX_MAX_RANK : 8], hi[KIND == REC_DELTA ? MIX_MAX_RANK : 8];
    __shared__ float red[2], red_o[RD_WAVES];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15;
    const int h = blockIdx.x, rep = a.heads / a.kv_heads, hk = h / rep, D = a.dim, Dv = a.vdim;
    // low-rank rows: four lanes per row, decay rows first
    const int cols = KIND == REC_MEMORY ? Dv + 1 : Dv;
    const int lr_rows = !DECAYS ? 0 : D + (KIND == REC_DELTA ? Dv : 0), lr_part = tid & 3;
    RowPart<BF16> lr;
    auto lr_start = [&](int r) {
        if (r < D) lr.start(a.w_lo, (size_t)h * D + r, a.r_lo, lr_part);
        else lr.start(a.w_hi, (size_t)h * Dv + (r - D), a.r_hi, lr_part);
    };
    if (DECAYS) lr_start(min(tid >> 2, lr_rows - 1));
    float *Sh = a.state + (size_t)h * cols * DP + i16 * KR;
    const int c0 = wave * 4 + (lane >> 4);
    float S[NT][KR];
#pragma unroll
    for (int n = 0; n < NT; ++n) load_kr<KR>(S[n], Sh + (size_t)min(n * RD_COLS + c0, cols - 1) * DP);
    // small things that are needed late, requested now (clamped where a thread has no use for them)
    const int own_row = min(tid >> 2, D - 1), own_col = min(tid, Dv - 1);
    const float bias0 = DECAYS ? a.bias[h * D + own_row] : 0.f, gain0 = a.gain[(a.gain_shared ? 0 : (size_t)h * Dv) + own_col];
    const float a_log = KIND == REC_DELTA ? a.a_log[h] : 0.f, b_raw = KIND == REC_DELTA ? a.proj[a.off_b + h] : 0.f;
    float u[KR];
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const int kc = i16 * KR + i;
        u[i] = 0.f;
        if (KIND == REC_WKV) {
            u[i] = a.u[h * D + min(kc, D - 1)];
            u[i] = kc < D ? u[i] : 0.f;
        }
    }

    float m_old = 0.f, raw_i = 0.f, raw_f = 0.f;
    if (KIND == REC_MEMORY) {
        m_old = a.m[h];
        raw_i = a.proj[a.off_i + h] + a.i_bias[h];
        raw_f = a.proj[a.off_f + h] + a.f_bias[h];
    }
    if (DECAYS)
        for (int i = tid; i < a.r_lo; i += RD_THREADS) {
            const float x = a.proj[a.off_lo + i];
            lo[i] = KIND != REC_DELTA ? tanhf(x) : x;
        }
    if (KIND == REC_DELTA)
        for (int i = tid; i < a.r_hi; i += RD_THREADS) hi[i] = a.proj[a.off_hi + i];
    if (KIND != REC_DELTA) {
        for (int i = tid; i < DP; i += RD_THREADS) {
            qs[i] = i < D ? a.proj[a.off_q + h * D + i] * (KIND == REC_MEMORY ? a.q_scale : 1.f) : 0.f;
            ks[i] = i < D ? a.proj[a.off_k + h * D + i] : 0.f;
            ws[i] = 0.f;
            if (KIND == REC_GENERAL) as[i] = i < D ? sigmoid_r(a.proj[a.off_a + h * D + i] + a.a_bias[h * D + i]) : 0.f;
        }
        for (int i = tid; i < Dv; i += RD_THREADS) {
            const float g = a.proj[a.off_gate + h * Dv + i];
            vs[i] = a.proj[a.off_v + h * Dv + i];
            gs[i] = KIND == REC_WKV ? silu_r(g) : sigmoid_r(g);
        }
        if (KIND == REC_MEMORY && tid == 0) vs[Dv] = 1.f;
    } else {
        const int nq = a.kv_heads * D, channels = 2 * nq + a.heads * Dv, keep = a.taps - 1;
        const unsigned slot = *a.step & 1u;
        const float *prev = a.conv + (size_t)slot * keep * channels;
        float *next = a.conv + (size_t)(slot ^ 1u) * keep * channels;
        for (int i = tid; i < 2 * DP + Dv; i += RD_THREADS) {
            const int part = i < DP ? 0 : i < 2 * DP ? 1 : 2;
            const int c = i - part * DP;
            if (part < 2 && c >= D) {
                (part ? ks : qs)[c] = 0.f;
                ws[c] = 0.f;
                continue;
            }
            const int ch = part == 2 ? 2 * nq + h * Dv + c : part * nq + hk * D + c;
            const float x = a.proj[part == 0 ? a.off_q + hk * D + c : part == 1 ? a.off_k + hk * D + c : a.off_v + h * Dv + c];
            const float *w = a.taps_w + (size_t)ch * a.taps;
            const bool keeper = part == 2 || h % rep == 0;  // one workgroup leaves a shared channel's inputs
            float acc = 0.f;
            for (int j0 = 0; j0 < keep; j0 += 3) {  // (three earlier inputs and their weights per trip to memory)
                float p[3], wj[3];
#pragma unroll
                for (int j = 0; j < 3; ++j) {
                    const int jc = min(j0 + j, keep - 1);
                    p[j] = prev[(size_t)jc * channels + ch];
                    wj[j] = w[jc];
                }
#pragma unroll
                for (int j = 0; j < 3; ++j) {
                    if (j0 + j < keep) {
                        acc = fmaf(wj[j], p[j], acc);
                        if (keeper && j0 + j > 0) next[(size_t)(j0 + j - 1) * channels + ch] = p[j];
                    }
                }
            }
            if (keeper && keep > 0) next[(size_t)(keep - 1) * channels + ch] = x;
            acc = silu_r(fmaf(w[keep], x, acc));
            (part == 0 ? qs : part == 1 ? ks : vs)[c] = acc;
        }
    }
    __syncthreads();
    const float decay_a = KIND == REC_DELTA ? expf(a_log) : KIND == REC_GENERAL ? a.z_scale : 0.f;
    if (KIND == REC_GENERAL && wave == 0) {  // the key's length
        float ss = 0.f;
        for (int c = lane; c < D; c += 64) ss = fmaf(ks[c], ks[c], ss);
        ss = wave_sum(ss);
        if (lane == 0) red[0] = 1.0f / sqrtf(ss + a.unit_eps);
    }
    if (KIND == REC_DELTA && wave < 2) {  // the sums of squares of q and of k
        const float *p = wave ? ks : qs;
        float ss = 0.f;
        for (int c = lane; c < D; c += 64) ss = fmaf(p[c], p[c], ss);
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = (wave ? 1.0f : a.q_scale) / sqrtf(ss + a.unit_eps);
    }
    for (int r0 = 0; r0 < lr_rows; r0 += RD_THREADS / 4) {  // (uniform trips, rows clamped: the lanes exchange parts)
        const int r = r0 + (tid >> 2), rc = min(r, lr_rows - 1);
        if (r0) lr_start(rc);
        const float z = lr.dot(rc < D ? lo : hi);
        if (lr_part == 0 && r < lr_rows) {
            if (r < D) ws[r] = decay_r<KIND>(z, r0 ? a.bias[h * D + r] : bias0, decay_a);
            else gs[r - D] = sigmoid_r(z);
        }
    }
    __syncthreads();
    float q[KR], k[KR], w[KR];
    load_kr<KR>(q, qs + i16 * KR);
    load_kr<KR>(k, ks + i16 * KR);
    load_kr<KR>(w, ws + i16 * KR);
    float beta = 0.f, ak[KR], keep = 0.f, m_new = 0.f;
    if (KIND == REC_GENERAL) {
        const float inv = red[0];
        load_kr<KR>(ak, as + i16 * KR);
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            u[i] = k[i] * inv;
            ak[i] *= u[i];
        }
    }
    if (KIND == REC_MEMORY) {
        const float li = memory_log_input(raw_i, a.cap), lf = memory_log_forget(raw_f, a.cap);
        m_new = fmaxf(lf + m_old, li);
        keep = expf(lf + m_old - m_new);
        const float add = expf(li - m_new);
#pragma unroll
        for (int i = 0; i < KR; ++i) k[i] *= add;
    }
    if (KIND == REC_DELTA) {
        const float iq = red[0], ik = red[1];
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            q[i] *= iq;
            k[i] *= ik;
        }
        beta = sigmoid_r(b_raw);
    }
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const int c = n * RD_COLS + c0;
        const float v = vs[min(c, cols - 1)];
        float o;
        if (KIND == REC_GENERAL) o = column_step_general<KR>(S[n], q, k, w, u, ak, v);
        else if (KIND == REC_MEMORY) o = column_step_memory<KR>(S[n], q, k, keep, v);
        else o = column_step<KIND, KR>(S[n], q, k, w, u, v, beta);
        if (c < cols) {
            store_kr<KR>(Sh + (size_t)c * DP, S[n]);
            if (i16 == 0) {
                os[c] = o;
                if (KIND != REC_MEMORY || c < Dv) ss = fmaf(o, o, ss);
            }
        }
    }
    ss = wave_sum(ss);
    if (lane == 0) red_o[wave] = ss;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int i = 0; i < RD_WAVES; ++i) tot += red_o[i];
    float read = 1.f;
    if (KIND == REC_MEMORY) {
        read = 1.0f / (fmaxf(fabsf(os[Dv]), expf(-m_new)) + a.den_eps);
        tot *= read * read;
        if (tid == 0) a.m[h] = m_new;
    }
    const float inv = 1.0f / sqrtf(tot / (float)Dv + a.norm_eps);
    if (tid < Dv) a.out[(size_t)h * Dv + tid] = os[tid] * read * inv * gain0 * gs[tid];
}

int launch_recurrence_decode(lumen_ctx *ctx, const RecurrenceDecodeArgs &a) {
    const int rows = recurrence_rows(a.dim), trips = (recurrence_columns(a.kind, a.vdim) + RD_COLS - 1) / RD_COLS;
    const int nt = trips <= 1 ? 1 : trips <= 2 ? 2 : trips <= 4 ? 4 : 5;  // (5: the matrix memory's widest heads and their normaliser)
    note_kernel(ctx, "recurrence_decode_kernel<%d, %d, %d, %s>", a.kind, rows / 16, nt, a.w_bf16 ? "true" : "false");
#define RD_LAUNCH(KIND, KR, NT)                                                                                           \
    do {                                                                                                                  \
        if (a.w_bf16) hipLaunchKernelGGL((recurrence_decode_kernel<KIND, KR, NT, true>), dim3(a.heads), dim3(RD_THREADS), 0, ctx->stream, a); \
        else hipLaunchKernelGGL((recurrence_decode_kernel<KIND, KR, NT, false>), dim3(a.heads), dim3(RD_THREADS), 0, ctx->stream, a);         \
    } while (0)
#define RD_TRIPS(KIND, KR)                     \
    do {                                       \
        if (nt == 1) RD_LAUNCH(KIND, KR, 1);   \
        else if (nt == 2) RD_LAUNCH(KIND, KR, 2); \
        else if (nt == 5 && KIND == REC_MEMORY) RD_LAUNCH(KIND, KR, (KIND == REC_MEMORY ? 5 : 4)); \
        else RD_LAUNCH(KIND, KR, 4);           \
    } while (0)
#define RD_KIND(KIND)                   \
    do {                                \
        if (rows == 64) RD_TRIPS(KIND, 4);  \
        else if (rows == 128) RD_TRIPS(KIND, 8); \
        else RD_TRIPS(KIND, 16);        \
    } while (0)
    if (a.kind == REC_WKV) RD_KIND(REC_WKV);
    else if (a.kind == REC_DELTA) RD_KIND(REC_DELTA);
    else if (a.kind == REC_GENERAL) RD_KIND(REC_GENERAL);
    else RD_KIND(REC_MEMORY);
#undef RD_KIND
#undef RD_TRIPS
#undef RD_LAUNCH
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

LUMEN_DEFINE_WARM(recurrence)
