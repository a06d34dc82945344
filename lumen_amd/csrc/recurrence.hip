// Matrix-state recurrences: the WKV time mixing and the channel-wise gated delta rule.  Both keep one f32 matrix
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

int recurrence_rows(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }

__device__ __forceinline__ float sigmoid_r(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_r(float z) { return z * sigmoid_r(z); }
__device__ __forceinline__ float softplus_r(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float gate_r(float z, int act) { return act == GATE_SILU ? silu_r(z) : act == GATE_SIGMOID ? sigmoid_r(z) : 1.0f; }

template <int KIND>
__device__ __forceinline__ float decay_r(float z, float bias, float a) {
    // WKV: exp(-exp(z + bias)); delta: exp(-a softplus(z + bias)) with a = exp(a_log)
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

// ------------------------------------------------------------------ prompt
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

int launch_recurrence(lumen_ctx *ctx, const RecurrenceArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    dim3 grid((a.vdim + REC_COLS - 1) / REC_COLS, a.heads);
    const int rows = recurrence_rows(a.dim);
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

// Causal convolution of one channel at token t of this portion: taps_w[taps - 1] is the current token's.
__device__ __forceinline__ float conv_at(const float *__restrict__ in, int stride, const float *__restrict__ w, int taps, int t,
                                         const float *__restrict__ prev, int channels, int ch) {
    float acc = 0.f;
    for (int j = 0; j < taps; ++j) {
        const int src = t - (taps - 1) + j;
        const float x = src >= 0 ? in[(size_t)src * stride] : prev[(size_t)(taps - 1 + src) * channels + ch];
        acc = fmaf(w[j], x, acc);
    }
    return acc;
}

// One workgroup per token: q and k of all kv heads go through LDS for their unit norms, v straight out.
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a) {
    LUMEN_DYNAMIC_LDS(float, qk);  // [2][kv_heads * dim]
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nq = a.kv_heads * a.dim, nv = a.heads * a.vdim, channels = 2 * nq + nv;
    for (int c = tid; c < channels; c += 256) {
        const int off = c < nq ? a.off_q + c : c < 2 * nq ? a.off_k + (c - nq) : a.off_v + (c - 2 * nq);
        const float y = silu_r(conv_at(a.in + off, a.stride, a.taps_w + (size_t)c * a.taps, a.taps, t, a.conv_prev, channels, c));
        if (c < 2 * nq) qk[c] = y;
        else a.v[(size_t)t * nv + (c - 2 * nq)] = y;
        if (t == a.s - 1) {  // the last taps - 1 inputs stay for the next portion
            for (int j = 0; j < a.taps - 1; ++j) {
                const int src = a.s - (a.taps - 1) + j;
                a.conv_next[(size_t)j * channels + c] = src >= 0 ? a.in[(size_t)src * a.stride + off]
                                                                 : a.conv_prev[(size_t)(a.taps - 1 + src) * channels + c];
            }
        }
    }
    const float *row = a.in + (size_t)t * a.stride;
    for (int i = tid; i < a.ra; i += 256) a.a1[(size_t)t * a.ra + i] = row[a.off_a1 + i];
    for (int i = tid; i < a.rg; i += 256) a.g1[(size_t)t * a.rg + i] = row[a.off_g1 + i];
    __syncthreads();
    for (int u = wave; u < 2 * a.kv_heads; u += 4) {  // head u of q (u < kv_heads) or of k
        const float *p = qk + (size_t)u * a.dim;
        float ss = 0.f;
        for (int c = lane; c < a.dim; c += 64) ss = fmaf(p[c], p[c], ss);
        ss = wave_sum(ss);
        const bool is_q = u < a.kv_heads;
        const float inv = (is_q ? a.q_scale : 1.0f) / sqrtf(ss + a.unit_eps);
        float *dst = is_q ? a.q + (size_t)t * nq + (size_t)u * a.dim : a.k + (size_t)t * nq + (size_t)(u - a.kv_heads) * a.dim;
        for (int c = lane; c < a.dim; c += 64) dst[c] = p[c] * inv;
    }
}

int launch_delta_prep(lumen_ctx *ctx, const DeltaPrepArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    const size_t lds = (size_t)2 * a.kv_heads * a.dim * sizeof(float);
    if (lds > 64 * 1024)
        HIP_TRY(hipFuncSetAttribute((const void *)delta_prep_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(delta_prep_kernel, dim3(a.s), dim3(256), lds, ctx->stream, a);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ------------------------------------------------------------------ decode
#define RD_THREADS 512
#define RD_WAVES (RD_THREADS / 64)

// dot product of a weight row of n (a multiple of 8) values with a vector in LDS
template <bool BF16>
__device__ __forceinline__ float row_dot(const void *w, size_t row, const float *xs, int n) {
    float s = 0.f;
    if (BF16) {
        const uint16_t *p = (const uint16_t *)w + row * n;
        for (int k = 0; k < n; k += 8) {
            const v4u r = *(const v4u *)(p + k);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s = fmaf(__uint_as_float(r[e] << 16), xs[k + 2 * e], s);
                s = fmaf(__uint_as_float(r[e] & 0xffff0000u), xs[k + 2 * e + 1], s);
            }
        }
    } else {
        const float *p = (const float *)w + row * n;
        for (int k = 0; k < n; k += 4) {
            const v4f r = *(const v4f *)(p + k);
#pragma unroll
            for (int e = 0; e < 4; ++e) s = fmaf(r[e], xs[k + e], s);
        }
    }
    return s;
}

// One workgroup per head, 32 state columns per trip.  The state is requested first (it depends on nothing), then the
// head's inputs are made: convolution and unit norms (delta), decay and gate rows of the low-rank products.
template <int KIND, int KR, bool BF16>
__global__ __launch_bounds__(RD_THREADS) void recurrence_decode_kernel(RecurrenceDecodeArgs a) {
    constexpr int DP = 16 * KR;
    __shared__ __align__(16) float qs[DP], ks[DP], ws[DP];
    __shared__ float vs[MIX_MAX_DIM], os[MIX_MAX_DIM], gs[MIX_MAX_DIM];
    __shared__ __align__(16) float lo[MIX_MAX_RANK], hi[MIX_MAX_RANK];
    __shared__ float red[2], red_o[RD_WAVES];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15;
    const int h = blockIdx.x, rep = a.heads / a.kv_heads, hk = h / rep, D = a.dim, Dv = a.vdim;
    float *Sh = a.state + (size_t)h * Dv * DP + i16 * KR;
    const int c0 = wave * 4 + (lane >> 4);
    float S[KR];
    load_kr<KR>(S, Sh + (size_t)min(c0, Dv - 1) * DP);

    for (int i = tid; i < a.r_lo; i += RD_THREADS) {
        const float x = a.proj[a.off_lo + i];
        lo[i] = KIND == REC_WKV ? tanhf(x) : x;
    }
    if (KIND == REC_DELTA)
        for (int i = tid; i < a.r_hi; i += RD_THREADS) hi[i] = a.proj[a.off_hi + i];
    if (KIND == REC_WKV) {
        for (int i = tid; i < DP; i += RD_THREADS) {
            qs[i] = i < D ? a.proj[a.off_q + h * D + i] : 0.f;
            ks[i] = i < D ? a.proj[a.off_k + h * D + i] : 0.f;
        }
        for (int i = tid; i < Dv; i += RD_THREADS) {
            vs[i] = a.proj[a.off_v + h * Dv + i];
            gs[i] = silu_r(a.proj[a.off_gate + h * Dv + i]);
        }
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
                continue;
            }
            const int ch = part == 2 ? 2 * nq + h * Dv + c : part * nq + hk * D + c;
            const float x = a.proj[part == 0 ? a.off_q + hk * D + c : part == 1 ? a.off_k + hk * D + c : a.off_v + h * Dv + c];
            const float *w = a.taps_w + (size_t)ch * a.taps;
            const bool keeper = part == 2 || h % rep == 0;  // one workgroup leaves a shared channel's inputs
            float acc = 0.f;
            for (int j = 0; j < keep; ++j) {
                const float p = prev[(size_t)j * channels + ch];
                acc = fmaf(w[j], p, acc);
                if (keeper && j > 0) next[(size_t)(j - 1) * channels + ch] = p;
            }
            if (keeper && keep > 0) next[(size_t)(keep - 1) * channels + ch] = x;
            acc = silu_r(fmaf(w[keep], x, acc));
            (part == 0 ? qs : part == 1 ? ks : vs)[c] = acc;
        }
    }
    __syncthreads();
    // decay and gate rows; the sums of squares of q and k meanwhile sit with the first two wavefronts
    const float decay_a = KIND == REC_DELTA ? expf(a.a_log[h]) : 0.f;
    if (KIND == REC_DELTA && wave < 2) {
        const float *p = wave ? ks : qs;
        float ss = 0.f;
        for (int c = lane; c < D; c += 64) ss = fmaf(p[c], p[c], ss);
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = (wave ? 1.0f : a.q_scale) / sqrtf(ss + a.unit_eps);
    }
    for (int i = tid; i < DP + (KIND == REC_DELTA ? Dv : 0); i += RD_THREADS) {
        if (i < D) ws[i] = decay_r<KIND>(row_dot<BF16>(a.w_lo, (size_t)h * D + i, lo, a.r_lo), a.bias[h * D + i], decay_a);
        else if (i < DP) ws[i] = 0.f;
        else gs[i - DP] = sigmoid_r(row_dot<BF16>(a.w_hi, (size_t)h * Dv + (i - DP), hi, a.r_hi));
    }
    __syncthreads();
    float q[KR], k[KR], w[KR], u[KR];
    load_kr<KR>(q, qs + i16 * KR);
    load_kr<KR>(k, ks + i16 * KR);
    load_kr<KR>(w, ws + i16 * KR);
    float beta = 0.f;
    if (KIND == REC_DELTA) {
        const float iq = red[0], ik = red[1];
#pragma unroll
        for (int i = 0; i < KR; ++i) {
            q[i] *= iq;
            k[i] *= ik;
        }
        beta = sigmoid_r(a.proj[a.off_b + h]);
    }
#pragma unroll
    for (int i = 0; i < KR; ++i) {
        const int kc = i16 * KR + i;
        u[i] = KIND == REC_WKV && kc < D ? a.u[h * D + kc] : 0.f;
    }
    float ss = 0.f;
    for (int cb = 0; cb < Dv; cb += RD_WAVES * 4) {  // (uniform trips: the lane exchanges need whole wavefronts)
        const int c = cb + c0;
        if (cb) load_kr<KR>(S, Sh + (size_t)min(c, Dv - 1) * DP);
        const float o = column_step<KIND, KR>(S, q, k, w, u, vs[min(c, Dv - 1)], beta);
        if (c < Dv) {
            store_kr<KR>(Sh + (size_t)c * DP, S);
            if (i16 == 0) {
                os[c] = o;
                ss = fmaf(o, o, ss);
            }
        }
    }
    ss = wave_sum(ss);
    if (lane == 0) red_o[wave] = ss;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int i = 0; i < RD_WAVES; ++i) tot += red_o[i];
    const float inv = 1.0f / sqrtf(tot / (float)Dv + a.norm_eps);
    const float *gain = a.gain + (a.gain_shared ? 0 : (size_t)h * Dv);
    for (int c = tid; c < Dv; c += RD_THREADS) a.out[(size_t)h * Dv + c] = os[c] * inv * gain[c] * gs[c];
}

int launch_recurrence_decode(lumen_ctx *ctx, const RecurrenceDecodeArgs &a) {
    const int rows = recurrence_rows(a.dim);
    note_kernel(ctx, "recurrence_decode_kernel<%d, %d, %s>", a.kind, rows / 16, a.w_bf16 ? "true" : "false");
#define RD_LAUNCH(KIND, KR)                                                                                               \
    do {                                                                                                                  \
        if (a.w_bf16) hipLaunchKernelGGL((recurrence_decode_kernel<KIND, KR, true>), dim3(a.heads), dim3(RD_THREADS), 0, ctx->stream, a); \
        else hipLaunchKernelGGL((recurrence_decode_kernel<KIND, KR, false>), dim3(a.heads), dim3(RD_THREADS), 0, ctx->stream, a);         \
    } while (0)
#define RD_KIND(KIND)                   \
    do {                                \
        if (rows == 64) RD_LAUNCH(KIND, 4);  \
        else if (rows == 128) RD_LAUNCH(KIND, 8); \
        else RD_LAUNCH(KIND, 16);       \
    } while (0)
    if (a.kind == REC_WKV) RD_KIND(REC_WKV);
    else RD_KIND(REC_DELTA);
#undef RD_KIND
#undef RD_LAUNCH
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

LUMEN_DEFINE_WARM(recurrence)
