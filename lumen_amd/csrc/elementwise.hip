// Small HBM-bound kernels of the path: RMSNorm, SiLU / add / mul / SwiGLU,
// embedding gather, greedy argmax and the tensor form of RoPE.
#include "internal.h"
#include "mixers.h"
#include "wave_reduce.h"

#include <cmath>

typedef float v4f __attribute__((ext_vector_type(4)));


// ------------------------------------------------------------------ RMSNorm
// One workgroup per row: sum of squares, rms = sqrt(ss/dim + eps), out = (x * inv) * w.
// src/layers/norm/rms_norm.rs:45-58
__global__ __launch_bounds__(256) void rmsnorm_kernel(const float *__restrict__ x, const float *__restrict__ w,
                                                      float *__restrict__ out, int dim, float eps) {
    __shared__ float red[4];
    const float *xr = x + (size_t)blockIdx.x * dim;
    float *o = out + (size_t)blockIdx.x * dim;
    const int tid = threadIdx.x;
    float ss = 0.f;
    for (int i = tid; i < dim; i += 256) {
        const float v = xr[i];
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float tot = (red[0] + red[1]) + (red[2] + red[3]);
    const float rms = sqrtf(tot / (float)dim + eps);
    const float inv = 1.0f / rms;
    for (int i = tid; i < dim; i += 256) o[i] = xr[i] * inv * w[i];
}

// The same for rows of up to 1024 * VPT floats that are 16-byte aligned: a thread requests all of its
// pieces of the row and of the gains at once (the scalar loop above takes a trip to memory per element
// and pass) and keeps the row in registers between the two passes.
template <int VPT>
__global__ __launch_bounds__(256) void rmsnorm_vec_kernel(const float *__restrict__ x, const float *__restrict__ w,
                                                          float *__restrict__ out, int dim, float eps) {
    __shared__ float red[4];
    const float *xr = x + (size_t)blockIdx.x * dim;
    float *o = out + (size_t)blockIdx.x * dim;
    const int tid = threadIdx.x;
    v4f v[VPT], g[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int k = (tid + i * 256) * 4;
        v[i] = v4f{0.f, 0.f, 0.f, 0.f};
        g[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (k < dim) {
            v[i] = *(const v4f *)(xr + k);
            g[i] = *(const v4f *)(w + k);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        ss = fmaf(v[i].x, v[i].x, ss);
        ss = fmaf(v[i].y, v[i].y, ss);
        ss = fmaf(v[i].z, v[i].z, ss);
        ss = fmaf(v[i].w, v[i].w, ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float tot = (red[0] + red[1]) + (red[2] + red[3]);
    const float rms = sqrtf(tot / (float)dim + eps);
    const float inv = 1.0f / rms;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int k = (tid + i * 256) * 4;
        if (k < dim) {
            v4f r;
            r.x = v[i].x * inv * g[i].x;
            r.y = v[i].y * inv * g[i].y;
            r.z = v[i].z * inv * g[i].z;
            r.w = v[i].w * inv * g[i].w;
            *(v4f *)(o + k) = r;
        }
    }
}

int launch_rmsnorm(lumen_ctx *ctx, const float *x, const float *w, float *out, int rows, int dim, float eps) {
    if (rows <= 0 || dim <= 0) return LUMEN_OK;
    const bool vec = dim % 4 == 0 && ((((uintptr_t)x | (uintptr_t)w | (uintptr_t)out) & 15) == 0);
    if (vec && dim <= 2048)
        hipLaunchKernelGGL(rmsnorm_vec_kernel<2>, dim3(rows), dim3(256), 0, ctx->stream, x, w, out, dim, eps);
    else if (vec && dim <= 4096)
        hipLaunchKernelGGL(rmsnorm_vec_kernel<4>, dim3(rows), dim3(256), 0, ctx->stream, x, w, out, dim, eps);
    else
        hipLaunchKernelGGL(rmsnorm_kernel, dim3(rows), dim3(256), 0, ctx->stream, x, w, out, dim, eps);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// -------------------------------------------------------------- elementwise
enum { OP_SILU, OP_ADD, OP_MUL, OP_SWIGLU, OP_COPY, OP_TANH, OP_GELU };

template <int OP>
__global__ __launch_bounds__(256) void ew_kernel(const float *__restrict__ a, const float *__restrict__ b,
                                                 float *__restrict__ out, size_t n) {
    const size_t stride = (size_t)gridDim.x * blockDim.x;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += stride) {
        const float x = a[i];
        float r;
        if (OP == OP_SILU) {
            const float sig = 1.0f / (1.0f + expf(-x));  // src/layers/activation.rs:143-146
            r = x * sig;
        } else if (OP == OP_COPY) {
            r = x;
        } else if (OP == OP_TANH) {
            r = tanhf(x);
        } else if (OP == OP_GELU) {
            r = 0.5f * x * (1.0f + erff(x * 0.70710678118654752f));
        } else if (OP == OP_ADD) {
            r = x + b[i];
        } else if (OP == OP_MUL) {
            r = x * b[i];
        } else {
            const float sig = 1.0f / (1.0f + expf(-x));
            r = (x * sig) * b[i];  // src/models/llama.rs:60-63
        }
        out[i] = r;
    }
}

template <int OP>
static int launch_ew(lumen_ctx *ctx, const float *a, const float *b, float *out, size_t n) {
    if (n == 0) return LUMEN_OK;
    size_t blocks = (n + 255) / 256;
    const size_t cap = (size_t)ctx->num_cus * 16;
    if (blocks > cap) blocks = cap;
    hipLaunchKernelGGL(ew_kernel<OP>, dim3((unsigned)blocks), dim3(256), 0, ctx->stream, a, b, out, n);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

int launch_silu(lumen_ctx *ctx, const float *x, float *out, size_t n) { return launch_ew<OP_SILU>(ctx, x, x, out, n); }
int launch_add(lumen_ctx *ctx, const float *a, const float *b, float *out, size_t n) { return launch_ew<OP_ADD>(ctx, a, b, out, n); }
int launch_mul(lumen_ctx *ctx, const float *a, const float *b, float *out, size_t n) { return launch_ew<OP_MUL>(ctx, a, b, out, n); }
int launch_swiglu(lumen_ctx *ctx, const float *g, const float *u, float *out, size_t n) { return launch_ew<OP_SWIGLU>(ctx, g, u, out, n); }
static int launch_copy(lumen_ctx *ctx, const float *x, float *out, size_t n) { return launch_ew<OP_COPY>(ctx, x, x, out, n); }

int launch_tanh(lumen_ctx *ctx, const float *x, float *out, size_t n) { return launch_ew<OP_TANH>(ctx, x, x, out, n); }

int launch_gelu(lumen_ctx *ctx, const float *x, float *out, size_t n) { return launch_ew<OP_GELU>(ctx, x, x, out, n); }

__global__ __launch_bounds__(256) void softcap_kernel(float *x, float cap, size_t n) {
    const size_t stride = (size_t)gridDim.x * blockDim.x;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += stride) x[i] = cap * tanhf(x[i] / cap);
}
int launch_softcap(lumen_ctx *ctx, float *x, float cap, size_t n) {
    if (n == 0) return LUMEN_OK;
    const size_t blocks = (n + 255) / 256, most = (size_t)ctx->num_cus * 16;
    hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)(blocks < most ? blocks : most)), dim3(256), 0, ctx->stream, x, cap, n);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ----------------------------------------------------- Dynamic Tanh, gated residual
__device__ __forceinline__ v4f dyt_row4(const v4f x, float alpha, const v4f g, const v4f b) {
    return v4f{fmaf(tanhf(alpha * x.x), g.x, b.x), fmaf(tanhf(alpha * x.y), g.y, b.y), fmaf(tanhf(alpha * x.z), g.z, b.z),
               fmaf(tanhf(alpha * x.w), g.w, b.w)};
}
__device__ __forceinline__ float sigmoid_e(float z) { return 1.0f / (1.0f + expf(-z)); }

__global__ __launch_bounds__(256) void dyt_kernel(const float *__restrict__ x, const float *__restrict__ alpha, const float *__restrict__ w,
                                                  const float *__restrict__ b, float *__restrict__ out, int dim) {
    const float al = *alpha;
    const size_t base = (size_t)blockIdx.x * dim;
    if (dim % 4 == 0) {
        for (int i = threadIdx.x * 4; i < dim; i += 1024)
            *(v4f *)(out + base + i) = dyt_row4(*(const v4f *)(x + base + i), al, *(const v4f *)(w + i), *(const v4f *)(b + i));
    } else {
        for (int i = threadIdx.x; i < dim; i += 256) out[base + i] = fmaf(tanhf(al * x[base + i]), w[i], b[i]);
    }
}
int launch_dyt(lumen_ctx *ctx, const float *x, const float *alpha, const float *w, const float *b, float *out, int rows, int dim) {
    if (rows <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(dyt_kernel, dim3(rows), dim3(256), 0, ctx->stream, x, alpha, w, b, out, dim);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// One workgroup per row of up to 4 * blockDim * GR_VPT elements: everything a thread needs is requested at once and stays
// in registers between the sums of squares and the result.
#define GR_VPT 4
__global__ __launch_bounds__(1024) void gated_residual_kernel(GatedResidualArgs a) {
    __shared__ float red[2][16];
    const int row = blockIdx.x, tid = threadIdx.x, nt = blockDim.x, waves = nt >> 6, W = a.dim;
    const size_t base = (size_t)row * W;
    v4f y[GR_VPT], y2[GR_VPT];
    float s1 = 0.f, s2 = 0.f;
#pragma unroll
    for (int i = 0; i < GR_VPT; ++i) {
        const int k = (tid + i * nt) * 4;
        y[i] = y2[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (k < W) {
            if (a.top > 0) {
                const size_t first = (size_t)row * a.top;
                for (int j = 0; j < a.top; ++j) {
                    const float f = a.sel_w[first + j];
                    const v4f v = *(const v4f *)(a.y + (first + j) * W + k);
#pragma unroll
                    for (int e = 0; e < 4; ++e) y[i][e] = fmaf(f, v[e], y[i][e]);
                }
            } else {
                y[i] = *(const v4f *)(a.y + base + k);
            }
            if (a.y2) {
                y2[i] = *(const v4f *)(a.y2 + base + k);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s1 = fmaf(y[i][e], y[i][e], s1);
                    s2 = fmaf(y2[i][e], y2[i][e], s2);
                }
            }
        }
    }
    float i1 = 0.f, i2 = 0.f;
    if (a.y2) {
        s1 = wave_sum(s1);
        s2 = wave_sum(s2);
        if ((tid & 63) == 0) {
            red[0][tid >> 6] = s1;
            red[1][tid >> 6] = s2;
        }
        __syncthreads();
        s1 = s2 = 0.f;
        for (int w = 0; w < waves; ++w) {
            s1 += red[0][w];
            s2 += red[1][w];
        }
        i1 = a.pair_scale / sqrtf(s1 / (float)a.width + a.eps);
        i2 = a.pair_scale / sqrtf(s2 / (float)a.width + a.eps);
    }
    const float alpha = a.norm_out ? *a.norm_alpha : 0.f;
#pragma unroll
    for (int i = 0; i < GR_VPT; ++i) {
        const int k = (tid + i * nt) * 4;
        if (k >= W) continue;
        v4f v = y[i];
        if (a.y2) {
            const v4f w1 = *(const v4f *)(a.w1 + k), w2 = *(const v4f *)(a.w2 + k);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = fmaf(y2[i][e] * i2, w2[e], v[e] * i1 * w1[e]);
        }
        v4f x = *(const v4f *)(a.x + base + k);
        const v4f gz = *(const v4f *)(a.gate + (size_t)row * a.gate_stride + k), gb = *(const v4f *)(a.gate_b + k);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = fmaf(sigmoid_e(gz[e] + gb[e]), v[e], x[e]);
        if (a.out) *(v4f *)(a.out + base + k) = x;
        if (a.norm_out) *(v4f *)(a.norm_out + base + k) = dyt_row4(x, alpha, *(const v4f *)(a.norm_w + k), *(const v4f *)(a.norm_b + k));
    }
}
int launch_gated_residual(lumen_ctx *ctx, const GatedResidualArgs &a) {
    if (a.rows <= 0) return LUMEN_OK;
    int threads = 256;
    while (threads < 1024 && (threads * 4 * GR_VPT < a.dim || (a.rows < 16 && threads * 4 < a.dim))) threads *= 2;
    if (threads * 4 * GR_VPT < a.dim) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "gated residual: rows of %d", a.dim);
    hipLaunchKernelGGL(gated_residual_kernel, dim3(a.rows), dim3(threads), 0, ctx->stream, a);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ----------------------------------------------------- PolyNorm, token shift, row helpers
// One workgroup per row; the row is read once for the three sums and once more (from cache) for the values.
__global__ __launch_bounds__(256) void polynorm_kernel(const float *z, const float *__restrict__ coef, float *out, int dim,
                                                       int stride, float eps) {
    __shared__ float red[3][4];
    const float *zr = z + (size_t)blockIdx.x * stride;
    float *o = out + (size_t)blockIdx.x * stride;
    const int tid = threadIdx.x;
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
    for (int i = tid; i < dim; i += 256) {
        const float v = zr[i], q = v * v, q2 = q * q;
        s1 += q;
        s2 += q2;
        s3 = fmaf(q2, q, s3);
    }
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    s3 = wave_sum(s3);
    if ((tid & 63) == 0) {
        red[0][tid >> 6] = s1;
        red[1][tid >> 6] = s2;
        red[2][tid >> 6] = s3;
    }
    __syncthreads();
    const float n = (float)dim;
    const float a1 = coef[0] / sqrtf(((red[0][0] + red[0][1]) + (red[0][2] + red[0][3])) / n + eps);
    const float a2 = coef[1] / sqrtf(((red[1][0] + red[1][1]) + (red[1][2] + red[1][3])) / n + eps);
    const float a3 = coef[2] / sqrtf(((red[2][0] + red[2][1]) + (red[2][2] + red[2][3])) / n + eps);
    const float c3 = coef[3];
    for (int i = tid; i < dim; i += 256) {
        const float v = zr[i];
        o[i] = fmaf(fmaf(fmaf(a3, v, a2), v, a1), v, c3);
    }
}

// The same for 16-byte aligned rows of up to 4096 VPT elements: read once, kept in registers between the two passes.
template <int VPT>
__global__ __launch_bounds__(1024) void polynorm_vec_kernel(const float *z, const float *__restrict__ coef, float *out, int dim,
                                                            int stride, float eps) {
    __shared__ float red[3][16];
    const float *zr = z + (size_t)blockIdx.x * stride;
    float *o = out + (size_t)blockIdx.x * stride;
    const int tid = threadIdx.x, nt = blockDim.x, nw = nt >> 6;
    v4f v[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int k = (tid + i * nt) * 4;
        v[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (k < stride) v[i] = *(const v4f *)(zr + k);
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (k + e >= dim) v[i][e] = 0.f;
    }
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float q = v[i][e] * v[i][e], q2 = q * q;
            s1 += q;
            s2 += q2;
            s3 = fmaf(q2, q, s3);
        }
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    s3 = wave_sum(s3);
    if ((tid & 63) == 0) {
        red[0][tid >> 6] = s1;
        red[1][tid >> 6] = s2;
        red[2][tid >> 6] = s3;
    }
    __syncthreads();
    s1 = s2 = s3 = 0.f;
    for (int w = 0; w < nw; ++w) {
        s1 += red[0][w];
        s2 += red[1][w];
        s3 += red[2][w];
    }
    const float n = (float)dim;
    const float a1 = coef[0] / sqrtf(s1 / n + eps), a2 = coef[1] / sqrtf(s2 / n + eps), a3 = coef[2] / sqrtf(s3 / n + eps), c3 = coef[3];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int k = (tid + i * nt) * 4;
        if (k < stride) {
            v4f r;
#pragma unroll
            for (int e = 0; e < 4; ++e) r[e] = k + e < dim ? fmaf(fmaf(fmaf(a3, v[i][e], a2), v[i][e], a1), v[i][e], c3) : 0.f;
            *(v4f *)(o + k) = r;
        }
    }
}

int launch_polynorm(lumen_ctx *ctx, const float *z, const float *coef, float *out, int rows, int dim, int stride, float eps) {
    if (rows <= 0 || dim <= 0) return LUMEN_OK;
    if (stride % 4 == 0 && stride <= 16384 && (((uintptr_t)z | (uintptr_t)out) & 15) == 0) {
        const int pieces = stride / 4, threads = pieces <= 256 ? 256 : pieces <= 512 ? 512 : 1024;
        if (pieces <= threads)
            hipLaunchKernelGGL(polynorm_vec_kernel<1>, dim3(rows), dim3(threads), 0, ctx->stream, z, coef, out, dim, stride, eps);
        else if (pieces <= 2 * threads)
            hipLaunchKernelGGL(polynorm_vec_kernel<2>, dim3(rows), dim3(threads), 0, ctx->stream, z, coef, out, dim, stride, eps);
        else
            hipLaunchKernelGGL(polynorm_vec_kernel<4>, dim3(rows), dim3(threads), 0, ctx->stream, z, coef, out, dim, stride, eps);
    } else {
        hipLaunchKernelGGL(polynorm_kernel, dim3(rows), dim3(256), 0, ctx->stream, z, coef, out, dim, stride, eps);
    }
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

__global__ __launch_bounds__(256) void token_shift_kernel(const float *__restrict__ h, const float *__restrict__ mu,
                                                          const float *__restrict__ prev, float *__restrict__ next,
                                                          float *__restrict__ mixes, int n, int s, int dim) {
    const int t = blockIdx.x;
    const float *cur = h + (size_t)t * dim, *bef = t ? cur - dim : prev;
    for (int i = threadIdx.x; i < dim; i += 256) {
        const float c = cur[i], d = bef[i] - c;
        for (int m = 0; m < n; ++m) mixes[((size_t)m * s + t) * dim + i] = fmaf(d, mu[(size_t)m * dim + i], c);
        if (t == s - 1) next[i] = c;
    }
}

// 16-byte pieces: workgroup (token, block of 1024 channels), all mixes' factors requested together
__global__ __launch_bounds__(256) void token_shift_vec_kernel(const float *__restrict__ h, const float *__restrict__ mu,
                                                              const float *__restrict__ prev, float *__restrict__ next,
                                                              float *__restrict__ mixes, int n, int s, int dim) {
    const int t = blockIdx.x, i = ((int)blockIdx.y * 256 + (int)threadIdx.x) * 4;
    if (i >= dim) return;
    const float *cur = h + (size_t)t * dim, *bef = t ? cur - dim : prev;
    const v4f c = *(const v4f *)(cur + i), d = *(const v4f *)(bef + i) - c;
#pragma unroll 5
    for (int m = 0; m < n; ++m) {
        const v4f f = *(const v4f *)(mu + (size_t)m * dim + i);
        v4f r;
#pragma unroll
        for (int e = 0; e < 4; ++e) r[e] = fmaf(d[e], f[e], c[e]);
        *(v4f *)(mixes + ((size_t)m * s + t) * dim + i) = r;
    }
    if (t == s - 1) *(v4f *)(next + i) = c;
}

int launch_token_shift(lumen_ctx *ctx, const float *h, const float *mu, const float *prev, float *next, float *mixes, int n,
                       int s, int dim) {
    if (s <= 0 || dim <= 0) return LUMEN_OK;
    const bool vec = dim % 4 == 0 && (((uintptr_t)h | (uintptr_t)mu | (uintptr_t)prev | (uintptr_t)next | (uintptr_t)mixes) & 15) == 0;
    if (vec)
        hipLaunchKernelGGL(token_shift_vec_kernel, dim3(s, (dim + 1023) / 1024), dim3(256), 0, ctx->stream, h, mu, prev, next, mixes, n, s, dim);
    else
        hipLaunchKernelGGL(token_shift_kernel, dim3(s), dim3(256), 0, ctx->stream, h, mu, prev, next, mixes, n, s, dim);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

__global__ __launch_bounds__(256) void add_steps_kernel(const float *__restrict__ base, const float *__restrict__ step,
                                                        float *__restrict__ out, int rows, int dim) {
    const size_t r = blockIdx.x;
    const int t = blockIdx.y;
    for (int i = threadIdx.x; i < dim; i += 256) out[((size_t)t * rows + r) * dim + i] = base[r * dim + i] + step[(size_t)t * dim + i];
}

int launch_add_steps(lumen_ctx *ctx, const float *base, const float *step, float *out, int times, int rows, int dim) {
    if (times <= 0 || rows <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(add_steps_kernel, dim3(rows, times), dim3(256), 0, ctx->stream, base, step, out, rows, dim);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

__global__ __launch_bounds__(256) void gather_rows_kernel(const float *__restrict__ x, const int *__restrict__ idx,
                                                          float *__restrict__ out, int dim) {
    const float *src = x + (size_t)idx[blockIdx.x] * dim;
    float *dst = out + (size_t)blockIdx.x * dim;
    for (int i = threadIdx.x; i < dim; i += 256) dst[i] = src[i];
}

int launch_gather_rows(lumen_ctx *ctx, const float *x, const int *idx, float *out, int n, int dim) {
    if (n <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(gather_rows_kernel, dim3(n), dim3(256), 0, ctx->stream, x, idx, out, dim);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// out [rows][n] = tanh of columns [0, n) of rows with the given stride
__global__ __launch_bounds__(256) void tanh_rows_kernel(const float *__restrict__ x, int stride, float *__restrict__ out, int rows, int n) {
    const size_t total = (size_t)rows * n;
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) out[i] = tanhf(x[i / n * stride + i % n]);
}
int launch_tanh_rows(lumen_ctx *ctx, const float *x, int stride, float *out, int rows, int n) {
    if (rows <= 0 || n <= 0) return LUMEN_OK;
    const size_t blocks = ((size_t)rows * n + 255) / 256, most = (size_t)ctx->num_cus * 8;
    hipLaunchKernelGGL(tanh_rows_kernel, dim3((unsigned)(blocks < most ? blocks : most)), dim3(256), 0, ctx->stream, x, stride, out, rows, n);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// Token vectors plus position vectors: row t is W[ids[t]] + P[pos0 + t] (pos0 from device memory where pos_dev is given);
// both indexes are clamped to their tables.
__global__ __launch_bounds__(256) void embedding_pos_kernel(const float *__restrict__ W, const int *__restrict__ ids, const float *__restrict__ P,
                                                            const int *__restrict__ pos_dev, int pos0, int dim, int vocab, int positions,
                                                            float *__restrict__ out) {
    const int id = min(max(ids[blockIdx.x], 0), vocab - 1);
    const int pos = min((pos_dev ? *pos_dev : pos0) + (int)blockIdx.x, positions - 1);
    const float *src = W + (size_t)id * dim, *add = P + (size_t)pos * dim;
    for (int i = threadIdx.x; i < dim; i += 256) out[(size_t)blockIdx.x * dim + i] = src[i] + add[i];
}
int launch_embedding_pos(lumen_ctx *ctx, const float *W, const int *ids_dev, const float *P, const int *pos_dev, int pos0, int n, int dim, int vocab,
                         int positions, float *out) {
    if (n <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(embedding_pos_kernel, dim3(n), dim3(256), 0, ctx->stream, W, ids_dev, P, pos_dev, pos0, dim, vocab, positions, out);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ---------------------------------------------------------------- embedding
// out[t, :] = W[ids[t], :], src/layers/basic/embedding.rs:47-57.  ids were
// range-checked on the host; the device clamps so that a stale id can never
// read outside the table.
__global__ __launch_bounds__(256) void embedding_kernel(const float *__restrict__ W, const int *__restrict__ ids,
                                                        int dim, int vocab, float *__restrict__ out) {
    int id = ids[blockIdx.x];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    const float *src = W + (size_t)id * dim;
    float *dst = out + (size_t)blockIdx.x * dim;
    for (int i = threadIdx.x; i < dim; i += 256) dst[i] = src[i];
}

int launch_embedding(lumen_ctx *ctx, const float *W, const int *ids_dev, int n, int dim, int vocab, float *out) {
    if (n <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(embedding_kernel, dim3(n), dim3(256), 0, ctx->stream, W, ids_dev, dim, vocab, out);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ------------------------------------------------------------------- argmax
// Single workgroup; first index of the maximum (lowest index wins ties).
__global__ __launch_bounds__(1024) void argmax_kernel(const float *__restrict__ x, int n, int *__restrict__ out,
                                                      int *__restrict__ pos_inc) {
    __shared__ float bv[16];
    __shared__ int bi[16];
    const int tid = threadIdx.x;
    float best = -INFINITY;
    int idx = 0x7fffffff;
    for (int i = tid; i < n; i += 1024) {
        const float v = x[i];
        if (v > best || (v == best && i < idx)) {
            best = v;
            idx = i;
        }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
        const float ov = __shfl_xor(best, off, 64);
        const int oi = __shfl_xor(idx, off, 64);
        if (ov > best || (ov == best && oi < idx)) {
            best = ov;
            idx = oi;
        }
    }
    if ((tid & 63) == 0) {
        bv[tid >> 6] = best;
        bi[tid >> 6] = idx;
    }
    __syncthreads();
    if (tid == 0) {
        for (int w = 1; w < 16; ++w)
            if (bv[w] > best || (bv[w] == best && bi[w] < idx)) {
                best = bv[w];
                idx = bi[w];
            }
        if (idx == 0x7fffffff) idx = 0;  // all NaN / -inf: index 0 like a sequential scan
        *out = idx;
        if (pos_inc) *pos_inc += 1;
    }
}

int launch_argmax(lumen_ctx *ctx, const float *x, int n, int *out_dev, int *pos_inc_dev) {
    hipLaunchKernelGGL(argmax_kernel, dim3(1), dim3(1024), 0, ctx->stream, x, n, out_dev, pos_inc_dev);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// --------------------------------------------------------------------- RoPE
// freq = 1 / theta^(2j/dim), val = pos * freq, cos/sin in f32, both halves
// alike: src/layers/attention/encoding.rs:29-54.  Computed on the host with
// libm so that the table holds the same values as the reference's.
void rope_tables_host(std::vector<float> &cos_t, std::vector<float> &sin_t, int dim, int max_seq, float theta) {
    const int half = dim / 2;
    cos_t.assign((size_t)max_seq * dim, 0.f);
    sin_t.assign((size_t)max_seq * dim, 0.f);
    std::vector<float> freq(half);
    for (int j = 0; j < half; ++j) freq[j] = 1.0f / powf(theta, ((float)j * 2.0f) / (float)dim);
    for (int i = 0; i < max_seq; ++i) {
        const float pos = (float)i;
        for (int j = 0; j < half; ++j) {
            const float val = pos * freq[j];
            const float c = cosf(val), s = sinf(val);
            cos_t[(size_t)i * dim + j] = c;
            cos_t[(size_t)i * dim + j + half] = c;
            sin_t[(size_t)i * dim + j] = s;
            sin_t[(size_t)i * dim + j + half] = s;
        }
    }
}

// x, out [B*H, S, D]: out[j] = x1*c - x2*s, out[j+half] = x2*c + x1*s (encoding.rs:103-116)
__global__ __launch_bounds__(256) void rope_bhsd_kernel(const float *__restrict__ x, float *__restrict__ out,
                                                        const float *__restrict__ cos_t,
                                                        const float *__restrict__ sin_t, int s, int d, int offset,
                                                        size_t npairs) {
    const int half = d / 2;
    const size_t stride = (size_t)gridDim.x * blockDim.x;
    for (size_t p = (size_t)blockIdx.x * blockDim.x + threadIdx.x; p < npairs; p += stride) {
        const int j = (int)(p % half);
        const size_t row = p / half;  // (b*h, s) flattened
        const int ss = (int)(row % s);
        const float *xr = x + row * d;
        const float x1 = xr[j], x2 = xr[j + half];
        const float c = cos_t[(size_t)(offset + ss) * d + j];
        const float sv = sin_t[(size_t)(offset + ss) * d + j];
        {
#pragma clang fp contract(off)  // separate multiplies and add, like the reference's compiled code
            out[row * d + j] = x1 * c - x2 * sv;
            out[row * d + j + half] = x2 * c + x1 * sv;
        }
    }
}

int launch_rope_bhsd(lumen_ctx *ctx, const float *x, float *out, const float *cos_t, const float *sin_t, int b, int h,
                     int s, int d, int offset) {
    const size_t npairs = (size_t)b * h * s * (d / 2);
    if (npairs == 0) return LUMEN_OK;
    size_t blocks = (npairs + 255) / 256;
    const size_t cap = (size_t)ctx->num_cus * 16;
    if (blocks > cap) blocks = cap;
    hipLaunchKernelGGL(rope_bhsd_kernel, dim3((unsigned)blocks), dim3(256), 0, ctx->stream, x, out, cos_t, sin_t, s, d,
                       offset, npairs);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ---------------------------------------------------------------------- C ABI
extern "C" int lumen_rmsnorm_f32(lumen_ctx *ctx, const float *x, const float *w, float *out, int rows, int dim,
                                 float eps) {
    if (!ctx || !x || !w || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "rmsnorm: null argument");
    if (rows < 0 || dim < 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "rmsnorm: negative dimension");
    return launch_rmsnorm(ctx, x, w, out, rows, dim, eps);
}

#define EW_ABI1(name, fn)                                                                 \
    extern "C" int name(lumen_ctx *ctx, const float *x, float *out, size_t n) {           \
        if (!ctx || ((!x || !out) && n)) LUMEN_FAIL(LUMEN_ERR_INVALID, #name ": null argument"); \
        return fn(ctx, x, out, n);                                                        \
    }
#define EW_ABI2(name, fn)                                                                         \
    extern "C" int name(lumen_ctx *ctx, const float *a, const float *b, float *out, size_t n) {   \
        if (!ctx || ((!a || !b || !out) && n)) LUMEN_FAIL(LUMEN_ERR_INVALID, #name ": null argument"); \
        return fn(ctx, a, b, out, n);                                                             \
    }
EW_ABI1(lumen_silu_f32, launch_silu)
EW_ABI1(lumen_copy_f32, launch_copy)
EW_ABI2(lumen_add_f32, launch_add)
EW_ABI2(lumen_mul_f32, launch_mul)
EW_ABI2(lumen_swiglu_f32, launch_swiglu)

extern "C" int lumen_embedding_f32(lumen_ctx *ctx, const float *W, const float *ids_host, int n_ids, int vocab,
                                   int dim, float *out) {
    if (!ctx || !W || (!ids_host && n_ids) || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "embedding: null argument");
    if (n_ids <= 0) return LUMEN_OK;
    std::vector<int> ids(n_ids);
    for (int t = 0; t < n_ids; ++t) {
        const float f = ids_host[t];
        // Rust `as usize`: truncates toward zero, saturates, NaN -> 0 (embedding.rs:50)
        long long idx = (f > 0.0f) ? (f >= 9.0e18f ? (long long)9e18 : (long long)f) : 0;
        if (idx >= vocab)  // embedding.rs:55
            LUMEN_FAIL(LUMEN_ERR_EMBED_OOB, "Embedding index out of bounds: %lld >= %d", idx, vocab);
        ids[t] = (int)idx;
    }
    int *ids_dev = nullptr;
    HIP_TRY(hipMalloc((void **)&ids_dev, sizeof(int) * (size_t)n_ids));
    hipError_t e = hipMemcpyAsync(ids_dev, ids.data(), sizeof(int) * (size_t)n_ids, hipMemcpyHostToDevice, ctx->stream);
    int rc = LUMEN_OK;
    if (e == hipSuccess) rc = launch_embedding(ctx, W, ids_dev, n_ids, dim, vocab, out);
    hipStreamSynchronize(ctx->stream);
    hipFree(ids_dev);
    if (e != hipSuccess) LUMEN_FAIL(LUMEN_ERR_HIP, "embedding: id upload failed: %s", hipGetErrorString(e));
    return rc;
}

extern "C" int lumen_argmax_f32(lumen_ctx *ctx, const float *x, int n, int *index_host_out) {
    if (!ctx || !x || !index_host_out) LUMEN_FAIL(LUMEN_ERR_INVALID, "argmax: null argument");
    if (n <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "argmax: empty input");
    LUMEN_TRY(launch_argmax(ctx, x, n, ctx->d_scratch_int, nullptr));
    HIP_TRY(hipMemcpyAsync(index_host_out, ctx->d_scratch_int, sizeof(int), hipMemcpyDeviceToHost, ctx->stream));
    HIP_TRY(hipStreamSynchronize(ctx->stream));
    return LUMEN_OK;
}

extern "C" int lumen_rope_create(lumen_ctx *ctx, int dim, int max_seq, float theta, lumen_rope **out) {
    if (!ctx || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "rope_create: null argument");
    if (dim <= 0 || (dim & 1) || max_seq <= 0) LUMEN_FAIL(LUMEN_ERR_SHAPE, "rope_create: dim=%d max_seq=%d", dim, max_seq);
    lumen_rope *r = new lumen_rope();
    r->ctx = ctx; r->dim = dim; r->max_seq = max_seq; r->theta = theta;
    rope_tables_host(r->cos_host, r->sin_host, dim, max_seq, theta);
    const size_t bytes = sizeof(float) * (size_t)max_seq * dim;
    if (hipMalloc((void **)&r->cos_dev, bytes) != hipSuccess || hipMalloc((void **)&r->sin_dev, bytes) != hipSuccess) {
        hipFree(r->cos_dev);
        delete r;
        LUMEN_FAIL(LUMEN_ERR_HIP, "rope_create: hipMalloc of %zu bytes failed", bytes);
    }
    int rc = lumen_upload(ctx, r->cos_dev, r->cos_host.data(), bytes);
    if (rc == LUMEN_OK) rc = lumen_upload(ctx, r->sin_dev, r->sin_host.data(), bytes);
    if (rc != LUMEN_OK) { lumen_rope_destroy(r); return rc; }
    *out = r;
    return LUMEN_OK;
}

extern "C" int lumen_rope_destroy(lumen_rope *r) {
    if (!r) return LUMEN_OK;
    hipStreamSynchronize(r->ctx->stream);
    hipFree(r->cos_dev);
    hipFree(r->sin_dev);
    delete r;
    return LUMEN_OK;
}

extern "C" int lumen_rope_tables_download(lumen_rope *r, float *cos_host, float *sin_host) {
    if (!r || !cos_host || !sin_host) LUMEN_FAIL(LUMEN_ERR_INVALID, "rope_tables_download: null argument");
    const size_t bytes = sizeof(float) * (size_t)r->max_seq * r->dim;
    LUMEN_TRY(lumen_download(r->ctx, cos_host, r->cos_dev, bytes));
    return lumen_download(r->ctx, sin_host, r->sin_dev, bytes);
}

extern "C" int lumen_rope_forward_f32(lumen_rope *r, const float *x, float *out, int b, int h, int s, int d, int offset) {
    if (!r || !x || !out) LUMEN_FAIL(LUMEN_ERR_INVALID, "rope_forward: null argument");
    if (d != r->dim) LUMEN_FAIL(LUMEN_ERR_SHAPE, "RoPE dimension mismatch: %d vs %d", d, r->dim);  // encoding.rs:60
    if (offset < 0 || s < 0 || offset + s > r->max_seq)  // encoding.rs:62-68
        LUMEN_FAIL(LUMEN_ERR_ROPE_RANGE, "RoPE index out of range: offset %d + len %d > max %d", offset, s, r->max_seq);
    return launch_rope_bhsd(r->ctx, x, out, r->cos_dev, r->sin_dev, b, h, s, d, offset);
}

extern "C" int lumen_rope_1token_copy_f32(lumen_rope *r, const float *src, float *dst, int d, int pos) {
    if (!r || !src || !dst) LUMEN_FAIL(LUMEN_ERR_INVALID, "rope_1token_copy: null argument");
    if (d != r->dim) LUMEN_FAIL(LUMEN_ERR_SHAPE, "RoPE src len mismatch: %d vs %d", d, r->dim);  // encoding.rs:174-175
    if (pos < 0 || pos >= r->max_seq)  // encoding.rs:176-181
        LUMEN_FAIL(LUMEN_ERR_ROPE_RANGE, "RoPE index out of range: pos %d >= max %d", pos, r->max_seq);
    return launch_rope_bhsd(r->ctx, src, dst, r->cos_dev, r->sin_dev, 1, 1, 1, d, pos);
}

LUMEN_DEFINE_WARM(elementwise)
