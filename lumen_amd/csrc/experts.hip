// Mixture of experts: the router's choice, the chosen experts' products for one token (decode), and for a prompt the
// tokens sorted by expert and multiplied tile by tile (launch_gemm_grouped).  Scores, weights and sums are f32.
#include <algorithm>

#include "mixers.h"
#include "wave_reduce.h"

typedef float v4f __attribute__((ext_vector_type(4)));
typedef unsigned int v4u __attribute__((ext_vector_type(4)));

// One wavefront's choice for one token: its LDS accesses execute in order, so its phases need no workgroup barrier (the wave
// barrier emits no instruction; it keeps the compiler from moving LDS accesses across it).  An expert's place is the number of
// better ones (ties: the lower index first), so no choice waits for the one before; every index in `sel` is valid
// whatever the logits are.
struct RouteLds {
    float s[EXPERTS_MAX], group[EXPERTS_MAX];
    int kept[EXPERTS_MAX];
    int sel[EXPERTS_MAX_TOP];
    float w[EXPERTS_MAX_TOP];
};
__device__ __forceinline__ void route_token(RouteLds &l, const RouterShape &r, const float *__restrict__ z) {
    const int lane = threadIdx.x & 63, size = r.experts / r.groups;
    for (int e = lane; e < r.experts; e += 64) l.s[e] = 1.0f / (1.0f + expf(-z[e]));
    if (lane < r.top) {
        l.sel[lane] = 0;
        l.w[lane] = 0.f;
    }
    __builtin_amdgcn_wave_barrier();
    if (r.groups > r.keep) {
        for (int g = lane; g < r.groups; g += 64) {
            float a = -INFINITY, b = 0.f;  // the two largest (a group of one counts its one)
            for (int i = 0; i < size; ++i) {
                const float v = l.s[g * size + i];
                b = v > a ? (i ? a : 0.f) : fmaxf(v, b);
                a = fmaxf(v, a);
            }
            l.group[g] = a + b;
        }
        __builtin_amdgcn_wave_barrier();
        for (int g = lane; g < r.groups; g += 64) {
            int better = 0;
            for (int o = 0; o < r.groups; ++o) better += l.group[o] > l.group[g] || (l.group[o] == l.group[g] && o < g);
            l.kept[g] = better < r.keep;
        }
        __builtin_amdgcn_wave_barrier();
        // (an expert that cannot be chosen: below every score)
        for (int e = lane; e < r.experts; e += 64)
            if (!l.kept[e / size]) l.s[e] = -1.f;
        __builtin_amdgcn_wave_barrier();
    }
    for (int e = lane; e < r.experts; e += 64) {
        const float mine = l.s[e];
        int better = 0;
#pragma unroll 8
        for (int o = 0; o < r.experts; ++o) better += l.s[o] > mine || (l.s[o] == mine && o < e);
        if (better < r.top && mine >= 0.f) {
            l.sel[better] = e;
            l.w[better] = mine;
        }
    }
    __builtin_amdgcn_wave_barrier();
    const float w = lane < r.top ? l.w[lane] : 0.f;
    const float sum = wave_sum(w);
    if (lane < r.top) l.w[lane] = w / (sum + 1e-20f) * r.scale;
    __builtin_amdgcn_wave_barrier();
}

__global__ __launch_bounds__(64) void route_kernel(RouterShape r, const float *__restrict__ z, int z_stride, int *__restrict__ sel,
                                                   float *__restrict__ sel_w) {
    __shared__ RouteLds l;
    route_token(l, r, z + (size_t)blockIdx.x * z_stride);
    for (int j = threadIdx.x; j < r.top; j += 64) {
        sel[(size_t)blockIdx.x * r.top + j] = l.sel[j];
        sel_w[(size_t)blockIdx.x * r.top + j] = l.w[j];
    }
}
int launch_route(lumen_ctx *ctx, const RouterShape &r, const float *z, int z_stride, int rows, int *sel, float *sel_w) {
    if (rows <= 0) return LUMEN_OK;
    hipLaunchKernelGGL(route_kernel, dim3(rows), dim3(64), 0, ctx->stream, r, z, z_stride, sel, sel_w);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

// ------------------------------------------------------------------ decode
#define ED_THREADS 256
#define ED_WAVES (ED_THREADS / 64)
#define ED_LOADS 8  // 16-byte loads in flight per lane

template <bool BF16>
__device__ __forceinline__ float dot16_e(const v4u raw, const float *xs) {
    const v4f a = *(const v4f *)xs;
    if (BF16) {
        const v4f b = *(const v4f *)(xs + 4);
        float s = __uint_as_float(raw.x << 16) * a.x;
        s = fmaf(__uint_as_float(raw.x & 0xffff0000u), a.y, s);
        s = fmaf(__uint_as_float(raw.y << 16), a.z, s);
        s = fmaf(__uint_as_float(raw.y & 0xffff0000u), a.w, s);
        s = fmaf(__uint_as_float(raw.z << 16), b.x, s);
        s = fmaf(__uint_as_float(raw.z & 0xffff0000u), b.y, s);
        s = fmaf(__uint_as_float(raw.w << 16), b.z, s);
        return fmaf(__uint_as_float(raw.w & 0xffff0000u), b.w, s);
    }
    float s = __uint_as_float(raw.x) * a.x;
    s = fmaf(__uint_as_float(raw.y), a.y, s);
    s = fmaf(__uint_as_float(raw.z), a.z, s);
    return fmaf(__uint_as_float(raw.w), a.w, s);
}

// A wavefront takes one (expert, channel) at a time: its gate and up rows, ED_LOADS / 2 pieces of each in flight.  Every
// workgroup routes (one wavefront) and normalises (the others) for itself; the first one leaves the choice for the down product.
template <bool BF16>
__global__ __launch_bounds__(ED_THREADS) void experts_up_kernel(ExpertsArgs a) {
    constexpr int VEC = BF16 ? 8 : 4, ESZ = BF16 ? 2 : 4, SWEEP = 64 * VEC, U = ED_LOADS / 2;
    __shared__ RouteLds l;
    LUMEN_DYNAMIC_LDS(float, xs);
    const int tid = threadIdx.x, lane = tid & 63, K = a.dim, F = a.ff, kpad = (K + SWEEP * U - 1) / (SWEEP * U) * (SWEEP * U);
    const float alpha = *a.norm_alpha;
    if (tid < 64) route_token(l, a.r, a.z);  // the first wavefront routes, the others normalise
    for (int k = (tid - 64) * 4; k < kpad && tid >= 64; k += (ED_THREADS - 64) * 4) {
        v4f v = {0.f, 0.f, 0.f, 0.f};
        if (k < K) {
            const v4f x = *(const v4f *)(a.x + k), g = *(const v4f *)(a.norm_w + k), b = *(const v4f *)(a.norm_b + k);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = fmaf(tanhf(alpha * x[e]), g[e], b[e]);
        }
        *(v4f *)(xs + k) = v;
    }
    __syncthreads();
    if (blockIdx.x == 0 && tid < a.r.top) a.sel[tid] = l.sel[tid];
    const int units = a.r.top * F, nw = gridDim.x * ED_WAVES;
    const size_t row_bytes = (size_t)K * ESZ;
    auto load = [&](int u, int k0, v4u (&raw)[2][U]) {
        const int j = u / F, f = u - j * F;
        const char *row = (const char *)a.w_up + ((size_t)l.sel[j] * 2 * F + 2 * f) * row_bytes;
#pragma unroll
        for (int r = 0; r < 2; ++r)
#pragma unroll
            for (int i = 0; i < U; ++i)
                raw[r][i] = __builtin_nontemporal_load((const v4u *)(row + r * row_bytes + (size_t)min(k0 + i * SWEEP + lane * VEC, K - VEC) * ESZ));
    };
    // two pieces in flight: while one is multiplied the next one travels
    v4u ra[2][U], rb[2][U];
    float acc[2] = {0.f, 0.f};
    int lu = blockIdx.x * ED_WAVES + (tid >> 6), lk = 0, u = lu, k0 = 0;
    auto advance = [&]() {
        lk += SWEEP * U;
        if (lk >= kpad) {
            lk = 0;
            lu += nw;
        }
    };
    auto consume = [&](const v4u (&raw)[2][U]) {
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
            for (int r = 0; r < 2; ++r) acc[r] += dot16_e<BF16>(raw[r][i], xs + k0 + i * SWEEP + lane * VEC);
        k0 += SWEEP * U;
        if (k0 >= kpad) {
            const float g = wave_sum(acc[0]), up = wave_sum(acc[1]);
            if (lane == 0) a.act[u] = expert_act(g, up, a.limit) * l.w[u / F];
            acc[0] = acc[1] = 0.f;
            k0 = 0;
            u += nw;
        }
    };
    if (lu >= units) return;
    load(lu, lk, ra);
    advance();
    while (u < units) {
        if (lu < units) load(lu, lk, rb);
        advance();
        consume(ra);
        if (u >= units) break;
        if (lu < units) load(lu, lk, ra);
        advance();
        consume(rb);
    }
}

// y = x + sigmoid(gate + gate_b) * sum over the chosen experts of W_down act (weights are in act): a wavefront per row, the
// experts' rows read as one of top * ff elements.
template <bool BF16>
__global__ __launch_bounds__(ED_THREADS) void experts_down_kernel(ExpertsArgs a) {
    constexpr int VEC = BF16 ? 8 : 4, ESZ = BF16 ? 2 : 4, SWEEP = 64 * VEC, U = ED_LOADS;
    __shared__ size_t base[EXPERTS_MAX_TOP];
    LUMEN_DYNAMIC_LDS(float, xs);
    const int tid = threadIdx.x, lane = tid & 63, F = a.ff, K = a.r.top * F, N = a.dim, kpad = (K + SWEEP * U - 1) / (SWEEP * U) * (SWEEP * U);
    if (tid < a.r.top) base[tid] = (size_t)a.sel[tid] * N * F;
    for (int k = tid * 4; k < kpad; k += ED_THREADS * 4) *(v4f *)(xs + k) = k < K ? *(const v4f *)(a.act + k) : v4f{0.f, 0.f, 0.f, 0.f};
    __syncthreads();
    const unsigned magic = 0xffffffffu / (unsigned)F + 1u;  // (p / F for p * F < 2^32; F = 1 never: a multiple of 8)
    auto load = [&](int n, int k0, v4u (&raw)[U]) {
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int p = min(k0 + i * SWEEP + lane * VEC, K - VEC), j = (int)__umulhi((unsigned)p, magic);
            raw[i] = __builtin_nontemporal_load((const v4u *)((const char *)a.w_down + (base[j] + (size_t)n * F + (p - j * F)) * ESZ));
        }
    };
    const int nw = gridDim.x * ED_WAVES;
    v4u ra[U], rb[U];
    float acc = 0.f;
    int ln = blockIdx.x * ED_WAVES + (tid >> 6), lk = 0, n = ln, k0 = 0;
    auto advance = [&]() {
        lk += SWEEP * U;
        if (lk >= kpad) {
            lk = 0;
            ln += nw;
        }
    };
    auto consume = [&](const v4u (&raw)[U]) {
#pragma unroll
        for (int i = 0; i < U; ++i) acc += dot16_e<BF16>(raw[i], xs + k0 + i * SWEEP + lane * VEC);
        k0 += SWEEP * U;
        if (k0 >= kpad) {
            acc = wave_sum(acc);
            if (lane == 0) a.y[n] = fmaf(1.0f / (1.0f + expf(-(a.gate[n] + a.gate_b[n]))), acc, a.x[n]);
            acc = 0.f;
            k0 = 0;
            n += nw;
        }
    };
    if (ln >= N) return;
    load(ln, lk, ra);
    advance();
    while (n < N) {
        if (ln < N) load(ln, lk, rb);
        advance();
        consume(ra);
        if (n >= N) break;
        if (ln < N) load(ln, lk, ra);
        advance();
        consume(rb);
    }
}

// Workgroups for `units` wavefront units: one round over the compute units, every wavefront the same number of units.
static int expert_blocks(const lumen_ctx *ctx, int units, size_t lds) {
    int per_cu = (int)((size_t)(160 * 1024) / (lds + 256));
    per_cu = per_cu > 4 ? 4 : per_cu < 1 ? 1 : per_cu;
    const int cap = ctx->num_cus * per_cu * ED_WAVES;
    const int per_wave = (units + cap - 1) / cap;
    return (units + per_wave * ED_WAVES - 1) / (per_wave * ED_WAVES);
}

template <typename K>
static int launch_expert_kernel(lumen_ctx *ctx, K kernel, const ExpertsArgs &a, int units, int k, int piece) {
    const size_t dyn = (size_t)((k + piece - 1) / piece * piece) * sizeof(float);
    if (dyn + sizeof(RouteLds) > 150 * 1024) LUMEN_FAIL(LUMEN_ERR_UNSUPPORTED, "experts: a vector of %d does not fit the stage", k);
    if (dyn + sizeof(RouteLds) > 64 * 1024)
        HIP_TRY(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)dyn));
    hipLaunchKernelGGL(kernel, dim3(expert_blocks(ctx, units, dyn + sizeof(RouteLds))), dim3(ED_THREADS), dyn, ctx->stream, a);
    LUMEN_CHECK_LAUNCH();
    return LUMEN_OK;
}

int launch_experts_up(lumen_ctx *ctx, const ExpertsArgs &a) {
    note_kernel(ctx, "experts_up_kernel<%s>", a.w_bf16 ? "true" : "false");
    const int units = a.r.top * a.ff, piece = 64 * (a.w_bf16 ? 8 : 4) * ED_LOADS / 2;
    return a.w_bf16 ? launch_expert_kernel(ctx, experts_up_kernel<true>, a, units, a.dim, piece)
                    : launch_expert_kernel(ctx, experts_up_kernel<false>, a, units, a.dim, piece);
}

int launch_experts_down(lumen_ctx *ctx, const ExpertsArgs &a) {
    note_kernel(ctx, "experts_down_kernel<%s>", a.w_bf16 ? "true" : "false");
    const int piece = 64 * (a.w_bf16 ? 8 : 4) * ED_LOADS;
    return a.w_bf16 ? launch_expert_kernel(ctx, experts_down_kernel<true>, a, a.dim, a.r.top * a.ff, piece)
                    : launch_expert_kernel(ctx, experts_down_kernel<false>, a, a.dim, a.r.top * a.ff, piece);
}

// ------------------------------------------------------------------ prompt
// plan: sel [s * top] | a_rows [s * top] | c_rows [s * top] | tiles [max_tiles][3]
// Rows of a tile by the mean number of tokens an expert gets: a few and the products are a matter of reading the experts'
// weights (the streaming kernel's 16 rows), more and the matrix cores' 128-row tiles take them (8 of 32 experts of width
// 512 on rows of 2048, prompt passes of 16 / 64 / 96 tokens: 2.8 / 3.9 / 4.5 ms with the former, 3.5 / 4.1 / 4.3 with the latter;
// 32 streamed rows are never the best).
#define EXPERTS_STREAM_ROWS 16
static int group_rows(int s, const RouterShape &r) { return (long)s * r.top <= (long)EXPERTS_STREAM_ROWS * r.experts ? 16 : 128; }
static int plan_tiles(int s, const RouterShape &r, int rows) { return (int)(((long)s * r.top + rows - 1) / rows) + std::min(r.experts, s * r.top); }
// (for up to s tokens)
size_t experts_plan_ints(int s, const RouterShape &r) { return (size_t)3 * s * r.top + (size_t)3 * plan_tiles(s, r, 16); }

// One workgroup: counts per expert, where each expert's rows start, the tiles, and every (token, choice)'s row.  The order
// of an expert's rows is whatever the counters give out; no row's values depend on it.
#define PLAN_THREADS 1024
__global__ __launch_bounds__(PLAN_THREADS) void experts_plan_kernel(int *plan, int n, int top, int experts, int max_tiles, int tile_rows) {
    __shared__ int count[EXPERTS_MAX], start[EXPERTS_MAX + 1], tile0[EXPERTS_MAX + 1];
    const int tid = threadIdx.x;
    const int *sel = plan;
    int *a_rows = plan + n, *c_rows = plan + 2 * (size_t)n, *tiles = plan + 3 * (size_t)n;
    for (int e = tid; e < experts; e += PLAN_THREADS) count[e] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += PLAN_THREADS) atomicAdd(&count[sel[i]], 1);
    __syncthreads();
    if (tid < 64) {  // prefix sums over the experts, 64 at a time
        int rows = 0, tl = 0;
        for (int e0 = 0; e0 < experts; e0 += 64) {
            const int e = e0 + tid, c = e < experts ? count[e] : 0, t = (c + tile_rows - 1) / tile_rows;
            int sc = c, st = t;
#pragma unroll
            for (int d = 1; d < 64; d <<= 1) {
                const int pc = __shfl_up(sc, d, 64), pt = __shfl_up(st, d, 64);
                if (tid >= d) {
                    sc += pc;
                    st += pt;
                }
            }
            if (e < experts) {
                start[e] = rows + sc - c;
                tile0[e] = tl + st - t;
            }
            rows += __shfl(sc, 63, 64);
            tl += __shfl(st, 63, 64);
        }
        if (tid == 0) tile0[experts] = tl;
    }
    __syncthreads();
    for (int e = tid; e < experts; e += PLAN_THREADS)
        for (int r = 0, t = tile0[e]; r < count[e] && t < max_tiles; r += tile_rows, ++t) {
            tiles[3 * t] = e;
            tiles[3 * t + 1] = start[e] + r;
            tiles[3 * t + 2] = min(tile_rows, count[e] - r);
        }
    for (int t = tile0[experts] + tid; t < max_tiles; t += PLAN_THREADS) tiles[3 * t] = tiles[3 * t + 1] = tiles[3 * t + 2] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += PLAN_THREADS) {
        const int row = atomicAdd(&start[sel[i]], 1);
        a_rows[row] = i / top;
        c_rows[row] = i;
    }
}

int launch_experts_prefill(lumen_ctx *ctx, const ExpertsArgs &a) {
    if (a.s <= 0) return LUMEN_OK;
    const int n = a.s * a.r.top, rows = group_rows(a.s, a.r), max_tiles = plan_tiles(a.s, a.r, rows);
    LUMEN_TRY(launch_route(ctx, a.r, a.z, a.z_stride, a.s, a.plan, a.sel_w));
    hipLaunchKernelGGL(experts_plan_kernel, dim3(1), dim3(PLAN_THREADS), 0, ctx->stream, a.plan, n, a.r.top, a.r.experts, max_tiles, rows);
    LUMEN_CHECK_LAUNCH();
    GemmArgs g = {};
    g.w_bf16 = a.w_bf16; g.group_rows = rows; g.M = n; g.tiles = a.plan + 3 * (size_t)n;
    g.A = a.rows; g.a_rows = a.plan + n; g.W = a.w_up; g.C = a.p_act; g.N = 2 * a.ff; g.K = a.dim; g.epi = EPI_EXPERT_ACT; g.limit = a.limit;
    LUMEN_TRY(launch_gemm_grouped(ctx, g, max_tiles));
    g.A = a.p_act; g.a_rows = nullptr; g.c_rows = a.plan + 2 * (size_t)n; g.W = a.w_down; g.C = a.out; g.N = a.dim; g.K = a.ff; g.epi = EPI_STORE;
    return launch_gemm_grouped(ctx, g, max_tiles);
}

LUMEN_DEFINE_WARM(experts)
