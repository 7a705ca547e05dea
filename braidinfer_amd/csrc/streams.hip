// Residual rows kept as several streams: a token's row is [S][W] floats.  A half of a layer reads one weighted sum of the
// streams and writes its output y back into all of them:
//
//     u = sum_s in[s] x_s;    x_t <- sum_s mix[s, t] x_s + out[t] y    (all t from the old streams)
//
// A connection's coefficients lie as floats in | out | mix, [S] + [S] + [S][S] (mix indexed [from][to]).  All of it is
// element by element over W, so writing a half's output back, the sum the next half reads and a norm that is element by
// element too, h = tanh(alpha u) w + b, are one pass over the row (`join`).
#include "common.h"

#define ST_MAX 16      // streams

// What follows the weighted sum: nothing (w null: h is u itself) or tanh(alpha u) w + b.
struct PointNorm { const float *alpha, *w, *b; };

template <typename T, int VEC>
__device__ __forceinline__ void st_norm_store(const PointNorm& p, int c, float* u, T* h) {
    if (p.w) {
        const float alpha = p.alpha[0];
        float w[VEC], b[VEC];
        ew_load<float, VEC>(p.w + c, w);
        ew_load<float, VEC>(p.b + c, b);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = fmaf(tanhf(alpha * u[e]), w[e], b[e]);
    }
    ew_store<T, VEC>(h, u);
}

// X[t][s] = x[t] for every stream.
template <int VEC>
__global__ __launch_bounds__(256) void streams_spread_kernel(const float* __restrict__ x, float* __restrict__ X, int S, int W, size_t n) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * VEC;
    if (i >= n) return;
    const size_t t = i / W, c = i - t * W;
    float v[VEC];
    ew_load<float, VEC>(x + i, v);
    for (int s = 0; s < S; ++s) ew_store<float, VEC>(X + (t * S + s) * W + c, v);
}

// h[r] = norm(sum_s in[s] X[row][s]) for row = rows[r] (or r); `in` null: the plain sum.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void streams_open_kernel(const float* __restrict__ X, const int* __restrict__ rows, const float* __restrict__ in,
                                                           PointNorm norm, T* __restrict__ h, int S, int W, size_t n) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * VEC;
    if (i >= n) return;
    const size_t r = i / W;
    const int c = (int)(i - r * W);
    const float* xr = X + (size_t)(rows ? rows[r] : (int)r) * S * W + c;
    float u[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) u[e] = 0.f;
    for (int s = 0; s < S; ++s) {
        float v[VEC];
        ew_load<float, VEC>(xr + (size_t)s * W, v);
        const float a = in ? in[s] : 1.0f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = fmaf(a, v[e], u[e]);
    }
    st_norm_store<T, VEC>(norm, c, u, h + i);
}

// A half's output: scale1 (y1 + bias1) + scale2 (y2 + bias2); biases [W] and y2 may be absent.
struct HalfOut { const float *y1, *b1, *y2, *b2; float s1, s2; };

template <int VEC>
__device__ __forceinline__ void st_add_branch(const float* __restrict__ y, const float* __restrict__ b, float scale, size_t i, int c, float* acc) {
    float v[VEC];
    ew_load<float, VEC>(y + i, v);
    if (b) {
        float bv[VEC];
        ew_load<float, VEC>(b + c, bv);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] += bv[e];
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = fmaf(scale, v[e], acc[e]);
}

// The half's output into the streams in place; with `h`, h = norm(sum_s next_in[s] x_s) of the new streams.  SN: streams
// (EXACT), or the most there may be.
template <int SN, bool EXACT, typename T, int VEC>
__global__ __launch_bounds__(256) void streams_join_kernel(float* __restrict__ X, const float* __restrict__ coef, HalfOut y,
                                                           const float* __restrict__ next_in, PointNorm norm, T* __restrict__ h, int S_, int W, size_t n) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * VEC;
    if (i >= n) return;
    const int S = EXACT ? SN : S_;
    const size_t t = i / W;
    const int c = (int)(i - t * W);
    float yv[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) yv[e] = 0.f;
    st_add_branch<VEC>(y.y1, y.b1, y.s1, i, c, yv);
    if (y.y2) st_add_branch<VEC>(y.y2, y.b2, y.s2, i, c, yv);
    float x[SN][VEC];
    float* xr = X + t * S * W + c;
#pragma unroll
    for (int s = 0; s < SN; ++s)
        if (EXACT || s < S) ew_load<float, VEC>(xr + (size_t)s * W, x[s]);
    float u[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) u[e] = 0.f;
    const float *out = coef + S, *mix = coef + 2 * S;
#pragma unroll
    for (int to = 0; to < SN; ++to) {
        if (!EXACT && to >= S) break;
        float v[VEC];
        const float o = out[to];
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = o * yv[e];
#pragma unroll
        for (int s = 0; s < SN; ++s) {
            if (!EXACT && s >= S) break;
            const float a = mix[s * S + to];
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[e] = fmaf(a, x[s][e], v[e]);
        }
        ew_store<float, VEC>(xr + (size_t)to * W, v);
        if (h) {
            const float a = next_in ? next_in[to] : 1.0f;
#pragma unroll
            for (int e = 0; e < VEC; ++e) u[e] = fmaf(a, v[e], u[e]);
        }
    }
    if (h) st_norm_store<T, VEC>(norm, c, u, h + i);
}

static inline bool st_at16(const void* a) { return ((uintptr_t)a % 16) == 0; }
static inline bool st_grid(size_t n, int vec, unsigned* blocks) {
    const size_t b = (n / (size_t)vec + 255) / 256;
    *blocks = (unsigned)b;
    return b > 0 && b <= 0x7fffffffULL;
}

extern "C" int br_streams_spread(const float* x, float* X, int T, int S, int W, hipStream_t s) {
    if (T <= 0) return BR_OK;
    if (S < 1 || S > ST_MAX || W <= 0) return BR_BAD_ARG;
    const size_t n = (size_t)T * W;
    const bool vec = W % 4 == 0 && st_at16(x) && st_at16(X);
    unsigned blocks;
    if (!st_grid(n, vec ? 4 : 1, &blocks)) return BR_BAD_ARG;
    if (vec) streams_spread_kernel<4><<<blocks, 256, 0, s>>>(x, X, S, W, n);
    else streams_spread_kernel<1><<<blocks, 256, 0, s>>>(x, X, S, W, n);
    return br_check_launch();
}

// R rows out; `rows` (or null) picks the streams' rows.
extern "C" int br_streams_open(const float* X, const int* rows, const float* in, const float* alpha, const float* w, const float* b, void* h,
                               int h_is_bf16, int R, int S, int W, hipStream_t s) {
    if (R <= 0) return BR_OK;
    if (S < 1 || S > ST_MAX || W <= 0 || (w && (!alpha || !b))) return BR_BAD_ARG;
    const size_t n = (size_t)R * W;
    const PointNorm norm = {alpha, w, b};
    const bool vec = W % 4 == 0 && st_at16(X) && st_at16(w) && st_at16(b) && st_at16(h);
    unsigned blocks;
    if (!st_grid(n, vec ? 4 : 1, &blocks)) return BR_BAD_ARG;
    if (h_is_bf16) {
        if (vec) streams_open_kernel<bf16, 4><<<blocks, 256, 0, s>>>(X, rows, in, norm, (bf16*)h, S, W, n);
        else streams_open_kernel<bf16, 1><<<blocks, 256, 0, s>>>(X, rows, in, norm, (bf16*)h, S, W, n);
    } else {
        if (vec) streams_open_kernel<float, 4><<<blocks, 256, 0, s>>>(X, rows, in, norm, (float*)h, S, W, n);
        else streams_open_kernel<float, 1><<<blocks, 256, 0, s>>>(X, rows, in, norm, (float*)h, S, W, n);
    }
    return br_check_launch();
}

// `h` null: nothing behind the streams; else with `next_in` (null: the plain sum) and the norm (w null: none).
extern "C" int br_streams_join(float* X, const float* coef, const float* y1, const float* b1, float s1, const float* y2, const float* b2,
                               float s2, const float* next_in, const float* alpha, const float* w, const float* b, void* h, int h_is_bf16,
                               int T, int S, int W, hipStream_t s) {
    if (T <= 0) return BR_OK;
    if (S < 1 || S > ST_MAX || W <= 0 || !y1 || !coef || (b2 && !y2) || (w && (!alpha || !b))) return BR_BAD_ARG;
    const size_t n = (size_t)T * W;
    const PointNorm norm = {alpha, w, b};
    const HalfOut y = {y1, b1, y2, b2, s1, s2};
    const bool vec = W % 4 == 0 && st_at16(X) && st_at16(y1) && st_at16(y2) && st_at16(b1) && st_at16(b2) && st_at16(w) && st_at16(b) && st_at16(h);
    unsigned blocks;
    if (!st_grid(n, vec ? 4 : 1, &blocks)) return BR_BAD_ARG;
#define ST_JOIN(SN, EX) do { \
        if (h_is_bf16) { \
            if (vec) streams_join_kernel<SN, EX, bf16, 4><<<blocks, 256, 0, s>>>(X, coef, y, next_in, norm, (bf16*)h, S, W, n); \
            else streams_join_kernel<SN, EX, bf16, 1><<<blocks, 256, 0, s>>>(X, coef, y, next_in, norm, (bf16*)h, S, W, n); \
        } else { \
            if (vec) streams_join_kernel<SN, EX, float, 4><<<blocks, 256, 0, s>>>(X, coef, y, next_in, norm, (float*)h, S, W, n); \
            else streams_join_kernel<SN, EX, float, 1><<<blocks, 256, 0, s>>>(X, coef, y, next_in, norm, (float*)h, S, W, n); \
        } \
    } while (0)
    switch (S) {
        case 1: ST_JOIN(1, true); break;
        case 2: ST_JOIN(2, true); break;
        case 3: ST_JOIN(3, true); break;
        case 4: ST_JOIN(4, true); break;
        default: if (S <= 8) ST_JOIN(8, false); else ST_JOIN(16, false);
    }
#undef ST_JOIN
    return br_check_launch();
}
