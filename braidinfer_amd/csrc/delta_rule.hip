// Recurrences over an outer-product state with one decay number per head and token, state in float:
// for a head with d key channels and e value channels (S is d x e, starts at zero),
//
//     gated delta rule:   S <- g_t S;  u_t = beta_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
//     decayed outer sum:  S <- g S + k_t v_t^T;                                            o_t = S^T q_t
//     weighted outer sum: S <- g_t S + b_t k_t v_t^T;                                      o_t = S^T q_t (+ D v_t)
//
// (the read-out sees the current token's write in all).  The delta rule's g_t is one number a head, or one a head and key
// channel (diag(g_t) S).  The weighted sum may carry one more column whose value is 1 for every token, i.e. the sum n of
// the weighted keys, and gives n^T q_t beside o_t.  Column c of S follows
// S[:, c] <- g S[:, c] + k (beta (v[c] - k . S[:, c])) and never meets another column, so the work is cut by
// (sequence, head, 16 columns) and walked like the other recurrences of this library: the state lies in a slot
// as `glr_scan_kernel` keeps it, a lane holds RPL rows of one column in registers, the tokens' rows come TC at a
// time through two LDS stages with the next chunk in flight, and a token costs a lane two sums over its 16 row
// groups (k . S for the correction, q . S for the read-out) by moves between neighbouring lanes in a fixed order.
//
// Beside the scan: `conv_prepare` (a short causal convolution over time per channel with the last inputs kept per
// sequence, silu, unit length per head, the decay and the write strength from their float sums), `ssm_prepare` (the
// convolution with a bias and silu alone, the decay and the step size of a state-space layer), `conv_keep` (the inputs a
// sequence's next step needs) and `exp_gates` (exponential input and sigmoid forget gates over a running maximum).
#include "common.h"

#define DR_MAX_EPL 8      // head widths up to 64 * DR_MAX_EPL
#define DR_MAX_TAPS 16

__device__ __forceinline__ float dr_row16_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));
    return v;
}

__device__ __forceinline__ float dr_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float dr_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ------------------------------------------------------------------- prepare -------
// rows [T, width] float, the projections' sums: q (G heads of d) | k (G of d) | v (H of e) | b (H) | a (H) | ...
// One wave per (token, head row) with head rows = G query heads, G key heads, H value heads; four waves a workgroup.  Channel ch of the
// C = 2 G d + H e convolved channels is column ch of `rows`; taps [C, n] float, the last column the current token's;
// `kept` holds per slot the last n - 1 inputs of every channel, [n - 1][C] (zeros in a new slot).
// Out: qo, ko [T, G d] (silu, unit length per head, q times d^-1/2), vo [T, H e] (silu), gb [T, 2 H]:
// g = exp(-exp(A_log) softplus(a + dt_bias)) then beta = sigmoid(b).
// With `z` (float rows `z_stride` apart, H heads of d) there is one decay a head and key channel: no a columns, dt_bias
// [H d], H more head rows turn z into gc [T, H d] = exp(-exp(A_log_head) softplus(z + dt_bias)), and gb holds beta alone (its
// second half).  A sequence that brings one token leaves its inputs in its slot here (only the lane that owns a channel
// reads or writes that channel's kept inputs); the others by `conv_keep` behind this kernel.
__global__ __launch_bounds__(256) void dr_conv_prepare_kernel(
    const float* __restrict__ rows, int width, const float* __restrict__ taps, int n_taps,
    float* kept, size_t kept_stride, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const int* __restrict__ seq_of_token, const int* __restrict__ cu_seqlens,
    const int* __restrict__ slots, float* __restrict__ qo, float* __restrict__ ko, float* __restrict__ vo,
    float* __restrict__ gb, int T, int G, int H, int d, int e, const float* __restrict__ z, size_t z_stride,
    float* __restrict__ gc) {
    const int n_hr = 2 * G + H + (z ? H : 0);
    const long long unit = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);          // a wave a (token, head row)
    if (unit >= (long long)T * n_hr) return;
    const int t = (int)(unit / n_hr), hr = (int)(unit - (long long)t * n_hr), lane = threadIdx.x & 63;
    if (hr >= 2 * G + H) {                          // a head's decays
        const int head = hr - 2 * G - H;
        const float a = expf(a_log[head]);
        for (int i = lane; i < d; i += 64)
            gc[((size_t)t * H + head) * d + i] = expf(-a * dr_softplus(z[(size_t)t * z_stride + head * d + i] + dt_bias[head * d + i]));
        return;
    }
    const bool is_q = hr < G, is_k = !is_q && hr < 2 * G;
    const int head = is_q ? hr : (is_k ? hr - G : hr - 2 * G);
    const int n = (is_q || is_k) ? d : e;
    const int C = 2 * G * d + H * e;
    const int col0 = is_q ? head * d : (is_k ? G * d + head * d : 2 * G * d + head * e);
    const int b = seq_of_token[t];
    const int slot = slots[b], t0 = cu_seqlens[b];
    const int i_in_step = t - t0;
    float v[DR_MAX_EPL];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < DR_MAX_EPL; ++j) {
        const int i = lane + 64 * j;
        v[j] = 0.f;
        if (i < n) {
            const int ch = col0 + i;
            float acc = 0.f;
            for (int x = 0; x < n_taps; ++x) {
                const int ii = i_in_step - (n_taps - 1) + x;          // the input's place in the step
                float in;
                if (ii >= 0) in = rows[(size_t)(t0 + ii) * width + ch];
                else in = slot >= 0 ? kept[(size_t)slot * kept_stride + (size_t)(n_taps - 1 + ii) * C + ch] : 0.f;
                acc = fmaf(taps[(size_t)ch * n_taps + x], in, acc);
            }
            if (slot >= 0 && cu_seqlens[b + 1] - t0 == 1 && n_taps > 1) {
                float* st = kept + (size_t)slot * kept_stride + ch;
                for (int x = 0; x + 1 < n_taps; ++x)
                    st[(size_t)x * C] = x + 2 < n_taps ? st[(size_t)(x + 1) * C] : rows[(size_t)t * width + ch];
            }
            v[j] = dr_silu(acc);
            ss = fmaf(v[j], v[j], ss);
        }
    }
    float mult = 1.f;
    if (is_q || is_k) {
        mult = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
        if (is_q) mult *= 1.0f / sqrtf((float)d);
    }
    float* dst = is_q ? qo + (size_t)t * G * d + head * d : (is_k ? ko + (size_t)t * G * d + head * d
                                                                   : vo + (size_t)t * H * e + head * e);
#pragma unroll
    for (int j = 0; j < DR_MAX_EPL; ++j) {
        const int i = lane + 64 * j;
        if (i < n) dst[i] = v[j] * mult;
    }
    if (!is_q && !is_k && lane == 0) {
        const float braw = rows[(size_t)t * width + C + head];
        if (!z) {
            const float araw = rows[(size_t)t * width + C + H + head] + dt_bias[head];
            gb[(size_t)t * 2 * H + head] = expf(-expf(a_log[head]) * dr_softplus(araw));
        }
        gb[(size_t)t * 2 * H + H + head] = 1.0f / (1.0f + expf(-braw));
    }
}

// The same with four channels a lane through 16-byte loads, for widths that are multiples of 4 (d, e, `width`, the kept
// rows' stride; 16-byte aligned pointers): `taps_t` [n, C] holds the taps with the channels side by side.  LPH lanes a
// (token, head row), 64 / LPH of them a wave: 16 lanes for heads of up to 64 channels, 32 up to 128, else 64.
template <int LPH>
__global__ __launch_bounds__(256) void dr_conv_prepare_vec_kernel(
    const float* __restrict__ rows, int width, const float* __restrict__ taps_t, int n_taps,
    float* kept, size_t kept_stride, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const int* __restrict__ seq_of_token, const int* __restrict__ cu_seqlens,
    const int* __restrict__ slots, float* __restrict__ qo, float* __restrict__ ko, float* __restrict__ vo,
    float* __restrict__ gb, int T, int G, int H, int d, int e, const float* __restrict__ z, size_t z_stride,
    float* __restrict__ gc) {
    constexpr int NJ = LPH == 64 ? DR_MAX_EPL / 4 : 1;
    const int n_hr = 2 * G + H + (z ? H : 0);
    const int lane = threadIdx.x & 63, l = lane % LPH;
    const long long unit = ((long long)blockIdx.x * 4 + (threadIdx.x >> 6)) * (64 / LPH) + lane / LPH;
    const bool on = unit < (long long)T * n_hr;          // lanes behind the last row go along for the sums and write nothing
    const int t = on ? (int)(unit / n_hr) : 0, hr = on ? (int)(unit - (long long)t * n_hr) : 0;
    const bool is_decay = hr >= 2 * G + H;          // a head's decays: its lanes go along for the sums with nothing in them
    if (on && is_decay) {
        const int head = hr - 2 * G - H;
        const float a = expf(a_log[head]);
        for (int i = 4 * l; i < d; i += 4 * LPH) {
            const f32x4 zv = *(const f32x4*)(z + (size_t)t * z_stride + head * d + i), bv = *(const f32x4*)(dt_bias + head * d + i);
            f32x4 out;
#pragma unroll
            for (int c = 0; c < 4; ++c) out[c] = expf(-a * dr_softplus(zv[c] + bv[c]));
            *(f32x4*)(gc + ((size_t)t * H + head) * d + i) = out;
        }
    }
    const bool is_q = hr < G, is_k = !is_q && hr < 2 * G;
    const int head = is_q ? hr : (is_k ? hr - G : hr - 2 * G);
    const int n = (is_q || is_k) ? d : e;
    const int C = 2 * G * d + H * e;
    const int col0 = is_q ? head * d : (is_k ? G * d + head * d : 2 * G * d + head * e);
    const int b = seq_of_token[t];
    const int slot = slots[b], t0 = cu_seqlens[b];
    const int i_in_step = t - t0;
    f32x4 v[NJ];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = 4 * l + 4 * LPH * j;
        v[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (on && !is_decay && i < n) {
            const int ch = col0 + i;
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
            for (int x = 0; x < n_taps; ++x) {
                const int ii = i_in_step - (n_taps - 1) + x;          // the input's place in the step
                f32x4 in = {0.f, 0.f, 0.f, 0.f};
                if (ii >= 0) in = *(const f32x4*)(rows + (size_t)(t0 + ii) * width + ch);
                else if (slot >= 0) in = *(const f32x4*)(kept + (size_t)slot * kept_stride + (size_t)(n_taps - 1 + ii) * C + ch);
                const f32x4 w = *(const f32x4*)(taps_t + (size_t)x * C + ch);
#pragma unroll
                for (int c = 0; c < 4; ++c) acc[c] = fmaf(w[c], in[c], acc[c]);
            }
            if (slot >= 0 && cu_seqlens[b + 1] - t0 == 1 && n_taps > 1) {
                float* st = kept + (size_t)slot * kept_stride + ch;
                for (int x = 0; x + 1 < n_taps; ++x)
                    *(f32x4*)(st + (size_t)x * C) = x + 2 < n_taps ? *(const f32x4*)(st + (size_t)(x + 1) * C) : *(const f32x4*)(rows + (size_t)t * width + ch);
            }
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                v[j][c] = dr_silu(acc[c]);
                ss = fmaf(v[j][c], v[j][c], ss);
            }
        }
    }
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);          // over the row's lanes, in a fixed order
    if (!on || is_decay) return;
    float mult = 1.f;
    if (is_q || is_k) {
        mult = 1.0f / sqrtf(ss + 1e-6f);
        if (is_q) mult *= 1.0f / sqrtf((float)d);
    }
    float* dst = is_q ? qo + (size_t)t * G * d + head * d : (is_k ? ko + (size_t)t * G * d + head * d
                                                                   : vo + (size_t)t * H * e + head * e);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = 4 * l + 4 * LPH * j;
        if (i < n) {
            f32x4 out;
#pragma unroll
            for (int c = 0; c < 4; ++c) out[c] = v[j][c] * mult;
            *(f32x4*)(dst + i) = out;
        }
    }
    if (!is_q && !is_k && l == 0) {
        const float braw = rows[(size_t)t * width + C + head];
        if (!z) {
            const float araw = rows[(size_t)t * width + C + H + head] + dt_bias[head];
            gb[(size_t)t * 2 * H + head] = expf(-expf(a_log[head]) * dr_softplus(araw));
        }
        gb[(size_t)t * 2 * H + H + head] = 1.0f / (1.0f + expf(-braw));
    }
}

// After the step: the last n - 1 inputs of every sequence that brought more than one token into its slot (one token's
// inputs are put there by the kernel that reads them).  grid (B, ceil(C / 256)).
__global__ __launch_bounds__(256) void dr_conv_keep_kernel(const float* __restrict__ rows, int width, int n_taps,
                                                           float* __restrict__ kept, size_t kept_stride,
                                                           const int* __restrict__ cu_seqlens,
                                                           const int* __restrict__ slots, int C) {
    const int b = blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
    const int slot = slots[b];
    if (ch >= C || slot < 0) return;
    const int t0 = cu_seqlens[b], n_new = cu_seqlens[b + 1] - t0, keep = n_taps - 1;
    if (n_new == 1) return;
    float* st = kept + (size_t)slot * kept_stride + ch;
    float old[DR_MAX_TAPS];
    for (int j = 0; j < keep; ++j) old[j] = st[(size_t)j * C];
    for (int j = 0; j < keep; ++j) {
        const int ii = n_new - keep + j;
        st[(size_t)j * C] = ii >= 0 ? rows[(size_t)(t0 + ii) * width + ch] : old[keep + ii];
    }
}

// `single_tokens`: no sequence brings more than one token (nothing is left to `conv_keep`).
extern "C" int br_dr_conv_prepare(const float* rows, int width, const float* taps, const float* taps_t, int n_taps, float* kept,
                                  size_t kept_stride, const float* a_log, const float* dt_bias, const int* seq_of_token,
                                  const int* cu_seqlens, const int* slots, float* qo, float* ko, float* vo, float* gb,
                                  const float* z, size_t z_stride, float* gc, int T, int B, int G, int H, int d, int e,
                                  int single_tokens, hipStream_t s) {
    if (T <= 0 || B <= 0) return BR_OK;
    const long long C = 2LL * G * d + (long long)H * e;
    if (G <= 0 || H <= 0 || H % G || d <= 0 || e <= 0 || d > 64 * DR_MAX_EPL || e > 64 * DR_MAX_EPL || n_taps < 1 ||
        n_taps > DR_MAX_TAPS || width < C + (z ? 1 : 2) * H || ((long long)T * (2 * G + 2 * H) + 3) / 4 > 0x7fffffffLL || B > 65535 ||
        (C + 255) / 256 > 65535 || (z && (!gc || z_stride < (size_t)H * d)) ||
        (n_taps > 1 && (!kept || kept_stride < (size_t)(n_taps - 1) * C)) || !a_log || !dt_bias)
        return BR_BAD_ARG;
    const long long head_rows = (long long)T * (2 * G + (z ? 2 : 1) * H);
    const unsigned blocks = (unsigned)((head_rows + 3) / 4);
    auto at16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool vec = taps_t && d % 4 == 0 && e % 4 == 0 && width % 4 == 0 && at16(rows) && at16(taps_t) && at16(qo) && at16(ko) &&
                     at16(vo) && (n_taps == 1 || (kept_stride % 4 == 0 && at16(kept))) &&
                     (!z || (at16(z) && at16(gc) && at16(dt_bias) && z_stride % 4 == 0));
    if (vec) {
        const int widest = d > e ? d : e, lph = widest <= 64 ? 16 : (widest <= 128 ? 32 : 64);
        const unsigned vblocks = (unsigned)((head_rows + 4 * (64 / lph) - 1) / (4 * (64 / lph)));
#define DR_PREP(L) dr_conv_prepare_vec_kernel<L><<<vblocks, 256, 0, s>>>(rows, width, taps_t, n_taps, kept, kept_stride, a_log, dt_bias, \
                                                                        seq_of_token, cu_seqlens, slots, qo, ko, vo, gb, T, G, H, d, e, z, z_stride, gc)
        if (lph == 16) DR_PREP(16); else if (lph == 32) DR_PREP(32); else DR_PREP(64);
#undef DR_PREP
    }
    else dr_conv_prepare_kernel<<<blocks, 256, 0, s>>>(rows, width, taps, n_taps, kept, kept_stride, a_log, dt_bias, seq_of_token,
                                                 cu_seqlens, slots, qo, ko, vo, gb, T, G, H, d, e, z, z_stride, gc);
    int rc = br_check_launch();
    if (rc != BR_OK || n_taps == 1 || single_tokens) return rc;
    dr_conv_keep_kernel<<<dim3(B, (unsigned)((C + 255) / 256)), 256, 0, s>>>(rows, width, n_taps, kept, kept_stride, cu_seqlens,
                                                                           slots, (int)C);
    return br_check_launch();
}

// ------------------------------------------------- a state-space layer's inputs -----
// x float rows `width` apart, C convolved channels (the caller's pointer stands at the first): out [T, C] = silu(the causal
// convolution over time per channel + bias), taps_t [n, C] with the current token's last, `kept` as in `conv_prepare`.
// dt float rows `width` apart, H heads: with s = softplus(dt + dt_bias), gb [T, 2 H] takes exp(-exp(A_log) s), then s.
// A thread VEC channels of a token, or a head of a token behind them.
template <int VEC>
__global__ __launch_bounds__(256) void ssm_prepare_kernel(
    const float* __restrict__ x, size_t width, const float* __restrict__ taps_t, const float* __restrict__ bias, int n_taps, float* kept,
    size_t kept_stride, const float* __restrict__ dt, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    const int* __restrict__ seq_of_token, const int* __restrict__ cu_seqlens, const int* __restrict__ slots, float* __restrict__ out,
    float* __restrict__ gb, int C, int H, size_t total) {
    typedef float vec_t __attribute__((ext_vector_type(VEC)));
    const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= total) return;
    const unsigned per = (unsigned)(C / VEC + H);
    const size_t t = idx / per;
    const int r = (int)(idx - t * per);
    if (r >= C / VEC) {
        const int h = r - C / VEC;
        const float s = dr_softplus(dt[t * width + h] + dt_bias[h]);
        gb[t * 2 * H + h] = expf(-expf(a_log[h]) * s);
        gb[t * 2 * H + H + h] = s;
        return;
    }
    const int ch = r * VEC;
    const int b = seq_of_token[t];
    const int slot = slots[b], t0 = cu_seqlens[b], t1 = cu_seqlens[b + 1];
    const int i_in_step = (int)t - t0;
    float acc[VEC];
#pragma unroll
    for (int c = 0; c < VEC; ++c) acc[c] = bias ? bias[ch + c] : 0.f;
    for (int j = 0; j < n_taps; ++j) {
        const int ii = i_in_step - (n_taps - 1) + j;
        float in[VEC];
#pragma unroll
        for (int c = 0; c < VEC; ++c) in[c] = 0.f;
        const float* src = ii >= 0 ? x + (size_t)(t0 + ii) * width + ch
                                   : (slot >= 0 ? kept + (size_t)slot * kept_stride + (size_t)(n_taps - 1 + ii) * C + ch : nullptr);
        if (src) {
            const vec_t v = *(const vec_t*)src;
#pragma unroll
            for (int c = 0; c < VEC; ++c) in[c] = ((const float*)&v)[c];
        }
        const vec_t w = *(const vec_t*)(taps_t + (size_t)j * C + ch);
#pragma unroll
        for (int c = 0; c < VEC; ++c) acc[c] = fmaf(((const float*)&w)[c], in[c], acc[c]);
    }
    if (slot >= 0 && t1 - t0 == 1 && n_taps > 1) {
        float* st = kept + (size_t)slot * kept_stride + ch;
        for (int j = 0; j + 1 < n_taps; ++j)
            *(vec_t*)(st + (size_t)j * C) = j + 2 < n_taps ? *(const vec_t*)(st + (size_t)(j + 1) * C) : *(const vec_t*)(x + t * width + ch);
    }
    vec_t o;
#pragma unroll
    for (int c = 0; c < VEC; ++c) ((float*)&o)[c] = dr_silu(acc[c]);
    *(vec_t*)(out + t * C + ch) = o;
}

extern "C" int br_ssm_prepare(const float* x, size_t width, const float* taps_t, const float* bias, int n_taps, float* kept,
                              size_t kept_stride, const float* dt, const float* a_log, const float* dt_bias,
                              const int* seq_of_token, const int* cu_seqlens, const int* slots, float* out, float* gb, int T, int B,
                              int C, int H, int single_tokens, hipStream_t s) {
    if (T <= 0 || B <= 0) return BR_OK;
    if (C <= 0 || H <= 0 || n_taps < 1 || n_taps > DR_MAX_TAPS || width < (size_t)C || width > 0x7fffffff || B > 65535 || (C + 255) / 256 > 65535 ||
        (n_taps > 1 && (!kept || kept_stride < (size_t)(n_taps - 1) * C)) || !dt || !a_log || !dt_bias)
        return BR_BAD_ARG;
    auto at16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool vec = C % 4 == 0 && width % 4 == 0 && at16(x) && at16(taps_t) && at16(out) &&
                     (n_taps == 1 || (kept_stride % 4 == 0 && at16(kept)));
    const size_t total = (size_t)T * (size_t)((vec ? C / 4 : C) + H), blocks = (total + 255) / 256;
    if (blocks > 0x7fffffffULL) return BR_BAD_ARG;
    if (vec) ssm_prepare_kernel<4><<<(unsigned)blocks, 256, 0, s>>>(x, width, taps_t, bias, n_taps, kept, kept_stride, dt, a_log, dt_bias, seq_of_token, cu_seqlens, slots, out, gb, C, H, total);
    else ssm_prepare_kernel<1><<<(unsigned)blocks, 256, 0, s>>>(x, width, taps_t, bias, n_taps, kept, kept_stride, dt, a_log, dt_bias, seq_of_token, cu_seqlens, slots, out, gb, C, H, total);
    int rc = br_check_launch();
    if (rc != BR_OK || n_taps == 1 || single_tokens) return rc;
    dr_conv_keep_kernel<<<dim3(B, (unsigned)((C + 255) / 256)), 256, 0, s>>>(x, (int)width, n_taps, kept, kept_stride, cu_seqlens, slots, C);
    return br_check_launch();
}

// ------------------------------------------------------- exponential gates ----------
// Per head the logarithms of an input and a forget gate from their float sums, i = cap tanh((zi + bi) / cap) and
// f = log sigmoid(cap tanh((zf + bf) / cap)), and the running maximum m_t = max(f_t + m_(t-1), i_t) that a memory of
// exponential gates is kept relative to (a slot keeps the last m; 0 in a new one).  gb [T, 2 H] takes
// exp(f_t + m_(t-1) - m_t), then exp(i_t - m_t); m [T, H] the maxima.  m is a prefix of the maps m -> max(m + a, b), one a
// token: composed across a wave's 64 tokens and, in long steps, across the WAVES waves of a workgroup (64 tokens each at a
// time) through LDS.  grid (B, H), 64 WAVES threads.
template <int WAVES>
__global__ __launch_bounds__(64 * WAVES) void exp_gates_kernel(const float* __restrict__ zi, const float* __restrict__ zf, size_t stride,
                                                               const float* __restrict__ bi, const float* __restrict__ bf, float cap,
                                                               float* kept, size_t kept_stride, const int* __restrict__ cu_seqlens,
                                                               const int* __restrict__ slots, float* __restrict__ gb,
                                                               float* __restrict__ m_out, int H) {
    __shared__ float wa[WAVES], wb[WAVES];
    const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int slot = slots[b], t0 = cu_seqlens[b], t1 = cu_seqlens[b + 1];
    float m0 = slot >= 0 ? kept[(size_t)slot * kept_stride + h] : 0.f;
    for (int tc = t0; tc < t1; tc += 64 * WAVES) {
        const int t = tc + (int)threadIdx.x;
        const bool on = t < t1;
        float i = -INFINITY, f = 0.f;
        if (on) {
            i = cap * tanhf((zi[(size_t)t * stride + h] + bi[h]) / cap);
            const float z = cap * tanhf((zf[(size_t)t * stride + h] + bf[h]) / cap);
            f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
        }
        float A = f, Bm = i;          // the map of the wave's tokens up to this one: m -> max(m + A, Bm)
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float pa = __shfl_up(A, o, WAVE), pb = __shfl_up(Bm, o, WAVE);
            if (lane >= o) { Bm = fmaxf(pb + A, Bm); A += pa; }
        }
        float start = m0;             // m in front of the wave's tokens
        if (WAVES > 1) {
            __syncthreads();
            if (lane == 63) { wa[wave] = A; wb[wave] = Bm; }
            __syncthreads();
#pragma unroll
            for (int w = 0; w < WAVES; ++w) {
                const float behind = fmaxf(m0 + wa[w], wb[w]);
                if (w < wave) start = behind;
                m0 = behind;
            }
        }
        const float m = fmaxf(start + A, Bm);
        float before = __shfl_up(m, 1, WAVE);
        if (lane == 0) before = start;
        if (on) {
            gb[(size_t)t * 2 * H + h] = expf(f + before - m);
            gb[(size_t)t * 2 * H + H + h] = expf(i - m);
            m_out[(size_t)t * H + h] = m;
        }
        if (WAVES == 1) m0 = __shfl(m, 63, WAVE);     // lanes behind the last token hold its m
    }
    if (threadIdx.x == 0 && slot >= 0) kept[(size_t)slot * kept_stride + h] = m0;
}

// `single_tokens`: no sequence brings more than one token (one wave a head).
extern "C" int br_exp_gates(const float* zi, const float* zf, size_t stride, const float* bi, const float* bf, float cap, float* kept,
                            size_t kept_stride, const int* cu_seqlens, const int* slots, float* gb, float* m_out, int B, int H,
                            int single_tokens, hipStream_t s) {
    if (B <= 0) return BR_OK;
    if (H <= 0 || H > 65535 || stride < (size_t)H || !(cap > 0.f) || !kept || kept_stride < (size_t)H || !bi || !bf) return BR_BAD_ARG;
    if (single_tokens) exp_gates_kernel<1><<<dim3(B, H), 64, 0, s>>>(zi, zf, stride, bi, bf, cap, kept, kept_stride, cu_seqlens, slots, gb, m_out, H);
    else exp_gates_kernel<16><<<dim3(B, H), 1024, 0, s>>>(zi, zf, stride, bi, bf, cap, kept, kept_stride, cu_seqlens, slots, gb, m_out, H);
    return br_check_launch();
}

// x[t, :n] <- silu(x[t, :n]) in place on float rows `stride` apart (projections' sums that go on as activations: done
// once here, not by every workgroup of a scan that reads them).  VEC: four a thread, for n, stride and pointer in fours.
template <bool VEC>
__global__ __launch_bounds__(256) void dr_silu_rows_kernel(float* __restrict__ x, size_t stride, int n, size_t total) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= total) return;
    if (VEC) {
        const size_t per = (size_t)n / 4, t = i / per, c = (i - t * per) * 4;
        f32x4* p = (f32x4*)(x + t * stride + c);
        f32x4 v = *p;
#pragma unroll
        for (int k = 0; k < 4; ++k) v[k] = dr_silu(v[k]);
        *p = v;
    } else {
        const size_t t = i / n, c = i - t * n;
        float* p = x + t * stride + c;
        *p = dr_silu(*p);
    }
}

extern "C" int br_silu_rows(float* x, size_t stride, int T, int n, hipStream_t s) {
    if (T <= 0 || n <= 0) return BR_OK;
    if (stride < (size_t)n) return BR_BAD_ARG;
    const bool vec = n % 4 == 0 && stride % 4 == 0 && ((uintptr_t)x % 16) == 0;
    const size_t total = vec ? (size_t)T * (n / 4) : (size_t)T * n;
    const size_t blocks = (total + 255) / 256;
    if (blocks > 0x7fffffffULL) return BR_BAD_ARG;
    if (vec) dr_silu_rows_kernel<true><<<(unsigned)blocks, 256, 0, s>>>(x, stride, n, total);
    else dr_silu_rows_kernel<false><<<(unsigned)blocks, 256, 0, s>>>(x, stride, n, total);
    return br_check_launch();
}

// q and k rows (float sums of their projections, rows `stride` apart, `heads` heads of d channels each) turned in place
// by their tokens' positions: of the first `rd` channels of a head, channel i < rd / 2 and channel i + rd / 2 form
// a pair that is turned by the angle whose cosine and sine are cs[t, i], sn[t, i] ((u, v) -> (u c - v s, v c + u s));
// the other channels pass.  Every channel of q is then multiplied by `q_mul` and every channel of k by `k_mul`.
// A thread a channel below rd / 2 (it owns the pair) or from rd on; grid over T * heads * (d - rd / 2) threads.
__global__ __launch_bounds__(256) void dr_rotate_rows_kernel(float* __restrict__ q, float* __restrict__ k, size_t stride,
                                                             const float* __restrict__ cs, const float* __restrict__ sn,
                                                             int rd, int heads, int d, float q_mul, float k_mul, size_t total) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= total) return;
    const int half = rd >> 1, per = d - half;
    const size_t th = i / per;
    const int j = (int)(i - th * per);
    const size_t t = th / heads;
    const int h = (int)(th - t * heads);
    float* qr = q + t * stride + (size_t)h * d;
    float* kr = k + t * stride + (size_t)h * d;
    if (j < half) {
        const float c = cs[t * half + j], s_ = sn[t * half + j];
        const float qu = qr[j], qv = qr[j + half], ku = kr[j], kv = kr[j + half];
        qr[j] = (qu * c - qv * s_) * q_mul;
        qr[j + half] = (qv * c + qu * s_) * q_mul;
        kr[j] = (ku * c - kv * s_) * k_mul;
        kr[j + half] = (kv * c + ku * s_) * k_mul;
    } else {
        const int ch = j + half;                    // channels from rd on
        qr[ch] *= q_mul;
        kr[ch] *= k_mul;
    }
}

extern "C" int br_dr_rotate_rows(float* q, float* k, size_t stride, const float* cs, const float* sn, int rd, int T, int heads,
                                 int d, float q_mul, float k_mul, hipStream_t s) {
    if (T <= 0) return BR_OK;
    if (heads <= 0 || d <= 0 || rd < 0 || (rd & 1) || rd > d || stride < (size_t)heads * d || (rd > 0 && (!cs || !sn))) return BR_BAD_ARG;
    const size_t total = (size_t)T * heads * (d - rd / 2);
    const size_t blocks = (total + 255) / 256;
    if (blocks > 0x7fffffffULL) return BR_BAD_ARG;
    dr_rotate_rows_kernel<<<(unsigned)blocks, 256, 0, s>>>(q, k, stride, cs, sn, rd, heads, d, q_mul, k_mul, total);
    return br_check_launch();
}

// ---------------------------------------------------------------------- scan -------
// q, k: float rows `qk_stride` apart, head kh's d channels at kh * d (kh = h / (H / G): G heads of keys serve H
// heads of values); v: rows `v_stride` apart, head h's e channels at h * e.  MODE:
//   DR_FIXED     the head's one decay `g_head[h]`, u = v
//   DR_DELTA     g and beta per token and head from `gb` (rows `gb_stride` apart, g at [h], beta at [H + h])
//   DR_CHANNELS  the delta rule with a decay per head and key channel from `gc` [T, H d], beta from `gb`
//   DR_WEIGHTED  g and the write's weight b from `gb`, u = b v; o gains skip[h] v where `skip` is given; with `ones` the
//                state has one column more, whose value is 1, and its read-out goes to `n_out` [T, H]
// SILU: q, k and v are the projections' float sums and pass silu on their way into LDS.
// grid (sequences, heads, ceil((e + ones) / 16)), 256 threads; a slot's state as `glr_state_shape` says for e + ones columns.
// LOCAL (the first pass over a long prompt cut into pieces, see `br_dr_scan_pieces`): the state starts at zero, nothing
// is written to o, and the last state goes to the piece's scratch; DR_WEIGHTED leaves the product of the piece's decays in
// `piece_decay` [sequences of the launch][H].
#define DR_FIXED 0
#define DR_DELTA 1
#define DR_WEIGHTED 2
#define DR_CHANNELS 3

struct DrScan {
    const float *q, *k, *v, *gb, *g_head, *gc, *skip;
    float *o, *n_out, *state, *piece_decay;
    const int *cu_seqlens, *slots;
    size_t qk_stride, v_stride, gb_stride, slot_stride;
    int H, G, d, e, ones;
};

template <int RPL, int TC, int MODE, bool SILU, bool LOCAL>
__global__ __launch_bounds__(256) void dr_scan_kernel(const DrScan p) {
    constexpr bool DELTA = MODE == DR_DELTA || MODE == DR_CHANNELS, CHAN = MODE == DR_CHANNELS;
    constexpr bool TOKEN_G = MODE != DR_FIXED;
    constexpr int DP = RPL * 16;
    constexpr int NL = TC * DP / 1024;
    extern __shared__ float lds[];
    float* kL = lds;                               // [2][TC][DP]
    float* qL = kL + 2 * TC * DP;                  // [2][TC][DP]
    float* vL = qL + 2 * TC * DP;                  // [2][TC][16]
    float* gL = vL + 2 * TC * 16;                  // [2][TC][2]
    float* cL = gL + 2 * TC * 2;                   // [2][TC][DP] (CHAN) the channels' decays
    const float* __restrict__ q = p.q;
    const float* __restrict__ k = p.k;
    const float* __restrict__ v = p.v;
    const float* __restrict__ gb = p.gb;
    const int H = p.H, d = p.d, e = p.e;
    const int s = blockIdx.x, h = blockIdx.y, cb16 = blockIdx.z;
    const int kh = h / (H / p.G);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cg = lane >> 4, g = lane & 15;
    const int cb4 = cb16 * 4 + wave, c = cb4 * 4 + cg;
    const int slot = p.slots[s];
    const int t0 = p.cu_seqlens[s], t1 = p.cu_seqlens[s + 1];
    const bool live = c < e, is_n = MODE == DR_WEIGHTED && p.ones && c == e;
    const int he = H * e;
    // where this lane's column is read out to: o's column, or the extra column's own array
    float* orow = is_n ? p.n_out + (size_t)t0 * H + h : p.o + (size_t)t0 * he + h * e + c;
    const size_t ostep = is_n ? H : he;
    const bool writes = !LOCAL && g == 0 && (live || is_n);
    if (slot < 0) {                                // padding: no state behind it; its rows of o are zero
        if (writes) for (int t = t0; t < t1; ++t, orow += ostep) orow[0] = 0.f;
        return;
    }
    const int ncb4 = (e + p.ones + 3) >> 2;
    float* S = p.state + (size_t)slot * p.slot_stride + (((size_t)h * ncb4 + cb4) * RPL) * 64 + lane;
    float st[RPL];
#pragma unroll
    for (int r = 0; r < RPL; ++r) st[r] = (!LOCAL && cb4 < ncb4) ? S[(size_t)r * 64] : 0.f;
    const float g_fixed = TOKEN_G ? 1.f : p.g_head[h];
    const float skip = (MODE == DR_WEIGHTED && p.skip && live) ? p.skip[h] : 0.f;
    float decayed = 1.f;                           // (LOCAL, DR_WEIGHTED) the product of the decays so far
    int l_tt[NL], l_r4[NL];
#pragma unroll
    for (int i = 0; i < NL; ++i) {
        const int idx = tid + 256 * i;
        l_tt[i] = idx / (DP / 4);
        l_r4[i] = (idx % (DP / 4)) * 4;
    }
    const int v_tt = tid >> 4, v_c = cb16 * 16 + (tid & 15);
    float rq[NL][4], rk[NL][4], rc[CHAN ? NL : 1][4], rv = 0.f, rg = 1.f;

    auto fetch = [&](int tc0) {
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            const int t = tc0 + l_tt[i];
            const float* qp = q + (size_t)t * p.qk_stride + kh * d + l_r4[i];
            const float* kp = k + (size_t)t * p.qk_stride + kh * d + l_r4[i];
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const bool ok = t < t1 && l_r4[i] + x < d;
                if (!LOCAL) rq[i][x] = ok ? qp[x] : 0.f;
                rk[i][x] = ok ? kp[x] : 0.f;
                if (CHAN) rc[CHAN ? i : 0][x] = ok ? p.gc[((size_t)t * H + h) * d + l_r4[i] + x] : 1.f;
            }
        }
        const int t = tc0 + v_tt;
        rv = (v_tt < TC && t < t1 && v_c < e) ? v[(size_t)t * p.v_stride + h * e + v_c] : 0.f;
        if (MODE == DR_WEIGHTED && p.ones && v_c == e) rv = 1.f;
        if (TOKEN_G) {
            // threads 0 .. 2 TC - 1 bring the chunk's decays and write strengths
            const int gt = tc0 + (tid >> 1);
            rg = (tid < 2 * TC && gt < t1) ? gb[(size_t)gt * p.gb_stride + (tid & 1) * H + h] : 1.f;
        }
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            f32x4 ko, qo, co;
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const bool real = l_r4[i] + x < d;       // rows behind d: key 0, query 0, so their state stays 0
                ko[x] = real ? (SILU ? dr_silu(rk[i][x]) : rk[i][x]) : 0.f;
                if (!LOCAL) qo[x] = real ? (SILU ? dr_silu(rq[i][x]) : rq[i][x]) : 0.f;
                if (CHAN) co[x] = rc[CHAN ? i : 0][x];
            }
            const size_t at = ((size_t)buf * TC + l_tt[i]) * DP + l_r4[i];
            *(f32x4*)(kL + at) = ko;
            if (!LOCAL) *(f32x4*)(qL + at) = qo;
            if (CHAN) *(f32x4*)(cL + at) = co;
        }
        if (v_tt < TC) vL[(buf * TC + v_tt) * 16 + (tid & 15)] = SILU ? dr_silu(rv) : rv;
        if (TOKEN_G && tid < 2 * TC) gL[buf * TC * 2 + tid] = rg;
    };

    fetch(t0);
    stage(0);
    __syncthreads();
    int buf = 0;
    for (int tc0 = t0; tc0 < t1; tc0 += TC) {
        const bool more = tc0 + TC < t1;
        if (more) fetch(tc0 + TC);
        const int nt = t1 - tc0 < TC ? t1 - tc0 : TC;
        const float* kp = kL + (size_t)buf * TC * DP + g * RPL;
        const float* qp = qL + (size_t)buf * TC * DP + g * RPL;
        const float* cp = cL + (size_t)buf * TC * DP + g * RPL;
        const float* vp = vL + buf * TC * 16 + wave * 4 + cg;
        const float* gp = gL + buf * TC * 2;
#pragma unroll 2
        for (int tt = 0; tt < nt; ++tt) {
            const float vc = vp[tt * 16];
            float kr[RPL];
#pragma unroll
            for (int k4 = 0; k4 < RPL / 4; ++k4) {
                const f32x4 kv4 = *(const f32x4*)(kp + (size_t)tt * DP + 4 * k4);
#pragma unroll
                for (int x = 0; x < 4; ++x) kr[4 * k4 + x] = kv4[x];
            }
            float u = vc;
            const float gt = CHAN ? 1.f : (TOKEN_G ? gp[2 * tt] : g_fixed);
            if (DELTA) {
                float part = 0.f;
#pragma unroll
                for (int k4 = 0; k4 < RPL / 4; ++k4) {
                    f32x4 gv = {gt, gt, gt, gt};
                    if (CHAN) gv = *(const f32x4*)(cp + (size_t)tt * DP + 4 * k4);
#pragma unroll
                    for (int x = 0; x < 4; ++x) {
                        const int r = 4 * k4 + x;
                        st[r] *= gv[x];
                        part = fmaf(st[r], kr[r], part);
                    }
                }
                u = gp[2 * tt + 1] * (vc - dr_row16_sum(part));
            } else if (MODE == DR_WEIGHTED) {
                u = gp[2 * tt + 1] * vc;
                if (LOCAL) decayed *= gt;
            }
            float sum = 0.f;
#pragma unroll
            for (int k4 = 0; k4 < RPL / 4; ++k4) {
                f32x4 qv4 = {0.f, 0.f, 0.f, 0.f};
                if (!LOCAL) qv4 = *(const f32x4*)(qp + (size_t)tt * DP + 4 * k4);
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    const int r = 4 * k4 + x;
                    st[r] = DELTA ? fmaf(kr[r], u, st[r]) : fmaf(gt, st[r], kr[r] * u);
                    if (!LOCAL) sum = fmaf(st[r], qv4[x], sum);
                }
            }
            if (!LOCAL) {
                sum = dr_row16_sum(sum);
                if (MODE == DR_WEIGHTED) sum = fmaf(skip, vc, sum);
                if (writes) orow[0] = sum;
                orow += ostep;
            }
        }
        if (more) stage(buf ^ 1);
        __syncthreads();
        buf ^= 1;
    }
    if (cb4 < ncb4) {
#pragma unroll
        for (int r = 0; r < RPL; ++r) S[(size_t)r * 64] = st[r];
    }
    if (LOCAL && MODE == DR_WEIGHTED && cb16 == 0 && tid == 0) p.piece_decay[(size_t)s * H + h] = decayed;
}

static inline int dr_rpl(int d) {
    const int r = (d + 15) / 16;
    return r <= 4 ? 4 : (r <= 8 ? 8 : (r <= 16 ? 16 : 32));
}

template <bool LOCAL>
static int dr_scan_launch(const DrScan& a, int B, int mode, int silu, hipStream_t s) {
    const int cols = a.e + a.ones, ncb4 = (cols + 3) / 4, rpl = dr_rpl(a.d);
    if (a.H <= 0 || a.H > 65535 || a.G <= 0 || a.H % a.G || a.d <= 0 || a.e <= 0 || a.d > 512 || (cols + 15) / 16 > 65535 || B > 0x7fffffff ||
        (a.ones != 0 && a.ones != 1) || a.qk_stride < (size_t)a.G * a.d || a.v_stride < (size_t)a.H * a.e ||
        a.slot_stride < (size_t)a.H * ncb4 * rpl * 64 || mode < 0 || mode > 3 ||
        (mode != DR_FIXED && (!a.gb || a.gb_stride < (size_t)2 * a.H)) || (mode == DR_FIXED && !a.g_head) || (mode == DR_CHANNELS && !a.gc) ||
        ((a.ones || a.skip) && mode != DR_WEIGHTED) || (a.ones && !LOCAL && !a.n_out) || (silu && mode != DR_FIXED) ||
        (LOCAL && (mode == DR_DELTA || mode == DR_CHANNELS)) || (LOCAL && mode == DR_WEIGHTED && !a.piece_decay))
        return BR_BAD_ARG;
    dim3 grid(B, a.H, (cols + 15) / 16);
#define DR_GO(R, TC, M, A) do { \
        const size_t lds = (size_t)((M == DR_CHANNELS ? 6 : 4) * TC * R * 16 + 2 * TC * 16 + 2 * TC * 2) * sizeof(float); \
        dr_scan_kernel<R, TC, M, A, LOCAL><<<grid, 256, lds, s>>>(a); \
    } while (0)
#define DR_SCAN(R, TC) do { \
        if (mode == DR_WEIGHTED) DR_GO(R, TC, DR_WEIGHTED, false); \
        else if (mode == DR_FIXED) { if (silu) DR_GO(R, TC, DR_FIXED, true); else DR_GO(R, TC, DR_FIXED, false); } \
        else if constexpr (!LOCAL) { if (mode == DR_DELTA) DR_GO(R, TC, DR_DELTA, false); else DR_GO(R, TC, DR_CHANNELS, false); } \
    } while (0)
    if (rpl == 4) DR_SCAN(4, 16);
    else if (rpl == 8) DR_SCAN(8, 16);
    else if (rpl == 16) DR_SCAN(16, 8);
    else DR_SCAN(32, 4);
#undef DR_SCAN
#undef DR_GO
    return br_check_launch();
}

// `mode`: DR_FIXED with `g_head`, DR_DELTA and DR_WEIGHTED with `gb`, DR_CHANNELS with `gb` and `gc`.  `silu` 1 (DR_FIXED):
// q, k, v pass silu.
extern "C" int br_dr_scan(const float* q, const float* k, size_t qk_stride, const float* v, size_t v_stride, const float* gb,
                          size_t gb_stride, const float* g_head, const float* gc, const float* skip, float* o, float* n_out,
                          float* state, size_t slot_stride, const int* cu_seqlens, const int* slots, int B, int H, int G, int d,
                          int e, int mode, int ones, int silu, hipStream_t s) {
    if (B <= 0) return BR_OK;
    const DrScan a = {q, k, v, gb, g_head, gc, skip, o, n_out, state, nullptr, cu_seqlens, slots, qk_stride, v_stride, gb_stride, slot_stride,
                      H, G, d, e, ones};
    return dr_scan_launch<false>(a, B, mode, silu, s);
}

// Between the two passes over a prompt cut into `pieces` pieces per sequence, for the outer sums: from the
// sequence's own state s_0 and every piece's local last state L_c, the state each piece starts from,
// s_(c+1) = D_c s_c + L_c with D_c the product of the piece's decays (`piece_decay` [B * pieces][H], or the head's one
// decay to the power of the piece's tokens), written over L_c; the last one becomes the sequence's state.
// grid (sequences, heads * column blocks of 4), block 64.
__global__ __launch_bounds__(64) void dr_carry_kernel(float* __restrict__ state, size_t slot_stride, const int* __restrict__ slots,
                                                      float* __restrict__ piece_state, size_t piece_stride,
                                                      const int* __restrict__ piece_cu, const float* __restrict__ g_head,
                                                      const float* __restrict__ piece_decay, int pieces, int H, int ncb4, int rpl) {
    const int b = blockIdx.x, hc = blockIdx.y, lane = threadIdx.x;
    const int slot = slots[b];
    if (slot < 0) return;
    const int h = hc / ncb4;
    const float decay = g_head ? g_head[h] : 0.f;
    for (int k = 0; k < rpl; ++k) {
        const size_t idx = ((size_t)hc * rpl + k) * 64 + lane;
        float sv = state[(size_t)slot * slot_stride + idx];
        for (int c = 0; c < pieces; ++c) {
            const size_t v = (size_t)b * pieces + c;
            const float local = piece_state[v * piece_stride + idx];
            piece_state[v * piece_stride + idx] = sv;
            const float D = piece_decay ? piece_decay[v * H + h] : powf(decay, (float)(piece_cu[v + 1] - piece_cu[v]));
            sv = fmaf(D, sv, local);
        }
        state[(size_t)slot * slot_stride + idx] = sv;
    }
}

// An outer sum (DR_FIXED or DR_WEIGHTED) over a step of long prompts with every sequence cut into `pieces` pieces that run
// side by side: the recurrence is linear in the state, so a piece can be walked from a zero state first (its last state
// L), the pieces' true first states follow from s_(c+1) = D_c s_c + L_c, and a second walk from those writes o.  Twice
// the arithmetic for `pieces` times the workgroups; results differ from the plain walk by the rounding of that one
// combination per piece.  `piece_cu` [B * pieces + 1] cuts the packed tokens (pieces of a sequence in order, empty
// ones allowed), `piece_slots` [B * pieces] is the piece's own number (or -1 for a padding sequence's),
// `piece_state` [B * pieces][state of a slot] and `piece_decay` [B * pieces][H] (DR_WEIGHTED) are scratch.
extern "C" int br_dr_scan_pieces(const float* q, const float* k, size_t qk_stride, const float* v, size_t v_stride,
                                 const float* gb, size_t gb_stride, const float* g_head, const float* skip, float* o, float* n_out,
                                 float* state, size_t slot_stride, const int* slots, const int* piece_cu, const int* piece_slots,
                                 float* piece_state, float* piece_decay, int B, int pieces, int H, int G, int d, int e, int mode,
                                 int ones, int silu, hipStream_t s) {
    if (B <= 0) return BR_OK;
    if (pieces <= 0 || (long long)B * pieces > 65535 || B > 65535 || H <= 0 || e <= 0 || d <= 0) return BR_BAD_ARG;
    const int ncb4 = (e + ones + 3) / 4, rpl = dr_rpl(d);
    const size_t piece_stride = (size_t)H * ncb4 * rpl * 64;
    if ((long long)H * ncb4 > 65535 || slot_stride < piece_stride) return BR_BAD_ARG;
    const DrScan a = {q, k, v, gb, g_head, nullptr, skip, o, n_out, piece_state, piece_decay, piece_cu, piece_slots, qk_stride, v_stride,
                      gb_stride, piece_stride, H, G, d, e, ones};
    int rc = dr_scan_launch<true>(a, B * pieces, mode, silu, s);
    if (rc != BR_OK) return rc;
    dr_carry_kernel<<<dim3(B, H * ncb4), 64, 0, s>>>(state, slot_stride, slots, piece_state, piece_stride, piece_cu, g_head,
                                                     mode == DR_WEIGHTED ? piece_decay : nullptr, pieces, H, ncb4, rpl);
    rc = br_check_launch();
    if (rc != BR_OK) return rc;
    return dr_scan_launch<false>(a, B * pieces, mode, silu, s);
}
