// A gated delta rule whose decay is a number a head and key channel, on a flat batch of segments.  A segment is the
// next tokens of one request; what a request carries from step to step lies in one float32 row of `state` per request
// (row state_slots[segment]):
//   [heads, P, DP] the memory, a column of P after the other (its D key channels, padded with zeros to DP = a multiple of
//   four), then [taps - 1, channels] the last inputs of the short convolutions (the oldest first).
// A fresh request's row is all zeros: the memory and what lies before the start.  Per head and token
//   S = diag(g) S;   u = beta (v - S^T k);   S = S + k u^T;   o = S^T q
// with k and q unit vectors (q times a factor).  Everything behind the projections and the convolutions is float32: unit
// norms, step sizes, decays, beta, the memory and every sum.
#include "common.h"
#include "short_conv.h"

// The sum over 32 lanes, within each half of the wavefront, in every lane of it; and the value of the lane 32 apart.
__device__ __forceinline__ float row_halves_sum(float v) {
    v = sum_across(v, 16);
    v += row_permuted<0x128>(v);
    v += row_permuted<0x124>(v);
    v += row_permuted<0x4E>(v);
    v += row_permuted<0xB1>(v);
    return v;
}
__device__ __forceinline__ float from_other_half(float v) {
    float a, b;                                  // the lower half's value and the upper half's, in both
    swap_halves(v, 32, a, b);
    return threadIdx.x % kWave < 32 ? b : a;
}

__device__ __forceinline__ float delta_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// ---- what the recurrence reads, from a token's projections:
//   q, k, v   silu(short convolution) of their bands of the row (`xqkv`: groups * D, groups * D, heads * P columns, in the
//             weights' order); q and k then unit vectors a head, x / sqrt(sum(x^2) + unit_eps), q times q_scale
//   kq        k . q of every group
//   f         exp(-rate * softplus(z + dt_bias)) a head and channel, rate = exp(A_log) of the head
//   beta      sigmoid of its projection
// qk float32 [2, tokens, groups * DP] (channels beyond D are zeros), kq float32 [tokens, groups], v T [tokens, heads * P],
// f float32 [tokens, heads * DP], beta float32 [tokens, heads].
// The grid is (token, piece): a wavefront takes one group's q and k, or 256 of the other results.  CARRY (a step of single
// tokens): the threads that read a request's carried rows move them up by one; else `conv_carry_kernel` does that. ----
constexpr int kDeltaWaves = 4;
constexpr int kDeltaPer = 4;                    // elements a lane: heads of up to 256 channels

struct DeltaInputs {
    const float* conv_w;                        // [taps, channels], a row a tap
    float* state;
    long long state_stride, carried_offset;
    const int* token_segment;
    const int* seg_q_start;
    const int* state_slots;
    const float* rate;
    const float* dt_bias;
    float* qk;
    float* kq;
    float* f;
    float* beta;
    float q_scale, unit_eps;
    int tokens, heads, groups, d, dp, p_dim, taps;
};

template <typename T, bool CARRY>
__global__ void __launch_bounds__(kWave * kDeltaWaves)
delta_inputs_kernel(const T* __restrict__ xqkv, long long x_stride, const T* __restrict__ z, long long z_stride,
                    const T* __restrict__ b, long long b_stride, T* __restrict__ v, DeltaInputs a) {
    const int token = blockIdx.x;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int seg = a.token_segment[token];
    const int local = token - a.seg_q_start[seg];
    const int channels = 2 * a.groups * a.d + a.heads * a.p_dim;
    float* carried = a.state + static_cast<size_t>(a.state_slots[seg]) * a.state_stride + a.carried_offset;
    const T* xt = xqkv + static_cast<size_t>(token) * x_stride;
    auto convolved = [&](int c) -> float {
        return short_conv<T, CARRY>(xt, x_stride, local, carried, a.conv_w, channels, a.taps, c);
    };
    int unit = blockIdx.y * kDeltaWaves + wave;
    if (unit < a.groups) {
        float q[kDeltaPer], k[kDeltaPer], qq = 0.f, kk = 0.f;
#pragma unroll
        for (int j = 0; j < kDeltaPer; ++j) {
            const int i = lane + kWave * j;
            q[j] = k[j] = 0.f;
            if (i < a.d) {
                q[j] = convolved(unit * a.d + i);
                k[j] = convolved((a.groups + unit) * a.d + i);
            }
            qq = fmaf(q[j], q[j], qq);
            kk = fmaf(k[j], k[j], kk);
        }
        const float q_inv = a.q_scale / sqrtf(wave_sum(qq) + a.unit_eps), k_inv = 1.f / sqrtf(wave_sum(kk) + a.unit_eps);
        const size_t width = static_cast<size_t>(a.groups) * a.dp;
        float* q_out = a.qk + static_cast<size_t>(token) * width + static_cast<size_t>(unit) * a.dp;
        float* k_out = q_out + static_cast<size_t>(a.tokens) * width;
        float dot = 0.f;
#pragma unroll
        for (int j = 0; j < kDeltaPer; ++j) {
            const int i = lane + kWave * j;
            q[j] *= q_inv;
            k[j] *= k_inv;
            dot = fmaf(q[j], k[j], dot);
            if (i < a.dp) {
                q_out[i] = q[j];
                k_out[i] = k[j];
            }
        }
        dot = wave_sum(dot);
        if (lane == 0) a.kq[static_cast<size_t>(token) * a.groups + unit] = dot;
        return;
    }
    unit -= a.groups;
    const int v_width = a.heads * a.p_dim, f_width = a.heads * a.dp;
#pragma unroll
    for (int j = 0; j < kDeltaPer; ++j) {
        int e = unit * kWave * kDeltaPer + kWave * j + lane;
        if (e < v_width) {
            v[static_cast<size_t>(token) * v_width + e] = from_float<T>(convolved(2 * a.groups * a.d + e));
            continue;
        }
        e -= v_width;
        if (e < f_width) {
            const int h = e / a.dp, i = e - h * a.dp;
            float f = 0.f;
            if (i < a.d) {
                const int c = h * a.d + i;
                f = expf(-a.rate[h] * delta_softplus(to_float(z[static_cast<size_t>(token) * z_stride + c]) + a.dt_bias[c]));
            }
            a.f[static_cast<size_t>(token) * f_width + e] = f;
            continue;
        }
        e -= f_width;
        if (e < a.heads)
            a.beta[static_cast<size_t>(token) * a.heads + e] = 1.f / (1.f + expf(-to_float(b[static_cast<size_t>(token) * b_stride + e])));
    }
}

// The same with four consecutive channels a lane (D, P, the rows' strides and the carried rows' place are multiples of
// four): lanes 0 .. 31 of a group's wavefront hold q, lanes 32 .. 63 k.  Many tokens: a wavefront takes GROUP tokens and keeps what
// they share in registers: up to four taps a channel, the decays' biases and, where the tokens and the inputs before them are
// all of one portion, the inputs, each of them asked for once and all of them before the first is waited for.
template <typename T> struct alignas(4 * sizeof(T)) DeltaFour { T v[4]; };

template <typename T>
__device__ __forceinline__ float4 four_floats(const T* p) {
    const DeltaFour<T> e = *reinterpret_cast<const DeltaFour<T>*>(p);
    return make_float4(to_float(e.v[0]), to_float(e.v[1]), to_float(e.v[2]), to_float(e.v[3]));
}
// Four elements as they lie in memory, and N of them in registers before the next statement (a compiler left alone asks
// for each where it is used and waits for every one).
template <typename T>
using RawFour = int __attribute__((ext_vector_type(sizeof(T))));
template <typename R, int N>
__device__ __forceinline__ void all_there(R (&x)[N]) {
#pragma unroll
    for (int i = 0; i < N; ++i) asm volatile("" : "+v"(x[i]));
}
template <typename T>
__device__ __forceinline__ float4 four_floats(const RawFour<T> raw) {
    const DeltaFour<T> e = __builtin_bit_cast(DeltaFour<T>, raw);
    return make_float4(to_float(e.v[0]), to_float(e.v[1]), to_float(e.v[2]), to_float(e.v[3]));
}
__device__ __forceinline__ float dot4(const float4 a, const float4 b) { return fmaf(a.w, b.w, fmaf(a.z, b.z, fmaf(a.y, b.y, a.x * b.x))); }

constexpr int kHeldTaps = 4;
constexpr int kDeltaGroup = 4;                  // tokens a wavefront, where there are many (eight: the last wavefronts wait)
struct HeldTaps {
    float4 w[kHeldTaps];                         // the first ones
    __device__ __forceinline__ void load(const float* from, int channels, int taps, int c) {
#pragma unroll
        for (int k = 0; k < kHeldTaps; ++k)
            w[k] = k < taps ? *reinterpret_cast<const float4*>(from + static_cast<size_t>(k) * channels + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
};

template <typename T, bool CARRY>
__device__ __forceinline__ float4 short_conv_four(const T* now, long long stride, int local, float* carried, const float* w,
                                                  const HeldTaps& held, int channels, int taps, int c) {
    float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
    auto tap = [&](int k, const float4 wv) {
        const int back = taps - 1 - k;           // how many tokens ago
        float4 x;
        if (back > 0 && (CARRY || local < back)) {
            x = *reinterpret_cast<const float4*>(carried + static_cast<size_t>(k + (CARRY ? 0 : local)) * channels + c);
            if (CARRY && k > 0) *reinterpret_cast<float4*>(carried + static_cast<size_t>(k - 1) * channels + c) = x;
        } else {
            x = four_floats(now + c - back * stride);
            if (CARRY && taps > 1) *reinterpret_cast<float4*>(carried + static_cast<size_t>(taps - 2) * channels + c) = x;
        }
        acc.x = fmaf(wv.x, x.x, acc.x);
        acc.y = fmaf(wv.y, x.y, acc.y);
        acc.z = fmaf(wv.z, x.z, acc.z);
        acc.w = fmaf(wv.w, x.w, acc.w);
    };
#pragma unroll
    for (int k = 0; k < kHeldTaps; ++k)
        if (k < taps) tap(k, held.w[k]);
    for (int k = kHeldTaps; k < taps; ++k) tap(k, *reinterpret_cast<const float4*>(w + static_cast<size_t>(k) * channels + c));
    acc.x /= 1.f + expf(-acc.x);
    acc.y /= 1.f + expf(-acc.y);
    acc.z /= 1.f + expf(-acc.z);
    acc.w /= 1.f + expf(-acc.w);
    return acc;
}

// The inputs of GROUP tokens and of the taps - 1 <= kHeldTaps - 1 before them, and the convolution of the token at place g.
// (what stands behind the last row is a copy of it; held taps beyond the last one are zeros)
template <typename T, int GROUP>
struct ConvWindow {
    RawFour<T> x[GROUP + kHeldTaps - 1];
    __device__ __forceinline__ void load(const T* xqkv, long long stride, int first, int last, int taps, int c) {
        const T* from = xqkv + static_cast<long long>(first - (taps - 1)) * stride + c;
        const int rows = last - first + taps - 1;
#pragma unroll
        for (int r = 0; r < GROUP + kHeldTaps - 1; ++r)
            x[r] = *reinterpret_cast<const RawFour<T>*>(from + static_cast<long long>(min(r, rows - 1)) * stride);
        all_there(x);
    }
    __device__ __forceinline__ float4 at(int g, const HeldTaps& held) const {
        float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int k = 0; k < kHeldTaps; ++k) {
            const float4 in = four_floats<T>(x[g + k]);
            acc.x = fmaf(held.w[k].x, in.x, acc.x);
            acc.y = fmaf(held.w[k].y, in.y, acc.y);
            acc.z = fmaf(held.w[k].z, in.z, acc.z);
            acc.w = fmaf(held.w[k].w, in.w, acc.w);
        }
        acc.x /= 1.f + expf(-acc.x);
        acc.y /= 1.f + expf(-acc.y);
        acc.z /= 1.f + expf(-acc.z);
        acc.w /= 1.f + expf(-acc.w);
        return acc;
    }
};

template <typename T, bool CARRY, int GROUP, int PER>
__global__ void __launch_bounds__(kWave * kDeltaWaves)
delta_inputs_four_kernel(const T* __restrict__ xqkv, long long x_stride, const T* __restrict__ z, long long z_stride,
                         const T* __restrict__ b, long long b_stride, T* __restrict__ v, DeltaInputs a) {
    const int first = blockIdx.x * GROUP, last = min(a.tokens, first + GROUP);
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int channels = 2 * a.groups * a.d + a.heads * a.p_dim;
    const int unit = blockIdx.y * kDeltaWaves + wave;
    // (a token's place in its segment and its request's carried rows)
    auto convolved = [&](int token, const HeldTaps& held, int c) {
        const int seg = a.token_segment[token];
        float* carried = a.state + static_cast<size_t>(a.state_slots[seg]) * a.state_stride + a.carried_offset;
        return short_conv_four<T, CARRY>(xqkv + static_cast<size_t>(token) * x_stride, x_stride, token - a.seg_q_start[seg], carried,
                                         a.conv_w, held, channels, a.taps, c);
    };
    bool inside = false;                         // the window of all the tokens lies in one portion
    if (GROUP > 1 && a.taps <= kHeldTaps) {
        const int seg = a.token_segment[first];
        inside = seg == a.token_segment[last - 1] && first - a.seg_q_start[seg] >= a.taps - 1;
    }
    if (unit < a.groups) {
        const int half = lane / 32;              // 0: q, 1: k
        HeldTaps held[PER];
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int i = 4 * (lane % 32 + 32 * j);
            held[j].load(a.conv_w, channels, i < a.d ? a.taps : 0, (half * a.groups + unit) * a.d + i);
        }
        auto finish = [&](int token, float4 (&x)[PER]) {
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < PER; ++j) ss += dot4(x[j], x[j]);
            ss = row_halves_sum(ss);
            const float inv = (half ? 1.f : a.q_scale) / sqrtf(ss + a.unit_eps);
            float* out = a.qk + (static_cast<size_t>(half) * a.tokens + token) * a.groups * a.dp + static_cast<size_t>(unit) * a.dp;
            float dot = 0.f;
#pragma unroll
            for (int j = 0; j < PER; ++j) {
                const int i = 4 * (lane % 32 + 32 * j);
                x[j].x *= inv;
                x[j].y *= inv;
                x[j].z *= inv;
                x[j].w *= inv;
                const float4 other = make_float4(from_other_half(x[j].x), from_other_half(x[j].y), from_other_half(x[j].z),
                                                 from_other_half(x[j].w));
                dot += dot4(x[j], other);
                if (i < a.d) *reinterpret_cast<float4*>(out + i) = x[j];
            }
            dot = row_halves_sum(dot);
            if (lane == 0) a.kq[static_cast<size_t>(token) * a.groups + unit] = dot;
        };
        if (GROUP > 1 && inside) {
            ConvWindow<T, GROUP> window[PER];
#pragma unroll
            for (int j = 0; j < PER; ++j)        // (a lane beyond the head reads its last channels: its taps are zeros)
                window[j].load(xqkv, x_stride, first, last, a.taps, (half * a.groups + unit) * a.d + min(4 * (lane % 32 + 32 * j), a.d - 4));
#pragma unroll
            for (int g = 0; g < GROUP; ++g) {
                if (first + g >= last) break;
                float4 x[PER];
#pragma unroll
                for (int j = 0; j < PER; ++j) x[j] = window[j].at(g, held[j]);
                finish(first + g, x);
            }
            return;
        }
        for (int token = first; token < last; ++token) {
            float4 x[PER];
#pragma unroll
            for (int j = 0; j < PER; ++j) {
                const int i = 4 * (lane % 32 + 32 * j);
                x[j] = make_float4(0.f, 0.f, 0.f, 0.f);
                if (i < a.d) x[j] = convolved(token, held[j], (half * a.groups + unit) * a.d + i);
            }
            finish(token, x);
        }
        return;
    }
    const int v_width = a.heads * a.p_dim, f_width = a.heads * a.d;
    int e = ((unit - a.groups) * kWave + lane) * 4;
    if (e < v_width) {
        const int c = 2 * a.groups * a.d + e;
        HeldTaps held;
        held.load(a.conv_w, channels, a.taps, c);
        auto write = [&](int token, const float4 x) {
            DeltaFour<T> r;
            r.v[0] = from_float<T>(x.x);
            r.v[1] = from_float<T>(x.y);
            r.v[2] = from_float<T>(x.z);
            r.v[3] = from_float<T>(x.w);
            *reinterpret_cast<DeltaFour<T>*>(v + static_cast<size_t>(token) * v_width + e) = r;
        };
        if (GROUP > 1 && inside) {
            ConvWindow<T, GROUP> window;
            window.load(xqkv, x_stride, first, last, a.taps, c);
#pragma unroll
            for (int g = 0; g < GROUP; ++g)
                if (first + g < last) write(first + g, window.at(g, held));
            return;
        }
        for (int token = first; token < last; ++token) write(token, convolved(token, held, c));
        return;
    }
    e -= v_width;
    if (e < f_width) {
        const float rate = a.rate[e / a.d];
        const float4 bias = *reinterpret_cast<const float4*>(a.dt_bias + e);
        RawFour<T> held[GROUP];
#pragma unroll
        for (int g = 0; g < GROUP; ++g)
            held[g] = *reinterpret_cast<const RawFour<T>*>(z + static_cast<size_t>(min(first + g, last - 1)) * z_stride + e);
        all_there(held);
#pragma unroll
        for (int g = 0; g < GROUP; ++g) {
            const int token = first + g;
            if (token >= last) break;
            const float4 zv = four_floats<T>(held[g]);
            float4 r;
            r.x = expf(-rate * delta_softplus(zv.x + bias.x));
            r.y = expf(-rate * delta_softplus(zv.y + bias.y));
            r.z = expf(-rate * delta_softplus(zv.z + bias.z));
            r.w = expf(-rate * delta_softplus(zv.w + bias.w));
            *reinterpret_cast<float4*>(a.f + static_cast<size_t>(token) * f_width + e) = r;
        }
        return;
    }
    e -= f_width;
    for (int token = first; token < last; ++token)
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (e + u < a.heads)
                a.beta[static_cast<size_t>(token) * a.heads + e + u] =
                    1.f / (1.f + expf(-to_float(b[static_cast<size_t>(token) * b_stride + e + u])));
}

WLLM_API int wllm_delta_inputs(const void* xqkv, long long x_stride, const void* z, long long z_stride, const void* b,
                               long long b_stride, const float* conv_w, const float* rate, const float* dt_bias, float* state,
                               long long state_stride, long long carried_offset, const int* token_segment, const int* seg_q_start,
                               const int* seg_q_len, const int* state_slots, float* qk, float* kq, void* v, float* f, float* beta,
                               float q_scale, float unit_eps, int is_bf16, int tokens, int segments, int heads, int groups, int d,
                               int p_dim, int taps, int single_tokens, hipStream_t stream) {
    if (tokens <= 0 || segments <= 0) return 0;
    if (heads <= 0 || groups <= 0 || heads % groups || d <= 0 || d > kWave * kDeltaPer || p_dim <= 0 || taps < 1 || taps > 64) return -1;
    if (single_tokens && tokens != segments) return -1;
    const int dp = (d + 3) / 4 * 4;
    const long long rest = static_cast<long long>(heads) * (p_dim + dp + 1);
    const long long units = groups + (rest + kWave * kDeltaPer - 1) / (kWave * kDeltaPer);
    const long long pieces = (units + kDeltaWaves - 1) / kDeltaWaves;
    if (pieces > 65535) return -1;
    const DeltaInputs a{conv_w, state, state_stride, carried_offset, token_segment, seg_q_start, state_slots, rate, dt_bias, qk, kq, f,
                        beta, q_scale, unit_eps, tokens, heads, groups, d, dp, p_dim, taps};
    const size_t four_bytes = 4 * (is_bf16 ? 2 : 4);
    const bool four = d % 4 == 0 && p_dim % 4 == 0 && x_stride % 4 == 0 && z_stride % 4 == 0 && state_stride % 4 == 0 &&
                      carried_offset % 4 == 0 && reinterpret_cast<uintptr_t>(xqkv) % four_bytes == 0 &&
                      reinterpret_cast<uintptr_t>(z) % four_bytes == 0 && reinterpret_cast<uintptr_t>(v) % four_bytes == 0 &&
                      reinterpret_cast<uintptr_t>(conv_w) % 16 == 0 && reinterpret_cast<uintptr_t>(dt_bias) % 16 == 0 &&
                      reinterpret_cast<uintptr_t>(state) % 16 == 0 && reinterpret_cast<uintptr_t>(qk) % 16 == 0 &&
                      reinterpret_cast<uintptr_t>(f) % 16 == 0;
    if (four) {
        const long long fours = rest / 4 + 1;    // (beta's last four may be partly there)
        const long long four_units = groups + (fours + kWave - 1) / kWave;
        const unsigned four_pieces = static_cast<unsigned>((four_units + kDeltaWaves - 1) / kDeltaWaves);
        // (about eight wavefronts a SIMD remain with four tokens each)
        const bool many = !single_tokens && static_cast<long long>(tokens) * four_pieces >= 8192;
#define LAUNCH(T, CARRY, GROUP, PER)                                                                                    \
    delta_inputs_four_kernel<T, CARRY, GROUP, PER>                                                                      \
        <<<dim3((tokens + GROUP - 1) / GROUP, four_pieces), kWave * kDeltaWaves, 0, stream>>>(                          \
            static_cast<const T*>(xqkv), x_stride, static_cast<const T*>(z), z_stride, static_cast<const T*>(b), b_stride, \
            static_cast<T*>(v), a)
#define BY_TOKENS(T, PER)                                                                                               \
    if (single_tokens) LAUNCH(T, true, 1, PER); else if (many) LAUNCH(T, false, kDeltaGroup, PER); else LAUNCH(T, false, 1, PER)
        if (is_bf16) { if (d <= 128) { BY_TOKENS(bf16, 1); } else { BY_TOKENS(bf16, 2); } }
        else { if (d <= 128) { BY_TOKENS(float, 1); } else { BY_TOKENS(float, 2); } }
#undef BY_TOKENS
#undef LAUNCH
    } else {
        const dim3 grid(tokens, static_cast<unsigned>(pieces));
#define LAUNCH(T, CARRY)                                                                                                \
        delta_inputs_kernel<T, CARRY><<<grid, kWave * kDeltaWaves, 0, stream>>>(                                        \
            static_cast<const T*>(xqkv), x_stride, static_cast<const T*>(z), z_stride, static_cast<const T*>(b), b_stride,\
            static_cast<T*>(v), a)
        if (is_bf16) { if (single_tokens) LAUNCH(bf16, true); else LAUNCH(bf16, false); }
        else { if (single_tokens) LAUNCH(float, true); else LAUNCH(float, false); }
#undef LAUNCH
    }
    if (const int err = launch_status()) return err;
    if (taps == 1 || single_tokens) return 0;
    const int channels = 2 * groups * d + heads * p_dim;
    const dim3 carry_grid(segments, (channels + 255) / 256 < 64 ? (channels + 255) / 256 : 64);
    if (is_bf16)
        conv_carry_kernel<bf16><<<carry_grid, 256, 0, stream>>>(static_cast<const bf16*>(xqkv), x_stride, state, state_stride,
                                                                carried_offset, seg_q_start, seg_q_len, state_slots, channels, taps);
    else
        conv_carry_kernel<float><<<carry_grid, 256, 0, stream>>>(static_cast<const float*>(xqkv), x_stride, state, state_stride,
                                                                 carried_offset, seg_q_start, seg_q_len, state_slots, channels, taps);
    return launch_status();
}

// ---- the recurrence.  The columns of a head's memory do not depend on each other, and a column's new write needs the
// sum over all its channels first: a column lies within 16 lanes, lane s of them holding the channels 4s .. 4s + 3 (and
// those 64, 128, 192 further on) in registers, and both sums of a token (S^T k and S^T q of the decayed memory) go
// through the 16 lanes by the vector unit's own permutations; the read-out behind the write is then S^T q + u (k . q).
// A wavefront is four columns, a workgroup's four wavefronts sixteen; nothing passes between them but the tokens' k, q
// and f, which go 16 tokens at a time through shared memory, the next 16 fetched into registers while these are
// walked.  A token's results are the same operations in the same order however the tokens are cut into steps. ----
constexpr int kScanTokens = 16;
constexpr int kScanWaves = 4;
constexpr int kScanLanes = 16;                               // lanes a column
constexpr int kScanCols = kWave / kScanLanes * kScanWaves;   // columns a workgroup
constexpr int kScanThreads = kWave * kScanWaves;

__device__ __forceinline__ float row_sum(float v) {          // over the 16 lanes of a row, in every lane
    v += row_permuted<0x128>(v);
    v += row_permuted<0x124>(v);
    v += row_permuted<0x4E>(v);
    v += row_permuted<0xB1>(v);
    return v;
}

template <typename T, int R>        // R: groups of four channels a lane (heads of up to 64 R channels)
__global__ void __launch_bounds__(kScanThreads)
delta_scan_kernel(const float* __restrict__ qk, const float* __restrict__ kq, const float* __restrict__ f,
                  const float* __restrict__ beta, const T* __restrict__ v, float* __restrict__ state, long long state_stride,
                  const int* __restrict__ seg_q_start, const int* __restrict__ seg_q_len, const int* __restrict__ state_slots,
                  float* __restrict__ y, int tokens, int heads, int groups, int dp, int p_dim, int shorter_than) {
    constexpr int kRow = 64 * R;                             // a token's k (q, f) in shared memory: DP channels and zeros
    constexpr int kFours = kScanTokens * kRow / 4 / kScanThreads;      // groups of four of each that a thread stages: R
    __shared__ __align__(16) float q_s[kScanTokens * kRow], k_s[kScanTokens * kRow], f_s[kScanTokens * kRow];
    __shared__ float v_s[kScanTokens * kScanCols];
    __shared__ float beta_s[kScanTokens], kq_s[kScanTokens];
    const int h = blockIdx.x, seg = blockIdx.y, p0 = blockIdx.z * kScanCols;
    const int q_len = seg_q_len[seg], q_start = seg_q_start[seg];
    if (q_len <= 0 || q_len >= shorter_than) return;
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int sl = lane % kScanLanes, col = wave * (kWave / kScanLanes) + lane / kScanLanes;
    const int p = p0 + col;
    const bool live = p < p_dim;
    const int g = h / (heads / groups);
    float* s_col = state + static_cast<size_t>(state_slots[seg]) * state_stride + (static_cast<size_t>(h) * p_dim + p) * dp;
    float4 s[R];
#pragma unroll
    for (int j = 0; j < R; ++j) {
        const int i = 64 * j + 4 * sl;
        s[j] = live && i < dp ? *reinterpret_cast<const float4*>(s_col + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const size_t q_width = static_cast<size_t>(groups) * dp, f_width = static_cast<size_t>(heads) * dp;
    const size_t k_plane = static_cast<size_t>(tokens) * q_width;
    float4 q_r[kFours], k_r[kFours], f_r[kFours];
    float v_r = 0.f, beta_r = 0.f, kq_r = 0.f;
    const int vt = tid / kScanCols, vc = tid % kScanCols;    // (16 tokens of 16 columns: one value a thread)
    auto fetch = [&](int t0) {
        const int count = min(kScanTokens, q_len - t0);
        const size_t first = static_cast<size_t>(q_start + t0);
#pragma unroll
        for (int u = 0; u < kFours; ++u) {
            const int four = tid + kScanThreads * u;
            const int t = four / (kRow / 4), i = four % (kRow / 4) * 4;
            q_r[u] = k_r[u] = f_r[u] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (t < count && i < dp) {
                const float* at = qk + (first + t) * q_width + static_cast<size_t>(g) * dp + i;
                q_r[u] = *reinterpret_cast<const float4*>(at);
                k_r[u] = *reinterpret_cast<const float4*>(at + k_plane);
                f_r[u] = *reinterpret_cast<const float4*>(f + (first + t) * f_width + static_cast<size_t>(h) * dp + i);
            }
        }
        v_r = vt < count && p0 + vc < p_dim ? to_float(v[(first + vt) * heads * p_dim + static_cast<size_t>(h) * p_dim + p0 + vc]) : 0.f;
        if (tid < count) {
            beta_r = beta[(first + tid) * heads + h];
            kq_r = kq[(first + tid) * groups + g];
        }
    };
    auto place = [&]() {
#pragma unroll
        for (int u = 0; u < kFours; ++u) {
            const int four = tid + kScanThreads * u;
            reinterpret_cast<float4*>(q_s)[four] = q_r[u];
            reinterpret_cast<float4*>(k_s)[four] = k_r[u];
            reinterpret_cast<float4*>(f_s)[four] = f_r[u];
        }
        v_s[tid] = v_r;
        if (tid < kScanTokens) {
            beta_s[tid] = beta_r;
            kq_s[tid] = kq_r;
        }
    };
    float kept = 0.f;                                        // lane sl of a column keeps the result of token sl of the 16
    struct Operands {
        float4 k[R], q[R], f[R];
        float v, beta, kq;
    };
    auto load = [&](int t) {
        Operands o;
#pragma unroll
        for (int j = 0; j < R; ++j) {
            const int at = t * kRow + 64 * j + 4 * sl;
            o.k[j] = *reinterpret_cast<const float4*>(k_s + at);
            o.q[j] = *reinterpret_cast<const float4*>(q_s + at);
            o.f[j] = *reinterpret_cast<const float4*>(f_s + at);
        }
        o.v = v_s[t * kScanCols + col];
        o.beta = beta_s[t];
        o.kq = kq_s[t];
        return o;
    };
    auto token = [&](int t, const Operands& o) {
        float seen[2] = {0.f, 0.f}, read[2] = {0.f, 0.f};    // two chains each
#pragma unroll
        for (int j = 0; j < R; ++j) {
            s[j].x *= o.f[j].x;
            s[j].y *= o.f[j].y;
            s[j].z *= o.f[j].z;
            s[j].w *= o.f[j].w;
            seen[0] = fmaf(s[j].x, o.k[j].x, seen[0]);
            seen[1] = fmaf(s[j].y, o.k[j].y, seen[1]);
            seen[0] = fmaf(s[j].z, o.k[j].z, seen[0]);
            seen[1] = fmaf(s[j].w, o.k[j].w, seen[1]);
            read[0] = fmaf(s[j].x, o.q[j].x, read[0]);
            read[1] = fmaf(s[j].y, o.q[j].y, read[1]);
            read[0] = fmaf(s[j].z, o.q[j].z, read[0]);
            read[1] = fmaf(s[j].w, o.q[j].w, read[1]);
        }
        const float u = o.beta * (o.v - row_sum(seen[0] + seen[1]));
        const float out = fmaf(u, o.kq, row_sum(read[0] + read[1]));
#pragma unroll
        for (int j = 0; j < R; ++j) {
            s[j].x = fmaf(o.k[j].x, u, s[j].x);
            s[j].y = fmaf(o.k[j].y, u, s[j].y);
            s[j].z = fmaf(o.k[j].z, u, s[j].z);
            s[j].w = fmaf(o.k[j].w, u, s[j].w);
        }
        if (sl == t) kept = out;
    };
    fetch(0);
    for (int t0 = 0; t0 < q_len; t0 += kScanTokens) {
        const int count = min(kScanTokens, q_len - t0);
        place();
        __syncthreads();
        if (t0 + kScanTokens < q_len) fetch(t0 + kScanTokens);
        if (count == kScanTokens) {
            Operands now = load(0);
#pragma unroll
            for (int t = 0; t < kScanTokens; ++t) {
                const Operands next = load(t + 1 < kScanTokens ? t + 1 : t);      // on their way while this token is worked on
                __builtin_amdgcn_sched_barrier(0);
                token(t, now);
                now = next;
            }
        } else {
            for (int t = 0; t < count; ++t) token(t, load(t));
        }
        if (live && sl < count)
            y[static_cast<size_t>(q_start + t0 + sl) * heads * p_dim + static_cast<size_t>(h) * p_dim + p] = kept;
        __syncthreads();                                     // the 16 tokens are read out
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < R; ++j) {
            const int i = 64 * j + 4 * sl;
            if (i < dp) *reinterpret_cast<float4*>(s_col + i) = s[j];
        }
    }
}

// Segments of `shorter_than` tokens and more are left alone (a caller that takes none of them away passes INT_MAX).
WLLM_API int wllm_delta_scan(const float* qk, const float* kq, const float* f, const float* beta, const void* v, float* state,
                             long long state_stride, const int* seg_q_start, const int* seg_q_len, const int* state_slots, float* y,
                             int is_bf16, int tokens, int segments, int heads, int groups, int d, int p_dim, int shorter_than,
                             hipStream_t stream) {
    if (tokens <= 0 || segments <= 0) return 0;
    if (heads <= 0 || groups <= 0 || heads % groups || d <= 0 || d > 256 || p_dim <= 0 || segments > 65535 ||
        (p_dim + kScanCols - 1) / kScanCols > 65535 || state_stride % 4 || reinterpret_cast<uintptr_t>(state) % 16)
        return -1;
    const int dp = (d + 3) / 4 * 4;
    const dim3 grid(heads, segments, (p_dim + kScanCols - 1) / kScanCols);
#define LAUNCH(T, R)                                                                                                   \
    delta_scan_kernel<T, R><<<grid, kScanThreads, 0, stream>>>(qk, kq, f, beta, static_cast<const T*>(v), state, state_stride, \
                                                               seg_q_start, seg_q_len, state_slots, y, tokens, heads, groups, dp, \
                                                               p_dim, shorter_than)
#define LAUNCH_R(T)                    \
    if (dp <= 64) LAUNCH(T, 1);        \
    else if (dp <= 128) LAUNCH(T, 2);  \
    else if (dp <= 192) LAUNCH(T, 3);  \
    else LAUNCH(T, 4);
    if (is_bf16) { LAUNCH_R(bf16) } else { LAUNCH_R(float) }
#undef LAUNCH_R
#undef LAUNCH
    return launch_status();
}

// ---- the same recurrence over many tokens, 16 at a time on the matrix cores.  With D_t the product of the decays of a
// chunk's tokens up to t (a number a channel), and every product of decays between two tokens formed from the decays
// between them (never as a quotient), the 16 tokens' writes are the solution of a triangular system:
//   W = V - (D K) S0;   U = M W;   O = (D Q) S0 + N W;   S = D_16 S0 + Kh^T U
// with (D K)_t = D_t k_t, (D Q)_t = D_t q_t, Kh_s = k_s times the decays behind s,
//   A_ts = k_t . (decays s < r <= t) k_s,   B_ts = q_t . (decays s < r <= t) k_s (s <= t),
//   M = (I + diag(beta) strictly_lower(A))^-1 diag(beta),   N = B M
// none of which depends on the memory: `delta_chunk_kernel` makes them for all chunks and heads at once, and
// `delta_chunk_scan_kernel` walks a segment's chunks in order with v_mfma_f32_16x16x4_f32 (float32 in and out).  A chunk
// begins every 16 tokens of a segment; the last one is filled with tokens that change nothing (k = q = 0, f = 1, beta = 0).
// Chunk c of segment s lies at place q_start / 16 + s + c of the scratch (no two chunks share one), its operands of head h
// as [16][C] D K, [16][C] D Q, [C][16] Kh, [C] D_16, [16][16] M, [16][16] N with C = the channels padded to a multiple of 64.
constexpr int kChunk = 16;

__host__ __device__ __forceinline__ size_t chunk_floats(int c) { return static_cast<size_t>(3 * kChunk + 1) * c + 2 * kChunk * kChunk; }

template <int R>        // C = 64 R
__global__ void __launch_bounds__(256)
delta_chunk_kernel(const float* __restrict__ qk, const float* __restrict__ f, const float* __restrict__ beta,
                   const int* __restrict__ token_segment, const int* __restrict__ seg_q_start, const int* __restrict__ seg_q_len,
                   float* __restrict__ chunks, int tokens, int heads, int groups, int dp, int from) {
    constexpr int C = 64 * R;
    __shared__ __align__(16) float k_s[kChunk * C], q_s[kChunk * C], f_s[kChunk * C];
    __shared__ float a_s[kChunk][kChunk + 1], b_s[kChunk][kChunk + 1], m_s[kChunk][kChunk + 1];
    __shared__ float beta_s[kChunk];
    const int h = blockIdx.y, g = h / (heads / groups);
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    // which of these 16 tokens begins a chunk (at most two do: a segment that is walked in chunks has 16 tokens or more)
    bool begins = false;
    {
        const int token = blockIdx.x * kChunk + lane;
        if (lane < kChunk && token < tokens) {
            const int seg = token_segment[token];
            begins = seg_q_len[seg] >= from && (token - seg_q_start[seg]) % kChunk == 0;
        }
    }
    unsigned long long starts = __ballot(begins);
    while (starts) {
        const int token = blockIdx.x * kChunk + __ffsll(starts) - 1;
        starts &= starts - 1;
        const int seg = token_segment[token], q_start = seg_q_start[seg];
        const int local = token - q_start, count = min(kChunk, seg_q_len[seg] - local);
        const size_t place = static_cast<size_t>(q_start / kChunk + seg + local / kChunk);
        float* out = chunks + (place * heads + h) * chunk_floats(C);
        const size_t q_width = static_cast<size_t>(groups) * dp, f_width = static_cast<size_t>(heads) * dp;
        __syncthreads();                          // the chunk before is read out
        for (int four = tid; four < kChunk * C / 4; four += 256) {
            const int t = four / (C / 4), i = four % (C / 4) * 4;
            float4 k = make_float4(0.f, 0.f, 0.f, 0.f), q = k, d = make_float4(1.f, 1.f, 1.f, 1.f);
            if (t < count && i < dp) {
                const float* at = qk + static_cast<size_t>(token + t) * q_width + static_cast<size_t>(g) * dp + i;
                q = *reinterpret_cast<const float4*>(at);
                k = *reinterpret_cast<const float4*>(at + static_cast<size_t>(tokens) * q_width);
                d = *reinterpret_cast<const float4*>(f + static_cast<size_t>(token + t) * f_width + static_cast<size_t>(h) * dp + i);
            }
            reinterpret_cast<float4*>(k_s)[four] = k;
            reinterpret_cast<float4*>(q_s)[four] = q;
            reinterpret_cast<float4*>(f_s)[four] = d;
        }
        if (tid < kChunk) beta_s[tid] = tid < count ? beta[static_cast<size_t>(token + tid) * heads + h] : 0.f;
        __syncthreads();
        // A and B: 16 lanes hold the key of token s, which decays as t goes on
        {
            const int s = tid / kChunk, sl = tid % kChunk;
            float4 r[R];
#pragma unroll
            for (int j = 0; j < R; ++j) r[j] = *reinterpret_cast<const float4*>(k_s + s * C + 64 * j + 4 * sl);
            const int first = wave * (kWave / kChunk);            // the wavefront's first s
            for (int t = 0; t < kChunk; ++t) {
                float a = 0.f, b = 0.f;
                if (t >= first) {
#pragma unroll
                    for (int j = 0; j < R; ++j) {
                        const int at = t * C + 64 * j + 4 * sl;
                        const float4 kt = *reinterpret_cast<const float4*>(k_s + at), qt = *reinterpret_cast<const float4*>(q_s + at);
                        if (t > s) {
                            const float4 ft = *reinterpret_cast<const float4*>(f_s + at);
                            r[j].x *= ft.x;
                            r[j].y *= ft.y;
                            r[j].z *= ft.z;
                            r[j].w *= ft.w;
                        }
                        a += dot4(r[j], kt);
                        b += dot4(r[j], qt);
                    }
                    a = row_sum(a);
                    b = row_sum(b);
                }
                if (sl == 0) {
                    a_s[t][s] = t > s ? a : 0.f;
                    b_s[t][s] = t >= s ? b : 0.f;
                }
            }
        }
        // the decays up to and behind every token, a channel a thread
        for (int c = tid; c < C; c += 256) {
            float decay = 1.f;
#pragma unroll
            for (int t = 0; t < kChunk; ++t) {
                decay *= f_s[t * C + c];
                out[t * C + c] = k_s[t * C + c] * decay;
                out[(kChunk + t) * C + c] = q_s[t * C + c] * decay;
            }
            out[3 * kChunk * C + c] = decay;
            float kh[kChunk], behind = 1.f;
#pragma unroll
            for (int t = kChunk - 1; t >= 0; --t) {
                kh[t] = k_s[t * C + c] * behind;
                behind *= f_s[t * C + c];
            }
#pragma unroll
            for (int t = 0; t < kChunk; t += 4)
                *reinterpret_cast<float4*>(out + 2 * kChunk * C + c * kChunk + t) = make_float4(kh[t], kh[t + 1], kh[t + 2], kh[t + 3]);
        }
        __syncthreads();
        float* mn = out + (3 * kChunk + 1) * C;
        if (tid < kChunk) {
            // a column of M: m_t = beta_t (delta_tj - sum over s < t of A_ts m_s)
            float m[kChunk];
#pragma unroll
            for (int t = 0; t < kChunk; ++t) {
                float sum = 0.f;
#pragma unroll
                for (int s = 0; s < t; ++s) sum = fmaf(a_s[t][s], m[s], sum);
                m[t] = beta_s[t] * ((t == tid ? 1.f : 0.f) - sum);
                m_s[t][tid] = m[t];
            }
        }
        __syncthreads();
        {
            const int t = tid / kChunk, j = tid % kChunk;
            float n = 0.f;
#pragma unroll
            for (int s = 0; s < kChunk; ++s) n = fmaf(b_s[t][s], m_s[s][j], n);
            mn[tid] = m_s[t][j];
            mn[kChunk * kChunk + tid] = n;
        }
    }
}

// A workgroup owns (head, segment, 16 value columns).  The channels are cut over its four wavefronts, each with TILES tiles
// of 16 of them: lane (i, g) holds the memory's channels 4g .. 4g + 3 of a tile in column i, which is what the product
// leaves and, channel by channel, what it takes (the k-th of four products takes the channels 4g + k), so the memory never
// moves between lanes.  The wavefronts' parts of (D K) S0 and (D Q) S0 meet in shared memory (two places in turn: one
// barrier a chunk); what follows every wavefront makes for itself.  The next chunk's operands are asked for first.
typedef float delta_float4 __attribute__((ext_vector_type(4)));

// (two workgroups a compute unit at least: the products then keep their sums in the registers the rest is in)
template <typename T, int TILES>
__global__ void __launch_bounds__(256, 2)
delta_chunk_scan_kernel(const float* chunks, const T* v, float* __restrict__ state,
                        long long state_stride, const int* __restrict__ seg_q_start, const int* __restrict__ seg_q_len,
                        const int* __restrict__ state_slots, float* __restrict__ y, int heads, int dp, int p_dim, int from) {
    constexpr int C = 64 * TILES;
    __shared__ delta_float4 part_s[2][4][2][kWave];
    const int h = blockIdx.x, seg = blockIdx.y, p0 = blockIdx.z * 16;
    const int q_len = seg_q_len[seg], q_start = seg_q_start[seg];
    if (q_len < from) return;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int i = lane % 16, g = lane / 16;
    const int p = p0 + i;
    const bool live = p < p_dim;
    float* s_col = state + static_cast<size_t>(state_slots[seg]) * state_stride + (static_cast<size_t>(h) * p_dim + p) * dp;
    const int ch0 = wave * 16 * TILES;
    delta_float4 s[TILES];
#pragma unroll
    for (int j = 0; j < TILES; ++j) {
        const int ch = ch0 + 16 * j + 4 * g;
        s[j] = live && ch < dp ? *reinterpret_cast<const delta_float4*>(s_col + ch) : delta_float4{0.f, 0.f, 0.f, 0.f};
    }
    struct Operands {
        delta_float4 k[TILES], q[TILES], kh[TILES], d[TILES], m, n;
        T v[4];
    };
    const float* base = chunks + (static_cast<size_t>(q_start / kChunk + seg) * heads + h) * chunk_floats(C);
    // where this lane's operands lie in a chunk's (unsigned: a lane's offset beside an address that is the same in all lanes)
    const unsigned k_at = i * C + ch0 + 4 * g, kh_at = 2 * kChunk * C + (ch0 + i) * kChunk + 4 * g, d_at = 3 * kChunk * C + ch0 + 4 * g;
    const unsigned m_at = (3 * kChunk + 1) * C + i * kChunk + 4 * g;
    const unsigned v_row = static_cast<unsigned>(heads) * p_dim, v_at = static_cast<unsigned>(min(p, p_dim - 1));
    const T* v_first = v + static_cast<size_t>(q_start) * v_row + static_cast<size_t>(h) * p_dim;
    float* y_first = y + static_cast<size_t>(q_start) * v_row + static_cast<size_t>(h) * p_dim;
    auto load = [&](int c) {
        Operands o;
        const float* at = base + static_cast<size_t>(c) * heads * chunk_floats(C);
#pragma unroll
        for (int j = 0; j < TILES; ++j) {
            o.k[j] = *reinterpret_cast<const delta_float4*>(at + k_at + 16 * j);
            o.q[j] = *reinterpret_cast<const delta_float4*>(at + k_at + kChunk * C + 16 * j);
            o.kh[j] = *reinterpret_cast<const delta_float4*>(at + kh_at + 16 * kChunk * j);
            o.d[j] = *reinterpret_cast<const delta_float4*>(at + d_at + 16 * j);
        }
        o.m = *reinterpret_cast<const delta_float4*>(at + m_at);
        o.n = *reinterpret_cast<const delta_float4*>(at + m_at + kChunk * kChunk);
        const T* v_chunk = v_first + static_cast<size_t>(c) * kChunk * v_row;
        const unsigned beyond = min(kChunk, q_len - c * kChunk) - 1;          // the chunk's last token
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            // (beyond the segment's last token, that token's once more: what it is multiplied by is zero.  Nothing is made of
            // the values here, and no branch stands before the loads: they are not waited for)
            o.v[u] = v_chunk[min(static_cast<unsigned>(4 * g + u), beyond) * v_row + v_at];
        }
        return o;
    };
    const int count = (q_len + kChunk - 1) / kChunk;
    auto walk = [&](int c, const Operands& now) {
        delta_float4 seen = {0.f, 0.f, 0.f, 0.f}, read = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < TILES; ++j)
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                seen = __builtin_amdgcn_mfma_f32_16x16x4f32(now.k[j][u], s[j][u], seen, 0, 0, 0);
                read = __builtin_amdgcn_mfma_f32_16x16x4f32(now.q[j][u], s[j][u], read, 0, 0, 0);
            }
        part_s[c % 2][wave][0][lane] = seen;
        part_s[c % 2][wave][1][lane] = read;
        // the memory decays while the parts meet
#pragma unroll
        for (int j = 0; j < TILES; ++j) s[j] *= now.d[j];
        // (a barrier for what lies in shared memory alone: the operands of the chunks ahead stay on their way)
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        seen = part_s[c % 2][0][0][lane];
        read = part_s[c % 2][0][1][lane];
#pragma unroll
        for (int w = 1; w < 4; ++w) {
            seen += part_s[c % 2][w][0][lane];
            read += part_s[c % 2][w][1][lane];
        }
        delta_float4 u4 = {0.f, 0.f, 0.f, 0.f}, left;
#pragma unroll
        for (int u = 0; u < 4; ++u) left[u] = (c * kChunk + 4 * g + u < q_len ? to_float(now.v[u]) : 0.f) - seen[u];
#pragma unroll
        for (int u = 0; u < 4; ++u) u4 = __builtin_amdgcn_mfma_f32_16x16x4f32(now.m[u], left[u], u4, 0, 0, 0);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int j = 0; j < TILES; ++j) s[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(now.kh[j][u], u4[u], s[j], 0, 0, 0);
#pragma unroll
        for (int u = 0; u < 4; ++u) read = __builtin_amdgcn_mfma_f32_16x16x4f32(now.n[u], left[u], read, 0, 0, 0);
        // wavefront w writes the tokens 4g + w
        const int t = 4 * g + wave;
        const float o = wave == 0 ? read[0] : wave == 1 ? read[1] : wave == 2 ? read[2] : read[3];
        if (live && c * kChunk + t < q_len) (y_first + static_cast<size_t>(c) * kChunk * v_row)[t * v_row + v_at] = o;
    };
    // two chunks' operands in turn, each asked for while the chunk before is walked (beyond the last: the last's once more)
    Operands a = load(0);
    int c = 0;
    for (; c + 1 < count; c += 2) {
        // (the loads stay where they are written: `chunks` and `v` may alias as far as the compiler knows, and the empty
        // statements touch memory)
        const Operands b = load(c + 1);
        asm volatile("" ::: "memory");
        walk(c, a);
        a = load(min(c + 2, count - 1));
        asm volatile("" ::: "memory");
        walk(c + 1, b);
    }
    if (c < count) walk(c, a);
    if (live) {
#pragma unroll
        for (int j = 0; j < TILES; ++j) {
            const int ch = ch0 + 16 * j + 4 * g;
            if (ch < dp) *reinterpret_cast<delta_float4*>(s_col + ch) = s[j];
        }
    }
}

// Floats of the scratch for a step of `tokens` tokens in `segments` segments.
WLLM_API long long wllm_delta_chunk_floats(int tokens, int segments, int heads, int d) {
    const int c = (d + 63) / 64 * 64;
    return static_cast<long long>(tokens / kChunk + segments + 1) * heads * static_cast<long long>(chunk_floats(c));
}

// Segments of `from` tokens (16 at least) and more; the others are left alone.
WLLM_API int wllm_delta_chunk_scan(const float* qk, const float* f, const float* beta, const void* v, float* state,
                                   long long state_stride, const int* token_segment, const int* seg_q_start, const int* seg_q_len,
                                   const int* state_slots, float* y, float* chunks, int is_bf16, int tokens, int segments, int heads,
                                   int groups, int d, int p_dim, int from, hipStream_t stream) {
    if (tokens <= 0 || segments <= 0) return 0;
    if (heads <= 0 || heads > 65535 || groups <= 0 || heads % groups || d <= 0 || d > 256 || p_dim <= 0 || segments > 65535 ||
        (p_dim + 15) / 16 > 65535 || from < kChunk || state_stride % 4 || reinterpret_cast<uintptr_t>(state) % 16 ||
        reinterpret_cast<uintptr_t>(chunks) % 16)
        return -1;
    const int dp = (d + 3) / 4 * 4, r = (d + 63) / 64;
    const dim3 chunk_grid((tokens + kChunk - 1) / kChunk, heads), grid(heads, segments, (p_dim + 15) / 16);
#define LAUNCH(T, R)                                                                                                   \
    delta_chunk_kernel<R><<<chunk_grid, 256, 0, stream>>>(qk, f, beta, token_segment, seg_q_start, seg_q_len, chunks, tokens,  \
                                                          heads, groups, dp, from);                                     \
    if (const int err = launch_status()) return err;                                                                   \
    delta_chunk_scan_kernel<T, R><<<grid, 256, 0, stream>>>(chunks, static_cast<const T*>(v), state, state_stride, seg_q_start, \
                                                            seg_q_len, state_slots, y, heads, dp, p_dim, from)
#define LAUNCH_R(T)                     \
    if (r == 1) { LAUNCH(T, 1); }       \
    else if (r == 2) { LAUNCH(T, 2); }  \
    else if (r == 3) { LAUNCH(T, 3); }  \
    else { LAUNCH(T, 4); }
    if (is_bf16) { LAUNCH_R(bf16) } else { LAUNCH_R(float) }
#undef LAUNCH_R
#undef LAUNCH
    return launch_status();
}
