// The residual stream's general norm step, for layers that put a norm behind a sublayer as well as
// before it:   x = norm_s(scale * x + norm_d(delta + extra));   out = norm_o(x)   (scale 1, no norm_s and no extra as a rule).
//
// x float32 [n, H] is the stream.  delta, what a sublayer left (a tensor of the activation type or a
// float32 stack of partial sums added in stack order), is normalised by a norm of its own before it is
// added: none, RMS (d / sqrt(mean(d^2) + eps) * (offset + w)) or layer norm without a bias
// ((d - mean) / sqrt(mean((d - mean)^2) + eps) * (offset + w)).  The sum is written back to x unless
// the rows are gathered (`rows`: logits of a few places; x is then left alone).  `out`, if asked
// for, is the new x under the second norm (the same three kinds; "none" is a cast), in the
// activation type.  Everything is float32: means, variances as means of squared deviations (two
// passes over a row held in shared memory), the sum.  One workgroup a row.
//
// `join` says how the sublayer's result meets the stream where it is not simply added: x is weighed before the sum
// (`scale`), the sum passes a norm of its own (`norm_s`: a layer that norms the sum of stream and sublayer), and the
// result may have a second term (`extra`, a tensor or a stack as delta is), whose rows are multiplied by a number a
// row (`extra_scale`: an expert that every token uses, behind its gate).
//
// `conv` (a step in which every row is its request's one new token): out is not a norm of the new x but the new x
// through a short convolution over time, out[c] = x[c] + sum_k w[k, c] * (the request's k-th carried row, the last tap
// x itself), and the carried rows (float32 [taps - 1, H] from `carried_offset` of row state_slots[row] of `state`)
// move up by one and take x: what `stream_conv` does for single tokens, in the launch that settles the stream.
#include "common.h"

struct NormJoin {
    float scale;               // of x before the sum
    int s_kind;                // the norm of the sum
    const float* s_weight;
    float s_eps, s_offset;
    const void* extra;         // null: none
    int extra_bf16, extra_splits;
    size_t extra_stride;
    const float* extra_scale;  // float32 [n], or null: 1
};

struct NormConv {
    const float* weight;       // [taps, H], a row a tap; null: no convolution
    float* state;
    long long state_stride;
    long long carried_offset;
    const int* state_slots;
    int taps;
};

constexpr int kNormNone = 0, kNormRms = 1, kNormLayer = 2;

// v (a thread's elements of the row, in shared memory `row`) under a norm; returns through `row`.
// Every thread of the workgroup calls it.
__device__ __forceinline__ void row_stats(const float* row, int hidden, int kind, float eps, float* scratch, float& mean,
                                          float& inv) {
    mean = 0.f;
    inv = 1.f;
    if (kind == kNormNone) return;
    const float count = static_cast<float>(hidden);
    if (kind == kNormLayer) {
        float s = 0.f;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) s += row[i];
        mean = block_sum(s, scratch) / count;
    }
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float d = row[i] - mean;
        ss += d * d;
    }
    inv = 1.f / sqrtf(block_sum(ss, scratch) / count + eps);
}

template <typename TD, typename TO>
__global__ void __launch_bounds__(1024)
norm_add_kernel(float* __restrict__ x, const TD* __restrict__ delta, int splits, size_t split_stride, int d_kind,
                const float* __restrict__ d_weight, float d_eps, float d_offset, const int* __restrict__ rows,
                TO* __restrict__ out, int o_kind, const float* __restrict__ o_weight, float o_eps, float o_offset,
                int hidden, NormConv conv, NormJoin join) {
    extern __shared__ float row[];
    __shared__ float scratch[16];
    const int orow = blockIdx.x;
    const int irow = rows ? rows[orow] : orow;
    float* xr = x + static_cast<size_t>(irow) * hidden;
    // The convolution's taps and the carried rows of this thread's (at most two) elements are asked for before anything
    // else, so that they arrive while the sublayer's product is normalised: a row's time is its chain of trips to memory.
    constexpr int kHeldTaps = 8;
    float held_w[2][kHeldTaps], held_c[2][kHeldTaps];
    const bool held = conv.weight && conv.taps <= kHeldTaps && hidden <= 2 * static_cast<int>(blockDim.x);
    if (held) {
        const float* carried = conv.state + static_cast<size_t>(conv.state_slots[orow]) * conv.state_stride + conv.carried_offset;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const int i = threadIdx.x + e * blockDim.x;
#pragma unroll
            for (int k = 0; k < kHeldTaps; ++k) {
                held_w[e][k] = (i < hidden && k < conv.taps) ? conv.weight[static_cast<size_t>(k) * hidden + i] : 0.f;
                held_c[e][k] = (i < hidden && k + 1 < conv.taps) ? carried[static_cast<size_t>(k) * hidden + i] : 0.f;
            }
        }
    }
    if (delta) {
        const TD* dr = delta + static_cast<size_t>(irow) * hidden;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            float d;
            if (sizeof(TD) == sizeof(float) && splits > 1) d = stack_sum(reinterpret_cast<const float*>(dr) + i, splits, split_stride);
            else d = to_float(dr[i]);
            if (join.extra) {
                const size_t at = static_cast<size_t>(irow) * hidden + i;
                float e;
                if (join.extra_bf16) e = to_float(static_cast<const bf16*>(join.extra)[at]);
                else e = stack_sum(static_cast<const float*>(join.extra) + at, join.extra_splits, join.extra_stride);
                d = fmaf(join.extra_scale ? join.extra_scale[irow] : 1.f, e, d);
            }
            row[i] = d;
        }
        __syncthreads();
        float mean, inv;
        row_stats(row, hidden, d_kind, d_eps, scratch, mean, inv);
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            float d = row[i];                       // this thread's own elements: no other thread writes them
            if (d_kind != kNormNone) d = (d - mean) * inv * (d_offset + d_weight[i]);
            const float v = fmaf(join.scale, xr[i], d);
            if (!rows && join.s_kind == kNormNone) xr[i] = v;
            row[i] = v;
        }
        if (join.s_kind != kNormNone) {
            __syncthreads();
            row_stats(row, hidden, join.s_kind, join.s_eps, scratch, mean, inv);
            for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
                const float v = (row[i] - mean) * inv * (join.s_offset + join.s_weight[i]);
                if (!rows) xr[i] = v;
                row[i] = v;
            }
        }
    } else {
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) row[i] = xr[i];
    }
    if (!out) return;
    TO* o = out + static_cast<size_t>(orow) * hidden;
    if (conv.weight) {
        // (a thread's own elements of the row, and its own columns of the carried rows)
        float* carried = conv.state + static_cast<size_t>(conv.state_slots[orow]) * conv.state_stride + conv.carried_offset;
        const int taps = conv.taps;
        if (held) {
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const int i = threadIdx.x + e * blockDim.x;
                if (i >= hidden) break;
                const float now = row[i];
                float acc = now;
#pragma unroll
                for (int k = 0; k < kHeldTaps; ++k) {
                    if (k + 1 < taps) {
                        acc = fmaf(held_w[e][k], held_c[e][k], acc);
                        if (k > 0) carried[static_cast<size_t>(k - 1) * hidden + i] = held_c[e][k];
                    } else if (k + 1 == taps) {
                        acc = fmaf(held_w[e][k], now, acc);
                    }
                }
                if (taps > 1) carried[static_cast<size_t>(taps - 2) * hidden + i] = now;
                o[i] = from_float<TO>(acc);
            }
            return;
        }
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            const float now = row[i];
            float acc = now;
            for (int k = 0; k + 1 < taps; ++k) {
                const float v = carried[static_cast<size_t>(k) * hidden + i];
                acc = fmaf(conv.weight[static_cast<size_t>(k) * hidden + i], v, acc);
                if (k > 0) carried[static_cast<size_t>(k - 1) * hidden + i] = v;
            }
            acc = fmaf(conv.weight[static_cast<size_t>(taps - 1) * hidden + i], now, acc);
            if (taps > 1) carried[static_cast<size_t>(taps - 2) * hidden + i] = now;
            o[i] = from_float<TO>(acc);
        }
        return;
    }
    __syncthreads();
    float mean, inv;
    row_stats(row, hidden, o_kind, o_eps, scratch, mean, inv);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float v = row[i];
        if (o_kind != kNormNone) v = (v - mean) * inv * (o_offset + o_weight[i]);
        o[i] = from_float<TO>(v);
    }
}

// The same for rows of a multiple of four elements, held in registers: a thread keeps G groups of four consecutive
// elements and moves 16 (bfloat16: 8) bytes at a time; everything a row needs is asked for before the first sum.
// CONV: the launch also convolves (`conv_aligned`: the carried rows begin at multiples of 16 bytes).
template <typename T> struct alignas(4 * sizeof(T)) NormFour { T v[4]; };

// Mean and 1 / sqrt(variance + eps) (a norm of kind RMS: mean 0) of the row that the workgroup's threads hold.
template <int G>
__device__ __forceinline__ void held_stats(const float (&v)[G][4], int hidden, int kind, float eps, float* scratch, float& mean,
                                           float& inv) {
    mean = 0.f;
    inv = 1.f;
    if (kind == kNormNone) return;
    const float count = static_cast<float>(hidden);
    if (kind == kNormLayer) {
        float s = 0.f;
#pragma unroll
        for (int e = 0; e < G; ++e) s += (v[e][0] + v[e][1]) + (v[e][2] + v[e][3]);       // (zeros beyond the row)
        mean = block_sum(s, scratch) / count;
    }
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < G; ++e) {
        if (static_cast<int>(threadIdx.x + e * blockDim.x) * 4 < hidden) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float d = v[e][u] - mean;
                ss += d * d;
            }
        }
    }
    inv = 1.f / sqrtf(block_sum(ss, scratch) / count + eps);
}

template <typename TD, typename TO, int G, bool CONV>
__global__ void __launch_bounds__(1024)
norm_add_four_kernel(float* __restrict__ x, const TD* __restrict__ delta, int splits, size_t split_stride, int d_kind,
                     const float* __restrict__ d_weight, float d_eps, float d_offset, const int* __restrict__ rows,
                     TO* __restrict__ out, int o_kind, const float* __restrict__ o_weight, float o_eps, float o_offset,
                     int hidden, NormJoin join, NormConv conv, int conv_aligned) {
    __shared__ float scratch[16];
    const int orow = blockIdx.x;
    const int irow = rows ? rows[orow] : orow;
    // the carried rows (and taps) of this thread's elements, the first ones asked for before anything else
    constexpr int kHeldTaps = CONV ? 4 : 1;
    float* carried = CONV ? conv.state + static_cast<size_t>(conv.state_slots[orow]) * conv.state_stride + conv.carried_offset : nullptr;
    NormFour<float> held_w[CONV ? G : 1][kHeldTaps], held_c[CONV ? G : 1][kHeldTaps];
    auto carried_four = [&](int k, int i) {
        const float* p = carried + static_cast<size_t>(k) * hidden + i;
        if (conv_aligned) return *reinterpret_cast<const NormFour<float>*>(p);
        return NormFour<float>{{p[0], p[1], p[2], p[3]}};
    };
    auto carry_four = [&](int k, int i, const NormFour<float>& t) {
        float* p = carried + static_cast<size_t>(k) * hidden + i;
        if (conv_aligned) {
            *reinterpret_cast<NormFour<float>*>(p) = t;
        } else {
#pragma unroll
            for (int u = 0; u < 4; ++u) p[u] = t.v[u];
        }
    };
    if (CONV) {
#pragma unroll
        for (int e = 0; e < G; ++e) {
            const int i = static_cast<int>(threadIdx.x + e * blockDim.x) * 4;
#pragma unroll
            for (int k = 0; k < kHeldTaps; ++k) {
                held_w[e][k] = held_c[e][k] = NormFour<float>{{0.f, 0.f, 0.f, 0.f}};
                if (i < hidden && k < conv.taps)
                    held_w[e][k] = *reinterpret_cast<const NormFour<float>*>(conv.weight + static_cast<size_t>(k) * hidden + i);
                if (i < hidden && k + 1 < conv.taps) held_c[e][k] = carried_four(k, i);
            }
        }
    }
    const size_t base = static_cast<size_t>(irow) * hidden;
    float xv[G][4], d[G][4], w[G][4];
    auto at = [&](int e) { return static_cast<int>(threadIdx.x + e * blockDim.x) * 4; };
    auto weights = [&](const float* from) {
#pragma unroll
        for (int e = 0; e < G; ++e) {
            NormFour<float> t = {{0.f, 0.f, 0.f, 0.f}};
            if (at(e) < hidden) t = *reinterpret_cast<const NormFour<float>*>(from + at(e));
#pragma unroll
            for (int u = 0; u < 4; ++u) w[e][u] = t.v[u];
        }
    };
    // a stack's slices at one place, added in order, several asked for at a time
    auto stack = [&](const float* from, int count, size_t stride, float (&sum)[4]) {
        NormFour<float> t = *reinterpret_cast<const NormFour<float>*>(from);
#pragma unroll
        for (int u = 0; u < 4; ++u) sum[u] = t.v[u];
        constexpr int kAhead = 8;
        for (int s0 = 1; s0 < count; s0 += kAhead) {
            NormFour<float> q[kAhead];
#pragma unroll
            for (int j = 0; j < kAhead; ++j)
                q[j] = *reinterpret_cast<const NormFour<float>*>(from + static_cast<size_t>(min(s0 + j, count - 1)) * stride);
#pragma unroll
            for (int j = 0; j < kAhead; ++j) {
                if (s0 + j >= count) break;
#pragma unroll
                for (int u = 0; u < 4; ++u) sum[u] += q[j].v[u];
            }
        }
    };
    const float extra_scale = join.extra && join.extra_scale ? join.extra_scale[irow] : 1.f;
    if (delta && d_kind != kNormNone) weights(d_weight);
    else if (delta && join.s_kind != kNormNone) weights(join.s_weight);
    else if (out && o_kind != kNormNone) weights(o_weight);
#pragma unroll
    for (int e = 0; e < G; ++e) {
        const int i = at(e);
#pragma unroll
        for (int u = 0; u < 4; ++u) xv[e][u] = d[e][u] = 0.f;
        if (i >= hidden) continue;
        const NormFour<float> t = *reinterpret_cast<const NormFour<float>*>(x + base + i);
#pragma unroll
        for (int u = 0; u < 4; ++u) xv[e][u] = t.v[u];
        if (!delta) continue;
        if (sizeof(TD) == sizeof(float)) {
            stack(reinterpret_cast<const float*>(delta) + base + i, splits, split_stride, d[e]);
        } else {
            const NormFour<TD> q = *reinterpret_cast<const NormFour<TD>*>(delta + base + i);
#pragma unroll
            for (int u = 0; u < 4; ++u) d[e][u] = to_float(q.v[u]);
        }
        if (join.extra) {
            float more[4];
            if (join.extra_bf16) {
                const NormFour<bf16> q = *reinterpret_cast<const NormFour<bf16>*>(static_cast<const bf16*>(join.extra) + base + i);
#pragma unroll
                for (int u = 0; u < 4; ++u) more[u] = to_float(q.v[u]);
            } else {
                stack(static_cast<const float*>(join.extra) + base + i, join.extra_splits, join.extra_stride, more);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) d[e][u] = fmaf(extra_scale, more[u], d[e][u]);
        }
    }
    float mean, inv;
    if (delta) {
        if (d_kind != kNormNone) {
            held_stats<G>(d, hidden, d_kind, d_eps, scratch, mean, inv);
#pragma unroll
            for (int e = 0; e < G; ++e)
#pragma unroll
                for (int u = 0; u < 4; ++u) d[e][u] = (d[e][u] - mean) * inv * (d_offset + w[e][u]);
            if (join.s_kind != kNormNone) weights(join.s_weight);
            else if (out && o_kind != kNormNone) weights(o_weight);
        }
#pragma unroll
        for (int e = 0; e < G; ++e)
#pragma unroll
            for (int u = 0; u < 4; ++u) xv[e][u] = at(e) < hidden ? fmaf(join.scale, xv[e][u], d[e][u]) : 0.f;
        if (join.s_kind != kNormNone) {
            held_stats<G>(xv, hidden, join.s_kind, join.s_eps, scratch, mean, inv);
#pragma unroll
            for (int e = 0; e < G; ++e)
#pragma unroll
                for (int u = 0; u < 4; ++u)
                    xv[e][u] = at(e) < hidden ? (xv[e][u] - mean) * inv * (join.s_offset + w[e][u]) : 0.f;
            if (out && o_kind != kNormNone) weights(o_weight);
        } else if (d_kind == kNormNone && out && o_kind != kNormNone) {
            weights(o_weight);
        }
        if (!rows) {
#pragma unroll
            for (int e = 0; e < G; ++e) {
                if (at(e) >= hidden) continue;
                NormFour<float> t;
#pragma unroll
                for (int u = 0; u < 4; ++u) t.v[u] = xv[e][u];
                *reinterpret_cast<NormFour<float>*>(x + base + at(e)) = t;
            }
        }
    }
    if (!out) return;
    if (CONV) {
        // (a thread's own columns of the carried rows: each moves up by one as it is read)
        const int taps = conv.taps;
#pragma unroll
        for (int e = 0; e < G; ++e) {
            const int i = at(e);
            if (i >= hidden) continue;
            NormFour<float> now, acc;
#pragma unroll
            for (int u = 0; u < 4; ++u) now.v[u] = acc.v[u] = xv[e][u];
            auto tap = [&](const NormFour<float>& wv, const NormFour<float>& v) {
#pragma unroll
                for (int u = 0; u < 4; ++u) acc.v[u] = fmaf(wv.v[u], v.v[u], acc.v[u]);
            };
#pragma unroll
            for (int k = 0; k < kHeldTaps; ++k) {
                if (k + 1 < taps) {
                    tap(held_w[e][k], held_c[e][k]);
                    if (k > 0) carry_four(k - 1, i, held_c[e][k]);
                } else if (k + 1 == taps) {
                    tap(held_w[e][k], now);
                }
            }
            for (int k = kHeldTaps; k < taps; ++k) {
                const NormFour<float> wv = *reinterpret_cast<const NormFour<float>*>(conv.weight + static_cast<size_t>(k) * hidden + i);
                if (k + 1 < taps) {
                    const NormFour<float> v = carried_four(k, i);
                    tap(wv, v);
                    carry_four(k - 1, i, v);
                } else {
                    tap(wv, now);
                }
            }
            if (taps > 1) carry_four(taps - 2, i, now);
            NormFour<TO> t;
#pragma unroll
            for (int u = 0; u < 4; ++u) t.v[u] = from_float<TO>(acc.v[u]);
            *reinterpret_cast<NormFour<TO>*>(out + static_cast<size_t>(orow) * hidden + i) = t;
        }
        return;
    }
    held_stats<G>(xv, hidden, o_kind, o_eps, scratch, mean, inv);
    TO* o = out + static_cast<size_t>(orow) * hidden;
#pragma unroll
    for (int e = 0; e < G; ++e) {
        if (at(e) >= hidden) continue;
        NormFour<TO> t;
#pragma unroll
        for (int u = 0; u < 4; ++u)
            t.v[u] = from_float<TO>(o_kind != kNormNone ? (xv[e][u] - mean) * inv * (o_offset + w[e][u]) : xv[e][u]);
        *reinterpret_cast<NormFour<TO>*>(o + at(e)) = t;
    }
}

// delta_type / out_type: 0 float32, 1 bfloat16.  Returns 0, a HIP error code, or -1 for sizes it does not take.
WLLM_API int wllm_norm_add(float* x, const void* delta, int delta_type, int splits, long long split_stride, int d_kind,
                           const float* d_weight, float d_eps, float d_offset, const int* rows, void* out, int out_type,
                           int o_kind, const float* o_weight, float o_eps, float o_offset, int num_rows, int hidden,
                           const float* conv_weight, int conv_taps, float* conv_state, long long conv_state_stride,
                           long long conv_carried_offset, const int* conv_state_slots, float x_scale, int s_kind,
                           const float* s_weight, float s_eps, float s_offset, const void* extra, int extra_bf16,
                           int extra_splits, long long extra_stride, const float* extra_scale, hipStream_t stream) {
    if (num_rows <= 0) return 0;
    if (conv_weight && (!out || rows || o_kind != kNormNone || conv_taps < 1 || conv_taps > 64 || !conv_state || !conv_state_slots))
        return -1;
    const NormConv conv{conv_weight, conv_state, conv_state_stride, conv_carried_offset, conv_state_slots, conv_taps};
    if (s_kind < 0 || s_kind > 2 || (s_kind != kNormNone && !s_weight)) return -1;
    // what joins the stream by a weight, a norm or a second term is a sublayer's result
    if (!delta && (extra || s_kind != kNormNone || x_scale != 1.f)) return -1;
    if (extra && extra_splits < 1) return -1;
    const NormJoin join{x_scale, s_kind, s_weight, s_eps, s_offset, extra, extra_bf16, extra_splits,
                        static_cast<size_t>(extra_stride), extra_scale};
    if (hidden <= 0 || hidden > 16384 || !x) return -1;
    if (d_kind < 0 || d_kind > 2 || o_kind < 0 || o_kind > 2) return -1;
    if (delta && d_kind != kNormNone && !d_weight) return -1;
    if (out && o_kind != kNormNone && !o_weight) return -1;
    if (!delta && !out) return 0;
    auto aligned = [](const void* p, size_t bytes) { return reinterpret_cast<uintptr_t>(p) % bytes == 0; };
    const bool four = hidden % 4 == 0 && hidden <= 4096 * 4 && (splits <= 1 || split_stride % 4 == 0) &&
                      (!extra || extra_splits <= 1 || extra_stride % 4 == 0) && aligned(x, 16) && aligned(delta, 16) && aligned(out, 16) &&
                      aligned(extra, 16) && aligned(d_weight, 16) && aligned(o_weight, 16) && aligned(s_weight, 16) && aligned(conv_weight, 16);
    const int conv_aligned = conv_state_stride % 4 == 0 && conv_carried_offset % 4 == 0 && aligned(conv_state, 16);
    if (four) {
        // many rows: groups of four a thread so that some workgroups share a compute unit; few rows: one, so that a row's
        // loads are all on their way at once
        const int quads = hidden / 4;
        const int groups = quads > 2048 ? 4 : quads > 1024 ? 2 : num_rows <= 256 || quads <= 256 ? 1 : 2;
        const int four_threads = ((quads + groups - 1) / groups + 63) / 64 * 64;
#define LAUNCH_C(TD, TO, G, CONV)                                                                                      \
    norm_add_four_kernel<TD, TO, G, CONV><<<num_rows, four_threads, 0, stream>>>(                                      \
        x, static_cast<const TD*>(delta), splits, static_cast<size_t>(split_stride), d_kind, d_weight, d_eps, d_offset, rows, \
        static_cast<TO*>(out), o_kind, o_weight, o_eps, o_offset, hidden, join, conv, conv_aligned)
#define LAUNCH_G(TD, TO, G) do { if (conv_weight) LAUNCH_C(TD, TO, G, true); else LAUNCH_C(TD, TO, G, false); } while (0)
#define LAUNCH(TD, TO)                          \
    if (groups == 1) LAUNCH_G(TD, TO, 1);       \
    else if (groups == 2) LAUNCH_G(TD, TO, 2);  \
    else LAUNCH_G(TD, TO, 4)
        if (delta_type && out_type) { LAUNCH(bf16, bf16); }
        else if (delta_type) { LAUNCH(bf16, float); }
        else if (out_type) { LAUNCH(float, bf16); }
        else { LAUNCH(float, float); }
#undef LAUNCH
#undef LAUNCH_G
#undef LAUNCH_C
        return launch_status();
    }
    const size_t smem = sizeof(float) * static_cast<size_t>(hidden);
    // The few rows of a decode step: a row's time is that of its chain of trips to memory (a stack of partial
    // sums to add, the stream, the weights), so as many threads as give each two elements; many rows: 256.
    int threads = 256;
    if (num_rows <= 256) {
        threads = (hidden / 2 + 63) / 64 * 64;
        threads = threads < 64 ? 64 : (threads > 1024 ? 1024 : threads);
    }
#define LAUNCH(TD, TO)                                                                                               \
    norm_add_kernel<TD, TO><<<num_rows, threads, smem, stream>>>(x, static_cast<const TD*>(delta), splits,            \
                                                              static_cast<size_t>(split_stride), d_kind, d_weight,   \
                                                              d_eps, d_offset, rows, static_cast<TO*>(out), o_kind,   \
                                                              o_weight, o_eps, o_offset, hidden, conv, join)
    if (delta_type && out_type) LAUNCH(bf16, bf16);
    else if (delta_type) LAUNCH(bf16, float);
    else if (out_type) LAUNCH(float, bf16);
    else LAUNCH(float, float);
#undef LAUNCH
    return launch_status();
}

// ---- RMS norm of a band of columns of every row, with a weight: out = v / sqrt(sum(v^2) / count + eps) * w,
// where v is the band, plus a bias (float32, one a column) if the band has one: a projection's bias that
// belongs in front of its norm.  The band [rows, cols] lies in a wider tensor (row stride); `count` is the number of elements the
// mean is taken over (less than cols where a band carries padding that is always zero); out may be
// the band itself or another band, and where it is wider than cols the further columns become zero.
// Up to two bands a launch (blockIdx.y), each with its own operands. ----
struct NormBand {
    const void* src;
    long long src_stride;
    int cols;
    const float* weight;
    float count;
    void* out;
    long long out_stride;
    int out_cols;
    const float* bias;
};

template <typename T>
__global__ void __launch_bounds__(256) band_norm_kernel(NormBand b0, NormBand b1, float eps) {
    __shared__ float scratch[16];
    const NormBand b = blockIdx.y == 0 ? b0 : b1;
    const T* s = static_cast<const T*>(b.src) + static_cast<size_t>(blockIdx.x) * b.src_stride;
    T* o = static_cast<T*>(b.out) + static_cast<size_t>(blockIdx.x) * b.out_stride;
    float ss = 0.f;
    for (int i = threadIdx.x; i < b.cols; i += blockDim.x) {
        const float v = to_float(s[i]) + (b.bias ? b.bias[i] : 0.f);
        ss += v * v;
    }
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / b.count + eps);
    for (int i = threadIdx.x; i < b.out_cols; i += blockDim.x)
        o[i] = from_float<T>(i < b.cols ? (to_float(s[i]) + (b.bias ? b.bias[i] : 0.f)) * inv * b.weight[i] : 0.f);
}

WLLM_API int wllm_band_norm(const void* src0, long long src_stride0, int cols0, const float* weight0, float count0,
                            void* out0, long long out_stride0, int out_cols0, const float* bias0, const void* src1,
                            long long src_stride1, int cols1, const float* weight1, float count1, void* out1,
                            long long out_stride1, int out_cols1, const float* bias1, float eps, int is_bf16, int rows,
                            hipStream_t stream) {
    if (rows <= 0) return 0;
    if (!src0 || !out0 || !weight0 || cols0 <= 0 || out_cols0 < cols0 || !(count0 > 0.f)) return -1;
    if (src1 && (!out1 || !weight1 || cols1 <= 0 || out_cols1 < cols1 || !(count1 > 0.f))) return -1;
    const NormBand b0{src0, src_stride0, cols0, weight0, count0, out0, out_stride0, out_cols0, bias0};
    const NormBand b1{src1, src_stride1, cols1, weight1, count1, out1, out_stride1, out_cols1, bias1};
    const dim3 grid(rows, src1 ? 2 : 1);
    if (is_bf16) band_norm_kernel<bf16><<<grid, 256, 0, stream>>>(b0, b1, eps);
    else band_norm_kernel<float><<<grid, 256, 0, stream>>>(b0, b1, eps);
    return launch_status();
}

// ---- out[r, c] = act(gate[r, c]) * table[ids[r], col0 + c]: a small projection of the stream,
// bent and multiplied by the token's own entry of a table (a band of `cols` columns of its row) ----
template <typename T, int ACT>
__global__ void gated_lookup_kernel(const T* __restrict__ gate, const int* __restrict__ ids, const T* __restrict__ table,
                                    long long table_stride, int col0, T* __restrict__ out, int rows, int cols) {
    const long long total = static_cast<long long>(rows) * cols;
    for (long long e = blockIdx.x * static_cast<long long>(blockDim.x) + threadIdx.x; e < total;
         e += static_cast<long long>(gridDim.x) * blockDim.x) {
        const int r = static_cast<int>(e / cols), c = static_cast<int>(e - static_cast<long long>(r) * cols);
        const float entry = to_float(table[static_cast<size_t>(ids[r]) * table_stride + col0 + c]);
        out[e] = from_float<T>(activate<ACT>(to_float(gate[e])) * entry);
    }
}

WLLM_API int wllm_gated_lookup(const void* gate, const int* ids, const void* table, long long table_stride, int col0,
                               void* out, int is_bf16, int activation, int rows, int cols, hipStream_t stream) {
    if (rows <= 0 || cols <= 0) return 0;
    if (activation < 0 || activation >= kActivations || col0 < 0 || col0 + cols > table_stride) return -1;
    const long long total = static_cast<long long>(rows) * cols;
    const int blocks = static_cast<int>(total / 256 + 1 < 4096 ? total / 256 + 1 : 4096);
#define LAUNCH(T)                                                                                                     \
    WLLM_BY_ACTIVATION(activation, (gated_lookup_kernel<T, ACT><<<blocks, 256, 0, stream>>>(                           \
                                       static_cast<const T*>(gate), ids, static_cast<const T*>(table), table_stride,  \
                                       col0, static_cast<T*>(out), rows, cols)))
    if (is_bf16) { LAUNCH(bf16); } else { LAUNCH(float); }
#undef LAUNCH
    return launch_status();
}

// ---- a product head by head: y[r, h * O + o] = sum_k x[r, h * K + k] * w[h, o, k].  x and y are
// bands of wider tensors (row strides); w is [heads, O, K].  float32 sums in ascending order of k,
// so a row's result does not depend on the rows beside it.  bfloat16 goes to the matrix cores (further
// below) where its rows are aligned; the kernels on the vector units here take everything.  A workgroup makes 32 rows by 64 outputs
// of one head, a thread 2 by 4 of them, from chunks of 32 keys staged in shared memory. ----
constexpr int kHlRows = 32, kHlOuts = 64, kHlKeys = 32;

template <typename T>
__global__ void __launch_bounds__(256)
head_linear_kernel(const T* __restrict__ x, long long x_stride, const T* __restrict__ w, T* __restrict__ y,
                   long long y_stride, int rows, int heads, int outs, int keys) {
    __shared__ float xs[kHlRows][kHlKeys + 1];
    __shared__ float ws[kHlOuts][kHlKeys + 1];
    const int h = blockIdx.y;
    const int r0 = blockIdx.x * kHlRows, o0 = blockIdx.z * kHlOuts;
    const int tx = threadIdx.x % 16, ty = threadIdx.x / 16;       // outputs 4 tx .. +4, rows 2 ty .. +2
    const T* wh = w + static_cast<size_t>(h) * outs * keys;
    float acc[2][4] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    for (int k0 = 0; k0 < keys; k0 += kHlKeys) {
        for (int e = threadIdx.x; e < kHlRows * kHlKeys; e += blockDim.x) {
            const int r = e / kHlKeys, k = e % kHlKeys;
            xs[r][k] = (r0 + r < rows && k0 + k < keys)
                           ? to_float(x[static_cast<size_t>(r0 + r) * x_stride + static_cast<size_t>(h) * keys + k0 + k]) : 0.f;
        }
        for (int e = threadIdx.x; e < kHlOuts * kHlKeys; e += blockDim.x) {
            const int o = e / kHlKeys, k = e % kHlKeys;
            ws[o][k] = (o0 + o < outs && k0 + k < keys) ? to_float(wh[static_cast<size_t>(o0 + o) * keys + k0 + k]) : 0.f;
        }
        __syncthreads();
#pragma unroll 8
        for (int k = 0; k < kHlKeys; ++k) {
            const float a0 = xs[2 * ty][k], a1 = xs[2 * ty + 1][k];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float b = ws[4 * tx + j][k];
                acc[0][j] = fmaf(a0, b, acc[0][j]);
                acc[1][j] = fmaf(a1, b, acc[1][j]);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int r = r0 + 2 * ty + i;
        if (r >= rows) continue;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int o = o0 + 4 * tx + j;
            if (o < outs) y[static_cast<size_t>(r) * y_stride + static_cast<size_t>(h) * outs + o] = from_float<T>(acc[i][j]);
        }
    }
}

// The few rows of a decode step: a workgroup takes one head and 64 outputs, all rows (at most 16).  Thread
// (o, q) multiplies the q-th quarter of output o's row of w (read once, in runs of consecutive elements) with
// every row of x, which lies in shared memory; the quarters are added in ascending order, so the sum's order
// is k ascending within a quarter and quarter by quarter.
constexpr int kHlFewRows = 16;

template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
head_linear_few_kernel(const T* __restrict__ x, long long x_stride, const T* __restrict__ w, T* __restrict__ y,
                       long long y_stride, int rows, int heads, int outs, int keys) {
    extern __shared__ float hl_smem[];
    float* xs = hl_smem;                                  // [rows][keys]
    float* part = hl_smem + rows * keys;                  // [4][rows][64]
    const int h = blockIdx.x, o0 = blockIdx.y * kHlOuts;
    for (int e = threadIdx.x; e < rows * keys; e += blockDim.x) {
        const int r = e / keys, k = e - r * keys;
        xs[e] = to_float(x[static_cast<size_t>(r) * x_stride + static_cast<size_t>(h) * keys + k]);
    }
    __syncthreads();
    const int o = threadIdx.x % kHlOuts, q = threadIdx.x / kHlOuts;
    const int per = (keys + 3) / 4, k_begin = q * per, k_end = min(keys, k_begin + per);
    float acc[kHlFewRows];
#pragma unroll
    for (int r = 0; r < kHlFewRows; ++r) acc[r] = 0.f;
    if (o0 + o < outs) {
        const T* wr = w + (static_cast<size_t>(h) * outs + o0 + o) * keys;
        if (VEC) {
            // the quarter is a whole number of 16-byte pieces that begin at multiples of 16 bytes: the row of w
            // streams in as such pieces, several asked for before the first is multiplied
            constexpr int kPiece = 16 / sizeof(T);
#pragma unroll 4
            for (int k = k_begin; k < k_end; k += kPiece) {
                const uint4 piece = load_streamed(wr + k);
                float wv[kPiece];
                if (sizeof(T) == 2) {
                    const uint32_t words[4] = {piece.x, piece.y, piece.z, piece.w};
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        wv[2 * j] = __uint_as_float(words[j] << 16);
                        wv[2 * j + 1] = __uint_as_float(words[j] & 0xffff0000u);
                    }
                } else {
                    wv[0] = __uint_as_float(piece.x);
                    wv[1] = __uint_as_float(piece.y);
                    wv[2] = __uint_as_float(piece.z);
                    wv[3] = __uint_as_float(piece.w);
                }
#pragma unroll
                for (int j = 0; j < kPiece; ++j)
#pragma unroll
                    for (int r = 0; r < kHlFewRows; ++r)
                        if (r < rows) acc[r] = fmaf(xs[r * keys + k + j], wv[j], acc[r]);
            }
        } else {
            for (int k = k_begin; k < k_end; ++k) {
                const float wv = to_float(wr[k]);
#pragma unroll
                for (int r = 0; r < kHlFewRows; ++r)
                    if (r < rows) acc[r] = fmaf(xs[r * keys + k], wv, acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < kHlFewRows; ++r)
        if (r < rows) part[(q * rows + r) * kHlOuts + o] = acc[r];
    __syncthreads();
    for (int e = threadIdx.x; e < rows * kHlOuts; e += blockDim.x) {
        const int r = e / kHlOuts, oo = e % kHlOuts;
        if (o0 + oo >= outs) continue;
        float total = part[r * kHlOuts + oo];
#pragma unroll
        for (int qq = 1; qq < 4; ++qq) total += part[(qq * rows + r) * kHlOuts + oo];
        y[static_cast<size_t>(r) * y_stride + static_cast<size_t>(h) * outs + o0 + oo] = from_float<T>(total);
    }
}

// The same for bfloat16 on the matrix cores (keys in multiples of 8, rows that begin at multiples of 16 bytes).  A
// wavefront makes 16 MT rows by 16 NT outputs of one head with v_mfma_f32_16x16x32_bf16: w is the A operand (lane
// (i, g) holds keys 8 g .. + 7 of output i), x the B operand (the same keys of row i), both straight from memory, 16
// bytes a lane; the result lands as four consecutive outputs of row i a lane.  The keys go by in steps of 32 from the
// first, the last step filled with zeros, whatever MT and NT are, so a row has the same bits in any batch.
typedef __bf16 hl_bf16x8 __attribute__((ext_vector_type(8)));
typedef float hl_float4 __attribute__((ext_vector_type(4)));
union HlFrag {
    uint4 u;
    hl_bf16x8 v;
};

template <int MT, int NT>
__global__ void __launch_bounds__(256)
head_linear_mfma_kernel(const bf16* __restrict__ x, long long x_stride, const bf16* __restrict__ w, bf16* __restrict__ y,
                        long long y_stride, int rows, int outs, int keys, int out_tiles, int tiles, int whole_stores) {
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int i = lane % 16, g = lane / 16;
    const int h = blockIdx.y, tile = blockIdx.x * (blockDim.x / kWave) + wave;
    if (tile >= tiles) return;
    const int o0 = (tile % out_tiles) * 16 * NT, r0 = (tile / out_tiles) * 16 * MT;
    // rows and outputs beyond the last read the last one: what comes of them is not written
    const bf16* wp[NT];
    const bf16* xp[MT];
#pragma unroll
    for (int a = 0; a < NT; ++a)
        wp[a] = w + (static_cast<size_t>(h) * outs + min(o0 + 16 * a + i, outs - 1)) * keys + 8 * g;
#pragma unroll
    for (int b = 0; b < MT; ++b)
        xp[b] = x + static_cast<size_t>(min(r0 + 16 * b + i, rows - 1)) * x_stride + static_cast<size_t>(h) * keys + 8 * g;
    hl_float4 acc[NT][MT];
#pragma unroll
    for (int a = 0; a < NT; ++a)
#pragma unroll
        for (int b = 0; b < MT; ++b) acc[a][b] = hl_float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 0; k < keys; k += 32) {
        const bool in = k + 8 * g < keys;
        HlFrag fw[NT], fx[MT];
#pragma unroll
        for (int a = 0; a < NT; ++a) fw[a].u = in ? *reinterpret_cast<const uint4*>(wp[a] + k) : make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int b = 0; b < MT; ++b) fx[b].u = in ? *reinterpret_cast<const uint4*>(xp[b] + k) : make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int a = 0; a < NT; ++a)
#pragma unroll
            for (int b = 0; b < MT; ++b)
                acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fw[a].v, fx[b].v, acc[a][b], 0, 0, 0);
    }
#pragma unroll
    for (int b = 0; b < MT; ++b) {
        const int r = r0 + 16 * b + i;
        if (r >= rows) continue;
        bf16* yr = y + static_cast<size_t>(r) * y_stride + static_cast<size_t>(h) * outs;
#pragma unroll
        for (int a = 0; a < NT; ++a) {
            const int o = o0 + 16 * a + 4 * g;
            if (whole_stores && o + 3 < outs) {
                uint2 p;
                p.x = pack2_bf16(acc[a][b][0], acc[a][b][1]);
                p.y = pack2_bf16(acc[a][b][2], acc[a][b][3]);
                *reinterpret_cast<uint2*>(yr + o) = p;
            } else {
#pragma unroll
                for (int v = 0; v < 4; ++v)
                    if (o + v < outs) yr[o + v] = from_float<bf16>(acc[a][b][v]);
            }
        }
    }
}

static int head_linear_mfma(const bf16* x, long long x_stride, const bf16* w, bf16* y, long long y_stride, int rows, int heads,
                            int outs, int keys, hipStream_t stream) {
    const int whole = outs % 4 == 0 && y_stride % 4 == 0 && reinterpret_cast<uintptr_t>(y) % 8 == 0;
    const int mt = rows <= 16 ? 1 : rows <= 32 ? 2 : 4;
    // four tiles of outputs a wavefront where about a thousand wavefronts remain
    const long long row_tiles = (rows + 16 * mt - 1) / (16 * mt);
    const int nt = mt == 4 && row_tiles * ((outs + 63) / 64) * heads >= 1024 ? 4 : 1;
    const int out_tiles = (outs + 16 * nt - 1) / (16 * nt);
    const long long tiles = row_tiles * out_tiles;
    const int waves = tiles * heads >= 1024 ? 4 : 1;
    if (tiles > 0x7fffffffLL) return -1;
    const dim3 grid(static_cast<unsigned>((tiles + waves - 1) / waves), heads);
#define LAUNCH(MT, NT)                                                                                                 \
    head_linear_mfma_kernel<MT, NT><<<grid, waves * kWave, 0, stream>>>(x, x_stride, w, y, y_stride, rows, outs, keys, \
                                                                        out_tiles, static_cast<int>(tiles), whole)
    if (mt == 1) LAUNCH(1, 1);
    else if (mt == 2) LAUNCH(2, 1);
    else if (nt == 1) LAUNCH(4, 1);
    else LAUNCH(4, 4);
#undef LAUNCH
    return launch_status();
}

WLLM_API int wllm_head_linear(const void* x, long long x_stride, const void* w, void* y, long long y_stride, int is_bf16,
                              int rows, int heads, int outs, int keys, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (heads <= 0 || outs <= 0 || keys <= 0 || heads > 65535) return -1;
    // (the last row's band may end where the tensor does: whole pieces of 8 keys stay inside it)
    if (is_bf16 && keys % 8 == 0 && x_stride % 8 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 &&
        reinterpret_cast<uintptr_t>(w) % 16 == 0)
        return head_linear_mfma(static_cast<const bf16*>(x), x_stride, static_cast<const bf16*>(w), static_cast<bf16*>(y), y_stride,
                                rows, heads, outs, keys, stream);
    const dim3 grid((rows + kHlRows - 1) / kHlRows, heads, (outs + kHlOuts - 1) / kHlOuts);
    if (grid.z > 65535) return -1;
    const size_t smem = sizeof(float) * (static_cast<size_t>(rows) * keys + 4 * static_cast<size_t>(rows) * kHlOuts);
    if (rows <= kHlFewRows && smem <= 48 * 1024) {
        const dim3 few(heads, (outs + kHlOuts - 1) / kHlOuts);
        // whole 16-byte pieces a quarter of a row of w, each at a multiple of 16 bytes
        const int piece = is_bf16 ? 8 : 4;
        const bool vec = keys % (4 * piece) == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0;
#define LAUNCH_FEW(T, V)                                                                                               \
    head_linear_few_kernel<T, V><<<few, 256, smem, stream>>>(static_cast<const T*>(x), x_stride, static_cast<const T*>(w), \
                                                             static_cast<T*>(y), y_stride, rows, heads, outs, keys)
        if (is_bf16) { if (vec) LAUNCH_FEW(bf16, true); else LAUNCH_FEW(bf16, false); }
        else { if (vec) LAUNCH_FEW(float, true); else LAUNCH_FEW(float, false); }
#undef LAUNCH_FEW
        return launch_status();
    }
    if (is_bf16)
        head_linear_kernel<bf16><<<grid, 256, 0, stream>>>(static_cast<const bf16*>(x), x_stride, static_cast<const bf16*>(w),
                                                           static_cast<bf16*>(y), y_stride, rows, heads, outs, keys);
    else
        head_linear_kernel<float><<<grid, 256, 0, stream>>>(static_cast<const float*>(x), x_stride,
                                                            static_cast<const float*>(w), static_cast<float*>(y), y_stride,
                                                            rows, heads, outs, keys);
    return launch_status();
}
