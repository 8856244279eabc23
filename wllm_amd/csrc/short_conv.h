// The short causal convolution over time on the channels of a flat batch of segments, for the kernels that need it: its
// value at one token and channel, and the rows that a request carries to its next step.
#pragma once
#include "common.h"

// silu(sum_k w[k, c] * in[t - (taps - 1) + k, c]) for channel `c` of the token whose inputs begin at `now` (place `local`
// of its segment; its neighbours' inputs lie `stride` elements before and behind); inputs before the segment's first
// token are the request's carried rows [taps - 1, channels], the oldest first.  w is a row a tap.  The sum runs over the
// taps in ascending order.  CARRY (the segment is this one token): the carried rows move up by one, this token's input
// behind them, each by the thread that reads its channel.
template <typename T, bool CARRY>
__device__ __forceinline__ float short_conv(const T* now, long long stride, int local, float* carried, const float* w,
                                            int channels, int taps, int c) {
    float acc = 0.f;
    const float mine = to_float(now[c]);
    for (int k = 0; k + 1 < taps; ++k) {
        const int back = taps - 1 - k;           // how many tokens ago
        float v;
        if (CARRY || local < back) {
            v = carried[static_cast<size_t>(k + (CARRY ? 0 : local)) * channels + c];
            if (CARRY && k > 0) carried[static_cast<size_t>(k - 1) * channels + c] = v;
        } else {
            v = to_float(now[c - back * stride]);
        }
        acc = fmaf(w[static_cast<size_t>(k) * channels + c], v, acc);
    }
    if (CARRY && taps > 1) carried[static_cast<size_t>(taps - 2) * channels + c] = mine;
    acc = fmaf(w[static_cast<size_t>(taps - 1) * channels + c], mine, acc);
    return acc / (1.f + expf(-acc));
}

// ---- after the convolution of a step: the carried rows take the segment's last taps - 1 inputs (of
// a segment shorter than that, the carried rows move up).  Row j's new value comes from a row above
// it or from the step's inputs, so a thread that walks j upwards never reads what it wrote. ----
template <typename T>
static __global__ void __launch_bounds__(256)
conv_carry_kernel(const T* __restrict__ in, long long in_stride, float* __restrict__ state, long long state_stride,
                  long long carried_offset, const int* __restrict__ seg_q_start, const int* __restrict__ seg_q_len,
                  const int* __restrict__ state_slots, int channels, int taps) {
    const int seg = blockIdx.x;
    const int q_len = seg_q_len[seg], q_start = seg_q_start[seg];
    if (q_len <= 0) return;
    float* carried = state + static_cast<size_t>(state_slots[seg]) * state_stride + carried_offset;
    for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < channels; c += gridDim.y * blockDim.x) {
        for (int j = 0; j < taps - 1; ++j) {
            const int src = q_len - (taps - 1) + j;
            carried[static_cast<size_t>(j) * channels + c] =
                src >= 0 ? to_float(in[static_cast<size_t>(q_start + src) * in_stride + c])
                         : carried[static_cast<size_t>(j + q_len) * channels + c];
        }
    }
}
