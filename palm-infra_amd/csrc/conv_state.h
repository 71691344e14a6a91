// The kept inputs of a short causal convolution over time, a channel at a time: [slots, taps - 1, channels], oldest first,
// zero for a sequence that has just begun.
#pragma once
#include "common.h"

constexpr int CONV_MAX_TAPS = 16;

// After the convolution has read the old state: the last taps-1 inputs of each sequence, old ones moved up.
template <typename T>
__global__ void conv_state_kernel(const T* __restrict__ x, int x_stride, float* __restrict__ conv_state,
                                  const int* __restrict__ seq_slot, const int* __restrict__ seq_new,
                                  const int* __restrict__ cu_new, int channels, int taps) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x, b = blockIdx.y;
    if (c >= channels) return;
    const int n_new = seq_new[b];
    if (n_new <= 0) return;
    const size_t row0 = (size_t)cu_new[b];
    float* st = conv_state + (size_t)seq_slot[b] * (taps - 1) * channels;
    float keep[CONV_MAX_TAPS];
#pragma unroll
    for (int j = 0; j < CONV_MAX_TAPS; ++j) {
        if (j < taps - 1) {
            const int at = n_new - (taps - 1) + j;
            keep[j] = at >= 0 ? to_float(x[(row0 + at) * x_stride + c]) : st[(size_t)(taps - 1 + at) * channels + c];
        }
    }
#pragma unroll
    for (int j = 0; j < CONV_MAX_TAPS; ++j)
        if (j < taps - 1) st[(size_t)j * channels + c] = keep[j];
}
