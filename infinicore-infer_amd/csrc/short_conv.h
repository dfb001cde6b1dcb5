// A short causal convolution per channel, shared by the kernels that apply it on the way in: the value at a token, and
// the move of the state (a request's last taps - 1 inputs, oldest first, float32 [taps - 1, C]).
#pragma once
#include "common.h"

constexpr int kConvMaxTaps = 8;

// sum_k w[c, k] in(t - (taps - 1 - k), c); inputs before the step's first row `start` of the request come from its state.
template <typename T>
__device__ __forceinline__ float conv_at(const T* __restrict__ x, int x_stride, const float* __restrict__ w, int taps, int C,
                                         const float* __restrict__ st, int t, int start, int c) {
    if (taps == 0) return to_f32(x[(size_t)t * x_stride + c]);         // no convolution
    float acc = 0.f;
    for (int k = 0; k < taps; ++k) {
        const int src = t - (taps - 1 - k);
        const float v = src >= start ? to_f32(x[(size_t)src * x_stride + c]) : st[(size_t)(taps - 1 - (start - src)) * C + c];
        acc += w[(size_t)c * taps + k] * v;
    }
    return acc;
}

// The state after a single token x of its request (the caller owns channel c and has read what it needs).
__device__ __forceinline__ void conv_shift(float* __restrict__ st, int taps, int C, int c, float x) {
    for (int k = 0; k + 2 < taps; ++k) st[(size_t)k * C + c] = st[(size_t)(k + 1) * C + c];
    if (taps > 1) st[(size_t)(taps - 2) * C + c] = x;
}

// The state after the step: the last taps-1 of (old state, the step's inputs).  One thread per (request, channel).
template <typename T>
static __global__ void __launch_bounds__(256)
conv_state_kernel(const T* __restrict__ xin, int xin_stride, const float* __restrict__ in_bias, int taps, int C,
                  float* __restrict__ state, long long state_stride, const int* __restrict__ req_start,
                  const int* __restrict__ state_slots) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x, r = blockIdx.y;
    if (c >= C) return;
    const int start = req_start[r], n = req_start[r + 1] - start;
    float* st = state + (long long)state_slots[r] * state_stride;
    const float ib = in_bias ? in_bias[c] : 0.f;
    float nv[kConvMaxTaps];
    for (int k = 0; k < taps - 1; ++k) {
        const int i = n + k;                      // index into (old state, inputs)
        nv[k] = i < taps - 1 ? st[(size_t)i * C + c]
                             : to_f32(xin[(size_t)(start + i - (taps - 1)) * xin_stride + c]) + ib;
    }
    for (int k = 0; k < taps - 1; ++k) st[(size_t)k * C + c] = nv[k];
}

// One channel's convolution over consecutive tokens, its weights and last inputs in registers (TMAX at least the taps; what a
// shorter convolution lacks has weight zero).
template <typename T, int TMAX> struct ConvWindow {
    float w[TMAX], x[TMAX];
    __device__ __forceinline__ void weights(const float* __restrict__ cw, int taps, int c) {
#pragma unroll
        for (int j = 0; j < TMAX; ++j) {
            const int k = j - (TMAX - taps);
            w[j] = k >= 0 ? cw[(size_t)c * taps + k] : 0.f;
            x[j] = 0.f;
        }
    }
    // The inputs before token t of a request that starts at row `start`: earlier rows of the step, then its state.
    __device__ __forceinline__ void restart(const T* __restrict__ rows, int stride, int taps, int C, const float* __restrict__ st, int t,
                                            int start, int c) {
#pragma unroll
        for (int j = 1; j < TMAX; ++j) {
            const int back = TMAX - j, src = t - back;
            float v = 0.f;
            if (back < taps) v = src >= start ? to_f32(rows[(size_t)src * stride + c]) : st[(size_t)(taps - 1 - (start - src)) * C + c];
            x[j] = v;
        }
    }
    __device__ __forceinline__ float next(float v) {
        float acc = 0.f;
#pragma unroll
        for (int j = 0; j + 1 < TMAX; ++j) {
            x[j] = x[j + 1];
            acc += w[j] * x[j];
        }
        x[TMAX - 1] = v;
        return acc + w[TMAX - 1] * v;
    }
};
