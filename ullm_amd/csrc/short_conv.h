// The state of a short causal convolution over time: the inputs of a request's last taps-1 tokens, moved on behind a
// step (shared by the kernels that convolve).
#pragma once
#include "common.h"

#define SHORT_CONV_MAX_TAPS 16

// Behind the convolution: the state row takes the inputs of the entry's last taps-1 tokens (older ones move up where
// the entry brought fewer).  A thread reads everything it needs before it writes.
template <typename TI>
__global__ void __launch_bounds__(256)
short_conv_carry_kernel(const TI* __restrict__ in, int in_stride, float* __restrict__ carry, long long carry_stride,
                        const int* __restrict__ q_start, const int* __restrict__ entry_slot, int channels, int taps) {
  const int b = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= channels) return;
  const int first = q_start[b], n = q_start[b + 1] - first;
  float* row = carry + (size_t)entry_slot[b] * carry_stride + c;
  float keep[SHORT_CONV_MAX_TAPS];
#pragma unroll
  for (int k = 0; k < SHORT_CONV_MAX_TAPS; ++k)
    if (k < taps - 1) {
      const int l = n - (taps - 1) + k;
      keep[k] = l >= 0 ? ld_f32(in + (size_t)(first + l) * in_stride + c) : row[(size_t)(k + n) * channels];
    }
#pragma unroll
  for (int k = 0; k < SHORT_CONV_MAX_TAPS; ++k)
    if (k < taps - 1) row[(size_t)k * channels] = keep[k];
}

template <typename TI>
static void launch_carry(const void* in, int in_stride, float* carry, long long carry_stride, const int* q_start,
                         const int* entry_slot, int B_, int channels, int taps, hipStream_t stream) {
  hipLaunchKernelGGL(short_conv_carry_kernel<TI>, dim3(B_, (channels + 255) / 256), dim3(256), 0, stream, (const TI*)in,
                     in_stride, carry, carry_stride, q_start, entry_slot, channels, taps);
}
