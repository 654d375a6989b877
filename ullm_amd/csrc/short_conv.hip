// A short causal convolution over time per channel, with the inputs of the last taps-1 tokens carried from step to
// step.  conv(i) = sum_j w[j, c] * in(i - (taps-1) + j) for the token's index i inside its entry, where in(l) is this
// step's input row q_start[b] + l for l >= 0 and otherwise what the entry's state row holds:
// carry[slot, (l + taps-1) * channels + c].  Weights lie tap by tap, [taps, channels].  What is stored:
//   CONV_SILU      silu(bias[c] + conv)
//   CONV_RESIDUAL  in(i) + conv
// All arithmetic is 32-bit; a token's sum has the same terms in the same order wherever its entry was cut.
#include "common.h"
#include "short_conv.h"

enum { CONV_SILU = 0, CONV_RESIDUAL = 1 };

template <int V>
struct ConvPiece {
  float v[V];
};
template <int V>
__device__ __forceinline__ ConvPiece<V> conv_load(const float* p) {
  ConvPiece<V> r;
  if constexpr (V == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    r.v[0] = t.x, r.v[1] = t.y, r.v[2] = t.z, r.v[3] = t.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V>
__device__ __forceinline__ ConvPiece<V> conv_load(const bf16_t* p) {
  ConvPiece<V> r;
  if constexpr (V == 4) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    r.v[0] = __uint_as_float(t.x << 16), r.v[1] = __uint_as_float(t.x & 0xffff0000u);
    r.v[2] = __uint_as_float(t.y << 16), r.v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else {
    r.v[0] = bf16_bits_to_f32(*p);
  }
  return r;
}
template <int V>
__device__ __forceinline__ void conv_store(float* p, const float* v) {
  if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else *p = v[0];
}
template <int V>
__device__ __forceinline__ void conv_store(bf16_t* p, const float* v) {
  if constexpr (V == 4) *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
  else *p = f32_to_bf16_bits(v[0]);
}

__device__ __forceinline__ float conv_silu_of(float z) { return z / (1.f + expf(-z)); }

// grid (runs of `tok` tokens, channel pieces).  A thread owns V neighbouring channels, keeps their weights and the last
// taps-1 inputs in registers and walks its run, RUN tokens' rows asked for at a time; at the run's start and at every
// entry's first token the inputs before come from the rows before or from the state row.  `update`: every entry brings
// one token, and the thread that has used its channels' state moves it on itself.
template <typename TI, typename TO, int TAPS, int V, int RUN>
__global__ void __launch_bounds__(256)
short_conv_kernel(const TI* __restrict__ in, int in_stride, const float* __restrict__ w, const float* __restrict__ bias,
                  float* __restrict__ carry, long long carry_stride, const int* __restrict__ token_entry,
                  const int* __restrict__ q_start, const int* __restrict__ entry_slot, TO* __restrict__ out, int T_,
                  int channels, int mode, int tok, int update) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= channels) return;
  ConvPiece<V> wt[TAPS], hist[TAPS];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) wt[j] = conv_load<V>(w + (size_t)j * channels + c);
  ConvPiece<V> b0;
#pragma unroll
  for (int u = 0; u < V; ++u) b0.v[u] = bias ? bias[c + u] : 0.f;
  const int t0 = blockIdx.x * tok;
  const int stop = t0 + tok < T_ ? t0 + tok : T_;
  for (int g0 = t0; g0 < stop; g0 += RUN) {
    ConvPiece<V> rows[RUN];
#pragma unroll
    for (int r = 0; r < RUN; ++r) rows[r] = conv_load<V>(in + (size_t)(g0 + r < stop ? g0 + r : stop - 1) * in_stride + c);
#pragma unroll
    for (int r = 0; r < RUN; ++r) {
      const int t = g0 + r;
      if (t >= stop) break;
      const int b = token_entry[t], first = q_start[b], i = t - first;
      if (t == t0 || i == 0) {
        const float* old = carry + (size_t)entry_slot[b] * carry_stride + c;
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k) {
          const int l = i - (TAPS - 1) + k;
          hist[k] = l >= 0 ? conv_load<V>(in + (size_t)(first + l) * in_stride + c)
                           : conv_load<V>(old + (size_t)(l + TAPS - 1) * channels);
        }
      }
      hist[TAPS - 1] = rows[r];
      float acc[V];
#pragma unroll
      for (int u = 0; u < V; ++u) acc[u] = b0.v[u];
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int u = 0; u < V; ++u) acc[u] += wt[j].v[u] * hist[j].v[u];
#pragma unroll
      for (int u = 0; u < V; ++u) acc[u] = mode == CONV_SILU ? conv_silu_of(acc[u]) : hist[TAPS - 1].v[u] + acc[u];
      conv_store<V>(out + (size_t)t * channels + c, acc);
#pragma unroll
      for (int k = 0; k < TAPS - 1; ++k) hist[k] = hist[k + 1];
      if (update) {
        float* row = carry + (size_t)entry_slot[b] * carry_stride + c;
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k) conv_store<V>(row + (size_t)k * channels, hist[k].v);
      }
    }
  }
}

// Any number of taps, one channel a thread, one token a block.
template <typename TI, typename TO>
__global__ void __launch_bounds__(256)
short_conv_general_kernel(const TI* __restrict__ in, int in_stride, const float* __restrict__ w,
                          const float* __restrict__ bias, const float* __restrict__ carry, long long carry_stride,
                          const int* __restrict__ token_entry, const int* __restrict__ q_start,
                          const int* __restrict__ entry_slot, TO* __restrict__ out, int channels, int taps, int mode) {
  const int t = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= channels) return;
  const int b = token_entry[t], first = q_start[b], i = t - first;
  const float* old = carry + (size_t)entry_slot[b] * carry_stride + c;
  float acc = bias ? bias[c] : 0.f, x = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int l = i - (taps - 1) + j;
    x = l >= 0 ? ld_f32(in + (size_t)(first + l) * in_stride + c) : old[(size_t)(l + taps - 1) * channels];
    acc += w[(size_t)j * channels + c] * x;
  }
  st_f32(out + (size_t)t * channels + c, mode == CONV_SILU ? conv_silu_of(acc) : x + acc);      // x: the token's own input
}

template <typename TI, typename TO>
static int launch_conv(const void* in, int in_stride, const float* w, const float* bias, float* carry,
                       long long carry_stride, const int* token_entry, const int* q_start, const int* entry_slot, void* out,
                       int T_, int B_, int channels, int taps, int mode, int single, int update, hipStream_t stream) {
  const int pad = 3;
  const bool by4 = channels % 4 == 0 && (in_stride & pad) == 0 && (carry_stride & pad) == 0 &&
                   ((uintptr_t)w | (uintptr_t)carry) % 16 == 0 && (uintptr_t)in % (4 * sizeof(TI)) == 0 &&
                   (uintptr_t)out % (4 * sizeof(TO)) == 0;
  bool moved = false;
  if (taps <= 4) {
    // a block walks several tokens where the step has many: weights and the overlap with the rows before cost less
    const int tok = single ? 1 : (T_ >= 1024 ? 8 : (T_ >= 256 ? 4 : 1));
    moved = single && update;
#define GO_R(TAPS, V, R) hipLaunchKernelGGL((short_conv_kernel<TI, TO, TAPS, V, R>), dim3((T_ + tok - 1) / tok, (channels / V + 255) / 256), \
    dim3(256), 0, stream, (const TI*)in, in_stride, w, bias, carry, carry_stride, token_entry, q_start, entry_slot, (TO*)out, T_,     \
    channels, mode, tok, moved ? 1 : 0)
#define GO(TAPS, V) do { if (tok >= 4) GO_R(TAPS, V, 4); else GO_R(TAPS, V, 1); } while (0)
#define GO_V(TAPS) do { if (by4) GO(TAPS, 4); else GO(TAPS, 1); } while (0)
    if (taps == 1) GO_V(1);
    else if (taps == 2) GO_V(2);
    else if (taps == 3) GO_V(3);
    else GO_V(4);
#undef GO_V
#undef GO
#undef GO_R
  } else {
    hipLaunchKernelGGL((short_conv_general_kernel<TI, TO>), dim3(T_, (channels + 255) / 256), dim3(256), 0, stream, (const TI*)in,
                       in_stride, w, bias, carry, carry_stride, token_entry, q_start, entry_slot, (TO*)out, channels, taps, mode);
  }
  if (update && !moved && taps > 1)
    launch_carry<TI>(in, in_stride, carry, carry_stride, q_start, entry_slot, B_, channels, taps, stream);
  ULLM_LAUNCH_CHECK();
}

extern "C" int ullm_short_conv(const void* in, int in_stride, const float* w, const float* bias, float* carry,
                               long long carry_stride, const int* token_entry, const int* q_start, const int* entry_slot,
                               void* out, int T_, int B_, int channels, int taps, int mode, int single, int update,
                               int in_dtype, int out_dtype, hipStream_t stream) {
  if (T_ <= 0 || B_ <= 0) return 0;
  if (channels <= 0 || taps < 1 || taps > SHORT_CONV_MAX_TAPS || in_stride < channels) return ULLM_ERR_SHAPE;
  if (mode != CONV_SILU && mode != CONV_RESIDUAL) return ULLM_ERR_UNSUPPORTED;
  if (single && T_ != B_) return ULLM_ERR_SHAPE;
#define CONV_ARGS in, in_stride, w, bias, carry, carry_stride, token_entry, q_start, entry_slot, out, T_, B_, channels, taps, mode, single, update, stream
  if (in_dtype == ULLM_F32 && out_dtype == ULLM_F32) return launch_conv<float, float>(CONV_ARGS);
  if (in_dtype == ULLM_F32 && out_dtype == ULLM_BF16) return launch_conv<float, bf16_t>(CONV_ARGS);
  if (in_dtype == ULLM_BF16 && out_dtype == ULLM_BF16) return launch_conv<bf16_t, bf16_t>(CONV_ARGS);
#undef CONV_ARGS
  return ULLM_ERR_DTYPE;
}
