// What lies between two sublayers of a model that norms what its sublayers put out (and nothing else): the stream takes
// the normed branch, and the next sublayer reads the stream itself, or the stream plus a short causal convolution of it.
//
//   y = a * branch (+ b * second),  stream += y / sqrt(mean(y^2) + eps) * gain
//   out = stream                                              in the compute dtype, or
//   out = stream + conv(stream)                               for steps of single tokens: the last taps rows per channel,
//                                                             those before the token's from its state row, which moves on
//
// A branch may be a stack of partial sums [S, T, H], added slice by slice.  Everything is 32-bit; a row's sums have a
// fixed order.
#include "common.h"

#define POST_MAX_TAPS 16
typedef __attribute__((ext_vector_type(4))) float post_f32x4;

template <int V>
__device__ __forceinline__ void post_load(const float* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const post_f32x4 t = *reinterpret_cast<const post_f32x4*>(p);
    v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
  } else v[0] = *p;
}
template <int V>
__device__ __forceinline__ void post_load(const bf16_t* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16), v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16), v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else v[0] = bf16_bits_to_f32(*p);
}
template <int V>
__device__ __forceinline__ void post_store(float* p, const float (&v)[V]) {
  if constexpr (V == 4) *reinterpret_cast<post_f32x4*>(p) = post_f32x4{v[0], v[1], v[2], v[3]};
  else *p = v[0];
}
template <int V>
__device__ __forceinline__ void post_store(bf16_t* p, const float (&v)[V]) {
  if constexpr (V == 4) *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
  else *p = f32_to_bf16_bits(v[0]);
}

struct PostConv {
  const float* w;             // [taps, H]; null: no convolution
  int taps;
  float* carry;               // state rows, oldest first
  long long carry_stride;
  const int* entry_slot;      // token t is entry t's only one
};

// One block per token; a thread owns K pieces of V neighbouring values.
// TAPS: the convolution's taps (0: none, or read one after the other).
template <typename TA, typename TB, typename TO, int V, int K, int TAPS>
__global__ void __launch_bounds__(256)
post_add_kernel(const TA* __restrict__ branch, int n_a, const TB* __restrict__ second, int n_b, float a, float b,
                const float* __restrict__ gain, float eps, float* __restrict__ stream_rows, TO* __restrict__ out, int T_, int H,
                PostConv conv) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const size_t row = (size_t)t * H, slice = (size_t)T_ * H;
  constexpr int HT = TAPS > 1 ? TAPS - 1 : 1, WT = TAPS > 0 ? TAPS : 1;
  float y[K][V], x[K][V], g[K][V], past[K][HT][V], w[K][WT][V];
  float* old = conv.w ? conv.carry + (size_t)conv.entry_slot[t] * conv.carry_stride : nullptr;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int c = V * (tid + 256 * k);
    if (c < H) {
      post_load<V>(stream_rows + row + c, x[k]);
      post_load<V>(gain + c, g[k]);
      if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) post_load<V>(old + (size_t)j * H + c, past[k][j]);
#pragma unroll
        for (int j = 0; j < TAPS; ++j) post_load<V>(conv.w + (size_t)j * H + c, w[k][j]);
      }
      float v[V];
      post_load<V>(branch + row + c, y[k]);
      for (int s = 1; s < n_a; ++s) {
        post_load<V>(branch + s * slice + row + c, v);
#pragma unroll
        for (int u = 0; u < V; ++u) y[k][u] += v[u];
      }
#pragma unroll
      for (int u = 0; u < V; ++u) y[k][u] *= a;
      if (n_b > 0) {
        float w2[V];
        post_load<V>(second + row + c, w2);
        for (int s = 1; s < n_b; ++s) {
          post_load<V>(second + s * slice + row + c, v);
#pragma unroll
          for (int u = 0; u < V; ++u) w2[u] += v[u];
        }
#pragma unroll
        for (int u = 0; u < V; ++u) y[k][u] += b * w2[u];
      }
#pragma unroll
      for (int u = 0; u < V; ++u) ss += y[k][u] * y[k][u];
    }
  }
  const float rs = 1.f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int c = V * (tid + 256 * k);
    if (c >= H) continue;
#pragma unroll
    for (int u = 0; u < V; ++u) x[k][u] += (y[k][u] * rs) * g[k][u];
    post_store<V>(stream_rows + row + c, x[k]);
    if (!out) continue;
    if (!conv.w) {
      post_store<V>(out + row + c, x[k]);
      continue;
    }
    float acc[V];
#pragma unroll
    for (int u = 0; u < V; ++u) acc[u] = 0.f;
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        if (j > 0) post_store<V>(old + (size_t)(j - 1) * H + c, past[k][j]);
#pragma unroll
        for (int u = 0; u < V; ++u) acc[u] += w[k][j][u] * past[k][j][u];
      }
      if (TAPS > 1) post_store<V>(old + (size_t)(TAPS - 2) * H + c, x[k]);
#pragma unroll
      for (int u = 0; u < V; ++u) acc[u] = x[k][u] + (acc[u] + w[k][TAPS - 1][u] * x[k][u]);
      post_store<V>(out + row + c, acc);
      continue;
    }
    float in[V], wj[V];
    for (int j = 0; j < conv.taps - 1; ++j) {
      post_load<V>(old + (size_t)j * H + c, in);
      post_load<V>(conv.w + (size_t)j * H + c, wj);
      if (j > 0) post_store<V>(old + (size_t)(j - 1) * H + c, in);          // the state moves up by one
#pragma unroll
      for (int u = 0; u < V; ++u) acc[u] += wj[u] * in[u];
    }
    post_load<V>(conv.w + (size_t)(conv.taps - 1) * H + c, wj);
    if (conv.taps > 1) post_store<V>(old + (size_t)(conv.taps - 2) * H + c, x[k]);
#pragma unroll
    for (int u = 0; u < V; ++u) acc[u] = x[k][u] + (acc[u] + wj[u] * x[k][u]);
    post_store<V>(out + row + c, acc);
  }
}

template <typename TA, typename TB, typename TO>
static int launch_post(const void* branch, int n_a, const void* second, int n_b, float a, float b, const float* gain, float eps,
                       float* stream_rows, void* out, int T_, int H, const PostConv& conv, hipStream_t stream) {
  const bool by4 = H % 4 == 0 && (uintptr_t)branch % (4 * sizeof(TA)) == 0 && (uintptr_t)second % (4 * sizeof(TB)) == 0 &&
                   (uintptr_t)out % (4 * sizeof(TO)) == 0 && ((uintptr_t)gain | (uintptr_t)stream_rows) % 16 == 0 &&
                   (!conv.w || ((uintptr_t)conv.w | (uintptr_t)conv.carry) % 16 == 0) && (!conv.w || conv.carry_stride % 4 == 0);
  const int pieces = ((by4 ? H / 4 : H) + 255) / 256;
#define GO_T(V, K, TAPS) hipLaunchKernelGGL((post_add_kernel<TA, TB, TO, V, K, TAPS>), dim3(T_), dim3(256), 0, stream, (const TA*)branch, n_a, \
    (const TB*)second, n_b, a, b, gain, eps, stream_rows, (TO*)out, T_, H, conv)
  // rows of up to 4096 values by fours with two to four taps: the convolution's operands wait in registers
#define GO(V, K) do { if constexpr (V == 4 && K <= 4) {                                                                   \
    if (conv.w && conv.taps == 2) GO_T(V, K, 2); else if (conv.w && conv.taps == 3) GO_T(V, K, 3);                          \
    else if (conv.w && conv.taps == 4) GO_T(V, K, 4); else GO_T(V, K, 0); } else GO_T(V, K, 0); } while (0)
#define GO_K(V) do { if (pieces <= 1) GO(V, 1); else if (pieces <= 2) GO(V, 2); else if (pieces <= 4) GO(V, 4); else if (pieces <= 8) GO(V, 8); \
    else if (pieces <= 16) GO(V, 16); else return ULLM_ERR_SHAPE; } while (0)
  if (by4) GO_K(4);
  else GO_K(1);
#undef GO_K
#undef GO
#undef GO_T
  ULLM_LAUNCH_CHECK();
}

extern "C" int ullm_post_add(const void* branch, int n_a, int a_dtype, const void* second, int n_b, int b_dtype, float a, float b,
                             const float* gain, float eps, float* stream_rows, void* out, int out_dtype, int T_, int H,
                             const float* conv_w, int taps, float* carry, long long carry_stride, const int* entry_slot,
                             hipStream_t stream) {
  if (T_ <= 0) return 0;
  if (H < 1 || n_a < 1 || n_b < 0 || (n_b > 0 && !second)) return ULLM_ERR_SHAPE;
  if (conv_w && (taps < 1 || taps > POST_MAX_TAPS || !carry || !entry_slot || !out)) return ULLM_ERR_SHAPE;
  const PostConv conv = {conv_w, taps, carry, carry_stride, entry_slot};
#define POST_ARGS branch, n_a, second, n_b, a, b, gain, eps, stream_rows, out, T_, H, conv, stream
#define GO_O(TA, TB) do { if (out_dtype == ULLM_F32) return launch_post<TA, TB, float>(POST_ARGS);            \
    if (out_dtype == ULLM_BF16) return launch_post<TA, TB, bf16_t>(POST_ARGS); return ULLM_ERR_DTYPE; } while (0)
  if (n_b == 0) b_dtype = a_dtype;
  if (a_dtype == ULLM_F32 && b_dtype == ULLM_F32) GO_O(float, float);
  if (a_dtype == ULLM_BF16 && b_dtype == ULLM_BF16) GO_O(bf16_t, bf16_t);
  if (a_dtype == ULLM_F32 && b_dtype == ULLM_BF16) GO_O(float, bf16_t);
  if (a_dtype == ULLM_BF16 && b_dtype == ULLM_F32) GO_O(bf16_t, float);
#undef GO_O
#undef POST_ARGS
  return ULLM_ERR_DTYPE;
}
