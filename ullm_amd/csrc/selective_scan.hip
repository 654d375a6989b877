// A selective scan with a state per channel (the Mamba form).  Per channel c and state n of an entry's tokens in order:
//   dt = softplus(raw[t, c] + dt_bias[c])
//   S[c, n] = exp(dt * A[c, n]) * S[c, n] + dt * x[t, c] * B[t, n]
//   y[t, c] = sum_n S[c, n] * C[t, n] + D[c] * x[t, c],   stored: y * silu(z[t, c])
// A is handed over as A * log2(e), so that a decay is one exponent of two.  The states are float32 and come from and
// go to the entry's state row (state[slot, off + c * N + n]).  Everything is 32-bit; x, z and the result are stored in
// the compute dtype.  A state element sees the same operations in the same order wherever its entry was cut.
#include "common.h"

#define SEL_THREADS 256
#define SEL_LANES 16          // lanes that share a channel
#define SEL_CH (SEL_THREADS / SEL_LANES)
#define SEL_CHUNK 16          // tokens staged at a time

__device__ __forceinline__ float sel_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// One block per (entry, SEL_CH channels).  Lane l of a channel's 16 owns the states l * NPT .. l * NPT + NPT - 1.  Per
// chunk of tokens: B and C, and per channel the step size, step size * x, x go to shared memory; then every lane walks
// the chunk's tokens, leaving its part of each token's sum in a register; the 16 lanes' parts are added by a
// butterfly in which a lane keeps half of its tokens in every round (lane l ends with token l's whole sum).
template <typename T, int NPT>
__global__ void __launch_bounds__(SEL_THREADS)
selective_scan_kernel(const T* __restrict__ x, int x_ld, const float* __restrict__ raw, int raw_ld,
                      const float* __restrict__ bc, int bc_ld, const T* __restrict__ z, int z_ld,
                      const float* __restrict__ a_log2, const float* __restrict__ dt_bias, const float* __restrict__ d_skip,
                      float* __restrict__ state, long long state_stride, long long state_off,
                      const int* __restrict__ q_start, const int* __restrict__ entry_slot, T* __restrict__ out, int inner,
                      int N, int write_state) {
  constexpr int NP = SEL_LANES * NPT;
  __shared__ __attribute__((aligned(16))) float s_b[SEL_CHUNK][NP], s_c[SEL_CHUNK][NP];
  __shared__ float s_dt[SEL_CHUNK][SEL_CH], s_dx[SEL_CHUNK][SEL_CH], s_x[SEL_CHUNK][SEL_CH];
  const int b = blockIdx.y, c0 = blockIdx.x * SEL_CH, tid = threadIdx.x;
  const int ch = tid / SEL_LANES, ln = tid % SEL_LANES, c = c0 + ch;
  const int first = q_start[b], end = q_start[b + 1];
  const bool live = c < inner;
  float* row = state + (size_t)entry_slot[b] * state_stride + state_off + (size_t)(live ? c : 0) * N;
  float s[NPT], a[NPT];
#pragma unroll
  for (int k = 0; k < NPT; ++k) {
    const int n = ln * NPT + k;
    const bool ok = live && n < N;
    s[k] = ok ? row[n] : 0.f;
    a[k] = ok ? a_log2[(size_t)c * N + n] : 0.f;
  }
  const int st = tid / SEL_CH, sc = tid % SEL_CH;                     // staging: token of the chunk, channel
  const bool s_live = c0 + sc < inner;
  const float s_bias = s_live ? dt_bias[c0 + sc] : 0.f, s_skip = s_live ? d_skip[c0 + sc] : 0.f;
  for (int t0 = first; t0 < end; t0 += SEL_CHUNK) {
    __syncthreads();
    for (int e = tid; e < SEL_CHUNK * NP; e += SEL_THREADS) {
      const int t = e / NP, n = e % NP;
      const bool ok = t0 + t < end && n < N;
      s_b[t][n] = ok ? bc[(size_t)(t0 + t) * bc_ld + n] : 0.f;
      s_c[t][n] = ok ? bc[(size_t)(t0 + t) * bc_ld + N + n] : 0.f;
    }
    {
      const bool ok = s_live && t0 + st < end;
      const float xv = ok ? ld_f32(x + (size_t)(t0 + st) * x_ld + c0 + sc) : 0.f;
      // past the entry's end the step size is zero: the state stands still
      const float dt = ok ? sel_softplus(raw[(size_t)(t0 + st) * raw_ld + c0 + sc] + s_bias) : 0.f;
      s_dt[st][sc] = dt;
      s_dx[st][sc] = dt * xv;
      s_x[st][sc] = xv;
    }
    __syncthreads();
    float part[SEL_CHUNK];
#pragma unroll
    for (int t = 0; t < SEL_CHUNK; ++t) {
      const float dt = s_dt[t][ch], dx = s_dx[t][ch];
      float acc = 0.f;
#pragma unroll
      for (int k = 0; k < NPT; ++k) {
        s[k] = __builtin_amdgcn_exp2f(dt * a[k]) * s[k] + dx * s_b[t][ln * NPT + k];
        acc += s[k] * s_c[t][ln * NPT + k];
      }
      part[t] = acc;
    }
#pragma unroll
    for (int m = SEL_CHUNK / 2; m >= 1; m >>= 1) {
      const bool upper = (ln & m) != 0;
#pragma unroll
      for (int u = 0; u < m; ++u) {
        const float give = upper ? part[u] : part[u + m], keep = upper ? part[u + m] : part[u];
        part[u] = keep + __shfl_xor(give, m, 64);
      }
    }
    // lane ln holds token ln's sum of its channel; the result goes out token by token through shared memory
    __syncthreads();
    s_dt[ln][ch] = part[0];
    __syncthreads();
    if (s_live && t0 + st < end) {
      const float y = s_dt[st][sc] + s_skip * s_x[st][sc];
      const float zv = ld_f32(z + (size_t)(t0 + st) * z_ld + c0 + sc);
      st_f32(out + (size_t)(t0 + st) * inner + c0 + sc, y * (zv / (1.f + expf(-zv))));
    }
  }
  if (write_state && live) {
#pragma unroll
    for (int k = 0; k < NPT; ++k) {
      const int n = ln * NPT + k;
      if (n < N) row[n] = s[k];
    }
  }
}

extern "C" int ullm_selective_scan(const void* x, int x_ld, const float* raw, int raw_ld, const float* bc, int bc_ld,
                                   const void* z, int z_ld, const float* a_log2, const float* dt_bias, const float* d_skip,
                                   float* state, long long state_stride, long long state_off, const int* q_start,
                                   const int* entry_slot, void* out, int B_, int inner, int N, int write_state, int dtype,
                                   hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (B_ > 65535 || inner < 1 || N < 1 || N > 16 * SEL_LANES || x_ld < inner || raw_ld < inner || z_ld < inner || bc_ld < 2 * N)
    return ULLM_ERR_SHAPE;
  const dim3 grid((inner + SEL_CH - 1) / SEL_CH, B_), block(SEL_THREADS);
  const int npt = (N + SEL_LANES - 1) / SEL_LANES;
#define GO(TT, NPT) hipLaunchKernelGGL((selective_scan_kernel<TT, NPT>), grid, block, 0, stream, (const TT*)x, x_ld, raw, raw_ld, bc,   \
    bc_ld, (const TT*)z, z_ld, a_log2, dt_bias, d_skip, state, state_stride, state_off, q_start, entry_slot, (TT*)out, inner, N, \
    write_state)
#define GO_N(TT) do { if (npt == 1) GO(TT, 1); else if (npt == 2) GO(TT, 2); else if (npt <= 4) GO(TT, 4); \
    else if (npt <= 8) GO(TT, 8); else GO(TT, 16); } while (0)
  if (dtype == ULLM_F32) GO_N(float);
  else if (dtype == ULLM_BF16) GO_N(bf16_t);
  else return ULLM_ERR_DTYPE;
#undef GO_N
#undef GO
  ULLM_LAUNCH_CHECK();
}
