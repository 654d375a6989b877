// A selective scan with a state per channel (the Mamba form).  Per channel c and state n of an entry's tokens in order:
//   dt = softplus(raw[t, c] + dt_bias[c])
//   S[c, :] = exp(dt * A[c, :]) * S[c, :] + (dt * x[t, c]) * B[t, :]
//   y       = S[c, :] . C[t, :] + D[c] * x[t, c],   stored: y * silu(z[t, c])
// A is handed over as A * log2(e), so that a decay is one exponent of two.  The states are float32 and come from and
// go to the entry's state row (state[slot, off + c * N + n]).  Everything is 32-bit; x, z and the result are stored in
// the compute dtype (B and C too: they are a projection's values).
//
// Three ways, by what the step holds:
//   portions of prompts, N <= 64   an entry's tokens are cut into segments ("items") that are walked side by side.  Over a
//                    segment the decays multiply up to exp(A * sum of its step sizes), so a first pass leaves every
//                    segment's states from zero and its sum of step sizes, a second small kernel chains them to every
//                    segment's first states, and the last pass walks the segments from there and stores the outputs.  A
//                    lane owns a channel with all its states in registers; B and C of a token are the same for the whole
//                    wave (scalar loads), and nothing moves between lanes.
//   a single token each            a lane owns four states of a channel (one where N is no multiple of four)
//   larger N                       a block walks an entry's tokens in order, sixteen lanes to a channel
#include "common.h"

__device__ __forceinline__ float sel_silu(float z) { return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }
// log(1 + e^v) = max(v, 0) + log(1 + e), e = e^-|v|; with u = 1 + e rounded, log(u) * e / (u - 1) is log(1 + e) to a few
// units in the last place for any e
__device__ __forceinline__ float sel_softplus(float v) {
  const float e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(v)), u = 1.f + e;
  const float l = u == 1.f ? e : 0.6931471805599453f * __builtin_amdgcn_logf(u) * (e / (u - 1.f));
  return fmaxf(v, 0.f) + l;
}

template <typename T>
struct ScanIn {
  const float* raw;           // [T, raw_ld]
  int raw_ld;
  const T* bc;                // [T, bc_ld]: B, then C
  int bc_ld;
  const float* a_log2;        // [inner, N]
  const float* dt_bias;
  const float* d_skip;
  int inner, N;
};

// ------------------------------------------------------------------ segments
// items [n][4] = (entry, first token, tokens, what it is): 0 an entry's only segment (its states come from and go to the
// state row), 1 one of several (its first states lie in `chain`), 2 the last of several (and its last states go to the
// state row).  chain float32 [n][N][inner], dt_sum float32 [n][inner].
#define SEG_AHEAD 8            // tokens whose step sizes and inputs are under way
// A token's N values of B (or C), the same address for the whole wave: whole words, so that they are wide scalar loads.
template <int N>
__device__ __forceinline__ void uniform_row(const float* p, float (&v)[N]) {
#pragma unroll
  for (int n = 0; n < N; ++n) v[n] = p[n];
}
template <int N>
__device__ __forceinline__ void uniform_row(const bf16_t* p, float (&v)[N]) {
  const uint32_t* w = reinterpret_cast<const uint32_t*>(p);
#pragma unroll
  for (int n = 0; n < N / 2; ++n) {
    v[2 * n] = __uint_as_float(w[n] << 16);
    v[2 * n + 1] = __uint_as_float(w[n] & 0xffff0000u);
  }
}

// FULL: the model has N states a channel, not fewer, and its rows of B and C are whole aligned words.
template <typename T, int N, bool OUT, bool FULL>
__global__ void __launch_bounds__(64)
scan_segment_kernel(const T* __restrict__ x, int x_ld, const T* __restrict__ z, int z_ld, ScanIn<T> in, const int* __restrict__ items,
                    float* __restrict__ chain, float* __restrict__ dt_sum, float* __restrict__ state, long long state_stride,
                    long long state_off, const int* __restrict__ entry_slot, T* __restrict__ out, int write_state) {
  const int item = blockIdx.y, what = items[4 * item + 3];
  if (!OUT && what != 1) return;                          // only segments with another behind them need their states
  const int b = items[4 * item], t0 = items[4 * item + 1], n_tok = items[4 * item + 2];
  const int c = blockIdx.x * 64 + threadIdx.x;
  const bool live = c < in.inner;
  const int cc = live ? c : in.inner - 1;
  const int n_states = FULL ? N : in.N;
  float* const row = state + (size_t)entry_slot[b] * state_stride + state_off + (size_t)cc * in.N;
  float* const link = chain + (size_t)item * in.N * in.inner + cc;
  float s[N], a[N];
#pragma unroll
  for (int n = 0; n < N; ++n) {
    const bool ok = n < n_states;
    a[n] = ok ? in.a_log2[(size_t)cc * in.N + n] : 0.f;
    s[n] = 0.f;
    if (OUT && ok) s[n] = what == 0 ? row[n] : link[(size_t)n * in.inner];
  }
  const float bias = in.dt_bias[cc], skip = in.d_skip[cc];
  const float* const raw = in.raw + (size_t)t0 * in.raw_ld + cc;
  const T* const xp = x + (size_t)t0 * x_ld + cc;
  const T* const zp = OUT ? z + (size_t)t0 * z_ld + cc : nullptr;
  float sum = 0.f;
  float r0[SEG_AHEAD], x0[SEG_AHEAD], z0[SEG_AHEAD];
  auto fetch = [&](int t) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < SEG_AHEAD; ++u) {
      const int tt = t + u < n_tok ? t + u : n_tok - 1;
      r0[u] = raw[(size_t)tt * in.raw_ld];
      x0[u] = ld_f32(xp + (size_t)tt * x_ld);
      if (OUT) z0[u] = ld_f32(zp + (size_t)tt * z_ld);
    }
  };
  fetch(0);
  for (int t = 0; t < n_tok; t += SEG_AHEAD) {
    float dt[SEG_AHEAD], xv[SEG_AHEAD], zv[SEG_AHEAD];
#pragma unroll
    for (int u = 0; u < SEG_AHEAD; ++u) {
      // past the segment's end the step size is zero: the state stands still
      dt[u] = t + u < n_tok ? sel_softplus(r0[u] + bias) : 0.f;
      xv[u] = x0[u];
      if (OUT) zv[u] = z0[u];
    }
    if (t + SEG_AHEAD < n_tok) fetch(t + SEG_AHEAD);
#pragma unroll
    for (int u = 0; u < SEG_AHEAD; ++u) {
      const int tt = t + u < n_tok ? t + u : n_tok - 1;
      const T* const bcr = in.bc + (size_t)(t0 + tt) * in.bc_ld;
      const float dx = dt[u] * xv[u];
      float acc = 0.f;
      if constexpr (FULL) {
        float bv[N], cv[N];
        uniform_row<N>(bcr, bv);
        if (OUT) uniform_row<N>(bcr + N, cv);
#pragma unroll
        for (int n = 0; n < N; ++n) {
          s[n] = __builtin_amdgcn_exp2f(dt[u] * a[n]) * s[n] + dx * bv[n];
          if (OUT) acc += s[n] * cv[n];
        }
      } else {
#pragma unroll
        for (int n = 0; n < N; ++n) {
          const int nn = n < n_states ? n : n_states - 1;   // states behind the last: no decay (a = 0), never stored
          s[n] = __builtin_amdgcn_exp2f(dt[u] * a[n]) * s[n] + dx * ld_f32(bcr + nn);
          if (OUT) acc += n < n_states ? s[n] * ld_f32(bcr + n_states + nn) : 0.f;
        }
      }
      if (OUT) {
        if (t + u < n_tok && live) st_f32(out + (size_t)(t0 + t + u) * in.inner + c, (acc + skip * xv[u]) * sel_silu(zv[u]));
      } else {
        sum += dt[u];
      }
    }
  }
  if (!live) return;
  if (!OUT) {
    dt_sum[(size_t)item * in.inner + c] = sum;
#pragma unroll
    for (int n = 0; n < N; ++n)
      if (n < n_states) link[(size_t)n * in.inner] = s[n];
  } else if (what != 1 && write_state) {
#pragma unroll
    for (int n = 0; n < N; ++n)
      if (n < n_states) row[n] = s[n];
  }
}

// Every segment's states from zero become its first states.  chains [n][3] = (entry, first item, items).
__global__ void __launch_bounds__(256)
scan_chain_kernel(const int* __restrict__ chains, float* __restrict__ chain, const float* __restrict__ dt_sum,
                  const float* __restrict__ a_log2, const float* __restrict__ state, long long state_stride, long long state_off,
                  const int* __restrict__ entry_slot, int inner, int N) {
  const int c = blockIdx.x * 256 + threadIdx.x, n = blockIdx.y;
  if (c >= inner) return;
  const int b = chains[3 * blockIdx.z], first = chains[3 * blockIdx.z + 1], count = chains[3 * blockIdx.z + 2];
  const float a = a_log2[(size_t)c * N + n];
  float s = state[(size_t)entry_slot[b] * state_stride + state_off + (size_t)c * N + n];
  const size_t step = (size_t)N * inner;
  float* link = chain + (size_t)first * step + (size_t)n * inner + c;
  const float* sum = dt_sum + (size_t)first * inner + c;
  constexpr int U = 8;
  for (int i = 0; i < count; i += U) {
    float h[U], d[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = i + u < count - 1 ? i + u : count - 2;          // the last segment left nothing behind
      h[u] = link[(size_t)k * step];
      d[u] = sum[(size_t)k * inner];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (i + u < count) {
        link[(size_t)(i + u) * step] = s;
        s = __builtin_amdgcn_exp2f(a * d[u]) * s + h[u];
      }
  }
}

extern "C" int ullm_selective_scan_segments(const void* x, int x_ld, const float* raw, int raw_ld, const void* bc, int bc_ld,
                                            const void* z, int z_ld, const float* a_log2, const float* dt_bias,
                                            const float* d_skip, float* state, long long state_stride, long long state_off,
                                            const int* entry_slot, const int* items, int n_items, const int* chains, int n_chains,
                                            float* chain, float* dt_sum, void* out, int inner, int N, int write_state, int dtype,
                                            hipStream_t stream) {
  if (n_items <= 0) return 0;
  if (n_items > 65535 || n_chains > 65535 || inner < 1 || N < 1 || N > 64 || x_ld < inner || raw_ld < inner || z_ld < inner ||
      bc_ld < 2 * N || (n_chains > 0 && (!chain || !dt_sum)))
    return ULLM_ERR_SHAPE;
  const bool words = dtype == ULLM_F32 || (bc_ld % 2 == 0 && (uintptr_t)bc % 4 == 0);
  const dim3 grid((inner + 63) / 64, n_items), block(64);
#define SCAN_IN(TT) ScanIn<TT>{raw, raw_ld, (const TT*)bc, bc_ld, a_log2, dt_bias, d_skip, inner, N}
#define GO_F(TT, NN, OUT, FULL) hipLaunchKernelGGL((scan_segment_kernel<TT, NN, OUT, FULL>), grid, block, 0, stream, (const TT*)x, x_ld, (const TT*)z, z_ld, \
    SCAN_IN(TT), items, chain, dt_sum, state, state_stride, state_off, entry_slot, (TT*)out, write_state)
#define GO(TT, NN, OUT) do { if (N == NN && words) GO_F(TT, NN, OUT, true); else GO_F(TT, NN, OUT, false); } while (0)
#define GO_N(TT, OUT) do { if (N <= 8) GO(TT, 8, OUT); else if (N <= 16) GO(TT, 16, OUT); else if (N <= 32) GO(TT, 32, OUT); else GO(TT, 64, OUT); } while (0)
#define GO_T(OUT) do { if (dtype == ULLM_F32) GO_N(float, OUT); else if (dtype == ULLM_BF16) GO_N(bf16_t, OUT); else return ULLM_ERR_DTYPE; } while (0)
  if (n_chains > 0) {
    GO_T(false);
    hipLaunchKernelGGL(scan_chain_kernel, dim3((inner + 255) / 256, N, n_chains), dim3(256), 0, stream, chains, chain, dt_sum, a_log2,
                       state, state_stride, state_off, entry_slot, inner, N);
  }
  GO_T(true);
#undef GO_T
#undef GO_N
#undef GO
#undef GO_F
  ULLM_LAUNCH_CHECK();
}

// ------------------------------------------------------------------ a single token of every entry
// `lanes` neighbouring lanes (a power of two, at most 64) share a channel and take its states V at a time.
template <typename T, int V>
__global__ void __launch_bounds__(256)
scan_step_kernel(const T* __restrict__ x, int x_ld, const T* __restrict__ z, int z_ld, ScanIn<T> in, float* __restrict__ state,
                 long long state_stride, long long state_off, const int* __restrict__ entry_slot, T* __restrict__ out, int lanes,
                 int write_state) {
  const int t = blockIdx.y, ln = threadIdx.x & (lanes - 1), c = blockIdx.x * (256 / lanes) + threadIdx.x / lanes;
  const bool live = c < in.inner;
  const int cc = live ? c : in.inner - 1;
  float* const row = state + (size_t)entry_slot[t] * state_stride + state_off + (size_t)cc * in.N;
  const float* const a = in.a_log2 + (size_t)cc * in.N;
  const T* const bcr = in.bc + (size_t)t * in.bc_ld;
  const float xv = ld_f32(x + (size_t)t * x_ld + cc), zv = ld_f32(z + (size_t)t * z_ld + cc);
  const float dt = sel_softplus(in.raw[(size_t)t * in.raw_ld + cc] + in.dt_bias[cc]), dx = dt * xv;
  float acc = 0.f;
  for (int n = V * ln; n < in.N; n += V * lanes) {
    if constexpr (V == 4) {
      float4 s = *reinterpret_cast<const float4*>(row + n);
      const float4 av = *reinterpret_cast<const float4*>(a + n);
      s.x = __builtin_amdgcn_exp2f(dt * av.x) * s.x + dx * ld_f32(bcr + n);
      s.y = __builtin_amdgcn_exp2f(dt * av.y) * s.y + dx * ld_f32(bcr + n + 1);
      s.z = __builtin_amdgcn_exp2f(dt * av.z) * s.z + dx * ld_f32(bcr + n + 2);
      s.w = __builtin_amdgcn_exp2f(dt * av.w) * s.w + dx * ld_f32(bcr + n + 3);
      const T* cr = bcr + in.N + n;
      acc += s.x * ld_f32(cr);
      acc += s.y * ld_f32(cr + 1);
      acc += s.z * ld_f32(cr + 2);
      acc += s.w * ld_f32(cr + 3);
      if (live && write_state) *reinterpret_cast<float4*>(row + n) = s;
    } else {
      const float s = __builtin_amdgcn_exp2f(dt * a[n]) * row[n] + dx * ld_f32(bcr + n);
      acc += s * ld_f32(bcr + in.N + n);
      if (live && write_state) row[n] = s;
    }
  }
  for (int m = lanes / 2; m > 0; m >>= 1) acc += __shfl_xor(acc, m, 64);
  if (ln == 0 && live) st_f32(out + (size_t)t * in.inner + c, (acc + in.d_skip[cc] * xv) * sel_silu(zv));
}

extern "C" int ullm_selective_scan_step(const void* x, int x_ld, const float* raw, int raw_ld, const void* bc, int bc_ld,
                                        const void* z, int z_ld, const float* a_log2, const float* dt_bias, const float* d_skip,
                                        float* state, long long state_stride, long long state_off, const int* entry_slot, void* out,
                                        int B_, int inner, int N, int write_state, int dtype, hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (B_ > 65535 || inner < 1 || N < 1 || x_ld < inner || raw_ld < inner || z_ld < inner || bc_ld < 2 * N) return ULLM_ERR_SHAPE;
  const bool by4 = N % 4 == 0 && state_stride % 4 == 0 && state_off % 4 == 0 && ((uintptr_t)state | (uintptr_t)a_log2) % 16 == 0;
  int lanes = 1;
  while (lanes < 64 && lanes * (by4 ? 4 : 1) < N) lanes *= 2;
  const int per = 256 / lanes;
#define GO(TT, V) hipLaunchKernelGGL((scan_step_kernel<TT, V>), dim3((inner + per - 1) / per, B_), dim3(256), 0, stream, (const TT*)x, x_ld, \
    (const TT*)z, z_ld, SCAN_IN(TT), state, state_stride, state_off, entry_slot, (TT*)out, lanes, write_state)
  if (dtype == ULLM_F32) { if (by4) GO(float, 4); else GO(float, 1); }
  else if (dtype == ULLM_BF16) { if (by4) GO(bf16_t, 4); else GO(bf16_t, 1); }
  else return ULLM_ERR_DTYPE;
#undef GO
  ULLM_LAUNCH_CHECK();
}

// ------------------------------------------------------------------ any N up to 256
#define SEL_THREADS 256
#define SEL_LANES 16          // lanes that share a channel
#define SEL_CH (SEL_THREADS / SEL_LANES)
#define SEL_CHUNK 16          // tokens staged at a time

// One block per (entry, SEL_CH channels).  Lane l of a channel's 16 owns the states l * NPT .. l * NPT + NPT - 1.  Per
// chunk of tokens: B and C, and per channel the step size, step size * x, x go to shared memory; then every lane walks
// the chunk's tokens, leaving its part of each token's sum in a register; the 16 lanes' parts are added by a
// butterfly in which a lane keeps half of its tokens in every round (lane l ends with token l's whole sum).
template <typename T, int NPT>
__global__ void __launch_bounds__(SEL_THREADS)
selective_scan_kernel(const T* __restrict__ x, int x_ld, const float* __restrict__ raw, int raw_ld,
                      const T* __restrict__ bc, int bc_ld, const T* __restrict__ z, int z_ld,
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
      s_b[t][n] = ok ? ld_f32(bc + (size_t)(t0 + t) * bc_ld + n) : 0.f;
      s_c[t][n] = ok ? ld_f32(bc + (size_t)(t0 + t) * bc_ld + N + n) : 0.f;
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
      st_f32(out + (size_t)(t0 + st) * inner + c0 + sc, y * sel_silu(zv));
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

extern "C" int ullm_selective_scan(const void* x, int x_ld, const float* raw, int raw_ld, const void* bc, int bc_ld,
                                   const void* z, int z_ld, const float* a_log2, const float* dt_bias, const float* d_skip,
                                   float* state, long long state_stride, long long state_off, const int* q_start,
                                   const int* entry_slot, void* out, int B_, int inner, int N, int write_state, int dtype,
                                   hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (B_ > 65535 || inner < 1 || N < 1 || N > 16 * SEL_LANES || x_ld < inner || raw_ld < inner || z_ld < inner || bc_ld < 2 * N)
    return ULLM_ERR_SHAPE;
  const dim3 grid((inner + SEL_CH - 1) / SEL_CH, B_), block(SEL_THREADS);
  const int npt = (N + SEL_LANES - 1) / SEL_LANES;
#define GO(TT, NPT) hipLaunchKernelGGL((selective_scan_kernel<TT, NPT>), grid, block, 0, stream, (const TT*)x, x_ld, raw, raw_ld, (const TT*)bc,   \
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
