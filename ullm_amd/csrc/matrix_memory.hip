// Recurrences over a matrix memory per head with one decay per token and head, and the passes ahead of them.
//
//   state   S [N, P] per head (N key channels, P value channels), float32, carried per request in a state row
//   RULE_DELTA  S <- g S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q        (the gated delta rule)
//   RULE_SUM    S <- g S + k (b v)^T;  o = S^T q, and the same with v = 1 for a normaliser n [N]: n <- g n + b k, n . q
//   g, b    float32 [T, heads], formed by a pass ahead: `delta_prepare` (with q, k, v through a short convolution over
//           time, silu and, q and k, over their length) or `exp_gates` (input and forget gates kept over e^m with a
//           running m)
//
// A batch is any mix of prompt portions and single tokens: entry b owns tokens q_start[b] .. q_start[b+1]-1 and the
// state row entry_slot[b]; rows of requests that start at their first token are zero when a step begins.  Everything
// is 32-bit.  A portion goes through the same operations in the same order wherever a prompt is cut; steps of single
// tokens add up in another order.
#include "common.h"
#include "short_conv.h"

typedef __attribute__((ext_vector_type(4))) float mem_f32x4;
typedef __attribute__((ext_vector_type(2))) float mem_f32x2;

#define MEMORY_MAX_KEYS 512

// A barrier for shared memory alone: loads and stores of global memory stay in flight.
__device__ __forceinline__ void memory_barrier_shared() {
#ifdef __HIP_DEVICE_COMPILE__
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
#endif
}

// The sum over a row of 16 lanes in every one of them, by four rotations inside the vector unit.
template <int CTRL>
__device__ __forceinline__ float row_rotated(float v) {
#ifdef __HIP_DEVICE_COMPILE__
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xf, 0xf, true));
#else
  return v;
#endif
}
template <int STEP>
__device__ __forceinline__ void row_sum_step(float& v) {
  if constexpr (STEP == 0) v += row_rotated<0x128>(v);
  if constexpr (STEP == 1) v += row_rotated<0x124>(v);
  if constexpr (STEP == 2) v += row_rotated<0x122>(v);
  if constexpr (STEP == 3) v += row_rotated<0x121>(v);
}
__device__ __forceinline__ float row_sum(float v) {
  row_sum_step<0>(v);
  row_sum_step<1>(v);
  row_sum_step<2>(v);
  row_sum_step<3>(v);
  return v;
}

struct MemoryArgs {
  const float* q;
  const float* k;
  const float* v;
  const float* keep;        // g [T, heads] (rows gate_ld apart)
  const float* take;        // b
  float* state;
  long long state_stride, state_off, norm_off;      // norm_off: the heads' normalisers [heads, N] (RULE_SUM)
  const int* q_start;
  const int* entry_slot;
  float* out;               // [T, heads * P]
  float* norm_out;          // [T, heads]: n . q (RULE_SUM)
  int q_ld, k_ld, v_ld, gate_ld;      // q_ld == k_ld in steps with portions
  int heads, kv_heads, N, P, write_state;
  float q_scale;
};

// ------------------------------------------------------------------ portions of prompts
// One block of four waves per (entry, head, slice of 16 value columns); with RULE_SUM the column behind the last is the
// normaliser.  Lane (r, c) = (lane % 16, lane / 16) of a wave keeps NPT rows of column c in registers; the sixteen lanes
// of a column hold its 16 NPT >= N rows and add up inside the wave, so no sum crosses waves and no token waits for a
// barrier.  An entry's tokens are walked in chunks of CH: the chunk's q, k, v, g and b lie in shared memory, the next
// chunk's are fetched into registers before the current one is worked on and put into the other buffer afterwards; a
// token's values are read two tokens ahead.  A token's read-out is formed while the next token's S^T k is on its way
// through the lanes (both read the same S), in an order the source fixes.  Lane r keeps token r's result until the chunk's end.  Tokens past the entry's end
// repeat its last token's values with b = 0 and g = 1, which changes nothing.
template <int NPT, bool DELTA, bool VEC>
__global__ void __launch_bounds__(256)
memory_scan_kernel(const MemoryArgs a) {
  constexpr int W = 4, LANES = 16;
  constexpr int NP = LANES * NPT;                    // padded key channels
  constexpr int CH = NP > 256 ? 4 : NP > 128 ? 8 : 16;
  constexpr int WC = 64 / LANES;                     // columns of a wave
  constexpr int COLS = WC * W, THREADS = 64 * W;
  constexpr int ROW = 2 * NP + COLS + 4;             // a token's q | k | v | g b
  constexpr int TOK_PIECES = NP / 2;                 // pieces of four channels of a token's q | k
  constexpr int PER = CH * TOK_PIECES > THREADS ? CH * TOK_PIECES / THREADS : 1;
  constexpr int STEP = THREADS / TOK_PIECES;         // tokens between a thread's pieces
  constexpr int V_PER = (CH * COLS + THREADS - 1) / THREADS;
  static_assert(THREADS % TOK_PIECES == 0, "a thread's pieces lie in one place of different tokens");
  static_assert(ROW % 4 == 0 && COLS % 4 == 0, "16-byte pieces");
  __shared__ __attribute__((aligned(16))) float buf[2][CH * ROW];
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * COLS;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane % LANES, cw = lane / LANES;
  const int N = a.N, P = a.P;
  const int kvh = h / (a.heads / a.kv_heads);
  const int col = c0 + WC * wave + cw;
  const bool live_col = col < P || (!DELTA && col == P);
  const int first = a.q_start[b], end = a.q_start[b + 1];
  if (first >= end) return;
  float* row = a.state + (size_t)a.entry_slot[b] * a.state_stride;
  // where this lane's column lies: rows of S are P apart, the normaliser's values side by side
  float* column = col < P ? row + a.state_off + (size_t)h * N * P + col : row + a.norm_off + (size_t)h * N;
  const int row_step = col < P ? P : 1;
  auto row_of = [&](int i) __attribute__((always_inline)) {
    return NPT % 4 == 0 ? (i / 4) * (4 * LANES) + 4 * r + i % 4 : r * NPT + i;
  };
  float s[NPT];
#pragma unroll
  for (int i = 0; i < NPT; ++i) {
    const int n = row_of(i);
    s[i] = (live_col && n < N) ? column[(size_t)n * row_step] : 0.f;
  }
  // staging: this thread brings channels n .. n + 3 of q or of k for the tokens tl, tl + STEP, ..
  const int tl = tid / TOK_PIECES, which = (tid / (NP / 4)) & 1, n = 4 * (tid % (NP / 4));
  const float* src = (which ? a.k : a.q) + (size_t)kvh * N;
  mem_f32x4 factor;                                  // q's scale, zero for channels past N
#pragma unroll
  for (int j = 0; j < 4; ++j) factor[j] = n + j < N ? (which ? 1.f : a.q_scale) : 0.f;
  if constexpr (VEC) src += n < N ? n : 0;
  const int v_col = c0 + tid % COLS;
  const float* src_v = a.v + (size_t)h * P + (v_col < P ? v_col : P - 1);
  const float* src_g = (tid & 1 ? a.take : a.keep) + h;
  mem_f32x4 raw[PER];
  float raw_v[V_PER], raw_g = 1.f;
  auto piece = [&](const float* p) __attribute__((always_inline)) {
    mem_f32x4 x;
    if constexpr (VEC) {
      x = *reinterpret_cast<const mem_f32x4*>(p);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = p[n + j < N ? n + j : N - 1];
    }
    return x;
  };
  // every load is issued whatever it is for, so that all of them are on their way at once; whole chunks step through
  // memory evenly, the last one may not read past the entry's end
  auto fetch = [&](int t0) __attribute__((always_inline)) {
    if (t0 + CH <= end) {
      const float* p = src + (size_t)(t0 + tl % CH) * a.q_ld;
#pragma unroll
      for (int i = 0; i < PER; ++i) raw[i] = piece(p + (size_t)(i * STEP) * a.q_ld);
      const float* pv = src_v + (size_t)(t0 + (tid / COLS) % CH) * a.v_ld;
#pragma unroll
      for (int i = 0; i < V_PER; ++i) raw_v[i] = pv[(size_t)(i * (THREADS / COLS)) * a.v_ld];
    } else {
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int tok = t0 + tl + i * STEP < end ? t0 + tl + i * STEP : end - 1;
        raw[i] = piece(src + (size_t)tok * a.q_ld);
      }
#pragma unroll
      for (int i = 0; i < V_PER; ++i) {
        const int tok = t0 + tid / COLS + i * (THREADS / COLS) < end ? t0 + tid / COLS + i * (THREADS / COLS) : end - 1;
        raw_v[i] = src_v[(size_t)tok * a.v_ld];
      }
    }
    if (tid < 2 * CH) {
      const int tok = t0 + (tid >> 1) < end ? t0 + (tid >> 1) : end - 1;
      raw_g = src_g[(size_t)tok * a.gate_ld];
    }
  };
  auto put = [&](int t0, float* dst) __attribute__((always_inline)) {
    float* to = dst + tl * ROW + which * NP + n;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (CH * TOK_PIECES >= THREADS || tl < CH) *reinterpret_cast<mem_f32x4*>(to + i * STEP * ROW) = raw[i] * factor;
#pragma unroll
    for (int i = 0; i < V_PER; ++i) {
      const int at = tid / COLS + i * (THREADS / COLS);
      if (CH * COLS >= THREADS || at < CH) dst[at * ROW + 2 * NP + tid % COLS] = (!DELTA && v_col == P) ? 1.f : raw_v[i];
    }
    if (tid < 2 * CH) dst[(tid >> 1) * ROW + 2 * NP + COLS + (tid & 1)] = t0 + (tid >> 1) < end ? raw_g : (tid & 1 ? 0.f : 1.f);
  };
  struct TokenIn {
    float q[NPT], k[NPT];
    float v, g, b;
  };
  auto read_token = [&](const float* from, TokenIn& in) __attribute__((always_inline)) {
    if constexpr (NPT % 4 == 0) {
#pragma unroll
      for (int i = 0; i < NPT; i += 4) {
        const mem_f32x4 kk = *reinterpret_cast<const mem_f32x4*>(from + NP + LANES * i + 4 * r);
        const mem_f32x4 qq = *reinterpret_cast<const mem_f32x4*>(from + LANES * i + 4 * r);
#pragma unroll
        for (int j = 0; j < 4; ++j) in.k[i + j] = kk[j], in.q[i + j] = qq[j];
      }
    } else {
#pragma unroll
      for (int i = 0; i < NPT; ++i) in.k[i] = from[NP + r * NPT + i], in.q[i] = from[r * NPT + i];
    }
    in.v = from[2 * NP + WC * wave + cw];
    const mem_f32x2 gb = *reinterpret_cast<const mem_f32x2*>(from + 2 * NP + COLS);
    in.g = gb.x, in.b = gb.y;
  };
  auto dot = [&](const float* x) __attribute__((always_inline)) {
    float lo = s[0] * x[0], hi = NPT > 1 ? s[NPT > 1 ? 1 : 0] * x[NPT > 1 ? 1 : 0] : 0.f;
#pragma unroll
    for (int i = 2; i < NPT; i += 2) lo += s[i] * x[i], hi += s[i + 1] * x[i + 1];
    return lo + hi;
  };
#define KEEP_ORDER __builtin_amdgcn_sched_barrier(0)
  // one token, and the read-out of the token before (the S it left is the one this token finds)
  auto move = [&](const TokenIn& in, const TokenIn& before) __attribute__((always_inline)) {
    float o;
    if constexpr (DELTA) {
      float p = dot(in.k);
      KEEP_ORDER;
      row_sum_step<0>(p);
      o = dot(before.q);
      KEEP_ORDER;
      row_sum_step<1>(p);
#pragma unroll
      for (int i = 0; i < NPT / 2; ++i) s[i] *= in.g;
      KEEP_ORDER;
      row_sum_step<2>(p);
#pragma unroll
      for (int i = NPT / 2; i < NPT; ++i) s[i] *= in.g;
      KEEP_ORDER;
      row_sum_step<3>(p);
      row_sum_step<0>(o);
      KEEP_ORDER;
      row_sum_step<1>(o);
      KEEP_ORDER;
      const float u = in.b * (in.v - in.g * p);
#pragma unroll
      for (int i = 0; i < NPT / 2; ++i) s[i] = fmaf(in.k[i], u, s[i]);
      row_sum_step<2>(o);
      KEEP_ORDER;
#pragma unroll
      for (int i = NPT / 2; i < NPT; ++i) s[i] = fmaf(in.k[i], u, s[i]);
      row_sum_step<3>(o);
      KEEP_ORDER;
    } else {
      o = dot(before.q);
      const float u = in.b * in.v;
#pragma unroll
      for (int i = 0; i < NPT; ++i) s[i] = fmaf(in.k[i], u, in.g * s[i]);
      o = row_sum(o);
    }
    return o;
  };
  fetch(first);
  put(first, buf[0]);
  memory_barrier_shared();
  int turn = 0;
  for (int t0 = first; t0 < end; t0 += CH) {
    const float* cur = buf[turn];
    const bool more = t0 + CH < end;
    if (more) fetch(t0 + CH);
    TokenIn in[4];
    float kept = 0.f;
    read_token(cur, in[0]);
    read_token(cur + ROW, in[1]);
#pragma unroll
    for (int t = 0; t < CH; ++t) {
      if (t == 0) in[3] = in[0];                       // no token before the chunk's first: what it reads is not kept
      if (t + 2 < CH) read_token(cur + (t + 2) * ROW, in[(t + 2) & 3]);
      const float o = move(in[t & 3], in[(t + 3) & 3]);
      if (t > 0) kept = r == t - 1 ? o : kept;
    }
    const float o = row_sum(dot(in[(CH - 1) & 3].q));
    kept = r == CH - 1 ? o : kept;
    if (more) put(t0 + CH, buf[1 - turn]);
    if (r < CH && t0 + r < end) {
      if (col < P) a.out[(size_t)(t0 + r) * a.heads * P + (size_t)h * P + col] = kept;
      else if (!DELTA && col == P) a.norm_out[(size_t)(t0 + r) * a.heads + h] = kept;
    }
    memory_barrier_shared();
    turn = 1 - turn;
  }
  if (a.write_state && live_col) {
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
      const int at = row_of(i);
      if (at < N) column[(size_t)at * row_step] = s[i];
    }
  }
#undef KEEP_ORDER
}

// ------------------------------------------------------------------ steps of single tokens
// One block per (entry, head, slice of PC value columns): thread (g, p) keeps the NPT rows n = g NPT .. of column p, all
// asked for at once; one round of partial sums (S^T k, S^T q and k . q; o = g S^T q + (k . q) u) through shared memory.
// With RULE_SUM the first slice's block also moves the normaliser on.
template <int PC, int NPT, bool DELTA>
__global__ void __launch_bounds__(256)
memory_step_kernel(const MemoryArgs a) {
  constexpr int R = 256 / PC, NP = R * NPT;
  __shared__ float part_k[DELTA ? R * PC : 1], part_q[R * PC], part_kq[R];
  __shared__ __attribute__((aligned(16))) float s_q[NP], s_k[NP];
  __shared__ float scratch[16];
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * PC;
  const int tid = threadIdx.x, p = tid % PC, gr = tid / PC;
  const int N = a.N, P = a.P;
  const int kvh = h / (a.heads / a.kv_heads);
  const int col = c0 + p, t = a.q_start[b];
  float* row = a.state + (size_t)a.entry_slot[b] * a.state_stride;
  float* column = row + a.state_off + (size_t)h * N * P + (col < P ? col : P - 1);
  float s[NPT];
#pragma unroll
  for (int i = 0; i < NPT; ++i) {
    const int n = gr * NPT + i;
    s[i] = column[(size_t)(n < N ? n : N - 1) * P];
  }
  const float g = a.keep[(size_t)t * a.gate_ld + h], take = a.take[(size_t)t * a.gate_ld + h];
  const float v = a.v[(size_t)t * a.v_ld + (size_t)h * P + (col < P ? col : P - 1)];
  for (int n = tid; n < NP; n += 256) {
    const int at = n < N ? n : N - 1;
    const float qv = a.q[(size_t)t * a.q_ld + (size_t)kvh * N + at] * a.q_scale;
    const float kv = a.k[(size_t)t * a.k_ld + (size_t)kvh * N + at];
    s_q[n] = n < N ? qv : 0.f;
    s_k[n] = n < N ? kv : 0.f;
  }
  float* norm = row + a.norm_off + (size_t)h * N;
  constexpr int NORM_PER = (NP + 255) / 256;
  float nv[NORM_PER];
  const bool norm_here = !DELTA && blockIdx.z == 0;
  if (norm_here) {
#pragma unroll
    for (int i = 0; i < NORM_PER; ++i) nv[i] = norm[tid + 256 * i < N ? tid + 256 * i : N - 1];
  }
  __syncthreads();
  float pk = 0.f, pq = 0.f, kq = 0.f;
#pragma unroll
  for (int i = 0; i < NPT; ++i) {
    const float kk = s_k[gr * NPT + i], qq = s_q[gr * NPT + i];
    if constexpr (DELTA) pk += s[i] * kk;
    pq += s[i] * qq;
    kq += kk * qq;
  }
  if constexpr (DELTA) part_k[gr * PC + p] = pk;
  part_q[gr * PC + p] = pq;
  if (p == 0) part_kq[gr] = kq;
  __syncthreads();
  pk = pq = kq = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    if constexpr (DELTA) pk += part_k[i * PC + p];
    pq += part_q[i * PC + p];
    kq += part_kq[i];
  }
  const float u = DELTA ? take * (v - g * pk) : take * v;
  if (gr == 0 && col < P) a.out[(size_t)t * a.heads * P + (size_t)h * P + col] = g * pq + kq * u;
  if (a.write_state && col < P) {
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
      const int n = gr * NPT + i;
      if (n < N) column[(size_t)n * P] = g * s[i] + s_k[n] * u;
    }
  }
  if (norm_here) {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NORM_PER; ++i) {
      const int n = tid + 256 * i;
      if (n < N) {
        const float x = g * nv[i] + take * s_k[n];
        sum += x * s_q[n];
        if (a.write_state) norm[n] = x;
      }
    }
    sum = block_sum(sum, scratch);
    if (tid == 0) a.norm_out[(size_t)t * a.heads + h] = sum;
  }
}

template <int NP, bool DELTA>
static int launch_scan(const MemoryArgs& a, int B_, hipStream_t stream) {
  const dim3 grid(B_, a.heads, (a.P + (DELTA ? 0 : 1) + 15) / 16);
  if (a.N % 4 == 0 && a.q_ld % 4 == 0 && ((uintptr_t)a.q | (uintptr_t)a.k) % 16 == 0)
    hipLaunchKernelGGL((memory_scan_kernel<NP / 16, DELTA, true>), grid, dim3(256), 0, stream, a);
  else
    hipLaunchKernelGGL((memory_scan_kernel<NP / 16, DELTA, false>), grid, dim3(256), 0, stream, a);
  ULLM_LAUNCH_CHECK();
}

template <int PC, int NPT, bool DELTA>
static int launch_step(const MemoryArgs& a, int B_, hipStream_t stream) {
  hipLaunchKernelGGL((memory_step_kernel<PC, NPT, DELTA>), dim3(B_, a.heads, (a.P + PC - 1) / PC), dim3(256), 0, stream, a);
  ULLM_LAUNCH_CHECK();
}

template <bool DELTA>
static int memory_any(const MemoryArgs& a, int B_, bool single, hipStream_t stream) {
  const int N = a.N;
  if (!single) {
    if (N <= 16) return launch_scan<16, DELTA>(a, B_, stream);
    if (N <= 32) return launch_scan<32, DELTA>(a, B_, stream);
    if (N <= 64) return launch_scan<64, DELTA>(a, B_, stream);
    if (N <= 128) return launch_scan<128, DELTA>(a, B_, stream);
    if (N <= 256) return launch_scan<256, DELTA>(a, B_, stream);
    return launch_scan<512, DELTA>(a, B_, stream);
  }
  // rows of 64 value channels a block (whole lines of state) where there are blocks enough without narrow slices
  if (a.P % 64 == 0 && N <= 128 && (long long)B_ * a.heads >= 1024) {
    if (N <= 32) return launch_step<64, 8, DELTA>(a, B_, stream);
    if (N <= 64) return launch_step<64, 16, DELTA>(a, B_, stream);
    return launch_step<64, 32, DELTA>(a, B_, stream);
  }
  if (N <= 16) return launch_step<16, 1, DELTA>(a, B_, stream);
  if (N <= 32) return launch_step<16, 2, DELTA>(a, B_, stream);
  if (N <= 64) return launch_step<16, 4, DELTA>(a, B_, stream);
  if (N <= 128) return launch_step<16, 8, DELTA>(a, B_, stream);
  if (N <= 256) return launch_step<16, 16, DELTA>(a, B_, stream);
  return launch_step<16, 32, DELTA>(a, B_, stream);
}

// rule 0: RULE_DELTA, 1: RULE_SUM.  `single`: every entry brings exactly one token.
extern "C" int ullm_matrix_memory(const float* q, int q_ld, const float* k, int k_ld, const float* v, int v_ld, const float* keep,
                                  const float* take, int gate_ld, int rule, float q_scale, float* state, long long state_stride,
                                  long long state_off, long long norm_off, const int* q_start, const int* entry_slot, float* out,
                                  float* norm_out, int B_, int heads, int kv_heads, int N, int P, int write_state, int single,
                                  hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (heads < 1 || kv_heads < 1 || heads % kv_heads || N < 1 || P < 1 || N > MEMORY_MAX_KEYS || heads > 65535) return ULLM_ERR_SHAPE;
  if ((P + 8) / 8 > 65535) return ULLM_ERR_SHAPE;
  if (!single && q_ld != k_ld) return ULLM_ERR_UNSUPPORTED;
  if (rule != 0 && (rule != 1 || norm_out == nullptr)) return ULLM_ERR_UNSUPPORTED;
  MemoryArgs a;
  a.q = q, a.k = k, a.v = v, a.keep = keep, a.take = take, a.state = state, a.state_stride = state_stride, a.state_off = state_off;
  a.norm_off = norm_off, a.q_start = q_start, a.entry_slot = entry_slot, a.out = out, a.norm_out = norm_out;
  a.q_ld = q_ld, a.k_ld = k_ld, a.v_ld = v_ld, a.gate_ld = gate_ld, a.heads = heads, a.kv_heads = kv_heads, a.N = N, a.P = P;
  a.write_state = write_state, a.q_scale = q_scale;
  return rule == 0 ? memory_any<true>(a, B_, single != 0, stream) : memory_any<false>(a, B_, single != 0, stream);
}

// ------------------------------------------------------------------ ahead of the delta rule
__device__ __forceinline__ float memory_silu(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float memory_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct PrepareArgs {
  const float* in;          // rows q (kv_heads * N) | k (kv_heads * N) | v (heads * P), in_ld apart
  const float* w;           // [taps, channels] in the same order of channels
  const float* raw_b;       // raw values [T, heads] of the write strength, and of the decay, in_ld apart
  const float* raw_a;
  const float* a_rate;      // [heads]: exp(A_log)
  const float* dt_bias;     // [heads]
  float* carry;             // a state row's last taps-1 inputs [taps-1, channels]
  long long carry_stride;
  const int* token_entry;
  const int* q_start;
  const int* entry_slot;
  float* out;               // [T, channels]
  float* gates;             // [T, 2, heads]: g, b
  int in_ld, T, heads, kv_heads, N, P, taps, run, update;
  float q_scale;
};

// A wave per (run of `run` tokens, item); items are the heads of q, of k and of v, and one more for the gates.  A lane
// owns the channels lane + 64 j of its head.  TAPS > 0: weights and the last inputs in registers, TAPS = 0: any number
// of taps, every input fetched for every tap.  `update`: every entry brings one token, and the wave that has read its channels'
// carried inputs moves them on itself.
template <int V, int TAPS>
__global__ void __launch_bounds__(256)
delta_prepare_kernel(const PrepareArgs a) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int items = 2 * a.kv_heads + a.heads + 1;
  if (item >= items) return;
  const int t0 = blockIdx.x * a.run, stop = t0 + a.run < a.T ? t0 + a.run : a.T;
  if (item == items - 1) {
    for (int e = lane; e < (stop - t0) * a.heads; e += 64) {
      const int t = t0 + e / a.heads, h = e % a.heads;
      const float za = a.raw_a[(size_t)t * a.in_ld + h] + a.dt_bias[h], zb = a.raw_b[(size_t)t * a.in_ld + h];
      a.gates[((size_t)t * 2) * a.heads + h] = expf(-a.a_rate[h] * memory_softplus(za));
      a.gates[((size_t)t * 2 + 1) * a.heads + h] = 1.f / (1.f + expf(-zb));
    }
    return;
  }
  const int qk = a.kv_heads * a.N, channels = 2 * qk + a.heads * a.P;
  const bool is_v = item >= 2 * a.kv_heads;
  const int size = is_v ? a.P : a.N;
  const int base = is_v ? 2 * qk + (item - 2 * a.kv_heads) * a.P : item * a.N;
  const float unit_scale = item < a.kv_heads ? a.q_scale : 1.f;
  constexpr int KEEP = TAPS > 1 ? TAPS - 1 : 1;
  float wt[V][TAPS > 0 ? TAPS : 1], hist[V][KEEP];
  int ch[V];
#pragma unroll
  for (int j = 0; j < V; ++j) {
    ch[j] = base + (lane + 64 * j < size ? lane + 64 * j : size - 1);
#pragma unroll
    for (int i = 0; i < TAPS; ++i) wt[j][i] = a.w[(size_t)i * channels + ch[j]];
  }
  for (int t = t0; t < stop; ++t) {
    const int b = a.token_entry[t], first = a.q_start[b], i = t - first;
    float* old = a.carry + (size_t)a.entry_slot[b] * a.carry_stride;
    float x[V], y[V];
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] = a.in[(size_t)t * a.in_ld + ch[j]], y[j] = 0.f;
    if constexpr (TAPS > 0) {
      if (t == t0 || i == 0) {
#pragma unroll
        for (int m = 0; m < TAPS - 1; ++m) {
          const int l = i - (TAPS - 1) + m;
#pragma unroll
          for (int j = 0; j < V; ++j)
            hist[j][m] = l >= 0 ? a.in[(size_t)(first + l) * a.in_ld + ch[j]] : old[(size_t)(l + TAPS - 1) * channels + ch[j]];
        }
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
#pragma unroll
        for (int m = 0; m < TAPS - 1; ++m) y[j] += wt[j][m] * hist[j][m];
        y[j] += wt[j][TAPS - 1] * x[j];
#pragma unroll
        for (int m = 0; m + 1 < TAPS - 1; ++m) hist[j][m] = hist[j][m + 1];
        if (TAPS > 1) hist[j][KEEP - 1] = x[j];
      }
      if (a.update) {
#pragma unroll
        for (int j = 0; j < V; ++j)
          if (lane + 64 * j < size) {
#pragma unroll
            for (int m = 0; m < TAPS - 1; ++m) old[(size_t)m * channels + ch[j]] = hist[j][m];
          }
      }
    } else {
      for (int m = 0; m < a.taps; ++m) {
        const int l = i - (a.taps - 1) + m;
#pragma unroll
        for (int j = 0; j < V; ++j)
          y[j] += a.w[(size_t)m * channels + ch[j]] *
                  (l >= 0 ? a.in[(size_t)(first + l) * a.in_ld + ch[j]] : old[(size_t)(l + a.taps - 1) * channels + ch[j]]);
      }
    }
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      y[j] = memory_silu(y[j]);
      if (lane + 64 * j < size) sq += y[j] * y[j];
    }
    float f = 1.f;
    if (!is_v) f = unit_scale / sqrtf(wave_sum(sq) + 1e-6f);
#pragma unroll
    for (int j = 0; j < V; ++j)
      if (lane + 64 * j < size) a.out[(size_t)t * channels + ch[j]] = y[j] * f;
  }
}

template <int V>
static void launch_prepare(const PrepareArgs& a, hipStream_t stream) {
  const dim3 grid((a.T + a.run - 1) / a.run, (2 * a.kv_heads + a.heads + 1 + 3) / 4);
  if (a.taps == 4) hipLaunchKernelGGL((delta_prepare_kernel<V, 4>), grid, dim3(256), 0, stream, a);
  else if (a.taps == 3) hipLaunchKernelGGL((delta_prepare_kernel<V, 3>), grid, dim3(256), 0, stream, a);
  else if (a.taps == 2) hipLaunchKernelGGL((delta_prepare_kernel<V, 2>), grid, dim3(256), 0, stream, a);
  else hipLaunchKernelGGL((delta_prepare_kernel<V, 0>), grid, dim3(256), 0, stream, a);
}

extern "C" int ullm_delta_prepare(const float* in, int in_ld, const float* w, const float* raw_b, const float* raw_a,
                                  const float* a_rate, const float* dt_bias, float* carry, long long carry_stride,
                                  const int* token_entry, const int* q_start, const int* entry_slot, float* out, float* gates,
                                  int T_, int B_, int heads, int kv_heads, int N, int P, int taps, float q_scale, int single,
                                  int update, hipStream_t stream) {
  if (T_ <= 0 || B_ <= 0) return 0;
  if (heads < 1 || kv_heads < 1 || heads % kv_heads || N < 1 || P < 1 || N > MEMORY_MAX_KEYS || P > MEMORY_MAX_KEYS || taps < 1 ||
      taps > SHORT_CONV_MAX_TAPS || (single && T_ != B_)) return ULLM_ERR_SHAPE;
  const int channels = 2 * kv_heads * N + heads * P;
  PrepareArgs a;
  a.in = in, a.w = w, a.raw_b = raw_b, a.raw_a = raw_a, a.a_rate = a_rate, a.dt_bias = dt_bias, a.carry = carry;
  a.carry_stride = carry_stride, a.token_entry = token_entry, a.q_start = q_start, a.entry_slot = entry_slot, a.out = out;
  a.gates = gates, a.in_ld = in_ld, a.T = T_, a.heads = heads, a.kv_heads = kv_heads, a.N = N, a.P = P, a.taps = taps;
  a.q_scale = q_scale;
  a.run = single ? 1 : (T_ >= 1024 ? 8 : (T_ >= 256 ? 4 : 1));
  const bool in_place = single && taps >= 2 && taps <= 4;
  a.update = in_place && update ? 1 : 0;
  const int big = N > P ? N : P;
  if (big <= 64) launch_prepare<1>(a, stream);
  else if (big <= 128) launch_prepare<2>(a, stream);
  else if (big <= 256) launch_prepare<4>(a, stream);
  else launch_prepare<8>(a, stream);
  if (update && !in_place && taps > 1) launch_carry<float>(in, in_ld, carry, carry_stride, q_start, entry_slot, B_, channels, taps, stream);
  ULLM_LAUNCH_CHECK();
}

// ------------------------------------------------------------------ exponential gates
// Per head: i = cap tanh((z_i + b_i) / cap), f = log sigmoid(cap tanh((z_f + b_f) / cap)); a running maximum
// m_t = max(f_t + m_(t-1), i_t) from the state row's m (0 at a request's start); keep = exp(f_t + m_(t-1) - m_t),
// take = exp(i_t - m_t), floor = exp(-m_t).  A token is the map m -> max(A + m, B) with (A, B) = (f, i); maps compose as
// (A1 + A2, max(B1 + A2, B2)), so a block of up to 1024 threads takes as many tokens of an (entry, head) at once.
__global__ void __launch_bounds__(1024)
exp_gates_kernel(const float* __restrict__ raw_i, const float* __restrict__ raw_f, int ld, const float* __restrict__ b_i,
                 const float* __restrict__ b_f, float cap, float* __restrict__ state, long long state_stride, long long m_off,
                 const int* __restrict__ q_start, const int* __restrict__ entry_slot, float* __restrict__ gates, int heads,
                 int write_state) {
  __shared__ float tot_a[16], tot_b[16];
  const int b = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, waves = (int)blockDim.x >> 6;
  const int first = q_start[b], end = q_start[b + 1];
  float* m_at = state + (size_t)entry_slot[b] * state_stride + m_off + h;
  float m0 = *m_at;
  const float bi = b_i[h], bf = b_f[h];
  for (int t0 = first; t0 < end; t0 += (int)blockDim.x) {
    const int t = t0 + tid;
    const bool live = t < end;
    const size_t at = (size_t)(live ? t : end - 1) * ld + h;
    const float gi = cap * tanhf((raw_i[at] + bi) / cap);
    const float gf = -memory_softplus(-(cap * tanhf((raw_f[at] + bf) / cap)));
    float A = live ? gf : 0.f, B = live ? gi : -INFINITY;       // past the end: the map that changes nothing
#pragma unroll
    for (int d = 1; d < 64; d *= 2) {
      const float pa = __shfl_up(A, d, 64), pb = __shfl_up(B, d, 64);
      if (lane >= d) {
        B = fmaxf(pb + A, B);
        A = pa + A;
      }
    }
    if (lane == 63) tot_a[wave] = A, tot_b[wave] = B;
    __syncthreads();
    float before = m0, after = m0;                              // m ahead of this wave's tokens, m behind the block's
    for (int w = 0; w < waves; ++w) {
      if (w == wave) before = after;
      after = fmaxf(tot_a[w] + after, tot_b[w]);
    }
    const float m = fmaxf(A + before, B);
    float prev = __shfl_up(m, 1, 64);
    if (lane == 0) prev = before;
    if (live) {
      float* g = gates + (size_t)t * 3 * heads + h;
      g[0] = expf(gf + prev - m);
      g[heads] = expf(gi - m);
      g[2 * heads] = expf(-m);
    }
    m0 = after;
    __syncthreads();
  }
  if (tid == 0 && write_state && first < end) *m_at = m0;
}

// gates [T, 3, heads]: keep, take, floor.
extern "C" int ullm_exp_gates(const float* raw_i, const float* raw_f, int ld, const float* b_i, const float* b_f, float cap,
                              float* state, long long state_stride, long long m_off, const int* q_start, const int* entry_slot,
                              float* gates, int B_, int heads, int max_len, int write_state, hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (heads < 1 || heads > 65535 || !(cap > 0.f)) return ULLM_ERR_SHAPE;
  int threads = 64;
  while (threads < max_len && threads < 1024) threads *= 2;
  hipLaunchKernelGGL(exp_gates_kernel, dim3(B_, heads), dim3(threads), 0, stream, raw_i, raw_f, ld, b_i, b_f, cap, state,
                     state_stride, m_off, q_start, entry_slot, gates, heads, write_state);
  ULLM_LAUNCH_CHECK();
}
