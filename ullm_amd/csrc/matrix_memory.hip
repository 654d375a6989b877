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
// is 32-bit, the matrix cores' products included.  A portion's chunks are counted from its first token, and steps of single
// tokens add up in another order: whole and cut prompts agree to rounding.
#include "common.h"
#include "short_conv.h"

typedef __attribute__((ext_vector_type(4))) float mem_f32x4;

#define MEMORY_MAX_KEYS 512

// A barrier for shared memory alone: loads and stores of global memory stay in flight.
__device__ __forceinline__ void memory_barrier_shared() {
#ifdef __HIP_DEVICE_COMPILE__
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
#endif
}

// D[i][j] = C[i][j] + sum_k A[i][k] B[k][j] for 16 x 4 by 4 x 16 in 32-bit: lane (c, g) = (lane % 16, lane / 16) holds A[c][k]
// and B[k][c] for its own k and D[4 g + r][c] in register r.  Which k a lane group stands for is free as long as A and B
// agree: a 16 x 16 result's register r is, as it lies, the B operand of the step whose groups stand for k = 4 g + r.
__device__ __forceinline__ mem_f32x4 mma(float a, float b, mem_f32x4 c) {
#ifdef __HIP_DEVICE_COMPILE__
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
#else
  return c;
#endif
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
  const int* items;         // the chunks of a step with portions: (first token, tokens) each, an entry's side by side
  const int* entry_item;    // [B]: an entry's first item
  float* chunks;            // [items, heads, CHUNK_FLOATS]
  float* out;               // [T, heads * P]
  float* norm_out;          // [T, heads]: n . q (RULE_SUM)
  int q_ld, k_ld, v_ld, gate_ld;
  int heads, kv_heads, N, P, write_state;
  float q_scale;
};

// ------------------------------------------------------------------ portions of prompts, in chunks of 16 tokens
// Inside a chunk, with S0 the memory it finds, G_ij = g_(j+1) .. g_i, c_i = g_1 .. g_i and d_j = g_(j+1) .. g_16:
//   u_i + b_i sum_(j<i) G_ij (k_i . k_j) u_j = b_i (v_i - c_i S0^T k_i)      (RULE_DELTA; u_i = b_i v_i with RULE_SUM)
//   o_i = c_i S0^T q_i + sum_(j<=i) G_ij (q_i . k_j) u_j,     S1 = c_16 S0 + sum_j d_j k_j u_j^T
// What does not depend on S0 is made for all chunks at once: the products of keys and queries, and the inverse of the
// unit lower triangle by substitution (memory_chunk_kernel).  What is left per chunk are products of 16-row tiles.
// Products of decays are formed as products: no logarithm, no quotient.  Tokens past an entry's end repeat its last
// token's vectors with g = 1 and b = 0, which changes nothing.
#define CHUNK_TOKENS 16
#define CHUNK_T 0          // [16][16]: inverse times b_j (RULE_DELTA)
#define CHUNK_M 256        // [16][16]: G_ij (q_i . k_j) for j <= i
#define CHUNK_C 512        // c_i
#define CHUNK_D 528        // d_j
#define CHUNK_B 544        // b_j
#define CHUNK_FLOATS 576

// Four neighbouring values of a row of N; past the end valid elements again (what meets them is zero).
template <bool VEC>
__device__ __forceinline__ mem_f32x4 row_piece(const float* row, int n, int N) {
  mem_f32x4 x;
  if constexpr (VEC) {
    x = *reinterpret_cast<const mem_f32x4*>(row + (n < N ? n : 0));
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j) x[j] = row[n + j < N ? n + j : N - 1];
  }
  return x;
}

// One wave per (chunk, head).
template <bool DELTA, bool VEC>
__global__ void __launch_bounds__(64)
memory_chunk_kernel(const MemoryArgs a) {
  __shared__ float s_g[16], s_b[16], s_l[16 * 20];
  const int item = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, c = lane & 15, g = lane >> 4;
  const int t0 = a.items[2 * item], n_tok = a.items[2 * item + 1], N = a.N;
  const int kvh = h / (a.heads / a.kv_heads);
  const int tok = t0 + (c < n_tok ? c : n_tok - 1);
  const float gm = c < n_tok ? a.keep[(size_t)tok * a.gate_ld + h] : 1.f;
  const float bm = c < n_tok ? a.take[(size_t)tok * a.gate_ld + h] : 0.f;
  const float* qr = a.q + (size_t)tok * a.q_ld + (size_t)kvh * N;
  const float* kr = a.k + (size_t)tok * a.k_ld + (size_t)kvh * N;
  mem_f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
#pragma unroll 4
  for (int n0 = 0; n0 < N; n0 += 16) {
    const int n = n0 + 4 * g;
    mem_f32x4 kv = row_piece<VEC>(kr, n, N);
    const mem_f32x4 qv = row_piece<VEC>(qr, n, N);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      kv[r] = n + r < N ? kv[r] : 0.f;
      qk = mma(qv[r], kv[r], qk);
      if constexpr (DELTA) kk = mma(kv[r], kv[r], kk);
    }
  }
  float before = gm, after = __shfl_down(gm, 1, 16);
  if (c == 15) after = 1.f;
#pragma unroll
  for (int d = 1; d < 16; d *= 2) {
    const float lo = __shfl_up(before, d, 16), hi = __shfl_down(after, d, 16);
    if (c >= d) before *= lo;
    if (c + d < 16) after *= hi;
  }
  if (g == 0) s_g[c] = gm, s_b[c] = bm;
  __syncthreads();
  // register r: row i = 4 g + r, column j = c
  float decay[4];
  float p = 1.f;
#pragma unroll
  for (int m = 1; m <= 12; ++m)
    if (m <= 4 * g && m > c) p *= s_g[m];
  decay[0] = p;
#pragma unroll
  for (int r = 1; r < 4; ++r) {
    if (4 * g + r > c) p *= s_g[4 * g + r];
    decay[r] = p;
  }
  float* to = a.chunks + ((size_t)item * a.heads + h) * CHUNK_FLOATS;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = 4 * g + r;
    to[CHUNK_M + i * 16 + c] = c <= i ? decay[r] * (qk[r] * a.q_scale) : 0.f;
    if constexpr (DELTA) s_l[i * 20 + c] = c < i ? s_b[i] * decay[r] * kk[r] : 0.f;
  }
  if (g == 0) to[CHUNK_C + c] = before, to[CHUNK_D + c] = after, to[CHUNK_B + c] = bm;
  if constexpr (DELTA) {
    __syncthreads();
    // the inverse column by column (the four lane groups do the same): x_i = (i == c) - sum_(m < i) L_im x_m
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == c ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v -= s_l[i * 20 + m] * x[m];
      x[i] = v;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (i / 4 == g) to[CHUNK_T + i * 16 + c] = x[i] * bm;
  }
}

// One block of four waves per (entry, head, slice of 16 value columns); with RULE_SUM the column behind the last is the
// normaliser.  Wave w keeps the RT row tiles w RT .. of S's slice in registers (64 RT >= N rows in all).  Per chunk it forms its
// rows' part of S0^T k and S0^T q; the parts of S0^T k meet in shared memory, then every wave forms u (the same in all four), adds
// a quarter of the tokens' part to its outputs, and moves its rows on.  The outputs' parts meet in the next chunk's
// exchange: one barrier a chunk.  A chunk's operands are asked for AHEAD chunks ahead, straight into registers; the keys pass
// through the wave's own shared memory once, to be read the other way round.
template <int RT, int AHEAD, bool DELTA, bool VEC>
__global__ void __launch_bounds__(256)
memory_scan_kernel(const MemoryArgs a) {
  constexpr int KT_ROW = 16 * RT + 4;
  __shared__ mem_f32x4 s_w[2][4][64], s_o[2][4][64];
  __shared__ __attribute__((aligned(16))) float s_kt[4][16 * KT_ROW];
  const int b = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int N = a.N, P = a.P, col = blockIdx.z * 16 + c;
  const int kvh = h / (a.heads / a.kv_heads);
  const bool live_col = col < P || (!DELTA && col == P);
  const int first = a.q_start[b], end = a.q_start[b + 1];
  if (first >= end) return;
  float* row = a.state + (size_t)a.entry_slot[b] * a.state_stride;
  // where this lane's column lies: rows of S are P apart, the normaliser's values side by side
  float* column = col < P ? row + a.state_off + (size_t)h * N * P + col : row + a.norm_off + (size_t)h * N;
  const int row_step = col < P ? P : 1;
  const int n_first = 16 * w * RT;                   // this wave's first row
  mem_f32x4 S[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = n_first + 16 * t + 4 * g + r;
      S[t][r] = (live_col && n < N) ? column[(size_t)n * row_step] : 0.f;
    }
  struct In {
    mem_f32x4 k[RT], q[RT];                          // token c's channels
    mem_f32x4 v, tri, cum, tail, take;               // tokens 4 g + r (tri: row c)
    float m, all;
  };
  // offsets inside a chunk, in values; the last chunk of an entry may not reach past its end and repeats the last token
  int last = CHUNK_TOKENS - 1;
  unsigned off_k, off_q, off_v[4];
  auto offsets = [&]() __attribute__((always_inline)) {
    const int tc = c < last ? c : last;
    off_k = (unsigned)(tc * a.k_ld), off_q = (unsigned)(tc * a.q_ld);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tr = 4 * g + r < last ? 4 * g + r : last;
      off_v[r] = (unsigned)(tr * a.v_ld) + (unsigned)(col < P ? col : P - 1);
    }
  };
  offsets();
  const float* kh = a.k + (size_t)kvh * N;
  const float* qh = a.q + (size_t)kvh * N;
  const float* vh = a.v + (size_t)h * P;
  const float* pre = a.chunks + ((size_t)a.entry_item[b] * a.heads + h) * CHUNK_FLOATS;
  const int last_chunk = first + (end - first - 1) / CHUNK_TOKENS * CHUNK_TOKENS;
  // always as many loads, whatever is left of the entry (behind its last chunk that one again): the waits for those asked
  // for earlier can then be counted
  auto fetch = [&](int t0, In& in) __attribute__((always_inline)) {
    t0 = t0 < last_chunk ? t0 : last_chunk;
    if (t0 + CHUNK_TOKENS > end) {
      last = end - 1 - t0;
      offsets();
    }
    const float* kr = kh + (size_t)t0 * a.k_ld;
    const float* qr = qh + (size_t)t0 * a.q_ld;
    const float* vr = vh + (size_t)t0 * a.v_ld;
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      const int n = n_first + 16 * t + 4 * g;
      if constexpr (VEC) {
        const unsigned at = (unsigned)(n < N ? n : 0);
        in.k[t] = *reinterpret_cast<const mem_f32x4*>(kr + (off_k + at));
        in.q[t] = *reinterpret_cast<const mem_f32x4*>(qr + (off_q + at));
      } else {
        in.k[t] = row_piece<false>(kr + off_k, n, N);
        in.q[t] = row_piece<false>(qr + off_q, n, N);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) in.v[r] = vr[off_v[r]];
    const float* at = pre + (size_t)((t0 - first) / CHUNK_TOKENS) * a.heads * CHUNK_FLOATS;
    if constexpr (DELTA) in.tri = *reinterpret_cast<const mem_f32x4*>(at + (CHUNK_T + 16 * c + 4 * g));
    else in.take = *reinterpret_cast<const mem_f32x4*>(at + (CHUNK_B + 4 * g));
    in.m = at[CHUNK_M + 16 * c + 4 * g + w];
    in.cum = *reinterpret_cast<const mem_f32x4*>(at + (CHUNK_C + 4 * g));
    in.tail = *reinterpret_cast<const mem_f32x4*>(at + (CHUNK_D + 4 * g));
    in.all = at[CHUNK_C + 15];
  };
  // the outputs of the chunk that began at t0: this wave adds up the parts of tokens 4 g + w
  const int o_step = col < P ? a.heads * P : a.heads;
  float* o_at = (col < P ? a.out + (size_t)h * P + col : a.norm_out + h) + (size_t)(first + 4 * g + w) * o_step;
  auto finish = [&](int t0, int turn) __attribute__((always_inline)) {
    float o = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) o += reinterpret_cast<const float*>(&s_o[turn][i][lane])[w];
    if (live_col && t0 + 4 * g + w < end) *o_at = o;
    o_at += (size_t)CHUNK_TOKENS * o_step;
  };
  float* kt_in = s_kt[w] + c * KT_ROW + 4 * g;
  const float* kt_out = s_kt[w] + 4 * g * KT_ROW + c;
#define KEEP_ORDER __builtin_amdgcn_sched_barrier(0)
  const bool whole = N == 64 * RT;
  const bool odd = threadIdx.x & 64, upper = threadIdx.x & 128;
  auto chunk = [&](int t0, int turn, In& in, In& later) __attribute__((always_inline)) {
    fetch(t0 + AHEAD * CHUNK_TOKENS, later);
    const mem_f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    mem_f32x4 sk = zero, sq = zero, kt[RT];
    if (!whole) {                                    // rows past N stay zero
#pragma unroll
      for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int j = 0; j < 4; ++j) in.k[t][j] = n_first + 16 * t + 4 * g + j < N ? in.k[t][j] : 0.f;
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) *reinterpret_cast<mem_f32x4*>(kt_in + 16 * t) = in.k[t];
    // S0^T k first: the other waves wait for it, and S0^T q is worked on while it is on its way
    if constexpr (DELTA) {
#pragma unroll
      for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) sk = mma(in.k[t][r], S[t][r], sk);
      KEEP_ORDER;
    }
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sq = mma(in.q[t][r], S[t][r], sq);
        if (t == 0 && r == 1) {
          KEEP_ORDER;
          if constexpr (DELTA) s_w[turn][w][lane] = sk;
#pragma unroll
          for (int i = 0; i < RT; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) kt[i][j] = kt_out[j * KT_ROW + 16 * i];
          KEEP_ORDER;
        }
      }
    memory_barrier_shared();
    if constexpr (DELTA) {
      sk = s_w[turn][0][lane];
#pragma unroll
      for (int i = 1; i < 4; ++i) sk += s_w[turn][i][lane];
    }
    mem_f32x4 u;
    if constexpr (DELTA) {
      u = zero;
#pragma unroll
      for (int r = 0; r < 4; ++r) u = mma(in.tri[r], in.v[r] - in.cum[r] * sk[r], u);
    } else {
      u = in.take * ((!DELTA && col == P) ? zero + 1.f : in.v);
    }
    const mem_f32x4 part = in.cum * (sq * a.q_scale);
#pragma unroll
    for (int t = 0; t < RT; ++t) S[t] *= in.all;
    const mem_f32x4 ut = u * in.tail;
    const float lo = odd ? u[1] : u[0], hi = odd ? u[3] : u[2];
    s_o[turn][w][lane] = mma(in.m, upper ? hi : lo, part);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int t = 0; t < RT; ++t) S[t] = mma(kt[t][r], ut[r], S[t]);
    if (t0 > first) finish(t0 - CHUNK_TOKENS, 1 - turn);
  };
  In in[AHEAD + 1];
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) fetch(first + i * CHUNK_TOKENS, in[i]);
  // the sets of registers take turns, and so do the halves of the exchange: both come round after ROUND chunks
  constexpr int ROUND = AHEAD == 1 ? 2 : 2 * (AHEAD + 1);
  int t0 = first;
  for (bool more = true; more;) {
#pragma unroll
    for (int i = 0; i < ROUND; ++i) {
      chunk(t0, i & 1, in[i % (AHEAD + 1)], in[(i + AHEAD) % (AHEAD + 1)]);
      t0 += CHUNK_TOKENS;
      if (t0 >= end) {
        more = false;
        break;
      }
    }
  }
#undef KEEP_ORDER
  memory_barrier_shared();
  finish(last_chunk, (last_chunk - first) / CHUNK_TOKENS & 1);
  if (a.write_state && live_col) {
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = n_first + 16 * t + 4 * g + r;
        if (n < N) column[(size_t)n * row_step] = S[t][r];
      }
  }
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

template <int RT, bool DELTA>
static int launch_scan(const MemoryArgs& a, int B_, int n_items, hipStream_t stream) {
  const dim3 grid(B_, a.heads, (a.P + (DELTA ? 0 : 1) + 15) / 16);
  if (a.N % 4 == 0 && a.q_ld % 4 == 0 && a.k_ld % 4 == 0 && ((uintptr_t)a.q | (uintptr_t)a.k) % 16 == 0) {
    hipLaunchKernelGGL((memory_chunk_kernel<DELTA, true>), dim3(n_items, a.heads), dim3(64), 0, stream, a);
    // few blocks: nothing else runs while a chunk's operands are on their way, so they are asked for two chunks ahead
    if (RT <= 4 && (long long)grid.x * grid.y * grid.z < 512)
      hipLaunchKernelGGL((memory_scan_kernel<RT, RT <= 4 ? 2 : 1, DELTA, true>), grid, dim3(256), 0, stream, a);
    else
      hipLaunchKernelGGL((memory_scan_kernel<RT, 1, DELTA, true>), grid, dim3(256), 0, stream, a);
  } else {
    hipLaunchKernelGGL((memory_chunk_kernel<DELTA, false>), dim3(n_items, a.heads), dim3(64), 0, stream, a);
    hipLaunchKernelGGL((memory_scan_kernel<RT, 1, DELTA, false>), grid, dim3(256), 0, stream, a);
  }
  ULLM_LAUNCH_CHECK();
}

template <int PC, int NPT, bool DELTA>
static int launch_step(const MemoryArgs& a, int B_, hipStream_t stream) {
  hipLaunchKernelGGL((memory_step_kernel<PC, NPT, DELTA>), dim3(B_, a.heads, (a.P + PC - 1) / PC), dim3(256), 0, stream, a);
  ULLM_LAUNCH_CHECK();
}

template <bool DELTA>
static int memory_any(const MemoryArgs& a, int B_, int n_items, bool single, hipStream_t stream) {
  const int N = a.N;
  if (!single) {
    if (N <= 64) return launch_scan<1, DELTA>(a, B_, n_items, stream);
    if (N <= 128) return launch_scan<2, DELTA>(a, B_, n_items, stream);
    if (N <= 256) return launch_scan<4, DELTA>(a, B_, n_items, stream);
    return launch_scan<8, DELTA>(a, B_, n_items, stream);
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

// rule 0: RULE_DELTA, 1: RULE_SUM.  `single`: every entry brings exactly one token; else `items` (first token, tokens) lists
// the step's chunks of up to 16 tokens, `entry_item` every entry's first, and `chunks` has room for what is made of them.
extern "C" int ullm_matrix_memory(const float* q, int q_ld, const float* k, int k_ld, const float* v, int v_ld, const float* keep,
                                  const float* take, int gate_ld, int rule, float q_scale, float* state, long long state_stride,
                                  long long state_off, long long norm_off, const int* q_start, const int* entry_slot, const int* items,
                                  const int* entry_item, int n_items, float* chunks, float* out, float* norm_out, int B_, int heads,
                                  int kv_heads, int N, int P, int write_state, int single, hipStream_t stream) {
  if (B_ <= 0) return 0;
  if (heads < 1 || kv_heads < 1 || heads % kv_heads || N < 1 || P < 1 || N > MEMORY_MAX_KEYS || heads > 65535) return ULLM_ERR_SHAPE;
  if ((P + 16) / 16 > 65535) return ULLM_ERR_SHAPE;
  if (!single && (q_ld > (1 << 26) || k_ld > (1 << 26) || v_ld > (1 << 26))) return ULLM_ERR_SHAPE;   // 32-bit offsets inside a chunk
  if (!single && (n_items < B_ || !items || !entry_item || !chunks || (uintptr_t)chunks % 16)) return ULLM_ERR_SHAPE;
  if (rule != 0 && (rule != 1 || norm_out == nullptr)) return ULLM_ERR_UNSUPPORTED;
  MemoryArgs a;
  a.q = q, a.k = k, a.v = v, a.keep = keep, a.take = take, a.state = state, a.state_stride = state_stride, a.state_off = state_off;
  a.norm_off = norm_off, a.q_start = q_start, a.entry_slot = entry_slot, a.items = items, a.entry_item = entry_item, a.chunks = chunks;
  a.out = out, a.norm_out = norm_out, a.q_ld = q_ld, a.k_ld = k_ld, a.v_ld = v_ld, a.gate_ld = gate_ld, a.heads = heads;
  a.kv_heads = kv_heads, a.N = N, a.P = P, a.write_state = write_state, a.q_scale = q_scale;
  return rule == 0 ? memory_any<true>(a, B_, n_items, single != 0, stream) : memory_any<false>(a, B_, n_items, single != 0, stream);
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
