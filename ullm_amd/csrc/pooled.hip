// Attention over a sliding window and, beyond it, over blocks of tokens seen as one key and value each: what happens
// around the products, and the general form of the attention itself.
//
//   conv_norm_write   q | k | v as projected pass a short causal convolution per channel; q and k are divided by the
//                     root mean square over all their values of a token and multiplied by a gain per value; q goes out,
//                     k and v go to the paged pools
//   block_means       a block's key is the mean of its tokens' keys as the pools hold them, its value the mean of the
//                     values; they go to paged pools of their own, one row per block
//   attention         scores q . k * scale, soft-capped, a number per head added; weights sigmoid(score), added over the
//                     keys as they are (nothing is normalised), or the softmax
//
// All arithmetic is 32-bit; T selects the storage type only.  Pools: keys [page, kv_head, row, hd], values
// [page, kv_head, hd, row].
#include "common.h"
#include "short_conv.h"

__device__ __forceinline__ void cnw_block_sum2(float& a, float& b, float* scratch /* 32 floats */) {
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, nwaves = (blockDim.x + WAVE - 1) / WAVE;
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if (lane == 0) {
    scratch[wave] = a;
    scratch[16 + wave] = b;
  }
  __syncthreads();
  float ra = 0.f, rb = 0.f;
  for (int w = 0; w < nwaves; ++w) {
    ra += scratch[w];
    rb += scratch[16 + w];
  }
  a = ra;
  b = rb;
}

template <typename T, int V>
__device__ __forceinline__ void cnw_load(const T* p, float (&v)[V]) {
  if constexpr (V == 4 && sizeof(T) == 2) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16), v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16), v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else if constexpr (V == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
  } else {
    v[0] = ld_f32(p);
  }
}
template <typename T, int V>
__device__ __forceinline__ void cnw_store(T* p, const float (&v)[V]) {
  if constexpr (V == 4 && sizeof(T) == 2) *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
  else if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else st_f32(p, v[0]);
}

// What block_means needs of one block; also used by conv_norm_write for a token that completes a block.
template <typename T>
__device__ __forceinline__ void write_block_mean(int block, int pool, const int* __restrict__ bt, const int* __restrict__ pooled_bt,
                                                 const T* k_pool, const T* v_pool, T* pk_pool, T* pv_pool, int page_size,
                                                 int nkv, int hd, int kvh, int tid, int nthreads) {
  const int to = pooled_bt[block / page_size];
  if (to < 0) return;
  const int slot = block % page_size;
  const float inv = 1.f / (float)pool;
  for (int d = tid; d < hd; d += nthreads) {
    float ks = 0.f, vs = 0.f;
    for (int j0 = 0; j0 < pool; j0 += 8) {                            // eight rows under way; added in order
      float kv[8], vv[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int pos = block * pool + (j0 + u < pool ? j0 + u : pool - 1), off = pos % page_size;
        const int page = max(bt[pos / page_size], 0);                 // (a block's tokens are held until it is complete)
        kv[u] = ld_f32(k_pool + (((size_t)page * nkv + kvh) * page_size + off) * hd + d);
        vv[u] = ld_f32(v_pool + (((size_t)page * nkv + kvh) * hd + d) * page_size + off);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (j0 + u < pool) ks += kv[u], vs += vv[u];
    }
    st_f32(pk_pool + (((size_t)to * nkv + kvh) * page_size + slot) * hd + d, ks * inv);
    st_f32(pv_pool + (((size_t)to * nkv + kvh) * hd + d) * page_size + slot, vs * inv);
  }
}

// One block of threads per run of RUN tokens.  A row of `proj` is q | k | v, (nq + 2 nkv) * hd = C values; weights lie tap
// by tap [taps, C]; the entry's state row holds the last taps-1 rows before the step, oldest first.  A thread owns PIECES
// pieces of V neighbouring channels: the run's rows are all asked for at once, and the last inputs stay in registers
// along the run.  Where the run's tokens lie side by side in a page, a channel's four values go out in one store.
// `single`: every entry brings one token: the thread moves its channels' state on itself, and a token that completes a
// block of `pool` tokens (pool > 0) leaves that block's mean behind.
template <typename T, int TAPS, int V, int PIECES, int RUN>
__global__ void __launch_bounds__(1024)
conv_norm_write_kernel(const T* __restrict__ proj, int ld, const float* __restrict__ w, int taps_rt, float* __restrict__ carry,
                       long long carry_stride, const float* __restrict__ q_gain, const float* __restrict__ k_gain, float eps,
                       float q_count, float k_count, const int* __restrict__ positions, const int* __restrict__ token_entry,
                       const int* __restrict__ q_start, const int* __restrict__ entry_slot, const int* __restrict__ block_table,
                       int bt_stride, T* __restrict__ q_out, T* k_pool, T* v_pool, int page_size, int nq, int nkv, int hd,
                       int T_, int single, int pool, const int* __restrict__ pooled_table, int pooled_stride,
                       T* pk_pool, T* pv_pool) {
  __shared__ float scratch[2][32];
  const int C = (nq + 2 * nkv) * hd, nqv = nq * hd, nkvv = nkv * hd, tid = threadIdx.x, nthreads = blockDim.x;
  constexpr int HT = TAPS > 0 ? TAPS : 1;
  const int taps = TAPS > 0 ? TAPS : taps_rt;
  const int t0 = blockIdx.x * RUN;
  float wt[PIECES][HT][V], hist[PIECES][HT][V], y[PIECES][RUN][V], gain[PIECES][V];
  int ent[RUN], pos[RUN], page[RUN];
#pragma unroll
  for (int r = 0; r < RUN; ++r) {
    const int t = t0 + r < T_ ? t0 + r : T_ - 1;
    ent[r] = token_entry[t];
    pos[r] = positions[t];
    page[r] = block_table[(size_t)ent[r] * bt_stride + pos[r] / page_size];
  }
#pragma unroll
  for (int p = 0; p < PIECES; ++p) {
    const int c = V * (tid + p * nthreads);
    if (c >= C) continue;
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int r = 0; r < RUN; ++r) cnw_load<T, V>(proj + (size_t)(t0 + r < T_ ? t0 + r : T_ - 1) * ld + c, y[p][r]);
#pragma unroll
      for (int j = 0; j < TAPS; ++j) cnw_load<float, V>(w + (size_t)j * C + c, wt[p][j]);
    }
    if (c < nqv + nkvv) cnw_load<float, V>(c < nqv ? q_gain + c : k_gain + (c - nqv), gain[p]);
  }
  const bool side_by_side = RUN == 4 && t0 + RUN <= T_ && ent[0] == ent[RUN - 1] && pos[0] % 4 == 0 && page_size % 4 == 0 && page[0] >= 0;
#pragma unroll
  for (int r = 0; r < RUN; ++r) {
    const int t = t0 + r;
    if (t >= T_) break;
    const int b = ent[r], first = q_start[b], i = t - first;
    float* old = carry + (size_t)entry_slot[b] * carry_stride;
    float ssq = 0.f, ssk = 0.f;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      const int c = V * (tid + p * nthreads);
      if (c >= C) continue;
      float out[V];
#pragma unroll
      for (int u = 0; u < V; ++u) out[u] = 0.f;
      if constexpr (TAPS > 0) {
        if (r == 0 || i == 0) {
#pragma unroll
          for (int k = 0; k < TAPS - 1; ++k) {
            const int l = i - (TAPS - 1) + k;
            if (l >= 0) cnw_load<T, V>(proj + (size_t)(first + l) * ld + c, hist[p][k]);
            else cnw_load<float, V>(old + (size_t)(l + TAPS - 1) * C + c, hist[p][k]);
          }
        }
#pragma unroll
        for (int u = 0; u < V; ++u) hist[p][TAPS - 1][u] = y[p][r][u];
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
          for (int u = 0; u < V; ++u) out[u] += wt[p][j][u] * hist[p][j][u];
        if (single) {
#pragma unroll
          for (int k = 0; k < TAPS - 1; ++k) cnw_store<float, V>(old + (size_t)k * C + c, hist[p][k + 1]);
        }
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
          for (int u = 0; u < V; ++u) hist[p][k][u] = hist[p][k + 1][u];
      } else {
        for (int j = 0; j < taps; ++j) {
          const int l = i - (taps - 1) + j;
          float in[V], ww[V];
          if (l >= 0) cnw_load<T, V>(proj + (size_t)(first + l) * ld + c, in);
          else cnw_load<float, V>(old + (size_t)(l + taps - 1) * C + c, in);
          cnw_load<float, V>(w + (size_t)j * C + c, ww);
#pragma unroll
          for (int u = 0; u < V; ++u) out[u] += ww[u] * in[u];
        }
      }
#pragma unroll
      for (int u = 0; u < V; ++u) {
        y[p][r][u] = out[u];
        if (c < nqv) ssq += out[u] * out[u];
        else if (c < nqv + nkvv) ssk += out[u] * out[u];
      }
    }
    cnw_block_sum2(ssq, ssk, scratch[r & 1]);
    const float rsq = 1.f / sqrtf(ssq / q_count + eps), rsk = 1.f / sqrtf(ssk / k_count + eps);
    const int slot = pos[r] % page_size;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      const int c = V * (tid + p * nthreads);
      if (c >= C) continue;
      if (c < nqv) {
        float o[V];
#pragma unroll
        for (int u = 0; u < V; ++u) o[u] = (y[p][r][u] * rsq) * gain[p][u];
        cnw_store<T, V>(q_out + (size_t)t * nqv + c, o);
      } else if (page[r] >= 0 && c < nqv + nkvv) {
        const int kc = c - nqv, kvh = kc / hd, d = kc % hd;
        float o[V];
#pragma unroll
        for (int u = 0; u < V; ++u) o[u] = (y[p][r][u] * rsk) * gain[p][u];
        cnw_store<T, V>(k_pool + (((size_t)page[r] * nkv + kvh) * page_size + slot) * hd + d, o);
      } else if (page[r] >= 0 && !side_by_side) {
        const int vc = c - nqv - nkvv, kvh = vc / hd, d = vc % hd;
        T* dst = v_pool + (((size_t)page[r] * nkv + kvh) * hd + d) * page_size + slot;
#pragma unroll
        for (int u = 0; u < V; ++u) st_f32(dst + (size_t)u * page_size, y[p][r][u]);
      }
    }
    if (single && pool > 0 && page[r] >= 0 && (pos[r] + 1) % pool == 0) {
      __threadfence_block();
      __syncthreads();                                      // the block's own stores of this token's key and value
      const int lane = tid & 63, wave = tid / 64, nwaves = nthreads / 64;
      for (int kvh = wave; kvh < nkv; kvh += nwaves)
        write_block_mean<T>(pos[r] / pool, pool, block_table + (size_t)b * bt_stride, pooled_table + (size_t)b * pooled_stride,
                            k_pool, v_pool, pk_pool, pv_pool, page_size, nkv, hd, kvh, lane, 64);
    }
  }
  if constexpr (RUN == 4) {
    if (!side_by_side) return;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      const int c = V * (tid + p * nthreads);
      if (c >= C || c < nqv + nkvv) continue;
      const int vc = c - nqv - nkvv, kvh = vc / hd, d = vc % hd;
      T* dst = v_pool + (((size_t)page[0] * nkv + kvh) * hd + d) * page_size + pos[0] % page_size;
#pragma unroll
      for (int u = 0; u < V; ++u) {
        float o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = y[p][r < RUN ? r : 0][u];
        cnw_store<T, 4>(dst + (size_t)u * page_size, o);
      }
    }
  }
}

extern "C" int ullm_conv_norm_write(const void* proj, int ld, const float* w, int taps, float* carry, long long carry_stride,
                                    const float* q_gain, const float* k_gain, float eps, float q_count, float k_count,
                                    const int* positions, const int* token_entry, const int* q_start, const int* entry_slot,
                                    const int* block_table, int bt_stride, void* q_out, void* k_pool, void* v_pool,
                                    int page_size, int nq, int nkv, int hd, int T_, int B_, int single, int pool,
                                    const int* pooled_table, int pooled_stride, void* pk_pool, void* pv_pool, int dtype,
                                    hipStream_t stream) {
  if (T_ <= 0) return 0;
  if (nq < 1 || nkv < 1 || hd < 1 || page_size < 1 || taps < 1 || taps > SHORT_CONV_MAX_TAPS || q_count <= 0.f || k_count <= 0.f || pool < 0)
    return ULLM_ERR_SHAPE;
  const int C = (nq + 2 * nkv) * hd;
  if (ld < C) return ULLM_ERR_SHAPE;
  if (pool > 0 && single && (!pooled_table || !pk_pool || !pv_pool)) return ULLM_ERR_UNSUPPORTED;
  const size_t item = dtype == ULLM_F32 ? 4 : 2;
  const bool by4 = hd % 4 == 0 && ld % 4 == 0 && carry_stride % 4 == 0 && (uintptr_t)proj % (4 * item) == 0 &&
                   (uintptr_t)carry % 16 == 0 && ((uintptr_t)w | (uintptr_t)q_gain | (uintptr_t)k_gain) % 16 == 0;
  const int pieces_all = by4 ? C / 4 : C;
  int pieces = 1;
  while (pieces * (T_ >= 64 ? 512 : 1024) < pieces_all) pieces *= 2;
  if (pieces > 16) return ULLM_ERR_SHAPE;                    // rows of up to 65536 values (16384 where not by fours)
  const int threads = ((pieces_all + pieces - 1) / pieces + 63) / 64 * 64;
  const bool runs = !single && T_ >= 512;
#define GO_R(TT, TAPS, V, P, R) hipLaunchKernelGGL((conv_norm_write_kernel<TT, TAPS, V, P, R>), dim3((T_ + R - 1) / R), dim3(threads), 0, \
    stream, (const TT*)proj, ld, w, taps, carry, carry_stride, q_gain, k_gain, eps, q_count, k_count, positions, token_entry,        \
    q_start, entry_slot, block_table, bt_stride, (TT*)q_out, (TT*)k_pool, (TT*)v_pool, page_size, nq, nkv, hd, T_, single,           \
    pool, pooled_table, pooled_stride, (TT*)pk_pool, (TT*)pv_pool)
#define GO(TT, TAPS, V, P) GO_R(TT, TAPS, V, P, 1)
#define GO_P(TT, TAPS, V) do { if (pieces <= 4 && runs && V == 4) { if (pieces == 1) GO_R(TT, TAPS, V, 1, 4); else if (pieces == 2) GO_R(TT, TAPS, V, 2, 4); else GO_R(TT, TAPS, V, 4, 4); } else if (pieces == 1) GO(TT, TAPS, V, 1); else if (pieces == 2) GO(TT, TAPS, V, 2); \
    else if (pieces == 4) GO(TT, TAPS, V, 4); else if (pieces == 8) GO(TT, 0, V, 8); else GO(TT, 0, V, 16); } while (0)
  // up to 4 taps with up to 4 pieces a thread the inputs are kept in registers; else every tap is read where it lies,
  // and the state is moved on by a kernel of its own
#define GO_T(TT) do {                                                                 \
    if (!by4) GO_P(TT, 0, 1);                                                         \
    else if (taps == 2) GO_P(TT, 2, 4);                                               \
    else if (taps == 3) GO_P(TT, 3, 4);                                               \
    else if (taps == 4) GO_P(TT, 4, 4);                                               \
    else GO_P(TT, 0, 4);                                                              \
  } while (0)
  if (dtype == ULLM_F32) GO_T(float);
  else if (dtype == ULLM_BF16) GO_T(bf16_t);
  else return ULLM_ERR_DTYPE;
#undef GO_T
#undef GO_P
#undef GO
#undef GO_R
  const bool moved = single && by4 && taps >= 2 && taps <= 4 && pieces <= 4;
  if (taps > 1 && !moved) {
    if (dtype == ULLM_F32) launch_carry<float>(proj, ld, carry, carry_stride, q_start, entry_slot, B_, C, taps, stream);
    else launch_carry<bf16_t>(proj, ld, carry, carry_stride, q_start, entry_slot, B_, C, taps, stream);
  }
  ULLM_LAUNCH_CHECK();
}

template <typename T>
__global__ void __launch_bounds__(128)
block_means_kernel(const int* __restrict__ blocks, const int* __restrict__ block_table, int bt_stride,
                   const int* __restrict__ pooled_table, int pooled_stride, const T* __restrict__ k_pool,
                   const T* __restrict__ v_pool, T* __restrict__ pk_pool, T* __restrict__ pv_pool, int pool, int page_size,
                   int nkv, int hd) {
  const int b = blocks[2 * blockIdx.x], block = blocks[2 * blockIdx.x + 1];
  write_block_mean<T>(block, pool, block_table + (size_t)b * bt_stride, pooled_table + (size_t)b * pooled_stride, k_pool, v_pool,
                      pk_pool, pv_pool, page_size, nkv, hd, blockIdx.y, threadIdx.x, blockDim.x);
}

extern "C" int ullm_block_means(const int* blocks, int n_blocks, const int* block_table, int bt_stride, const int* pooled_table,
                                int pooled_stride, const void* k_pool, const void* v_pool, void* pk_pool, void* pv_pool,
                                int pool, int page_size, int nkv, int hd, int dtype, hipStream_t stream) {
  if (n_blocks <= 0) return 0;
  if (pool < 1 || page_size < 1 || nkv < 1 || hd < 1) return ULLM_ERR_SHAPE;
#define GO(TT) hipLaunchKernelGGL(block_means_kernel<TT>, dim3(n_blocks, nkv), dim3(128), 0, stream, blocks, block_table, bt_stride, \
    pooled_table, pooled_stride, (const TT*)k_pool, (const TT*)v_pool, (TT*)pk_pool, (TT*)pv_pool, pool, page_size, nkv, hd)
  if (dtype == ULLM_F32) GO(float);
  else if (dtype == ULLM_BF16) GO(bf16_t);
  else return ULLM_ERR_DTYPE;
#undef GO
  ULLM_LAUNCH_CHECK();
}

// ------------------------------------------------------------------ the general form of the attention
// One block per (token, query head), any head size up to 1024; keys are visited in tiles of the block size in a fixed
// order (first the blocks, then the window's tokens) that depends on the token's position alone.
#define PAG_THREADS 128
#define PAG_MAX_HD 1024
template <typename T>
__global__ void __launch_bounds__(PAG_THREADS)
pooled_attention_general_kernel(const T* __restrict__ q, int q_stride, T* __restrict__ out, const T* __restrict__ k_pool,
                                const T* __restrict__ v_pool, const int* __restrict__ block_table, int bt_stride,
                                const T* __restrict__ pk_pool, const T* __restrict__ pv_pool,
                                const int* __restrict__ pooled_table, int pooled_stride, const int* __restrict__ positions,
                                const int* __restrict__ token_entry, int page_size, int nq, int nkv, int hd, float scale,
                                float softcap, const float* __restrict__ head_bias, int window, int pool, int softmax) {
  __shared__ float q_s[PAG_MAX_HD];
  __shared__ float p_s[PAG_THREADS];
  __shared__ long long row_s[PAG_THREADS];
  __shared__ float scratch[16];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, kvh = h / (nq / nkv);
  const int pos = positions[t], b = token_entry[t];
  const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
  // blocks wholly before the window: (block + 1) * pool <= lo, where the window has a first token behind position 0
  const int n_blocks = pool > 0 ? lo / pool : 0;
  const int n_keys = n_blocks + pos - lo + 1;
  for (int i = tid; i < hd; i += PAG_THREADS) q_s[i] = ld_f32(q + (size_t)t * q_stride + (size_t)h * hd + i);
  __syncthreads();
  constexpr int DPT = PAG_MAX_HD / PAG_THREADS;
  float acc[DPT];
#pragma unroll
  for (int r = 0; r < DPT; ++r) acc[r] = 0.f;
  const float add = head_bias ? head_bias[h] : 0.f;
  float m = -INFINITY, l = 0.f;
  for (int base = 0; base < n_keys; base += PAG_THREADS) {
    const int j = base + tid;
    float s = -INFINITY;
    long long row = -1;
    const bool in_block = j < n_blocks;
    if (j < n_keys) {
      const int key = in_block ? j : lo + j - n_blocks;
      const int page = in_block ? pooled_table[(size_t)b * pooled_stride + key / page_size] : block_table[(size_t)b * bt_stride + key / page_size];
      if (page >= 0) {
        row = ((long long)page * nkv + kvh) * page_size + key % page_size;
        const T* kp = (in_block ? pk_pool : k_pool) + row * hd;
        float d = 0.f;
        for (int i = 0; i < hd; ++i) d += q_s[i] * ld_f32(kp + i);
        d *= scale;
        if (softcap > 0.f) d = softcap * tanhf(d / softcap);
        s = d + add;
      }
    }
    float alpha = 1.f, p;
    if (softmax) {
      const float m_new = fmaxf(m, block_max(s, scratch));
      p = row >= 0 ? expf(s - m_new) : 0.f;
      alpha = m == -INFINITY ? 0.f : expf(m - m_new);
      l = l * alpha + block_sum(p, scratch);
      if (m_new > -INFINITY) m = m_new;
    } else {
      p = row >= 0 ? 1.f / (1.f + expf(-s)) : 0.f;
    }
    __syncthreads();
    p_s[tid] = p;
    row_s[tid] = row;
    __syncthreads();
    const int n_tile = n_keys - base < PAG_THREADS ? n_keys - base : PAG_THREADS;
#pragma unroll
    for (int r = 0; r < DPT; ++r) {
      const int d = tid + r * PAG_THREADS;
      if (d < hd) {
        float a = acc[r] * alpha;
        for (int jj = 0; jj < n_tile; ++jj) {
          const long long vr = row_s[jj];
          if (vr >= 0)
            a += p_s[jj] * ld_f32((base + jj < n_blocks ? pv_pool : v_pool) + (vr / page_size) * page_size * hd + (size_t)d * page_size + vr % page_size);
        }
        acc[r] = a;
      }
    }
  }
  const float inv = softmax ? (l > 0.f ? 1.f / l : 0.f) : 1.f;
#pragma unroll
  for (int r = 0; r < DPT; ++r) {
    const int d = tid + r * PAG_THREADS;
    if (d < hd) st_f32(out + ((size_t)t * nq + h) * hd + d, acc[r] * inv);
  }
}

extern "C" int ullm_pooled_attention_general(const void* q, int q_stride, void* out, const void* k_pool, const void* v_pool,
                                             const int* block_table, int bt_stride, const void* pk_pool, const void* pv_pool,
                                             const int* pooled_table, int pooled_stride, const int* positions,
                                             const int* token_entry, int page_size, int T_, int nq, int nkv, int hd,
                                             float scale, float softcap, const float* head_bias, int window, int pool,
                                             int softmax, int dtype, hipStream_t stream) {
  if (T_ <= 0) return 0;
  if (hd < 1 || hd > PAG_MAX_HD || nq < 1 || nq > 65535 || nkv < 1 || nq % nkv || page_size < 1 || window < 0 || pool < 0 ||
      (pool > 0 && (window < 1 || !pk_pool || !pv_pool || !pooled_table)))
    return ULLM_ERR_SHAPE;
#define GO(TT) hipLaunchKernelGGL(pooled_attention_general_kernel<TT>, dim3(T_, nq), dim3(PAG_THREADS), 0, stream, (const TT*)q, q_stride, \
    (TT*)out, (const TT*)k_pool, (const TT*)v_pool, block_table, bt_stride, (const TT*)pk_pool, (const TT*)pv_pool, pooled_table,     \
    pooled_stride, positions, token_entry, page_size, nq, nkv, hd, scale, softcap, head_bias, window, pool, softmax)
  if (dtype == ULLM_F32) GO(float);
  else if (dtype == ULLM_BF16) GO(bf16_t);
  else return ULLM_ERR_DTYPE;
#undef GO
  ULLM_LAUNCH_CHECK();
}
