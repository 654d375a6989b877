// Attention over a sliding window and, beyond it, over blocks of tokens seen as one key and value each, with sigmoid
// weights, on the matrix cores (bfloat16 operands, 32-bit accumulation): for decoded tokens and for prompt portions.
//
//   weight(key) = sigmoid(cap * tanh(q . k * scale / cap) + bias[head])   (without a cap: sigmoid(q . k * scale + bias))
//   out = sum over the visible keys of weight * value
//
// Nothing is normalised over the keys, so there is no running maximum, no rescaling and partial results simply add.
// One wave owns 16 "columns" per group (decode: the query heads of one token that share a kv head; prompts: 16
// consecutive tokens of one head).  Per 32 keys:
//   S^T[key, col]   = K[key, :] . Q[col, :]          (v_mfma_f32_16x16x32_bf16: A = K rows, B = Q columns)
//   O^T[dim, col]  += V^T[dim, key] * P^T[key, col]  (A = values, transposed inside the page, B = P)
// and a lane's weights are the ones it feeds as the B operand of the second product.
//
// A query's keys are two ranges: rows [0, n_blocks) of the pooled pools, with n_blocks = lo / pool and lo the window's
// first token, then tokens [lo, pos].  Both are walked as one list of 32-key tiles.
// Pools: keys [page, kv_head, row, hd], values [page, kv_head, hd, row]; the page size is a multiple of 16.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
union Pack8 {
  bf16x8_t v;
  uint4 u4;
  uint2 u2[2];
  uint32_t w[4];
  bf16_t h[8];
};

// The weight of a raw product s, with the constants folded into exponents of two.  With a cap c:
//   tanh(y) = 1 - 2 / (1 + e^(2y)), so -(c tanh(y) + bias) log2(e) = k1 + k2 / (1 + 2^(k0 s)),
//   k0 = 2 scale log2(e) / c, k1 = -(c + bias) log2(e), k2 = 2 c log2(e); without one the exponent is k0 s + k1 with
//   k0 = -scale log2(e), k1 = -bias log2(e).  An exponent of two that overflows is an infinity whose reciprocal is 0.
struct WeightConsts {
  float k0, k1, k2;
};
__device__ __forceinline__ WeightConsts weight_consts(float scale, float cap, float bias) {
  constexpr float L2E = 1.4426950408889634f;
  if (cap > 0.f) return {2.f * scale * L2E / cap, -(cap + bias) * L2E, 2.f * cap * L2E};
  return {-scale * L2E, -bias * L2E, 0.f};
}
template <bool CAP>
__device__ __forceinline__ float key_weight(float s, const WeightConsts& k) {
  if constexpr (CAP) {
    const float r = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(k.k0 * s));
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fmaf(k.k2, r, k.k1)));
  } else {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fmaf(k.k0, s, k.k1)));
  }
}

// Both ranges of one request as seen by the kernels.
struct KeyRanges {
  const bf16_t* k_pool;
  const bf16_t* v_pool;
  const bf16_t* pk_pool;
  const bf16_t* pv_pool;
  const int* bt;              // the request's rows of the two block tables
  const int* pbt;
  int page_size, nkv, kvh;
};

// ------------------------------------------------------------------------------- decode
template <int NQK>
struct Tile {
  Pack8 k[2][NQK];
  uint2 v[2 * NQK][2];
};

// Pages of up to 64 consecutive 16-key pieces of the tile list, one per lane.
struct PieceWindow {
  int base;                   // first piece (tile * 2 + half) held
  int page, off;              // lane i: page id of piece base + i (-1: none) and the row of its first key there
};

// Tiles [0, n_pool_tiles) are blocks, tile n_pool_tiles + j holds tokens first + 32 j ...
__device__ __forceinline__ PieceWindow load_pieces(int piece, int n_blocks, int n_pool_tiles, int first, int pos, const KeyRanges& r) {
  PieceWindow w;
  w.base = piece;
  const int at = piece + (int)(threadIdx.x & 63);
  const bool pooled = at < 2 * n_pool_tiles;
  const int key = pooled ? 16 * at : first + 16 * (at - 2 * n_pool_tiles);
  const bool in = pooled ? key < n_blocks : key <= pos;
  w.page = in ? (pooled ? r.pbt : r.bt)[key / r.page_size] : -1;
  w.off = key % r.page_size;
  return w;
}

template <int NQK>
__device__ __forceinline__ void load_tile(Tile<NQK>& t, int tile, int n_pool_tiles, const PieceWindow& w, const KeyRanges& r) {
  constexpr int HD = 32 * NQK;
  const int lane = threadIdx.x & 63, g = lane >> 4, c = lane & 15;
  const bool pooled = tile < n_pool_tiles;
  const bf16_t* const kb = pooled ? r.pk_pool : r.k_pool;
  const bf16_t* const vb = pooled ? r.pv_pool : r.v_pool;
#pragma unroll
  for (int sb = 0; sb < 2; ++sb) {
    const int page = __builtin_amdgcn_readlane(w.page, 2 * tile + sb - w.base);
    const int off = __builtin_amdgcn_readlane(w.off, 2 * tile + sb - w.base);
    if (page >= 0) {
      const bf16_t* kp = kb + (((size_t)page * r.nkv + r.kvh) * r.page_size + off + c) * HD + 8 * g;
#pragma unroll
      for (int ch = 0; ch < NQK; ++ch) t.k[sb][ch].u4 = ld16(kp + 32 * ch);
      const bf16_t* vp = vb + (((size_t)page * r.nkv + r.kvh) * HD + c) * r.page_size + off + 4 * g;
#pragma unroll
      for (int n = 0; n < 2 * NQK; ++n) t.v[n][sb] = ld_stream8(vp + (size_t)16 * n * r.page_size);
    } else {
#pragma unroll
      for (int ch = 0; ch < NQK; ++ch) t.k[sb][ch].u4 = make_uint4(0, 0, 0, 0);
#pragma unroll
      for (int n = 0; n < 2 * NQK; ++n) t.v[n][sb] = make_uint2(0, 0);
    }
  }
}

// Keys key0 .. key0 + 31 of one range; the columns see lo .. hi of it (the same for all columns: one token).
template <int NQK, bool CAP>
__device__ __forceinline__ void work_tile(const Tile<NQK>& t, int key0, int lo, int hi, const Pack8 (&q)[NQK], const WeightConsts& kc,
                                          f32x4_t (&acc)[2 * NQK]) {
  const int g = (threadIdx.x & 63) >> 4;
  const bool whole = key0 >= lo && key0 + 31 <= hi;
  f32x4_t s[2];
#pragma unroll
  for (int sb = 0; sb < 2; ++sb) {
    s[sb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ch = 0; ch < NQK; ++ch) s[sb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(t.k[sb][ch].v, q[ch].v, s[sb], 0, 0, 0);
  }
  Pack8 p;
#pragma unroll
  for (int sb = 0; sb < 2; ++sb) {
    float e[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      e[r] = key_weight<CAP>(s[sb][r], kc);
      if (!whole) {
        const int kk = key0 + 16 * sb + 4 * g + r;
        if (kk < lo || kk > hi) e[r] = 0.f;
      }
    }
    p.w[2 * sb] = pack2_bf16(e[0], e[1]);
    p.w[2 * sb + 1] = pack2_bf16(e[2], e[3]);
  }
#pragma unroll
  for (int n = 0; n < 2 * NQK; ++n) {
    Pack8 v;
    v.u2[0] = t.v[n][0];
    v.u2[1] = t.v[n][1];
    if (!whole) {
      // rows of the tile behind the data hold whatever was there before: not to be multiplied, even by zero
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (key0 + 16 * (j >> 2) + 4 * g + (j & 3) > hi) v.h[j] = 0;
    }
    acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, p.v, acc[n], 0, 0, 0);
  }
}

// grid (num_splits, nkv * col_groups, n_tokens), block 64 * WAVES.  A token's tiles are cut into num_splits * WAVES
// equal shares (a cut that depends on the token's own position); the waves' outputs are added pairwise through shared
// memory in a fixed order, the splits' by a second small kernel in split order.
template <int NQK, int WAVES, bool CAP>
__global__ void __launch_bounds__(64 * WAVES)
pooled_decode_kernel(const bf16_t* __restrict__ q, int q_stride, bf16_t* __restrict__ out, const bf16_t* __restrict__ k_pool,
                     const bf16_t* __restrict__ v_pool, const int* __restrict__ block_table, int bt_stride,
                     const bf16_t* __restrict__ pk_pool, const bf16_t* __restrict__ pv_pool,
                     const int* __restrict__ pooled_table, int pooled_stride, const int* __restrict__ token_list,
                     const int* __restrict__ positions, const int* __restrict__ token_entry, int page_size, int nq, int nkv,
                     float scale, float cap, const float* __restrict__ head_bias, int window, int pool, int num_splits,
                     float* __restrict__ part) {
  constexpr int HD = 32 * NQK;
  __shared__ float merge[WAVES > 1 ? (WAVES / 2) * 8 * NQK * 64 : 1];      // [writer][value][lane]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
  const int G = nq / nkv, groups = (G + 15) / 16;
  const int kvh = blockIdx.y / groups, in_group = (blockIdx.y % groups) * 16 + c;
  const int item = blockIdx.z, t = token_list ? token_list[item] : item;
  const bool col_ok = in_group < G;
  const int head = kvh * G + (col_ok ? in_group : 0);
  Pack8 qreg[NQK];
#pragma unroll
  for (int ch = 0; ch < NQK; ++ch) qreg[ch].u4 = ld16(q + (size_t)t * q_stride + (size_t)head * HD + 32 * ch + 8 * g);
  const int pos = positions[t], b = token_entry[t];
  const KeyRanges r = {k_pool, v_pool, pk_pool, pv_pool, block_table + (size_t)b * bt_stride,
                       pool > 0 ? pooled_table + (size_t)b * pooled_stride : nullptr, page_size, nkv, kvh};
  const WeightConsts kc = weight_consts(scale, cap, head_bias ? head_bias[head] : 0.f);
  const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
  const int n_blocks = pool > 0 ? lo / pool : 0, pt = (n_blocks + 31) / 32;
  const int first = lo & ~31, tiles = pt + (pos - first) / 32 + 1;
  const int share = (tiles + num_splits * WAVES - 1) / (num_splits * WAVES);
  const int begin = ((int)blockIdx.x * WAVES + wave) * share, stop = begin + share < tiles ? begin + share : tiles;
  f32x4_t acc[2 * NQK];
#pragma unroll
  for (int n = 0; n < 2 * NQK; ++n) acc[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#define TILE_WORK(T, I)                                                                                      \
  do {                                                                                                       \
    if ((I) < pt) work_tile<NQK, CAP>(T, 32 * (I), 0, n_blocks - 1, qreg, kc, acc);                           \
    else work_tile<NQK, CAP>(T, first + 32 * ((I) - pt), lo, pos, qreg, kc, acc);                             \
  } while (0)
  for (int base = begin; base < stop; base += 32) {
    const PieceWindow w = load_pieces(2 * base, n_blocks, pt, first, pos, r);
    const int end = base + 32 < stop ? base + 32 : stop;
    Tile<NQK> t0, t1;                                     // in turns: one is worked on while the other loads
    load_tile<NQK>(t0, base, pt, w, r);
    for (int i = base; i < end; i += 2) {
      if (i + 1 < end) load_tile<NQK>(t1, i + 1, pt, w, r);
      TILE_WORK(t0, i);
      if (i + 1 >= end) break;
      if (i + 2 < end) load_tile<NQK>(t0, i + 2, pt, w, r);
      TILE_WORK(t1, i + 1);
    }
  }
#undef TILE_WORK
#pragma unroll
  for (int half = WAVES / 2; half >= 1; half >>= 1) {
    if (wave >= half && wave < 2 * half) {
      float* m = merge + (size_t)(wave - half) * 8 * NQK * 64 + lane;
#pragma unroll
      for (int n = 0; n < 2 * NQK; ++n)
#pragma unroll
        for (int e = 0; e < 4; ++e) m[(4 * n + e) * 64] = acc[n][e];
    }
    __syncthreads();
    if (wave < half) {
      const float* m = merge + (size_t)wave * 8 * NQK * 64 + lane;
#pragma unroll
      for (int n = 0; n < 2 * NQK; ++n)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[n][e] += m[(4 * n + e) * 64];
    }
    __syncthreads();
  }
  if (wave != 0 || !col_ok) return;
  if (num_splits == 1) {
    bf16_t* op = out + ((size_t)t * nq + head) * HD;
#pragma unroll
    for (int n = 0; n < 2 * NQK; ++n)
      *reinterpret_cast<uint2*>(op + 16 * n + 4 * g) = make_uint2(pack2_bf16(acc[n][0], acc[n][1]), pack2_bf16(acc[n][2], acc[n][3]));
    return;
  }
  float* pp = part + (((size_t)item * nq + head) * num_splits + blockIdx.x) * HD;
#pragma unroll
  for (int n = 0; n < 2 * NQK; ++n)
    *reinterpret_cast<float4*>(pp + 16 * n + 4 * g) = make_float4(acc[n][0], acc[n][1], acc[n][2], acc[n][3]);
}

// out[token, head] = the splits' partial outputs added in split order.  grid (n_items, nq).
__global__ void __launch_bounds__(64)
pooled_reduce_kernel(const float* __restrict__ part, bf16_t* __restrict__ out, const int* __restrict__ token_list, int nq, int hd,
                     int num_splits) {
  const int item = blockIdx.x, head = blockIdx.y, t = token_list ? token_list[item] : item;
  const float* pp = part + ((size_t)item * nq + head) * num_splits * hd;
  for (int d = 4 * threadIdx.x; d < hd; d += 256) {
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int s = 0; s < num_splits; ++s) {
      const float4 v = *reinterpret_cast<const float4*>(pp + (size_t)s * hd + d);
      a.x += v.x, a.y += v.y, a.z += v.z, a.w += v.w;
    }
    *reinterpret_cast<uint2*>(out + ((size_t)t * nq + head) * hd + d) = make_uint2(pack2_bf16(a.x, a.y), pack2_bf16(a.z, a.w));
  }
}

// ------------------------------------------------------------------------------- prompt portions
// A tile = (first token, number of tokens <= 32) of one request.  A block of four waves works on one tile and one kv
// head; its units (query head of the kv head's group, half of the tile's tokens) go to the waves, NG to each, so that
// every 32-key tile of keys and values is fetched once per block and shared through LDS:
//   keys   LDS row = one key, hd values + 32 bytes of padding
//   values LDS row = one dim, its 32 keys in the order [g][half][4] (the 8 keys lane group g feeds to one product are 16
//          adjacent bytes) + 32 bytes of padding
// Two LDS tiles take turns, and the loads of the next two tiles are in flight during the products of the current one (the
// barrier between tiles waits for shared memory alone).
// grid (n_tiles * nkv, unit chunks); kv heads vary fastest, so that a kv head's keys stay in one die's cache where the
// number of kv heads is a multiple of the dies'.
__device__ __forceinline__ void lds_barrier() {
#ifdef __HIP_DEVICE_COMPILE__
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
#endif
}

#define PF_WAVES 4
#define PF_THREADS (64 * PF_WAVES)

template <int NQK, int NG, bool CAP>
__global__ void __launch_bounds__(PF_THREADS)
pooled_prefill_kernel(const bf16_t* __restrict__ q, int q_stride, bf16_t* __restrict__ out, const bf16_t* __restrict__ k_pool,
                      const bf16_t* __restrict__ v_pool, const int* __restrict__ block_table, int bt_stride,
                      const bf16_t* __restrict__ pk_pool, const bf16_t* __restrict__ pv_pool,
                      const int* __restrict__ pooled_table, int pooled_stride, const int* __restrict__ tile_list, int n_tiles,
                      const int* __restrict__ positions, const int* __restrict__ token_entry, int page_size, int nq, int nkv,
                      float scale, float cap, const float* __restrict__ head_bias, int window, int pool) {
  constexpr int HD = 32 * NQK;
  constexpr int KROW = 2 * HD + 32, VROW = 64 + 32, KBYTES = 32 * KROW, VBYTES = HD * VROW;
  constexpr int PIECES = (4 * HD + PF_THREADS - 1) / PF_THREADS;     // 16-byte pieces a thread brings, of keys and of values
  __shared__ __attribute__((aligned(16))) char lds[2 * (KBYTES + VBYTES)];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
  const int kvh = blockIdx.x % nkv, item = n_tiles - 1 - blockIdx.x / nkv;       // the tiles with the most keys first
  const int t0 = tile_list[2 * item], count = tile_list[2 * item + 1];
  const int G = nq / nkv, b = token_entry[t0], p_first = positions[t0], p_last = p_first + count - 1;
  const int* const bt = block_table + (size_t)b * bt_stride;
  const int* const pbt = pool > 0 ? pooled_table + (size_t)b * pooled_stride : nullptr;
  // this wave's units
  Pack8 qreg[NG][NQK];
  WeightConsts kc[NG];
  int lo[NG], hi[NG], nb[NG], head[NG], tok[NG];
  bool any = false;
#pragma unroll
  for (int u = 0; u < NG; ++u) {
    const int unit = ((int)blockIdx.y * PF_WAVES + wave) * NG + u;
    const int h = unit >> 1, ti = 16 * (unit & 1) + c;
    const bool ok = h < G && ti < count;
    head[u] = kvh * G + (h < G ? h : 0);
    tok[u] = ok ? t0 + ti : -1;
    hi[u] = ok ? p_first + ti : -1;                                              // a padding column sees no key
    lo[u] = (window > 0 && hi[u] - window + 1 > 0) ? hi[u] - window + 1 : 0;
    nb[u] = ok && pool > 0 ? lo[u] / pool : 0;
    any = any || (h < G && 16 * (unit & 1) < count);
    kc[u] = weight_consts(scale, cap, head_bias ? head_bias[head[u]] : 0.f);
#pragma unroll
    for (int ch = 0; ch < NQK; ++ch)
      qreg[u][ch].u4 = ld16(q + (size_t)(ok ? tok[u] : t0) * q_stride + (size_t)head[u] * HD + 32 * ch + 8 * g);
  }
  const int lo_first = (window > 0 && p_first - window + 1 > 0) ? p_first - window + 1 : 0;
  const int lo_last = (window > 0 && p_last - window + 1 > 0) ? p_last - window + 1 : 0;
  const int nb_min = pool > 0 ? lo_first / pool : 0, nb_max = pool > 0 ? lo_last / pool : 0;
  const int pt = (nb_max + 31) / 32, first = lo_first & ~31, tiles = pt + (p_last - first) / 32 + 1;
  f32x4_t acc[NG][2 * NQK];
#pragma unroll
  for (int u = 0; u < NG; ++u)
#pragma unroll
    for (int n = 0; n < 2 * NQK; ++n) acc[u][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  const KeyRanges ranges = {k_pool, v_pool, pk_pool, pv_pool, bt, pbt, page_size, nkv, kvh};
  struct Stage {                                          // a tile on its way from the cache to LDS
    uint4 k[PIECES], v[PIECES];
  };
  PieceWindow win = load_pieces(0, nb_max, pt, first, p_last, ranges);
  auto fetch = [&](int i, Stage& st) __attribute__((always_inline)) {
    if (2 * i + 1 >= win.base + 64) win = load_pieces(2 * i, nb_max, pt, first, p_last, ranges);
    const bool pooled = i < pt;
    const bf16_t* const kb = pooled ? pk_pool : k_pool;
    const bf16_t* const vb = pooled ? pv_pool : v_pool;
#pragma unroll
    for (int j = 0; j < PIECES; ++j) {
      const int piece = tid + j * PF_THREADS;
      const int sb = piece / (2 * HD), rem = piece % (2 * HD);            // the half is the same for a whole wave
      st.k[j] = st.v[j] = make_uint4(0, 0, 0, 0);
      if (piece >= 4 * HD) continue;
      const int at = __builtin_amdgcn_readfirstlane(2 * i + sb - win.base);
      const int page = __builtin_amdgcn_readlane(win.page, at), off = __builtin_amdgcn_readlane(win.off, at);
      if (page < 0) continue;
      st.k[j] = ld16(kb + (((size_t)page * nkv + kvh) * page_size + off + rem / (HD / 8)) * HD + 8 * (rem % (HD / 8)));
      st.v[j] = ld16(vb + (((size_t)page * nkv + kvh) * HD + rem / 2) * page_size + off + 8 * (rem % 2));
    }
  };
  auto put = [&](int i, Stage& st, char* buf) __attribute__((always_inline)) {
    const bool pooled = i < pt;
    const int key0 = pooled ? 32 * i : first + 32 * (i - pt), limit = pooled ? nb_max - 1 : p_last;
#pragma unroll
    for (int j = 0; j < PIECES; ++j) {
      const int piece = tid + j * PF_THREADS;
      if (piece >= 4 * HD) continue;
      const int sb = piece / (2 * HD), rem = piece % (2 * HD);
      if (key0 + 31 > limit) {
        // values of rows behind the data are not to be multiplied, even by zero
        const int over = key0 + 16 * sb + 8 * (rem % 2) + 7 - limit;                // how many of the eight lie behind
        Pack8 v;
        v.u4 = st.v[j];
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (e >= 8 - over) v.h[e] = 0;
        st.v[j] = v.u4;
      }
      *reinterpret_cast<uint4*>(buf + (16 * sb + rem / (HD / 8)) * KROW + 16 * (rem % (HD / 8))) = st.k[j];
      char* v = buf + KBYTES + (rem / 2) * VROW + 8 * sb + 32 * (rem % 2);
      *reinterpret_cast<uint2*>(v) = make_uint2(st.v[j].x, st.v[j].y);
      *reinterpret_cast<uint2*>(v + 16) = make_uint2(st.v[j].z, st.v[j].w);
    }
  };
  auto work = [&](int i, const char* buf) __attribute__((always_inline)) {
    if (!any) return;
    const bool pooled = i < pt;
    const int key0 = pooled ? 32 * i : first + 32 * (i - pt);
    const bool whole = pooled ? key0 + 32 <= nb_min : (key0 >= lo_last && key0 + 31 <= p_first);   // every column sees every key
    Pack8 p[NG];
    {
      f32x4_t s[NG][2];
#pragma unroll
      for (int u = 0; u < NG; ++u) s[u][0] = s[u][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ch = 0; ch < NQK; ++ch)
#pragma unroll
        for (int sb = 0; sb < 2; ++sb) {
          Pack8 k;
          k.u4 = *reinterpret_cast<const uint4*>(buf + (16 * sb + c) * KROW + 64 * ch + 16 * g);
#pragma unroll
          for (int u = 0; u < NG; ++u) s[u][sb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k.v, qreg[u][ch].v, s[u][sb], 0, 0, 0);
        }
#pragma unroll
      for (int u = 0; u < NG; ++u)
#pragma unroll
        for (int sb = 0; sb < 2; ++sb) {
          float e[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) e[r] = key_weight<CAP>(s[u][sb][r], kc[u]);
          if (!whole) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int kk = key0 + 16 * sb + 4 * g + r;
              const bool ok = pooled ? kk < nb[u] : (kk >= lo[u] && kk <= hi[u]);
              if (!ok) e[r] = 0.f;
            }
          }
          p[u].w[2 * sb] = pack2_bf16(e[0], e[1]);
          p[u].w[2 * sb + 1] = pack2_bf16(e[2], e[3]);
        }
    }
#pragma unroll
    for (int n = 0; n < 2 * NQK; ++n) {
      Pack8 v;
      v.u4 = *reinterpret_cast<const uint4*>(buf + KBYTES + (16 * n + c) * VROW + 16 * g);
#pragma unroll
      for (int u = 0; u < NG; ++u) acc[u][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, p[u].v, acc[u][n], 0, 0, 0);
    }
  };
  char* const buf0 = lds;
  char* const buf1 = lds + KBYTES + VBYTES;
  Stage s0, s1;
  fetch(0, s0);
  if (tiles > 1) fetch(1, s1);
  put(0, s0, buf0);
  lds_barrier();
  for (int i = 0; i < tiles; i += 2) {
    if (i + 2 < tiles) fetch(i + 2, s0);
    work(i, buf0);
    if (i + 1 >= tiles) break;
    put(i + 1, s1, buf1);
    lds_barrier();
    if (i + 3 < tiles) fetch(i + 3, s1);
    work(i + 1, buf1);
    if (i + 2 >= tiles) break;
    put(i + 2, s0, buf0);
    lds_barrier();
  }
#pragma unroll
  for (int u = 0; u < NG; ++u) {
    if (tok[u] < 0) continue;
    bf16_t* op = out + ((size_t)tok[u] * nq + head[u]) * HD;
#pragma unroll
    for (int n = 0; n < 2 * NQK; ++n)
      *reinterpret_cast<uint2*>(op + 16 * n + 4 * g) = make_uint2(pack2_bf16(acc[u][n][0], acc[u][n][1]), pack2_bf16(acc[u][n][2], acc[u][n][3]));
  }
}

extern "C" int ullm_pooled_mfma_supports(int hd, int page_size, int nq, int nkv) {
  return (hd == 32 || hd == 64 || hd == 96 || hd == 128 || hd == 256) && page_size >= 16 && page_size % 16 == 0 && nkv >= 1 && nq % nkv == 0;
}

static bool bad_shape(int hd, int page_size, int nq, int nkv, int window, int pool, const void* pk, const void* pv, const int* table) {
  return !ullm_pooled_mfma_supports(hd, page_size, nq, nkv) || window < 0 || pool < 0 || (pool > 0 && (window < 1 || !pk || !pv || !table));
}

#define BY_SIZE(M, CAPPED) do { if (hd == 32) M(1, CAPPED); else if (hd == 64) M(2, CAPPED); else if (hd == 96) M(3, CAPPED); \
    else if (hd == 128) M(4, CAPPED); else M(8, CAPPED); } while (0)

extern "C" int ullm_pooled_decode(const void* q, int q_stride, void* out, const void* k_pool, const void* v_pool,
                                  const int* block_table, int bt_stride, const void* pk_pool, const void* pv_pool,
                                  const int* pooled_table, int pooled_stride, const int* token_list, int n_items,
                                  const int* positions, const int* token_entry, int page_size, int nq, int nkv, int hd,
                                  float scale, float cap, const float* head_bias, int window, int pool, int num_splits, int waves,
                                  float* part, hipStream_t stream) {
  if (n_items <= 0) return 0;
  const int groups = (nq / (nkv > 0 ? nkv : 1) + 15) / 16;
  if (bad_shape(hd, page_size, nq, nkv, window, pool, pk_pool, pv_pool, pooled_table) || num_splits < 1 || n_items > 65535 ||
      nkv * groups > 65535 || (num_splits > 1 && !part) || (waves != 1 && waves != 4))
    return ULLM_ERR_SHAPE;
#define GO_W(NQK, W, CAPPED) hipLaunchKernelGGL((pooled_decode_kernel<NQK, W, CAPPED>), dim3(num_splits, nkv * groups, n_items),      \
    dim3(64 * W), 0, stream, (const bf16_t*)q, q_stride, (bf16_t*)out, (const bf16_t*)k_pool, (const bf16_t*)v_pool, block_table,   \
    bt_stride, (const bf16_t*)pk_pool, (const bf16_t*)pv_pool, pooled_table, pooled_stride, token_list, positions, token_entry,     \
    page_size, nq, nkv, scale, cap, head_bias, window, pool, num_splits, part)
#define GO(NQK, CAPPED) do { if (waves == 4) GO_W(NQK, 4, CAPPED); else GO_W(NQK, 1, CAPPED); } while (0)
  if (cap > 0.f) BY_SIZE(GO, true);
  else BY_SIZE(GO, false);
#undef GO
#undef GO_W
  if (num_splits > 1)
    hipLaunchKernelGGL(pooled_reduce_kernel, dim3(n_items, nq), dim3(64), 0, stream, part, (bf16_t*)out, token_list, nq, hd, num_splits);
  ULLM_LAUNCH_CHECK();
}

extern "C" int ullm_pooled_prefill(const void* q, int q_stride, void* out, const void* k_pool, const void* v_pool,
                                   const int* block_table, int bt_stride, const void* pk_pool, const void* pv_pool,
                                   const int* pooled_table, int pooled_stride, const int* tiles, int n_tiles,
                                   const int* positions, const int* token_entry, int page_size, int nq, int nkv, int hd,
                                   float scale, float cap, const float* head_bias, int window, int pool, hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (bad_shape(hd, page_size, nq, nkv, window, pool, pk_pool, pv_pool, pooled_table)) return ULLM_ERR_SHAPE;
  const int G = nq / nkv, units = 2 * G, ng = G >= 3 ? 2 : 1, chunks = (units + PF_WAVES * ng - 1) / (PF_WAVES * ng);
#define GO_G(NQK, NG, CAPPED) hipLaunchKernelGGL((pooled_prefill_kernel<NQK, NG, CAPPED>), dim3(n_tiles * nkv, chunks), dim3(PF_THREADS), \
    0, stream, (const bf16_t*)q, q_stride, (bf16_t*)out, (const bf16_t*)k_pool, (const bf16_t*)v_pool, block_table, bt_stride,      \
    (const bf16_t*)pk_pool, (const bf16_t*)pv_pool, pooled_table, pooled_stride, tiles, n_tiles, positions, token_entry, page_size, \
    nq, nkv, scale, cap, head_bias, window, pool)
#define GO(NQK, CAPPED) do { if (ng == 2) GO_G(NQK, 2, CAPPED); else GO_G(NQK, 1, CAPPED); } while (0)
  if (cap > 0.f) BY_SIZE(GO, true);
  else BY_SIZE(GO, false);
#undef GO
#undef GO_G
  ULLM_LAUNCH_CHECK();
}
