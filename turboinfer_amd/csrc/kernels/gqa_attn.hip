// gqa_attn.hip -- grouped-query attention of the layer-stack models (ti_stack.h): keys and values cached
// as MFMA fragments, so that every operand load of a wave is one contiguous KiB.
//
//   * gqa_prep_kernel: RMS norms of the whole query and key projections, query scale by position, cache
//     append -- one launch per layer.
//   * gqa_decode_kernel: the query heads that share a key/value head are the MFMA columns; a workgroup
//     takes 64-position blocks, its waves split the positions for the scores and the value dimensions for
//     the sums; keys are split over workgroups, merged by gqa_merge_kernel.
//   * gqa_prefill_kernel: prompt chunks; a workgroup owns MQ tiles of 16 rows of one key/value head's query
//     heads (heads of the same rows first), its waves split the key blocks.
// Scores, softmax and sums are fp32; the denominator holds exp(sink) of the head once.
#include <algorithm>

#include "elem.hpp"

namespace ti {

// Elements of a 64-position block; the key part comes first.
template <class T>
__host__ __device__ __forceinline__ int gqa_dim_p(int dim) {
  return (dim + El<T>::KT - 1) / El<T>::KT * El<T>::KT;
}
__host__ __device__ __forceinline__ int gqa_vdim_p(int vdim) { return (vdim + 15) / 16 * 16; }

template <class T>
__global__ __launch_bounds__(512) void gqa_prep_kernel(const ti_gqa_prep_args a) {
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC;
  extern __shared__ float r[];   // the queries' and keys' row
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x, pos = a.pos[m], nq = a.heads * a.dim, dim_p = gqa_dim_p<T>(a.dim);
  const int nkey = a.k_off >= 0 ? a.kv_heads * a.dim : 0, vdim_p = gqa_vdim_p(a.vdim);
  const float* src = a.a32 + (size_t)m * a.lda;
  float q2 = 0.0f, k2 = 0.0f;
  for (int i = tid; i < nq; i += 512) {
    const float v = src[i];
    r[i] = v;
    q2 = fmaf(v, v, q2);
  }
  for (int i = tid; i < nkey; i += 512) {
    const float v = src[a.k_off + i];
    r[nq + i] = v;
    k2 = fmaf(v, v, k2);
  }
  float qi = 1.0f / sqrtf(block_sum(q2, red) / (float)nq + a.eps);   // (the sum's barriers publish r)
  if (a.q_scale) qi *= a.q_scale[pos];
  T* q = (T*)a.q + (size_t)m * a.heads * dim_p;
  for (int i = tid; i < a.heads * dim_p; i += 512) {
    const int h = i / dim_p, d = i - h * dim_p, c = h * a.dim + d;
    q[i] = d < a.dim ? (T)(r[c] * qi * a.q_w[c]) : (T)0.0f;
  }
  if (!nkey) return;
  const float ki = 1.0f / sqrtf(block_sum(k2, red) / (float)nkey + a.eps);
  const int be = 64 * (dim_p + vdim_p), p = pos & 63, nkt = dim_p / KT;
  T* blk = (T*)a.cache + (size_t)(a.slot ? a.slot[m] : m) * a.slot_stride + (size_t)(pos >> 6) * be;
  const size_t hs = (size_t)(a.seq_p >> 6) * be;
  for (int c = tid; c < nkey; c += 512) {
    const int h = c / a.dim, d = c - h * a.dim;
    blk[h * hs + ((size_t)((p >> 4) * nkt + d / KT) * 64 + (d % KT) / VEC * 16 + (p & 15)) * VEC + d % VEC] =
        (T)(r[nq + c] * ki * a.k_w[c]);
  }
  for (int c = tid; c < a.kv_heads * a.vdim; c += 512) {
    const int h = c / a.vdim, d = c - h * a.vdim;
    blk[h * hs + 64 * dim_p + ((size_t)((d >> 4) * (64 / KT) + p / KT) * 64 + ((p & 15) >> 2) * 16 + (d & 15)) * VEC +
        (p % KT >> 4) * 4 + (p & 3)] = (T)src[a.v_off + c];
  }
}

// The same with head and value sizes that are multiples of 4 and at most NC * 2048 projected values: a thread
// holds its quads in registers, every load in flight before the sums.
template <class T, int NC>
__global__ __launch_bounds__(512) void gqa_prep_vec_kernel(const ti_gqa_prep_args a) {
  typedef typename El<T>::Q Q;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC;
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x, nq4 = a.heads * a.dim >> 2, dim_p = gqa_dim_p<T>(a.dim), vdim_p = gqa_vdim_p(a.vdim);
  const bool kv = a.k_off >= 0;
  const int nk4 = kv ? a.kv_heads * a.dim >> 2 : 0, n4 = nq4 + nk4 + (kv ? a.kv_heads * a.vdim >> 2 : 0);
  const int pos = a.pos[m], slot = a.slot ? a.slot[m] : m;
  const float* src = a.a32 + (size_t)m * a.lda;
  f32x4 x[NC], w[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = tid + 512 * c, k = i - nq4, v = k - nk4;
    const float* s = i < nq4 ? src + 4 * i : v < 0 ? src + a.k_off + 4 * k : src + a.v_off + 4 * v;
    const float* ws = i < nq4 ? a.q_w + 4 * i : a.k_w + 4 * k;
    x[c] = w[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (i < n4) x[c] = *(const f32x4*)s;
    if (i < nq4 + nk4) w[c] = *(const f32x4*)ws;
  }
  const float temp = a.q_scale ? a.q_scale[pos] : 1.0f;
  float q2 = 0.0f, k2 = 0.0f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = tid + 512 * c;
    const float s = (x[c][0] * x[c][0] + x[c][1] * x[c][1]) + (x[c][2] * x[c][2] + x[c][3] * x[c][3]);
    if (i < nq4) q2 += s;
    else if (i < nq4 + nk4) k2 += s;
  }
  const float qi = temp / sqrtf(block_sum(q2, red) / (float)(4 * nq4) + a.eps);
  const float ki = kv ? 1.0f / sqrtf(block_sum(k2, red) / (float)(4 * nk4) + a.eps) : 0.0f;
  const int be = 64 * (dim_p + vdim_p), p = pos & 63, nkt = dim_p / KT;
  T* blk = (T*)a.cache + (size_t)slot * a.slot_stride + (size_t)(pos >> 6) * be;
  const size_t hs = (size_t)(a.seq_p >> 6) * be;
  T* q = (T*)a.q + (size_t)m * a.heads * dim_p;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = tid + 512 * c, k = i - nq4, v = k - nk4;
    if (i < nq4) {
      const int h = 4 * i / a.dim, d = 4 * i - h * a.dim;
      *(Q*)(q + h * dim_p + d) = quad<T>(x[c] * qi * w[c]);
    } else if (v < 0) {
      const int h = 4 * k / a.dim, d = 4 * k - h * a.dim;
      *(Q*)(blk + h * hs + ((size_t)((p >> 4) * nkt + d / KT) * 64 + (d % KT) / VEC * 16 + (p & 15)) * VEC + d % VEC) =
          quad<T>(x[c] * ki * w[c]);
    } else if (i < n4) {
      const int h = 4 * v / a.vdim, d = 4 * v - h * a.vdim;
      T* o = blk + h * hs + 64 * dim_p + ((size_t)((d >> 4) * (64 / KT) + p / KT) * 64 + ((p & 15) >> 2) * 16 + (d & 15)) * VEC +
             (p % KT >> 4) * 4 + (p & 3);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e * VEC] = (T)x[c][e];
    }
  }
  const int pad = dim_p - a.dim;   // (the queries' k padding)
  for (int i = tid; i < a.heads * pad; i += 512) q[i / pad * dim_p + a.dim + i % pad] = (T)0.0f;
}

// The weights' operand fragment of one KT span: row[] holds 64 positions' weights of this lane's column.
__device__ __forceinline__ bf16x8 weight_frag(const bf16* row, int g) {
  const bf16x4 lo = *(const bf16x4*)(row + 4 * g), hi = *(const bf16x4*)(row + 16 + 4 * g);
  return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
}
__device__ __forceinline__ f32x4 weight_frag(const float* row, int g) { return *(const f32x4*)(row + 4 * g); }

// Grid (splits, kv heads * tiles of 16 query heads, rows).
template <class T, int NVW>
__global__ __launch_bounds__(256, NVW > 2 || sizeof(T) > 2 ? 2 : 4) void gqa_decode_kernel(const ti_gqa_attn_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, VB = 64 / KT, PLD = 64 + 16 / (int)sizeof(T), NKU = 8;
  extern __shared__ char lds[];
  const int split = blockIdx.x, m = blockIdx.z, rep = a.heads / a.kv_heads, tiles = (rep + 15) >> 4;
  const int kvh = blockIdx.y / tiles, h0 = (blockIdx.y - kvh * tiles) * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int dim_p = gqa_dim_p<T>(a.dim), vdim_p = gqa_vdim_p(a.vdim), nkt = dim_p / KT, nv = vdim_p >> 4;
  V* qf = (V*)lds;                          // [nkt][64]
  T* pb = (T*)(lds + (size_t)nkt * 1024);   // [16][PLD]
  float* sm = (float*)(pb + 16 * PLD);      // [4][16] wave maxima, then wave sums
  const int pos = a.pos[m], head = kvh * rep + h0 + col;
  const bool live = h0 + col < rep;
  const size_t be = (size_t)64 * (dim_p + vdim_p);
  const T* cache = (const T*)a.cache + (size_t)(a.slot ? a.slot[m] : m) * a.slot_stride + (size_t)kvh * (a.seq_p >> 6) * be;
  const int nb = (pos >> 6) + 1, bps = (nb + a.splits - 1) / a.splits, b0 = split * bps, b1 = min(nb, b0 + bps);
  V k[NKU], v[NVW][VB];
  auto load_k = [&](int b, int kt0) {
    const V* kp = (const V*)(cache + b * be) + (size_t)wave * nkt * 64 + lane;
#pragma unroll
    for (int u = 0; u < NKU; ++u) k[u] = kp[min(kt0 + u, nkt - 1) * 64];
  };
  auto load_v = [&](int b) {   // (value tiles past the last: clamped, not stored)
    const V* vp = (const V*)(cache + b * be + 64 * dim_p) + lane;
#pragma unroll
    for (int i = 0; i < NVW; ++i)
#pragma unroll
      for (int u = 0; u < VB; ++u) v[i][u] = vp[(size_t)(min(wave + 4 * i, nv - 1) * VB + u) * 64];
  };
  if (b0 < b1) {
    load_k(b0, 0);
    load_v(b0);
  }
  for (int kt = wave; kt < nkt; kt += 4) {
    V x = {};
    if (live) x = *(const V*)((const T*)a.q + ((size_t)m * a.heads + head) * dim_p + kt * KT + g * VEC);
    qf[kt * 64 + lane] = x;
  }
  f32x4 o[NVW];
#pragma unroll
  for (int i = 0; i < NVW; ++i) o[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float mr = -INFINITY, lr = 0.0f;
  lds_sync();
  for (int b = b0; b < b1; ++b) {
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    for (int kt0 = 0; kt0 < nkt; kt0 += NKU) {
      if (kt0) load_k(b, kt0);
#pragma unroll
      for (int u = 0; u < NKU; ++u)
        if (kt0 + u < nkt) s = mma(k[u], qf[(kt0 + u) * 64 + lane], s);
    }
    if (b + 1 < b1) load_k(b + 1, 0);   // the next block's keys fly through the softmax and the sums
    const int k0 = b * 64 + wave * 16 + 4 * g;
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = k0 + r <= pos ? s[r] * a.scale : -INFINITY;
      mx = fmaxf(mx, s[r]);
    }
    mx = xor32_max(xor16_max(mx));
    if (lane < 16) sm[wave * 16 + col] = mx;
    lds_sync();
    const float mn = fmaxf(fmaxf(mr, fmaxf(sm[col], sm[16 + col])), fmaxf(sm[32 + col], sm[48 + col]));
    const float alpha = expf(mr - mn);   // (every block holds a visible key: mn is finite)
    mr = mn;
    lr *= alpha;
    f32x4 p;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      p[r] = expf(s[r] - mn);
      lr += p[r];
    }
    *(typename El<T>::Q*)(pb + col * PLD + wave * 16 + 4 * g) = quad<T>(p);
    lds_sync();
    V pf[VB];
#pragma unroll
    for (int u = 0; u < VB; ++u) pf[u] = weight_frag(pb + col * PLD + u * KT, g);
#pragma unroll
    for (int i = 0; i < NVW; ++i) {
      o[i] *= alpha;
#pragma unroll
      for (int u = 0; u < VB; ++u) o[i] = mma(v[i][u], pf[u], o[i]);
    }
    if (b + 1 < b1) load_v(b + 1);
  }
  lr += lane_xor<16>(lr);
  lr += lane_xor<32>(lr);
  __syncthreads();
  if (lane < 16) sm[wave * 16 + col] = lr;
  __syncthreads();
  float l = sm[col] + sm[16 + col] + sm[32 + col] + sm[48 + col];
  if (!live) return;
  if (a.splits > 1) {
    const size_t row = ((size_t)m * a.splits + split) * a.heads + head;
    if (wave == 0 && lane < 16) *(float2*)(a.part_ml + row * 2) = make_float2(mr, l);
    if (b0 >= b1) return;
    const float inv = 1.0f / l;
#pragma unroll
    for (int i = 0; i < NVW; ++i)
      if (wave + 4 * i < nv) *(f32x4*)(a.part_o + row * vdim_p + (wave + 4 * i) * 16 + 4 * g) = o[i] * inv;
    return;
  }
  if (a.sink) l += expf(a.sink[head] - mr);   // (a huge sink gives inf: weights 0)
  const float inv = 1.0f / l;
#pragma unroll
  for (int i = 0; i < NVW; ++i) {
    const int d0 = (wave + 4 * i) * 16 + 4 * g;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (d0 + r >= a.vdim) continue;
      const int c = head * a.vdim + d0 + r;
      const float gt = a.gate ? fast_sigmoid(a.gate[(size_t)m * a.ldg + c]) : 1.0f;
      ((T*)a.out)[(size_t)m * a.ldo + c] = (T)(o[i][r] * inv * gt);
    }
  }
}

constexpr int kGqaSplits = 64;

// Grid (heads, rows), one wave per 64 value dimensions.
template <class T>
__global__ __launch_bounds__(256) void gqa_merge_kernel(const ti_gqa_attn_args a) {
  __shared__ float wt[kGqaSplits];
  const int h = blockIdx.x, m = blockIdx.y, tid = threadIdx.x, vdim_p = gqa_vdim_p(a.vdim);
  const size_t row0 = (size_t)m * a.splits * a.heads + h;
  if (tid < 64) {
    float mx = -INFINITY, l = 0.0f;
    if (tid < a.splits) {
      const float2 ml = *(const float2*)(a.part_ml + (row0 + (size_t)tid * a.heads) * 2);
      mx = ml.x;
      l = ml.y;
    }
    const float sink = a.sink ? a.sink[h] : -INFINITY, mm = fmaxf(wave_max(mx), sink);
    const float e = l > 0.0f ? l * expf(mx - mm) : 0.0f;
    wt[tid] = e / (group_sum<64>(e) + expf(sink - mm));
  }
  __syncthreads();
  for (int d = tid; d < a.vdim; d += blockDim.x) {
    float acc = 0.0f;
    for (int s0 = 0; s0 < a.splits; s0 += 8) {
      float x[8];
#pragma unroll
      for (int u = 0; u < 8; ++u)
        x[u] = a.part_o[(row0 + (size_t)min(s0 + u, a.splits - 1) * a.heads) * vdim_p + d];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float f = s0 + u < a.splits ? wt[s0 + u] : 0.0f;
        if (f != 0.0f) acc = fmaf(f, x[u], acc);   // (a split without keys holds no partial)
      }
    }
    const int c = h * a.vdim + d;
    const float gt = a.gate ? fast_sigmoid(a.gate[(size_t)m * a.ldg + c]) : 1.0f;
    ((T*)a.out)[(size_t)m * a.ldo + c] = (T)(acc * gt);
  }
}

// ------------------------------------------------------------------ prompt chunks
// Weights of 64 keys (4 key tiles, lane: query column, keys t * 16 + 4 g + r) x value fragments.
__device__ __forceinline__ void gqa_pv(f32x4& acc, const bf16x8* vf, const f32x4* p) {
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    bf16x8 pf;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      pf[r] = (bf16)p[2 * b][r];
      pf[4 + r] = (bf16)p[2 * b + 1][r];
    }
    acc = mma(vf[b], pf, acc);
  }
}
__device__ __forceinline__ void gqa_pv(f32x4& acc, const f32x4* vf, const f32x4* p) {
#pragma unroll
  for (int t = 0; t < 4; ++t) acc = mma(vf[t], p[t], acc);
}

// Tile j of a key/value head: query head j % rep of it, rows 16 (j / rep)...  A workgroup owns tiles
// [MQ i, +MQ); its waves take the 64-key blocks in turn and merge at the end.  Each XCD gets a contiguous
// run of the (kv head, tile group) list; a head's last groups (most keys) start first.
template <class T, int MQ, int NV>
__global__ __launch_bounds__(256, NV * MQ > 16 ? 1 : 2) void gqa_prefill_kernel(const ti_gqa_attn_args a, int groups) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, VB = 64 / KT;
  extern __shared__ char lds[];
  __shared__ float ml[2][4][MQ * 16];   // the waves' maxima, sums
  const int list = groups * a.kv_heads, per = (list + 7) >> 3;
  const int id = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per || id >= list) return;
  const int kvh = id / groups, j0 = (groups - 1 - id % groups) * MQ, rep = a.heads / a.kv_heads, tiles = (a.M + 15) / 16 * rep;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int dim_p = gqa_dim_p<T>(a.dim), vdim_p = gqa_vdim_p(a.vdim), nkt = dim_p / KT, nv = vdim_p >> 4;
  auto tile_row = [&](int q) { return min(j0 + q, tiles - 1) / rep * 16; };
  auto tile_head = [&](int q) { return kvh * rep + min(j0 + q, tiles - 1) % rep; };
  V* qf = (V*)lds;
  for (int i = wave; i < nkt * MQ; i += 4) {
    const int m = min(tile_row(i % MQ) + col, a.M - 1);
    qf[i * 64 + lane] = *(const V*)((const T*)a.q + ((size_t)m * a.heads + tile_head(i % MQ)) * dim_p + i / MQ * KT + g * VEC);
  }
  __syncthreads();
  const size_t be = (size_t)64 * (dim_p + vdim_p);
  const T* cache = (const T*)a.cache + (size_t)kvh * (a.seq_p >> 6) * be;
  f32x4 o[MQ][NV];
  float mr[MQ], lr[MQ];
#pragma unroll
  for (int q = 0; q < MQ; ++q) {
    // the sink: weight exp(sink - max), no value; counted by one wave
    mr[q] = a.sink ? a.sink[tile_head(q)] : -1e30f;
    lr[q] = a.sink && wave == 0 && g == 0 ? 1.0f : 0.0f;
#pragma unroll
    for (int v = 0; v < NV; ++v) o[q][v] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  const int last = a.pos0 + min(tile_row(MQ - 1) + 16, a.M) - 1;   // the tiles' last position
  for (int k0 = wave * 64; k0 <= last; k0 += 256) {
    const V* kf = (const V*)(cache + (k0 >> 6) * be) + lane;
    const V* vf = (const V*)(cache + (k0 >> 6) * be + 64 * dim_p) + lane;
    f32x4 s[MQ][4];
#pragma unroll
    for (int q = 0; q < MQ; ++q)
#pragma unroll
      for (int t = 0; t < 4; ++t) s[q][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int kt = 0; kt < nkt; ++kt) {
      V k[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) k[t] = kf[(size_t)(t * nkt + kt) * 64];
#pragma unroll
      for (int q = 0; q < MQ; ++q) {
        const V qv = qf[(kt * MQ + q) * 64 + lane];
#pragma unroll
        for (int t = 0; t < 4; ++t) s[q][t] = mma(k[t], qv, s[q][t]);
      }
    }
#pragma unroll
    for (int q = 0; q < MQ; ++q) {
      const int p = a.pos0 + tile_row(q) + col;
      float mx = mr[q];
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[q][t][r] = k0 + t * 16 + 4 * g + r <= p ? s[q][t][r] * a.scale : -INFINITY;
          mx = fmaxf(mx, s[q][t][r]);
        }
      mx = xor32_max(xor16_max(mx));
      const float alpha = expf(mr[q] - mx);
      mr[q] = mx;
      float l = 0.0f;
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[q][t][r] = expf(s[q][t][r] - mx);
          l += s[q][t][r];
        }
      lr[q] = lr[q] * alpha + l;
#pragma unroll
      for (int v = 0; v < NV; ++v) o[q][v] *= alpha;
    }
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      if (v < nv) {
        V vv[VB];
#pragma unroll
        for (int b = 0; b < VB; ++b) vv[b] = vf[(size_t)(v * VB + b) * 64];
#pragma unroll
        for (int q = 0; q < MQ; ++q) gqa_pv(o[q][v], vv, s[q]);
      }
    }
  }
#pragma unroll
  for (int q = 0; q < MQ; ++q) {
    float l = lr[q];
    l += lane_xor<16>(l);
    l += lane_xor<32>(l);
    if (lane < 16) {
      ml[0][wave][q * 16 + col] = mr[q];
      ml[1][wave][q * 16 + col] = l;
    }
  }
  __syncthreads();   // (and the last reads of qf)
  f32x4* ob = (f32x4*)lds;   // [4][NV][64]
#pragma unroll
  for (int q = 0; q < MQ; ++q) {
    const int m = tile_row(q) + col, h = tile_head(q);
    float mx = ml[0][0][q * 16 + col], l = 0.0f;
#pragma unroll
    for (int w = 1; w < 4; ++w) mx = fmaxf(mx, ml[0][w][q * 16 + col]);
#pragma unroll
    for (int w = 0; w < 4; ++w) l += ml[1][w][q * 16 + col] * expf(ml[0][w][q * 16 + col] - mx);
    const float f = expf(mr[q] - mx);
#pragma unroll
    for (int v = 0; v < NV; ++v) ob[(wave * NV + v) * 64 + lane] = o[q][v] * f;
    __syncthreads();
    if (m < a.M && j0 + q < tiles) {
      const float inv = 1.0f / l;
#pragma unroll
      for (int v0 = 0; v0 < NV; v0 += 4) {
        const int v = v0 + wave, d = v * 16 + 4 * g;
        if (d >= a.vdim) continue;
        f32x4 x = ob[v * 64 + lane];
#pragma unroll
        for (int w = 1; w < 4; ++w) x += ob[(w * NV + v) * 64 + lane];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (d + r >= a.vdim) continue;
          const int c = h * a.vdim + d + r;
          const float gt = a.gate ? fast_sigmoid(a.gate[(size_t)m * a.ldg + c]) : 1.0f;
          ((T*)a.out)[(size_t)m * a.ldo + c] = (T)(x[r] * inv * gt);
        }
      }
    }
    if (q + 1 < MQ) __syncthreads();
  }
}

template <class T>
int launch_gqa_decode(const ti_gqa_attn_args& a, hipStream_t s) {
  const int nkt = gqa_dim_p<T>(a.dim) / El<T>::KT, nvw = (gqa_vdim_p(a.vdim) / 16 + 3) / 4, rep = a.heads / a.kv_heads;
  const size_t lds = (size_t)nkt * 1024 + (size_t)16 * (64 + 16 / sizeof(T)) * sizeof(T) + 64 * 4;
  const dim3 grid(a.splits, a.kv_heads * ((rep + 15) / 16), a.M), blk(256);
  if (nvw == 1) hipLaunchKernelGGL((gqa_decode_kernel<T, 1>), grid, blk, lds, s, a);
  else if (nvw == 2) hipLaunchKernelGGL((gqa_decode_kernel<T, 2>), grid, blk, lds, s, a);
  else hipLaunchKernelGGL((gqa_decode_kernel<T, 4>), grid, blk, lds, s, a);
  TI_LAUNCH_CHECK("gqa_decode_kernel");
  if (a.splits > 1) {
    hipLaunchKernelGGL(gqa_merge_kernel<T>, dim3(a.heads, a.M), dim3(a.vdim <= 64 ? 64 : a.vdim <= 128 ? 128 : 256), 0, s, a);
    TI_LAUNCH_CHECK("gqa_merge_kernel");
  }
  return TI_OK;
}

template <class T>
int launch_gqa_prefill(const ti_gqa_attn_args& a, hipStream_t s) {
  const int nkt = gqa_dim_p<T>(a.dim) / El<T>::KT, nv = gqa_vdim_p(a.vdim) / 16, rep = a.heads / a.kv_heads;
  const long tiles = (long)((a.M + 15) / 16) * rep;
  // two tiles per workgroup where they still give every CU two workgroups
  const bool two = nkt <= 32 && nv <= 8 && (tiles + 1) / 2 * a.kv_heads >= 512;
  const int mq = two ? 2 : 1, groups = (int)((tiles + mq - 1) / mq), nvp = nv <= 4 ? 4 : nv <= 8 ? 8 : 16;
  const size_t lds = (size_t)std::max(nkt * mq, 4 * nvp) * 1024;
  const dim3 grid((unsigned)(((long)groups * a.kv_heads + 7) / 8 * 8)), blk(256);
#define TI_GP(MQ, NV) hipLaunchKernelGGL((gqa_prefill_kernel<T, MQ, NV>), grid, blk, lds, s, a, groups)
  if (two && nv <= 4) TI_GP(2, 4);
  else if (two) TI_GP(2, 8);
  else if (nv <= 4) TI_GP(1, 4);
  else if (nv <= 8) TI_GP(1, 8);
  else TI_GP(1, 16);
#undef TI_GP
  TI_LAUNCH_CHECK("gqa_prefill_kernel");
  return TI_OK;
}

int gqa_check(const ti_gqa_attn_args* a, const char* what) {
  if (!a || !a->q || !a->cache || !a->out || a->M < 1 || a->M > 65535 || a->heads < 1 || a->kv_heads < 1 || a->heads % a->kv_heads ||
      a->dim < 1 || a->vdim < 1 || a->seq_p < 64 || a->seq_p % 64 || (a->dtype != TI_DT_BF16 && a->dtype != TI_DT_F32) ||
      a->ldo < a->heads * a->vdim || (a->gate && a->ldg < a->heads * a->vdim))
    return ti_set_error(TI_ERR_ARG, "%s: bad arguments", what);
  if (a->vdim > 256 || a->dim > 1024)
    return ti_set_error(TI_ERR_UNSUPPORTED, "%s: head of %d, values of %d (at most 1024, 256)", what, a->dim, a->vdim);
  return TI_OK;
}

// Kernels whose dynamic LDS can pass 64 KiB.
template <class T>
int gqa_prepare() {
  const void* k[] = {(const void*)gqa_decode_kernel<T, 1>,     (const void*)gqa_decode_kernel<T, 2>,
                     (const void*)gqa_decode_kernel<T, 4>,     (const void*)gqa_prefill_kernel<T, 2, 4>,
                     (const void*)gqa_prefill_kernel<T, 2, 8>, (const void*)gqa_prefill_kernel<T, 1, 4>,
                     (const void*)gqa_prefill_kernel<T, 1, 8>, (const void*)gqa_prefill_kernel<T, 1, 16>,
                     (const void*)gqa_prep_kernel<T>};
  for (const void* f : k)
    TI_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 131072), "grouped-query attention LDS");
  return TI_OK;
}

int gqa_prepare_all() {
  const int rc = gqa_prepare<bf16>();
  return rc ? rc : gqa_prepare<float>();
}

}  // namespace ti

extern "C" int ti_gqa_block_elems(int dtype, int dim, int vdim) {
  if (dim < 1 || vdim < 1) return 0;
  return 64 * ((dtype == TI_DT_BF16 ? ti::gqa_dim_p<ti::bf16>(dim) : ti::gqa_dim_p<float>(dim)) + ti::gqa_vdim_p(vdim));
}

extern "C" int ti_gqa_prep(const ti_gqa_prep_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->a32 || !a->q_w || !a->pos || !a->q || a->M < 1 || a->heads < 1 || a->kv_heads < 1 || a->dim < 1 || a->vdim < 1 ||
      a->seq_p < 64 || a->seq_p % 64 || (a->dtype != TI_DT_BF16 && a->dtype != TI_DT_F32) || a->lda < a->heads * a->dim ||
      (a->k_off >= 0 && (!a->k_w || !a->cache || a->lda < a->k_off + a->kv_heads * a->dim || a->lda < a->v_off + a->kv_heads * a->vdim)))
    return ti_set_error(TI_ERR_ARG, "ti_gqa_prep: bad arguments");
  const int n = (a->heads + (a->k_off >= 0 ? a->kv_heads : 0)) * a->dim + (a->k_off >= 0 ? a->kv_heads * a->vdim : 0);
  if (((a->dim | a->vdim | a->lda) & 3) == 0 && (a->k_off < 0 || ((a->k_off | a->v_off) & 3) == 0) && n <= 4 * 2048) {
    hipStream_t s = (hipStream_t)stream;
    auto launch = [&]<int NC>() {
      if (a->dtype == TI_DT_BF16) hipLaunchKernelGGL((gqa_prep_vec_kernel<bf16, NC>), dim3(a->M), dim3(512), 0, s, *a);
      else hipLaunchKernelGGL((gqa_prep_vec_kernel<float, NC>), dim3(a->M), dim3(512), 0, s, *a);
    };
    if (n <= 2048) launch.template operator()<1>();
    else if (n <= 2 * 2048) launch.template operator()<2>();
    else launch.template operator()<4>();
    TI_LAUNCH_CHECK("gqa_prep_vec_kernel");
    return TI_OK;
  }
  const size_t lds = (size_t)(a->heads + a->kv_heads) * a->dim * 4;
  if (lds > 131072) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_gqa_prep: %d + %d heads of %d", a->heads, a->kv_heads, a->dim);
  if (a->dtype == TI_DT_BF16)
    hipLaunchKernelGGL(gqa_prep_kernel<bf16>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  else
    hipLaunchKernelGGL(gqa_prep_kernel<float>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  TI_LAUNCH_CHECK("gqa_prep_kernel");
  return TI_OK;
}

extern "C" int ti_gqa_splits(int M, int heads, int kv_heads, int max_seq) {
  // four workgroups per CU (splits cost a merge), none with less than one 64-position block
  const int rep = heads / std::max(1, kv_heads), wgs = M * kv_heads * ((rep + 15) / 16), cap = std::max(1, (max_seq + 63) / 64);
  return std::max(1, std::min({cap, ti::kGqaSplits, (1024 + wgs - 1) / std::max(1, wgs)}));
}

extern "C" int ti_gqa_decode(const ti_gqa_attn_args* a, ti_stream_t stream) {
  using namespace ti;
  const int rc = gqa_check(a, "ti_gqa_decode");
  if (rc) return rc;
  if (!a->pos || a->splits < 1 || a->splits > kGqaSplits || (a->splits > 1 && (!a->part_o || !a->part_ml)))
    return ti_set_error(TI_ERR_ARG, "ti_gqa_decode: %d splits", a->splits);
  return a->dtype == TI_DT_BF16 ? launch_gqa_decode<bf16>(*a, (hipStream_t)stream) : launch_gqa_decode<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_gqa_prefill(const ti_gqa_attn_args* a, ti_stream_t stream) {
  using namespace ti;
  const int rc = gqa_check(a, "ti_gqa_prefill");
  if (rc) return rc;
  if (a->pos0 < 0 || a->pos0 + a->M > a->seq_p) return ti_set_error(TI_ERR_ARG, "ti_gqa_prefill: %d rows at %d", a->M, a->pos0);
  return a->dtype == TI_DT_BF16 ? launch_gqa_prefill<bf16>(*a, (hipStream_t)stream) : launch_gqa_prefill<float>(*a, (hipStream_t)stream);
}
