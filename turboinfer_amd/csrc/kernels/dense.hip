// dense.hip -- matrix products of the layer-stack models (ti_stack.h ti_dense): fragment-ordered
// weights x row-major activations on MFMA, bf16 or fp32, with the consumer's first step fused into
// the epilogue (SiLU * up, rotary pairs, head gates, logits + argmax, key / value fragments).
//
// Two kernels share the epilogue:
//   * dense_skinny_kernel (M <= 64): HBM-bound weight streaming.  One workgroup per 16 output columns,
//     its waves split k; each weight fragment is one contiguous KiB read once and multiplied with up
//     to 4 row tiles; the waves' partial sums meet in LDS.
//   * dense_tile_kernel (more rows): 4 waves side by side over a BM x BN tile, activations staged through
//     double-buffered LDS in fragment order, each wave's weight fragments straight from L2 into
//     registers; both 2 or 4 k-stages (128 bytes each) ahead of their use.
// Both take independent batches (per-head products) or grouped tiles (experts: a tile is up to
// tile_rows entries of one expert's list, rows gathered and scattered through the list).
#include <algorithm>

#include "elem.hpp"

namespace ti {

__device__ __forceinline__ unsigned long long logit_key(float v, int n) {
  return ((unsigned long long)float_order_key(v) << 32) | (unsigned long long)(0xFFFFFFFFu - (uint32_t)n);
}

__device__ __forceinline__ float activate(int act, float z) {
  if (act == TI_ACT_GELU_ERF) return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f));
  // (1 + tanh x) / 2 is the logistic function of 2 x
  if (act == TI_ACT_GELU_TANH) return z * fast_sigmoid(1.59576912160573072f * fmaf(0.044715f * z * z, z, z));
  return z;
}

// Four consecutive output columns n0.. of row m (out row mo); rows >= rows are padding.
template <class T, int EPI>
__device__ __forceinline__ void dense_store(const ti_dense_args& a, int batch, int m, int mo, int rows, int n0, f32x4 v) {
  constexpr int VEC = El<T>::VEC, KT = El<T>::KT;
  const bool live = m < rows;
  switch (EPI) {
    case TI_DE_F32: {
      if (!live) return;
      float* o = (float*)a.out + (size_t)batch * a.o_batch + (size_t)mo * a.ldo + n0;
      if (a.add)
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] += a.add[min(n0 + i, a.N - 1)];
      if (n0 + 4 <= a.N && ((a.ldo | a.o_batch) & 3) == 0) {
        *(f32x4*)o = v;
        return;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < a.N) o[i] = v[i];
      return;
    }
    case TI_DE_T: {
      if (!live) return;
      T* o = (T*)a.out + (size_t)batch * a.o_batch + (size_t)mo * a.ldo + n0;
      if (n0 + 4 <= a.N && ((a.ldo | a.o_batch) & 3) == 0) {
        *(typename El<T>::Q*)o = quad<T>(v);
        return;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < a.N) o[i] = (T)v[i];
      return;
    }
    case TI_DE_SWIGLU: {
      if (!live) return;
      T* o = (T*)a.out + (size_t)mo * a.ldo + (n0 >> 1);
#pragma unroll
      for (int i = 0; i < 2; ++i)
        if (n0 + 2 * i < a.N) o[i] = (T)(v[2 * i] * sigmoidf(v[2 * i]) * v[2 * i + 1]);
      return;
    }
    case TI_DE_ROPE: {
      if (!live || n0 >= a.N) return;
      const int r = n0 % a.head_w - a.rot_off;
      if (r >= 0) {
        const int pairs = (a.head_w - a.rot_off) >> 1;
        const float* cs = a.rope_cs + ((size_t)a.pos[m] * pairs + (r >> 1)) * 2;
        const f32x4 t = *(const f32x4*)cs;
        v = (f32x4){v[0] * t[0] - v[1] * t[1], v[1] * t[0] + v[0] * t[1], v[2] * t[2] - v[3] * t[3],
                    v[3] * t[2] + v[2] * t[3]};
      }
      *(typename El<T>::Q*)((T*)a.out + (size_t)mo * a.ldo + n0) = quad<T>(v);
      return;
    }
    case TI_DE_GATE: {
      if (!live) return;
      const float g = a.gate[(size_t)m * a.gate_ld + batch];
      T* o = (T*)a.out + (size_t)mo * a.ldo + (size_t)batch * a.N + n0;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < a.N) o[i] = (T)(v[i] * g);
      return;
    }
    case TI_DE_KFRAG: {   // every row of the tile is written (padding rows repeat the last key)
      if (n0 >= a.N) return;
      const int h = n0 / a.head_w, d = n0 - h * a.head_w, dt = a.head_w / KT;
      T* o = (T*)a.out + ((((size_t)h * a.key_blocks + (m >> 4)) * dt + d / KT) * 64 + ((d % KT) / VEC) * 16 + (m & 15)) * VEC +
             d % VEC;
      *(typename El<T>::Q*)o = quad<T>(v);
      return;
    }
    case TI_DE_ACT: {
      if (!live) return;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (a.add) v[i] += a.add[min(n0 + i, a.N - 1)];
        if (n0 + i < a.act_cols) v[i] = activate(a.act, v[i]);
      }
      T* o = (T*)a.out + (size_t)mo * a.ldo + n0;
      if (n0 + 4 <= a.t_cols && (a.ldo & 3) == 0) {
        *(typename El<T>::Q*)o = quad<T>(v);
        return;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int n = n0 + i;
        if (n < a.t_cols) o[i] = (T)v[i];
        else if (n < a.N) a.out2[(size_t)mo * a.ld2 + n - a.t_cols] = v[i];
      }
      return;
    }
    case TI_DE_LRU: {
      if (!live || n0 >= a.N) return;
      const int per = a.N >> 1, channels = per * a.batch;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int j = (n0 >> 1) + i, c = batch * per + j;
        if (j >= per) return;
        const float* gb = a.add + (size_t)batch * a.N + n0 + 2 * i;
        const float u = (float)((const T*)a.a)[(size_t)m * a.lda + (size_t)batch * a.a_batch + j];
        *(float2*)((float*)a.out + ((size_t)m * channels + c) * 2) = lru_coef(v[2 * i] + gb[0], v[2 * i + 1] + gb[1], a.lru_rate[c], u);
      }
      return;
    }
    default: return;
  }
}

// TI_DE_VFRAG: four consecutive keys m0.. of column n.
template <class T>
__device__ __forceinline__ void dense_store_v(const ti_dense_args& a, int m0, int n, f32x4 v) {
  constexpr int VEC = El<T>::VEC, KT = El<T>::KT;
  if (n >= a.N) return;
  const int h = n / a.head_w, d = n - h * a.head_w;
  const int kb = m0 / KT, t = (m0 % KT) >> 4, g = (m0 & 15) >> 2, nkb = a.key_blocks * 16 / KT;
  T* o = (T*)a.out + ((((size_t)h * (a.head_w >> 4) + (d >> 4)) * nkb + kb) * 64 + g * 16 + (d & 15)) * VEC + t * 4;
  *(typename El<T>::Q*)o = quad<T>(v);
}

// Greedy argmax keys of a 16-column tile: lane l holds columns n0.. of row m = its (l & 15).
__device__ __forceinline__ void dense_argmax(const ti_dense_args& a, int m, int rows, int n0, f32x4 v, int lane, int slot) {
  unsigned long long key = 0ull;
  if (m < rows) {
    float* o = (float*)a.out + (size_t)m * a.ldo + n0;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n0 + i < a.N) {
        o[i] = v[i];
        const unsigned long long k = logit_key(v[i], n0 + i);
        key = k > key ? k : key;
      }
  }
#pragma unroll
  for (int o = 16; o < 64; o <<= 1) {
    const unsigned long long other = __shfl_xor(key, o, kWave);
    key = other > key ? other : key;
  }
  if (lane < 16 && key) atomicMax(a.argmax + (size_t)m * TI_ARGMAX_SLOTS + (slot & (TI_ARGMAX_SLOTS - 1)), key);
}

struct DenseSpan {   // what a workgroup works on
  int rows, first, batch;
  const void* w;
};

__device__ __forceinline__ bool dense_span(const ti_dense_args& a, int y, DenseSpan& s, size_t esize) {
  s.batch = 0;
  int e = 0;
  if (a.tile_rows == 1) {
    s.first = y;
    s.rows = 1;
    e = a.tiles[y];
    e = __builtin_amdgcn_readfirstlane(e);
  } else if (a.tile_rows) {
    if (y >= *a.n_tiles) return false;
    e = a.tiles[4 * y];
    s.first = a.tiles[4 * y + 1];
    s.rows = a.tiles[4 * y + 2];
  } else {
    s.first = 0;
    s.rows = a.M;
    s.batch = e = y;
  }
  s.w = (const char*)a.w + (size_t)e * a.w_batch * esize;
  return true;
}
__device__ __forceinline__ int row_in(const ti_dense_args& a, int p) {
  const int r = a.rows_in ? a.rows_in[p] : p;
  return a.row_div > 1 ? r / a.row_div : r;
}
__device__ __forceinline__ int row_out(const ti_dense_args& a, int p) { return a.rows_out ? a.rows_out[p] : p; }

template <class T, int MT, int W, int EPI>
__global__ __launch_bounds__(64 * W) void dense_skinny_kernel(const ti_dense_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, U = 8;
  __shared__ f32x4 red[W][MT][64];
  DenseSpan sp;
  if (!dense_span(a, blockIdx.y, sp, sizeof(T))) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nt = blockIdx.x, nk = a.K / KT, z0 = blockIdx.z * MT * 16;
  const V* wp = (const V*)sp.w + (size_t)nt * nk * 64 + lane;
  const V* ap[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int p = sp.first + min(z0 + mt * 16 + (lane & 15), sp.rows - 1);
    ap[mt] = (const V*)((const T*)a.a + (size_t)sp.batch * a.a_batch + (size_t)row_in(a, p) * a.lda) + (lane >> 4);
  }
  f32x4 acc[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) acc[mt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // n k-tiles of this wave: their weight fragments in flight together (kept to ~64 VGPRs: workgroups
  // per CU hide more latency than a deeper wave)
  auto batch = [&]<int N>(int kt) {
    V wf[N];
#pragma unroll
    for (int u = 0; u < N; ++u) wf[u] = wp[(size_t)(kt + u * W) * 64];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      V af[N];
#pragma unroll
      for (int u = 0; u < N; ++u) af[u] = ap[mt][(kt + u * W) * (KT / VEC)];
#pragma unroll
      for (int u = 0; u < N; ++u) acc[mt] = mma(wf[u], af[u], acc[mt]);
    }
  };
  int kt = wave;
  for (; kt + (U - 1) * W < nk; kt += U * W) batch.template operator()<U>(kt);
  if (kt + 3 * W < nk) {
    batch.template operator()<4>(kt);
    kt += 4 * W;
  }
  if (kt + W < nk) {
    batch.template operator()<2>(kt);
    kt += 2 * W;
  }
  if (kt < nk) batch.template operator()<1>(kt);
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) red[wave][mt][lane] = acc[mt];
  __syncthreads();
  for (int mt = wave; mt < MT; mt += W) {
    f32x4 v = red[0][mt][lane];
#pragma unroll
    for (int w = 1; w < W; ++w) v += red[w][mt][lane];
    const int m = z0 + mt * 16 + (lane & 15), n0 = nt * 16 + 4 * (lane >> 4);
    if constexpr (EPI == TI_DE_LOGITS)
      dense_argmax(a, m, sp.rows, n0, v, lane, nt);
    else
      dense_store<T, EPI>(a, sp.batch, m, m < sp.rows ? row_out(a, sp.first + m) : 0, sp.rows, n0, v);
  }
  if (EPI == TI_DE_LOGITS && a.step_ctr && nt == 0 && blockIdx.z == 0 && tid == 0) *a.step_ctr += a.advance;
}

template <class T, int BM, int BN, int D, int EPI>
__global__ __launch_bounds__(256, BM * BN > 16384 ? 1 : 2) void dense_tile_kernel(const ti_dense_args a, int m_tiles, int n_tiles) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, FM = BM / 16, FN = BN / 64, NA = BM / 32;
  constexpr bool VF = EPI == TI_DE_VFRAG;
  __shared__ V as[2][FM * 2][64];
  // Consecutive workgroups go to the 8 XCDs in turn; each XCD gets a contiguous run of the work list,
  // ordered so that neighbours share weight columns (its L2 holds them once): row tiles fastest, for
  // grouped products 4 tiles (mostly one expert's) fastest, then the columns.
  const int list = a.tile_rows ? (*a.n_tiles + 3) / 4 * 4 * n_tiles : m_tiles * n_tiles, per = (list + 7) >> 3;
  const int id = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per || id >= list) return;
  int mtile, ntile, y;
  if (a.tile_rows) {
    const int b = id / (4 * n_tiles), r = id - b * 4 * n_tiles;
    mtile = 0;
    ntile = r >> 2;
    y = b * 4 + (r & 3);
  } else {
    mtile = id % m_tiles;
    ntile = id / m_tiles;
    y = blockIdx.y;
  }
  const int m_base = mtile * BM;
  DenseSpan sp;
  if (!dense_span(a, y, sp, sizeof(T))) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int nk = a.K / KT, nst = nk >> 1, NT = (a.N + 15) >> 4;
  const V* ap[NA];
#pragma unroll
  for (int i = 0; i < NA; ++i) {
    const int f = i * 4 + wave;   // fragment (row tile f >> 1, k-tile f & 1) of the stage
    const int p = sp.first + min(m_base + (f >> 1) * 16 + (lane & 15), sp.rows - 1);
    ap[i] = (const V*)((const T*)a.a + (size_t)sp.batch * a.a_batch + (size_t)row_in(a, p) * a.lda) + (f & 1) * (KT / VEC) +
            (lane >> 4);
  }
  const V* wp[FN];
#pragma unroll
  for (int j = 0; j < FN; ++j)
    wp[j] = (const V*)sp.w + (size_t)min(ntile * (BN / 16) + wave * FN + j, NT - 1) * nk * 64 + lane;
  f32x4 acc[FM][FN];
#pragma unroll
  for (int i = 0; i < FM; ++i)
#pragma unroll
    for (int j = 0; j < FN; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // rings of D stages in registers: weights of stage s in set s % D, activations likewise until they
  // move to LDS one stage before their use
  V ar[D][NA], w[D][FN][2];
  auto load_a = [&](V (&d)[NA], int s) {
#pragma unroll
    for (int i = 0; i < NA; ++i) d[i] = ap[i][min(s, nst - 1) * 2 * (KT / VEC)];
  };
  auto load_w = [&](V (&d)[FN][2], int s) {
#pragma unroll
    for (int j = 0; j < FN; ++j) {
      d[j][0] = wp[j][(size_t)min(s, nst - 1) * 128];
      d[j][1] = wp[j][(size_t)min(s, nst - 1) * 128 + 64];
    }
  };
  auto store_a = [&](int buf, const V (&d)[NA]) {
#pragma unroll
    for (int i = 0; i < NA; ++i) as[buf][i * 4 + wave][lane] = d[i];
  };
  // s % 4 == B.  A stage's operand reads all go out first (left alone, the scheduler keeps two in
  // flight and waits for LDS between products), the hand-over of the next stage's activations next.
  auto stage = [&]<int B>(int s) {
    V af[2][FM];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < FM; ++i) af[kk][i] = as[B & 1][i * 2 + kk][lane];
    __builtin_amdgcn_sched_barrier(0);
    store_a((B + 1) & 1, ar[(B + 1) % D]);
    load_a(ar[(B + 1) % D], s + 1 + D);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < FM; ++i)
#pragma unroll
        for (int j = 0; j < FN; ++j)
          acc[i][j] = VF ? mma(af[kk][i], w[B % D][j][kk], acc[i][j]) : mma(w[B % D][j][kk], af[kk][i], acc[i][j]);
    load_w(w[B % D], s + D);
    lds_sync();
  };
  load_a(ar[0], 0);
#pragma unroll
  for (int d = 0; d < D; ++d) {
    load_w(w[d], d);
    if (d == 0) {
      store_a(0, ar[0]);
      load_a(ar[0], D);
    } else {
      load_a(ar[d], d);
    }
  }
  lds_sync();
  for (int s = 0; s < nst; s += 4) {
    stage.template operator()<0>(s);
    if (s + 1 < nst) stage.template operator()<1>(s + 1);
    if (s + 2 < nst) stage.template operator()<2>(s + 2);
    if (s + 3 < nst) stage.template operator()<3>(s + 3);
  }
#pragma unroll
  for (int i = 0; i < FM; ++i) {
    const int mt = m_base + i * 16;
    const int m = mt + (lane & 15);
    const int mo = m < sp.rows ? row_out(a, sp.first + m) : 0;
#pragma unroll
    for (int j = 0; j < FN; ++j) {
      const int nt = ntile * (BN / 16) + wave * FN + j;
      if (nt >= NT) continue;
      if constexpr (VF)
        dense_store_v<T>(a, mt + 4 * (lane >> 4), nt * 16 + (lane & 15), acc[i][j]);
      else if constexpr (EPI == TI_DE_LOGITS)
        dense_argmax(a, m, sp.rows, nt * 16 + 4 * (lane >> 4), acc[i][j], lane, nt);
      else
        dense_store<T, EPI>(a, sp.batch, m, mo, sp.rows, nt * 16 + 4 * (lane >> 4), acc[i][j]);
    }
  }
  if (EPI == TI_DE_LOGITS && a.step_ctr && id == 0 && tid == 0) *a.step_ctr += a.advance;
}

template <class T, int MT, int EPI>
int launch_skinny(const ti_dense_args& a, hipStream_t s) {
  const int NT = (a.N + 15) / 16, y = a.tile_rows ? a.max_tiles : a.batch, nk = a.K / El<T>::KT;
  const int z = a.tile_rows ? 1 : (a.M + 16 * MT - 1) / (16 * MT);
  if (nk >= 32)
    hipLaunchKernelGGL((dense_skinny_kernel<T, MT, 8, EPI>), dim3(NT, y, z), dim3(512), 0, s, a);
  else
    hipLaunchKernelGGL((dense_skinny_kernel<T, MT, 4, EPI>), dim3(NT, y, z), dim3(256), 0, s, a);
  TI_LAUNCH_CHECK("dense_skinny_kernel");
  return TI_OK;
}

template <class T, int BM, int BN, int D, int EPI>
int launch_tile(const ti_dense_args& a, hipStream_t s) {
  const int mt = (a.M + BM - 1) / BM, nt = (a.N + BN - 1) / BN;
  const int list = a.tile_rows ? (a.max_tiles + 3) / 4 * 4 * nt : mt * nt;
  hipLaunchKernelGGL((dense_tile_kernel<T, BM, BN, D, EPI>), dim3((list + 7) / 8 * 8, a.tile_rows ? 1 : a.batch), dim3(256), 0,
                     s, a, mt, nt);
  TI_LAUNCH_CHECK("dense_tile_kernel");
  return TI_OK;
}

// up to 64 rows: as many row tiles per workgroup as still leave two workgroups per CU
template <class T, int EPI>
int skinny(const ti_dense_args& a, hipStream_t s) {
  const long g = (long)((a.N + 15) / 16) * a.batch;
  const int mt = (a.M + 15) / 16;
  if (a.tile_rows || mt == 1 || g < 256) return launch_skinny<T, 1, EPI>(a, s);
  if (mt == 2 || g < 512) return launch_skinny<T, 2, EPI>(a, s);
  return launch_skinny<T, 4, EPI>(a, s);
}

// More rows: the tile whose rounds over the 256 CUs cost least, by the time of one round of each tile
// (us at K 2048, measured).
template <class T, int EPI>
int tiled(const ti_dense_args& a, hipStream_t s) {
  auto cost = [&](int bm, int bn, float us) {
    const long wgs = (long)((a.M + bm - 1) / bm) * ((a.N + bn - 1) / bn) * a.batch;
    return (float)((wgs + 255) / 256) * us;
  };
  const float c[4] = {cost(128, 256, 37.f), cost(64, 256, 27.f), cost(64, 128, 15.f), cost(32, 128, 11.5f)};
  switch (std::min_element(c, c + 4) - c) {
    case 0: return launch_tile<T, 128, 256, 2, EPI>(a, s);
    case 1: return launch_tile<T, 64, 256, 2, EPI>(a, s);
    case 2: return launch_tile<T, 64, 128, 4, EPI>(a, s);
    default: return launch_tile<T, 32, 128, 4, EPI>(a, s);
  }
}

template <class T>
int dispatch_dense(const ti_dense_args& a, hipStream_t s) {
  const bool few = a.tile_rows == 1 || a.tile_rows == 16 || (!a.tile_rows && a.M <= 64);
  switch (a.epi) {
    case TI_DE_F32: return few ? skinny<T, TI_DE_F32>(a, s) : tiled<T, TI_DE_F32>(a, s);
    case TI_DE_ROPE: return few ? skinny<T, TI_DE_ROPE>(a, s) : tiled<T, TI_DE_ROPE>(a, s);
    case TI_DE_ACT: return few ? skinny<T, TI_DE_ACT>(a, s) : tiled<T, TI_DE_ACT>(a, s);
    case TI_DE_LRU: return few ? skinny<T, TI_DE_LRU>(a, s) : launch_tile<T, 64, 128, 4, TI_DE_LRU>(a, s);   // (short k: the epilogue decides)
    case TI_DE_LOGITS: return few ? skinny<T, TI_DE_LOGITS>(a, s) : launch_tile<T, 64, 64, 4, TI_DE_LOGITS>(a, s);
    case TI_DE_GATE: return few ? skinny<T, TI_DE_GATE>(a, s) : launch_tile<T, 64, 64, 4, TI_DE_GATE>(a, s);
    case TI_DE_SWIGLU:
      if (few) return skinny<T, TI_DE_SWIGLU>(a, s);
      if (a.tile_rows == 128) return launch_tile<T, 128, 256, 2, TI_DE_SWIGLU>(a, s);
      return launch_tile<T, 64, 256, 2, TI_DE_SWIGLU>(a, s);
    case TI_DE_T:
      if (few) return skinny<T, TI_DE_T>(a, s);
      if (a.tile_rows == 128) return launch_tile<T, 128, 256, 2, TI_DE_T>(a, s);
      if (a.tile_rows) return launch_tile<T, 64, 256, 2, TI_DE_T>(a, s);
      return launch_tile<T, 64, 64, 4, TI_DE_T>(a, s);
    // (every row of a 128-row tile is written by the fragment epilogues)
    case TI_DE_KFRAG: return launch_tile<T, 128, 128, 2, TI_DE_KFRAG>(a, s);
    default: return launch_tile<T, 128, 128, 2, TI_DE_VFRAG>(a, s);
  }
}

template <class T>
__global__ __launch_bounds__(256) void stack_fill_kernel(uint64_t stream, uint64_t n, float scale, T* out) {
  for (uint64_t i = (uint64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (uint64_t)gridDim.x * 256)
    out[i] = (T)(scale * synth_unit(stream, i));
}

// fp32 source elements into fragment order (ti_stack_pack)
template <class T>
__global__ __launch_bounds__(256) void stack_pack_kernel(const float* src, int64_t rs, int64_t ks, int rows, int K, int nk,
                                                         const int32_t* map, T* dst) {
  constexpr int VEC = El<T>::VEC, KT = El<T>::KT;
  const int64_t n = (int64_t)rows * K;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int r = (int)(i / K), k = (int)(i - (int64_t)r * K), d = map ? map[r] : r;
    dst[(((int64_t)(d >> 4) * nk + k / KT) * 64 + ((k % KT) / VEC) * 16 + (d & 15)) * VEC + k % VEC] = (T)src[r * rs + k * ks];
  }
}
template <class T>
__global__ __launch_bounds__(256) void stack_convert_kernel(const float* src, uint64_t n, T* dst) {
  for (uint64_t i = (uint64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (uint64_t)gridDim.x * 256) dst[i] = (T)src[i];
}

}  // namespace ti

extern "C" int ti_stack_kpad(int dtype, int K) {
  const int u = dtype == TI_DT_BF16 ? 64 : 32;
  return (K + u - 1) / u * u;
}

extern "C" size_t ti_stack_weight_bytes(int dtype, int N, int K) {
  if (N < 1 || K < 1) return 0;
  return (size_t)((N + 15) / 16 * 16) * ti_stack_kpad(dtype, K) * (dtype == TI_DT_BF16 ? 2 : 4);
}

extern "C" int ti_stack_pack(const float* src, int64_t rs, int64_t ks, int rows, int K, const int32_t* map, int dtype,
                             void* dst, ti_stream_t stream) {
  using namespace ti;
  if (!src || !dst || rows < 1 || K < 1 || (dtype != TI_DT_BF16 && dtype != TI_DT_F32))
    return ti_set_error(TI_ERR_ARG, "ti_stack_pack: bad arguments");
  const unsigned g = (unsigned)std::min<int64_t>(((int64_t)rows * K + 255) / 256, 8192);
  const int kp = ti_stack_kpad(dtype, K);
  if (dtype == TI_DT_BF16)
    hipLaunchKernelGGL(stack_pack_kernel<bf16>, dim3(g), dim3(256), 0, (hipStream_t)stream, src, rs, ks, rows, K,
                       kp / El<bf16>::KT, map, (bf16*)dst);
  else
    hipLaunchKernelGGL(stack_pack_kernel<float>, dim3(g), dim3(256), 0, (hipStream_t)stream, src, rs, ks, rows, K,
                       kp / El<float>::KT, map, (float*)dst);
  TI_LAUNCH_CHECK("stack_pack_kernel");
  return TI_OK;
}

extern "C" int ti_stack_convert(const float* src, uint64_t n, int dtype, void* dst, ti_stream_t stream) {
  using namespace ti;
  if (!src || !dst || (dtype != TI_DT_BF16 && dtype != TI_DT_F32)) return ti_set_error(TI_ERR_ARG, "ti_stack_convert: bad arguments");
  if (n == 0) return TI_OK;
  const unsigned g = (unsigned)std::min<uint64_t>((n + 255) / 256, 4096);
  if (dtype == TI_DT_BF16)
    hipLaunchKernelGGL(stack_convert_kernel<bf16>, dim3(g), dim3(256), 0, (hipStream_t)stream, src, n, (bf16*)dst);
  else
    hipLaunchKernelGGL(stack_convert_kernel<float>, dim3(g), dim3(256), 0, (hipStream_t)stream, src, n, (float*)dst);
  TI_LAUNCH_CHECK("stack_convert_kernel");
  return TI_OK;
}

extern "C" size_t ti_dense_args_bytes(void) { return sizeof(ti_dense_args); }

extern "C" int ti_dense(const ti_dense_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->w || !a->a || !a->out || a->M < 1 || a->N < 1 || a->K < 1 || a->batch < 1)
    return ti_set_error(TI_ERR_ARG, "ti_dense: bad arguments");
  if (a->dtype != TI_DT_BF16 && a->dtype != TI_DT_F32) return ti_set_error(TI_ERR_ARG, "ti_dense: dtype %d", a->dtype);
  const int vec = a->dtype == TI_DT_BF16 ? 8 : 4;
  if (a->K != ti_stack_kpad(a->dtype, a->K) || a->lda % vec || a->a_batch % vec)
    return ti_set_error(TI_ERR_ARG, "ti_dense: K %d / lda %d not padded", a->K, a->lda);
  if ((!a->tile_rows && !a->rows_in && a->lda < a->K) || a->batch > 65535)
    return ti_set_error(TI_ERR_ARG, "ti_dense: lda %d < K %d or batch %d", a->lda, a->K, a->batch);
  const bool rows_ok = a->tile_rows == 1 || a->tile_rows == 16 || a->tile_rows == 64 || a->tile_rows == 128;
  if (a->tile_rows && (a->epi == TI_DE_F32 || a->epi > TI_DE_SWIGLU || !rows_ok || a->max_tiles < 1 || a->max_tiles > 65535 ||
                       a->batch != 1 || (a->rows_in && a->row_div < 1) || !a->tiles ||
                       (a->tile_rows == 1 ? a->rows_in || a->rows_out : !a->n_tiles)))
    return ti_set_error(TI_ERR_ARG, "ti_dense: grouped arguments");
  if (!a->tile_rows && (a->rows_in || a->rows_out)) return ti_set_error(TI_ERR_ARG, "ti_dense: row lists need grouped tiles");
  switch (a->epi) {
    case TI_DE_F32: case TI_DE_T: break;
    case TI_DE_SWIGLU:
      if (a->N % 2 || a->batch != 1) return ti_set_error(TI_ERR_ARG, "ti_dense: SWIGLU N %d", a->N);
      break;
    case TI_DE_ROPE:
      if (!a->rope_cs || !a->pos || a->head_w < 1 || a->N % a->head_w || a->head_w % 4 || a->rot_off % 4 || a->ldo % 4 ||
          a->rot_off > a->head_w || a->batch != 1)
        return ti_set_error(TI_ERR_ARG, "ti_dense: ROPE arguments");
      break;
    case TI_DE_GATE:
      if (!a->gate || a->gate_ld < a->batch) return ti_set_error(TI_ERR_ARG, "ti_dense: GATE arguments");
      break;
    case TI_DE_LOGITS:
      if (!a->argmax || a->batch != 1) return ti_set_error(TI_ERR_ARG, "ti_dense: LOGITS arguments");
      break;
    case TI_DE_KFRAG: case TI_DE_VFRAG: {
      const int unit = a->epi == TI_DE_KFRAG ? 4 * vec : 16;
      if (a->head_w < 1 || a->N % a->head_w || a->head_w % unit || a->batch != 1 || a->key_blocks % 8 ||
          (long)a->key_blocks * 16 < ((long)a->M + 127) / 128 * 128)
        return ti_set_error(TI_ERR_ARG, "ti_dense: key / value fragments: head_w %d, key_blocks %d, M %d", a->head_w,
                            a->key_blocks, a->M);
      break;
    }
    case TI_DE_ACT:
      if (a->batch != 1 || a->t_cols < 0 || a->t_cols > a->N || (a->t_cols < a->N && !a->out2) || a->ldo < a->t_cols ||
          a->act < TI_ACT_NONE || a->act > TI_ACT_GELU_ERF)
        return ti_set_error(TI_ERR_ARG, "ti_dense: ACT arguments");
      break;
    case TI_DE_LRU:
      if (a->N % 2 || !a->add || !a->lru_rate)
        return ti_set_error(TI_ERR_ARG, "ti_dense: LRU arguments");
      break;
    default: return ti_set_error(TI_ERR_ARG, "ti_dense: epilogue %d", a->epi);
  }
  return a->dtype == TI_DT_BF16 ? dispatch_dense<bf16>(*a, (hipStream_t)stream) : dispatch_dense<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_stack_fill(uint64_t seed, uint32_t tid, uint64_t n, float scale, int dtype, void* out, ti_stream_t stream) {
  using namespace ti;
  if (!out || (dtype != TI_DT_BF16 && dtype != TI_DT_F32)) return ti_set_error(TI_ERR_ARG, "ti_stack_fill: bad arguments");
  if (n == 0) return TI_OK;
  const unsigned g = (unsigned)std::min<uint64_t>((n + 255) / 256, 4096);
  const uint64_t st = synth_stream(seed, tid);
  if (dtype == TI_DT_BF16)
    hipLaunchKernelGGL(stack_fill_kernel<bf16>, dim3(g), dim3(256), 0, (hipStream_t)stream, st, n, scale, (bf16*)out);
  else
    hipLaunchKernelGGL(stack_fill_kernel<float>, dim3(g), dim3(256), 0, (hipStream_t)stream, st, n, scale, (float*)out);
  TI_LAUNCH_CHECK("stack_fill_kernel");
  return TI_OK;
}
