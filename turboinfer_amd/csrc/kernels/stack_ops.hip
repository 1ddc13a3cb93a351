// stack_ops.hip -- row kernels of the layer-stack models (ti_stack.h): residual + norms, expert
// routing.  All arithmetic fp32.
#include <algorithm>

#include "elem.hpp"

namespace ti {

// A row of H values in LDS, normalised: mean and inverse deviation (layer norm) or inverse root mean
// square (mean = 0).  The variance is the mean of the squared deviations (second pass over LDS).
__device__ __forceinline__ float2 row_stats(const float* row, int H, float eps, int kind, float* red) {
  float mean = 0.0f;
  if (kind == TI_NORM_LAYER) {
    float s = 0.0f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) s += row[i];
    mean = block_sum(s, red) / (float)H;
  }
  float q = 0.0f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float d = row[i] - mean;
    q = fmaf(d, d, q);
  }
  const float var = block_sum(q, red) / (float)H;
  return make_float2(mean, 1.0f / sqrtf(var + eps));
}

template <class T>
__global__ __launch_bounds__(512) void rownorm_kernel(const ti_rownorm_args a) {
  extern __shared__ float row[];
  __shared__ float red[8];
  const int m = blockIdx.x, H = a.H;
  float* x = a.x + (size_t)m * H;
  // (each thread touches only its own elements of `row` outside the reductions, which hold barriers)
  if (a.y || a.parts) {
    if (a.parts) {
      const T* p = (const T*)a.parts + (size_t)m * a.top * a.ldy;
      for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = 0.0f;
        for (int k = 0; k < a.top; ++k) v = fmaf(a.part_w[(size_t)m * a.top + k], (float)p[(size_t)k * a.ldy + i], v);
        row[i] = v;
      }
    } else {
      for (int i = threadIdx.x; i < H; i += blockDim.x) row[i] = a.y[(size_t)m * a.ldy + i];
    }
    if (a.post_w) {
      const float2 st = row_stats(row, H, a.eps, a.kind, red);
      for (int i = threadIdx.x; i < H; i += blockDim.x) {
        const float b = a.kind == TI_NORM_LAYER ? a.post_b[i] : 0.0f;
        row[i] = x[i] + ((row[i] - st.x) * st.y * a.post_w[i] + b);
      }
    } else {
      for (int i = threadIdx.x; i < H; i += blockDim.x) row[i] += x[i];
    }
    for (int i = threadIdx.x; i < H; i += blockDim.x) x[i] = row[i];
  } else {
    for (int i = threadIdx.x; i < H; i += blockDim.x) row[i] = x[i];
  }
  if (a.cat) {
    T* c = (T*)a.cat + (size_t)m * a.ldc;
    const float* x0 = a.x0 + (size_t)m * H;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
      c[i] = (T)row[i];
      c[H + i] = (T)x0[i];
    }
  }
  if (a.xn && !a.w) {
    T* o = (T*)a.xn + (size_t)m * a.ldn;
    for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = (T)row[i];
  } else if (a.xn) {
    const float2 st = row_stats(row, H, a.eps, a.kind, red);
    T* o = (T*)a.xn + (size_t)m * a.ldn;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
      const float b = a.kind == TI_NORM_LAYER ? a.b[i] : 0.0f;
      o[i] = (T)((row[i] - st.x) * st.y * a.w[i] + b);
    }
  }
}

// The same with H % 4 == 0 and H <= 4 * TH * NC: each thread holds NC float4 of the row in registers and
// every load (residual, sublayer output, both norms' weights) is in flight before the first reduction.
// ROUTE: the same workgroup multiplies the normalised row with the router's weights (its first
// fragments in flight through the norms) and picks the row's experts.
template <class T, int TH, int NC, bool ROUTE>
__global__ __launch_bounds__(TH) void rownorm_vec_kernel(const ti_rownorm_args a) {
  typedef typename El<T>::Q Q;
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, NW = TH / 64, PF = 4;
  __shared__ float red[TH / 64];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int nk = ROUTE ? ti_kpad<T>(a.H) / KT : 0, nt = ROUTE ? (a.route_e + 15) >> 4 : 0;
  const V* rw = (const V*)a.route_w + lane;
  V rf[ROUTE ? PF : 1][4];
  const int m = blockIdx.x, tid = threadIdx.x, H4 = a.H >> 2;
  const bool ln = a.kind == TI_NORM_LAYER, add = a.y || a.parts;
  f32x4* x = (f32x4*)(a.x + (size_t)m * a.H);
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 v[NC], y[NC], pw[NC], pb[NC], w[NC], b[NC], z[NC];
  bool live[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = min(tid + c * TH, H4 - 1);
    live[c] = tid + c * TH < H4;
    v[c] = x[i];
    y[c] = a.y ? *(const f32x4*)(a.y + (size_t)m * a.ldy + 4 * i) : zero;
    pw[c] = add && a.post_w ? *(const f32x4*)(a.post_w + 4 * i) : zero;
    pb[c] = add && a.post_w && ln ? *(const f32x4*)(a.post_b + 4 * i) : zero;
    w[c] = a.w ? *(const f32x4*)(a.w + 4 * i) : zero;
    b[c] = a.w && ln ? *(const f32x4*)(a.b + 4 * i) : zero;
    z[c] = a.cat ? *(const f32x4*)(a.x0 + (size_t)m * a.H + 4 * i) : zero;
  }
  if (a.parts) {
    const T* p = (const T*)a.parts + (size_t)m * a.top * a.ldy;
    for (int k0 = 0; k0 < a.top; k0 += 4) {
      Q q[4][NC];
      float pk[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = min(k0 + u, a.top - 1);
        pk[u] = k0 + u < a.top ? a.part_w[(size_t)m * a.top + k] : 0.0f;
#pragma unroll
        for (int c = 0; c < NC; ++c) q[u][c] = *(const Q*)(p + (size_t)k * a.ldy + 4 * min(tid + c * TH, H4 - 1));
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (k0 + u < a.top)
#pragma unroll
          for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int e = 0; e < 4; ++e) y[c][e] = fmaf(pk[u], (float)q[u][c][e], y[c][e]);
    }
  }
  if constexpr (ROUTE) {   // (behind the row's own loads, in flight through the norms)
#pragma unroll
    for (int i = 0; i < PF; ++i)
#pragma unroll
      for (int t = 0; t < 4; ++t) rf[i][t] = rw[((size_t)min(t, nt - 1) * nk + min(wave + i * NW, nk - 1)) * 64];
  }
  // mean and inverse deviation of the row held in r
  auto stats = [&](const f32x4* r) -> float2 {
    float mean = 0.0f;
    if (ln) {
      float s = 0.0f;
#pragma unroll
      for (int c = 0; c < NC; ++c)
        if (live[c]) s += (r[c][0] + r[c][1]) + (r[c][2] + r[c][3]);
      mean = block_sum(s, red) / (float)a.H;
    }
    float q = 0.0f;
#pragma unroll
    for (int c = 0; c < NC; ++c)
      if (live[c])
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float d = r[c][e] - mean;
          q = fmaf(d, d, q);
        }
    return make_float2(mean, 1.0f / sqrtf(block_sum(q, red) / (float)a.H + a.eps));
  };
  if (add) {
    float2 st = make_float2(0.0f, 1.0f);
    if (a.post_w) st = stats(y);
#pragma unroll
    for (int c = 0; c < NC; ++c) {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[c][e] += a.post_w ? (y[c][e] - st.x) * st.y * pw[c][e] + pb[c][e] : y[c][e];
      if (live[c]) x[tid + c * TH] = v[c];
    }
  }
  if (a.cat) {
    T* cr = (T*)a.cat + (size_t)m * a.ldc;
#pragma unroll
    for (int c = 0; c < NC; ++c)
      if (live[c]) {
        *(Q*)(cr + 4 * (tid + c * TH)) = quad<T>(v[c]);
        *(Q*)(cr + a.H + 4 * (tid + c * TH)) = quad<T>(z[c]);
      }
  }
  if (a.xn) {
    float2 st = make_float2(0.0f, 1.0f);
    if (a.w) st = stats(v);
    T* o = (T*)a.xn + (size_t)m * a.ldn;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      f32x4 r;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = a.w ? (v[c][e] - st.x) * st.y * w[c][e] + b[c][e] : v[c][e];
      if (live[c]) *(Q*)(o + 4 * (tid + c * TH)) = quad<T>(r);
      if constexpr (ROUTE) {   // (the row's k padding: zeros)
        extern __shared__ float row[];
        if (4 * (tid + c * TH) < nk * KT) *(Q*)((T*)row + 4 * (tid + c * TH)) = live[c] ? quad<T>(r) : quad<T>(zero);
      }
    }
    if constexpr (ROUTE) {
      extern __shared__ float row[];
      __shared__ float zr[NW][64];
      lds_sync();
      f32x4 acc[4] = {zero, zero, zero, zero};
      const T* xr = (const T*)row + (lane >> 4) * VEC;   // every operand column is this row
#pragma unroll
      for (int i = 0; i < PF; ++i)
        if (wave + i * NW < nk) {
          const V x = *(const V*)(xr + (wave + i * NW) * KT);
#pragma unroll
          for (int t = 0; t < 4; ++t) acc[t] = mma(rf[i][t], x, acc[t]);
        }
      for (int kt = wave + PF * NW; kt < nk; kt += NW) {
        const V x = *(const V*)(xr + kt * KT);
#pragma unroll
        for (int t = 0; t < 4; ++t) acc[t] = mma(rw[((size_t)min(t, nt - 1) * nk + kt) * 64], x, acc[t]);
      }
      if ((lane & 15) == 0)
#pragma unroll
        for (int t = 0; t < 4; ++t) *(f32x4*)&zr[wave][t * 16 + 4 * (lane >> 4)] = acc[t];
      lds_sync();
      if (wave == 0) {
        float zl = 0.0f;
#pragma unroll
        for (int w = 0; w < NW; ++w) zl += zr[w][lane];
        route_top64(zl, a.route_e, a.route_top, a.route_idx + (size_t)m * a.route_top, a.route_wgt + (size_t)m * a.route_top);
      }
    }
  }
}

template <class T>
int launch_rownorm(const ti_rownorm_args& a, hipStream_t s) {
  const bool vec = a.H % 4 == 0 && a.H <= 8192 && a.ldy % 4 == 0 && a.ldn % 4 == 0 && a.ldc % 4 == 0;
  if (a.route_w) {
    if (!vec) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_rownorm: routing needs H %% 4 == 0, H <= 8192");
    const size_t lds = (size_t)ti_kpad<T>(a.H) * sizeof(T);
    if (a.H <= 1024) hipLaunchKernelGGL((rownorm_vec_kernel<T, 512, 1, true>), dim3(a.M), dim3(512), lds, s, a);
    else if (a.H <= 4096) hipLaunchKernelGGL((rownorm_vec_kernel<T, 1024, 1, true>), dim3(a.M), dim3(1024), lds, s, a);
    else hipLaunchKernelGGL((rownorm_vec_kernel<T, 1024, 2, true>), dim3(a.M), dim3(1024), lds, s, a);
  } else if (vec && a.H <= 1024) {
    hipLaunchKernelGGL((rownorm_vec_kernel<T, 256, 1, false>), dim3(a.M), dim3(256), 0, s, a);
  } else if (vec && a.H <= 2048) {
    hipLaunchKernelGGL((rownorm_vec_kernel<T, 512, 1, false>), dim3(a.M), dim3(512), 0, s, a);
  } else if (vec && a.H <= 4096) {
    hipLaunchKernelGGL((rownorm_vec_kernel<T, 1024, 1, false>), dim3(a.M), dim3(1024), 0, s, a);
  } else if (vec) {
    hipLaunchKernelGGL((rownorm_vec_kernel<T, 1024, 2, false>), dim3(a.M), dim3(1024), 0, s, a);
  } else {
    hipLaunchKernelGGL(rownorm_kernel<T>, dim3(a.M), dim3(a.H <= 1024 ? 256 : 512), (size_t)a.H * 4, s, a);
  }
  TI_LAUNCH_CHECK("rownorm_kernel");
  return TI_OK;
}

// ------------------------------------------------------------------ expert routing
constexpr int kMaxE = 1024, kMaxTop = 64;

// One wave per row: softmax over the experts, the top scores (lowest index first among equals).
// Repeated maxima; E <= 64: lane l holds expert l, more experts: lane l holds experts l, l + 64, ...
__device__ __forceinline__ void route_row(const ti_route_args& a, int m) {
  constexpr int PER = kMaxE / 64;
  const int lane = threadIdx.x & 63;
  const float* z = a.logits + (size_t)m * a.ld;
  if (a.E <= 64) {
    route_top64(lane < a.E ? z[lane] : 0.0f, a.E, a.top, a.idx + (size_t)m * a.top, a.wgt + (size_t)m * a.top);
    return;
  }
  float s[PER];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = lane + 64 * i;
    s[i] = e < a.E ? z[e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  mx = wave_max_xor<64>(mx);
  float sum = 0.0f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    s[i] = lane + 64 * i < a.E ? expf(s[i] - mx) : -1.0f;
    sum += s[i] >= 0.0f ? s[i] : 0.0f;
  }
  sum = group_sum<64>(sum);
  for (int k = 0; k < a.top; ++k) {
    unsigned long long best = 0ull;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (s[i] >= 0.0f) {
        const unsigned long long key = ((unsigned long long)float_order_key(s[i]) << 32) |
                                       (unsigned long long)(0xFFFFFFFFu - (uint32_t)(lane + 64 * i));
        best = key > best ? key : best;
      }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const unsigned long long other = __shfl_xor(best, o, kWave);
      best = other > best ? other : best;
    }
    // (no comparable score left, NaN logits: expert 0, never an index outside the table)
    const int e = best ? (int)(0xFFFFFFFFu - (uint32_t)(best & 0xFFFFFFFFull)) : 0;
    float v = 0.0f;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (lane + 64 * i == e) {
        v = s[i];
        s[i] = -1.0f;
      }
    if (lane == (e & 63)) {
      a.idx[(size_t)m * a.top + k] = e;
      a.wgt[(size_t)m * a.top + k] = v / sum;
    }
  }
}

// One workgroup groups the M * top entries by expert: counts, a scan over the experts of entries and
// tiles, then the lists.
__device__ __forceinline__ void route_group(const ti_route_args& a) {
  __shared__ int cnt[kMaxE], at[kMaxE], tl[kMaxE];
  const int tid = threadIdx.x, nt = blockDim.x, n = a.M * a.top;
  for (int e = tid; e < a.E; e += nt) cnt[e] = 0;
  __syncthreads();
  for (int p = tid; p < n; p += nt) atomicAdd(&cnt[a.idx[p]], 1);
  __syncthreads();
  if (tid < 64) {   // wave 0: exclusive scans over the experts, 64 at a time
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < a.E; e0 += 64) {
      const int e = e0 + tid, c = e < a.E ? cnt[e] : 0, t = (c + a.tile_rows - 1) / a.tile_rows;
      int ic = c, it = t;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int uc = __shfl_up(ic, o, 64), ut = __shfl_up(it, o, 64);
        if (tid >= o) {
          ic += uc;
          it += ut;
        }
      }
      if (e < a.E) {
        at[e] = base + ic - c;
        tl[e] = tbase + it - t;
      }
      base += __shfl(ic, 63, 64);
      tbase += __shfl(it, 63, 64);
    }
    if (tid == 0) *a.n_tiles = tbase;
  }
  __syncthreads();
  for (int e = tid; e < a.E; e += nt)
    for (int i = 0, c = cnt[e]; i < c; i += a.tile_rows) {
      int* t = a.tiles + 4 * (tl[e] + i / a.tile_rows);
      t[0] = e;
      t[1] = at[e] + i;
      t[2] = min(a.tile_rows, c - i);
      t[3] = 0;
    }
  __syncthreads();
  for (int p = tid; p < n; p += nt) a.list[atomicAdd(&at[a.idx[p]], 1)] = p;
}

__global__ __launch_bounds__(256) void route_kernel(const ti_route_args a) {
  const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (m < a.M) route_row(a, m);
}
__global__ __launch_bounds__(1024) void route_group_kernel(const ti_route_args a) { route_group(a); }
// few rows: both steps in one workgroup
__global__ __launch_bounds__(1024) void route_both_kernel(const ti_route_args a) {
  if (a.logits)
    for (int m = threadIdx.x >> 6; m < a.M; m += 16) route_row(a, m);
  __threadfence_block();
  __syncthreads();
  route_group(a);
}

}  // namespace ti

extern "C" int ti_rownorm(const ti_rownorm_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->x || a->M < 1 || a->H < 1 || a->H > 16128 || (a->kind != TI_NORM_LAYER && a->kind != TI_NORM_RMS) ||
      (a->dtype != TI_DT_BF16 && a->dtype != TI_DT_F32))
    return ti_set_error(TI_ERR_ARG, "ti_rownorm: bad arguments");
  if ((a->y && a->parts) || ((a->y || a->parts) && a->ldy < a->H) || (a->parts && (!a->part_w || a->top < 1)) ||
      (a->post_w && a->kind == TI_NORM_LAYER && !a->post_b) ||
      (a->w && !a->xn) || (a->xn && (a->ldn < a->H || (a->w && a->kind == TI_NORM_LAYER && !a->b))) ||
      (a->cat && (!a->x0 || a->ldc < 2 * a->H)))
    return ti_set_error(TI_ERR_ARG, "ti_rownorm: inconsistent arguments");
  if (a->route_w && (!a->xn || !a->w || !a->route_idx || !a->route_wgt || a->route_e < 1 || a->route_e > 64 || a->route_top < 1 ||
                     a->route_top > a->route_e))
    return ti_set_error(TI_ERR_ARG, "ti_rownorm: routing arguments");
  return a->dtype == TI_DT_BF16 ? launch_rownorm<bf16>(*a, (hipStream_t)stream) : launch_rownorm<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_rownorm_routes(int H, int E) { return H % 4 == 0 && H <= 8192 && E >= 1 && E <= 64; }

extern "C" int ti_route_max_tiles(int M, int E, int top, int tile_rows) {
  if (M < 1 || E < 1 || top < 1 || tile_rows < 1) return 0;
  const long n = (long)M * top;
  // every expert with entries has at most one partly filled tile
  return (int)(std::min<long>(E, n) + n / tile_rows);
}

extern "C" int ti_route(const ti_route_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || (!a->logits && !a->tile_rows) || !a->idx || !a->wgt || a->M < 1 || a->E < 1 || a->E > kMaxE || a->top < 1 || a->top > kMaxTop ||
      a->top > a->E || (a->logits && a->ld < a->E))
    return ti_set_error(TI_ERR_ARG, "ti_route: bad arguments (1 <= top <= experts <= %d, top <= %d)", kMaxE, kMaxTop);
  if (a->tile_rows && (!a->list || !a->tiles || !a->n_tiles || a->tile_rows < 1))
    return ti_set_error(TI_ERR_ARG, "ti_route: list / tiles");
  hipStream_t s = (hipStream_t)stream;
  if (a->tile_rows && a->M <= 16) {
    hipLaunchKernelGGL(route_both_kernel, dim3(1), dim3(1024), 0, s, *a);
  } else {
    if (a->logits) hipLaunchKernelGGL(route_kernel, dim3((a->M + 3) / 4), dim3(256), 0, s, *a);
    if (a->tile_rows) hipLaunchKernelGGL(route_group_kernel, dim3(1), dim3(1024), 0, s, *a);
  }
  TI_LAUNCH_CHECK("route_kernel");
  return TI_OK;
}
