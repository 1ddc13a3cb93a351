// recurrent.hip -- recurrent mixers of the layer-stack models (ti_stack.h): short causal convolutions, the
// state-space recurrence (SSD) and the gated linear recurrence over prompt chunks and single tokens.
//
//   * conv_kernel: convolution over rows and the slot's ring of earlier inputs.
//   * ssd_step_kernel: one token per row: convolution, step size, state update and output of a slice of
//     one head; the state is streamed once (read, update, write).
//   * ssd_scan_kernel: a prompt chunk in blocks of 64 tokens: scores C B^T under the decay mask, the state
//     carried in MFMA accumulators; products that involve decays or the state are fp32 MFMA.
//   * ssd_norm_kernel: SiLU gate and grouped RMS norm.
//   * lru_scan_kernel: S = a S + b per channel, the chunk cut into 64 segments scanned side by side.
// Step sizes, decays, states and sums are fp32 (cumulated log decays fp64).
#include <algorithm>

#include "elem.hpp"

namespace ti {

__device__ __forceinline__ float siluf(float z) { return z * sigmoidf(z); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

// ------------------------------------------------------------------ short convolution
constexpr int kConvRows = 4;

// A thread owns VQ consecutive output places of kConvRows rows.
template <class T, int VQ>
__global__ __launch_bounds__(256) void conv_kernel(const ti_conv_args a, int places) {
  const int i0 = ((int)blockIdx.x * 256 + (int)threadIdx.x) * VQ;
  if (i0 >= places) return;
  int c0 = i0;   // first channel; -1: places no channel has
  if (i0 >= a.c0) {
    const int s = i0 - a.o0, r = s % a.bwp;
    c0 = s >= 0 && r < a.bw ? a.c0 + s / a.bwp * a.bw + r : -1;
    if (s < 0 && i0 < a.o0) return;   // (between the plain part and the sections: unused)
  }
  typedef T TV __attribute__((ext_vector_type(VQ)));
  for (int r = 0; r < kConvRows; ++r) {
    const int m = blockIdx.y * kConvRows + r;
    if (m >= a.M) return;
    TV o;
    if (c0 < 0) {
#pragma unroll
      for (int e = 0; e < VQ; ++e) o[e] = (T)0.0f;
    } else {
      const int pos = a.pos[m];
      T* ring = (T*)a.ring + (size_t)(a.chunk ? a.slot0 : a.slot ? a.slot[m] : m) * a.taps * a.channels + c0;
      float acc[VQ];
#pragma unroll
      for (int e = 0; e < VQ; ++e) acc[e] = a.b[c0 + e];
      TV cur;
      for (int back = a.taps - 1; back >= 0; --back) {
        const int p = pos - back;
        if (p < 0) continue;
        const T* src = back == 0 || (a.chunk && m >= back) ? (const T*)a.x + (size_t)(m - back) * a.ldx + c0
                                                           : ring + (size_t)(p % a.taps) * a.channels;
        cur = *(const TV*)src;
#pragma unroll
        for (int e = 0; e < VQ; ++e) acc[e] = fmaf(a.w[(size_t)(c0 + e) * a.taps + a.taps - 1 - back], (float)cur[e], acc[e]);
      }
      if (!a.chunk) *(TV*)(ring + (size_t)(pos % a.taps) * a.channels) = cur;
#pragma unroll
      for (int e = 0; e < VQ; ++e) o[e] = (T)(a.act == TI_CONV_SILU ? siluf(acc[e]) : acc[e]);
    }
    *(TV*)((T*)a.out + (size_t)m * a.ldo + i0) = o;
  }
}

// ------------------------------------------------------------------ SSD, one token per row
// Grid (slices of ps value dimensions, heads, rows).  LPR lanes share a state row (4 elements each).
template <class T, int LPR>
__global__ __launch_bounds__(256) void ssd_step_kernel(const ti_ssd_args a, int ps) {
  constexpr int RW = 64 / LPR, PF = 4;
  extern __shared__ float sh[];
  const int h = blockIdx.y, m = blockIdx.z, p0 = blockIdx.x * ps, N = a.state_n, np = (N + 3) & ~3, n4 = np >> 2;
  const int np_ = min(ps, a.vdim - p0), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l = lane % LPR;
  const int hpg = a.heads / a.groups, grp = h / hpg, inner = a.heads * a.vdim, channels = inner + 2 * a.groups * N;
  const int pos = a.pos[m], slot = a.slot ? a.slot[m] : m;
  float *xs = sh, *bs = sh + ((ps + 3) & ~3), *cs = bs + np;
  f32x4* st = (f32x4*)(a.state + (((size_t)slot * a.heads + h) * a.vdim + p0) * np);
  const int q0 = min(l, n4 - 1), pr = wave * RW + lane / LPR;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  // the first state rows fly through the convolution
  f32x4 s[PF];
  auto load = [&](int base, int q) {
#pragma unroll
    for (int u = 0; u < PF; ++u) s[u] = pos > 0 ? st[(size_t)min(base + u * 4 * RW, np_ - 1) * n4 + q] : zero;
  };
  load(pr, q0);
  const T* raw = (const T*)a.a + (size_t)m * a.lda + inner;
  T* ring = (T*)a.ring + (size_t)slot * a.taps * channels;
  for (int i = tid; i < np_ + 2 * np; i += 256) {
    int c, own;
    float* dst;
    if (i < np_) {
      c = h * a.vdim + p0 + i;
      own = 1;
      dst = xs + i;
    } else {
      const int j = i - np_, isc = j >= np, n = j - isc * np;
      c = n < N ? inner + (isc * a.groups + grp) * N + n : -1;
      own = blockIdx.x == 0 && h == grp * hpg;
      dst = (isc ? cs : bs) + n;
    }
    float v = 0.0f;
    if (c >= 0) {
      v = a.conv_b[c];
      const T cur = raw[c];
      for (int back = a.taps - 1; back > 0; --back)
        if (pos >= back)
          v = fmaf(a.conv_w[(size_t)c * a.taps + a.taps - 1 - back], (float)ring[(size_t)((pos - back) % a.taps) * channels + c], v);
      v = fmaf(a.conv_w[(size_t)c * a.taps + a.taps - 1], (float)cur, v);
      // (the place written is read by no one: it held position pos - taps)
      if (own) ring[(size_t)(pos % a.taps) * channels + c] = cur;
      v = (float)(T)siluf(v);
    }
    *dst = v;
  }
  const float dt = softplusf(a.dt[(size_t)m * a.heads + h] + a.dt_bias[h]), decay = expf(-expf(a.a_log[h]) * dt), D = a.d[h];
  lds_sync();
  for (int base = pr; base - pr < np_; base += PF * 4 * RW) {
    float acc[PF] = {};
    for (int q = l; q - l < n4; q += LPR) {   // (one pass unless the state is longer than 256)
      if (base != pr || q != l) load(base, min(q, n4 - 1));
      const bool on = q < n4;
      const f32x4 bq = *(const f32x4*)(bs + 4 * min(q, n4 - 1)) * dt, cq = *(const f32x4*)(cs + 4 * min(q, n4 - 1));
#pragma unroll
      for (int u = 0; u < PF; ++u) {
        const int p = base + u * 4 * RW;
        const float x = xs[min(p, np_ - 1)];
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          v[e] = fmaf(decay, s[u][e], bq[e] * x);
          if (on) acc[u] = fmaf(v[e], cq[e], acc[u]);
        }
        if (on && p < np_) st[(size_t)p * n4 + q] = v;
      }
    }
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      const int p = base + u * 4 * RW;
      const float y = group_sum<LPR>(acc[u]);
      if (l == 0 && p < np_) a.y[(size_t)m * a.ldy + h * a.vdim + p0 + p] = fmaf(D, xs[p], y);
    }
  }
}

// ------------------------------------------------------------------ SSD over a prompt chunk
__device__ __forceinline__ f32x4 widen4(const bf16* p) {
  const bf16x4 v = *(const bf16x4*)p;
  return (f32x4){(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
__device__ __forceinline__ f32x4 widen4(const float* p) { return *(const f32x4*)p; }

constexpr int kSsdTok = 64;

// Grid (slices of 16 value dimensions, heads).  Blocks of 64 tokens one after another; per block, with
// L(t, s) = exp(cum_t - cum_s):
//   y_t = sum_{s <= t} (C_t . B_s) L(t, s) dt_s x_s + exp(cum_t) S^T C_t + D x_t
//   S  <- exp(cum_last) S + sum_t L(last, t) dt_t B_t x_t^T
// Wave w owns tokens [16 w, +16) of the outputs and the state tiles w, w + 4, ... of 16 state rows; the
// accumulator of a product is the operand fragment of the next one (scores, state).
template <class T, int NTW>
__global__ __launch_bounds__(256, 1) void ssd_scan_kernel(const ti_ssd_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, PF = 4, XLD = kSsdTok + 4;
  extern __shared__ char lds[];
  const int N = a.state_n, nk = (N + KT - 1) / KT * KT, ld = nk + 16 / (int)sizeof(T), np = (N + 3) & ~3, nt = (N + 15) >> 4;
  T* Bs = (T*)lds;                       // [64][ld]
  T* Cs = Bs + kSsdTok * ld;             // [64][ld]
  float* xt = (float*)(Cs + kSsdTok * ld);   // [16][XLD] values, transposed
  f32x4* red = (f32x4*)(xt + 16 * XLD);  // [4][4][64] the waves' state outputs
  double* cum = (double*)(red + 16 * 64);
  float* dts = (float*)(cum + kSsdTok);  // [64]
  float* wl = dts + kSsdTok;             // [64] L(last, t) dt_t
  float* ec = wl + kSsdTok;              // [64] exp(cum_t)
  const int h = blockIdx.y, p0 = blockIdx.x * 16, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int grp = h / (a.heads / a.groups);
  const T* src = (const T*)a.a;
  const T* bsrc = src + a.o0 + (size_t)grp * nk;
  const T* csrc = bsrc + (size_t)a.groups * nk;
  const int ppr = nk / VEC, pieces = kSsdTok * ppr;   // 16-byte pieces per row, per block
  const float A = -expf(a.a_log[h]), bias = a.dt_bias[h], D = a.d[h];
  float* state = a.state + (((size_t)a.slot0 * a.heads + h) * a.vdim + p0) * np;
  const bool prow = p0 + col < a.vdim;
  f32x4 S[NTW];   // tile i: state rows n0 + 4 g + r, value dimension col
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int n = (wave + 4 * i) * 16 + 4 * g;
    S[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (a.pos[0] > 0 && prow && n < np) S[i] = *(const f32x4*)(state + (size_t)col * np + n);
  }
  V rb[PF], rc[PF];
  float rx[4], rdt = 0.0f;
  const V vz = {};
  auto piece = [&](const T* s, int m0, int i) -> V {
    const int t = i / ppr, c = i - t * ppr;
    return i < pieces && m0 + t < a.M ? *(const V*)(s + (size_t)(m0 + t) * a.lda + c * VEC) : vz;
  };
  auto load = [&](int m0) {
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      rb[u] = piece(bsrc, m0, tid + u * 256);
      rc[u] = piece(csrc, m0, tid + u * 256);
    }
    const int m = m0 + (tid >> 2), p = p0 + (tid & 3) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) rx[e] = m < a.M && p + e < a.vdim ? (float)src[(size_t)m * a.lda + h * a.vdim + p + e] : 0.0f;
    if (wave == 0) rdt = m0 + lane < a.M ? a.dt[(size_t)(m0 + lane) * a.heads + h] : 0.0f;
  };
  auto put = [&](T* d, int i, V v) {
    const int t = i / ppr, c = i - t * ppr;
    if (i < pieces) *(V*)(d + t * ld + c * VEC) = v;
  };
  load(0);
  for (int m0 = 0; m0 < a.M; m0 += kSsdTok) {
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      put(Bs, tid + u * 256, rb[u]);
      put(Cs, tid + u * 256, rc[u]);
    }
    for (int i = tid + PF * 256; i < pieces; i += 256) {   // (long states)
      put(Bs, i, piece(bsrc, m0, i));
      put(Cs, i, piece(csrc, m0, i));
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) xt[((tid & 3) * 4 + e) * XLD + (tid >> 2)] = rx[e];
    if (wave == 0) {
      const float dt = m0 + lane < a.M ? softplusf(rdt + bias) : 0.0f;   // (past the end: no decay, no input)
      double c = (double)(A * dt);
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double v = __shfl_up(c, o, 64);
        if (lane >= o) c += v;
      }
      cum[lane] = c;
      dts[lane] = dt;
      wl[lane] = expf((float)(__shfl(c, 63, 64) - c)) * dt;
      ec[lane] = expf((float)c);
    }
    lds_sync();
    if (m0 + kSsdTok < a.M) load(m0 + kSsdTok);
    // the carried state's share of every token, over this wave's state rows
    f32x4 yi[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) yi[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int tile = wave + 4 * i;
      if (tile < nt)
#pragma unroll
        for (int t = 0; t < 4; ++t) yi[t] = mma(S[i], widen4(Cs + (t * 16 + col) * ld + tile * 16 + 4 * g), yi[t]);
    }
#pragma unroll
    for (int t = 0; t < 4; ++t) red[(wave * 4 + t) * 64 + lane] = yi[t];
    // scores of this wave's tokens with the block's earlier ones, decayed, times their inputs
    f32x4 y = {0.f, 0.f, 0.f, 0.f};
    const int tok = wave * 16 + col;
    const double ct = cum[tok];
    for (int st = 0; st <= wave; ++st) {
      f32x4 sc = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < nk; k += KT)
        sc = mma(*(const V*)(Bs + (st * 16 + col) * ld + k + g * VEC), *(const V*)(Cs + tok * ld + k + g * VEC), sc);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = st * 16 + 4 * g + r;
        sc[r] = s <= tok ? sc[r] * expf((float)(ct - cum[s])) * dts[s] : 0.0f;
      }
      y = mma(*(const f32x4*)(xt + col * XLD + st * 16 + 4 * g), sc, y);
    }
    // the state over the block
    const float last = ec[kSsdTok - 1];
    f32x4 wx[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      const f32x4 w = *(const f32x4*)(wl + t * 16 + 4 * g), x = *(const f32x4*)(xt + col * XLD + t * 16 + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) wx[t][r] = w[r] * x[r];
    }
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int tile = wave + 4 * i;
      if (tile >= nt) continue;
#pragma unroll
      for (int r = 0; r < 4; ++r) S[i][r] *= last;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        f32x4 b;
#pragma unroll
        for (int r = 0; r < 4; ++r) b[r] = (float)Bs[(t * 16 + 4 * g + r) * ld + tile * 16 + col];
        S[i] = mma(b, wx[t], S[i]);
      }
    }
    lds_sync();
    // out: tokens this wave's, dimensions 4 g + r
    f32x4 z = red[wave * 64 + lane];
#pragma unroll
    for (int w = 1; w < 4; ++w) z += red[(w * 4 + wave) * 64 + lane];
    if (m0 + tok < a.M) {
      float* o = a.y + (size_t)(m0 + tok) * a.ldy + h * a.vdim + p0 + 4 * g;
      const float e = ec[tok];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (p0 + 4 * g + r < a.vdim) o[r] = fmaf(e, z[r], y[r]) + D * xt[(4 * g + r) * XLD + tok];
    }
    lds_sync();   // (the block's LDS is free)
  }
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int n = (wave + 4 * i) * 16 + 4 * g;
    if (prow && n < np) *(f32x4*)(state + (size_t)col * np + n) = S[i];
  }
}

// ------------------------------------------------------------------ gate and norm
template <class T>
__global__ __launch_bounds__(512) void ssd_norm_kernel(const ti_ssd_norm_args a) {
  extern __shared__ float v[];
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x, per = a.inner / a.groups;
  const float* y = a.y + (size_t)m * a.ldy;
  const T* raw = (const T*)a.raw + (size_t)m * a.lda;
  T* out = (T*)a.out + (size_t)m * a.ldo;
  for (int gr = 0; gr < a.groups; ++gr) {
    float q = 0.0f;
    for (int i = gr * per + tid; i < (gr + 1) * per; i += 512) {
      const float x = y[i] * siluf((float)raw[i]);
      v[i] = x;
      q = fmaf(x, x, q);
    }
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)per + a.eps);
    for (int i = gr * per + tid; i < (gr + 1) * per; i += 512) out[i] = (T)(v[i] * inv * a.w[i]);
  }
  if (a.ring && m >= a.M - (a.taps - 1)) {
    T* ring = (T*)a.ring + ((size_t)a.slot0 * a.taps + a.pos[m] % a.taps) * a.channels;
    for (int i = tid; i < a.channels; i += 512) ring[i] = raw[a.inner + i];
  }
}

// ------------------------------------------------------------------ gated linear recurrence over a chunk
// 16 channels x 64 segments of the rows: every segment's product and end value from zero, one scan over
// the segments, then the segments again from their start values.
constexpr int kLruSeg = 64;
template <class T>
__global__ __launch_bounds__(1024) void lru_scan_kernel(const ti_lru_scan_args a) {
  __shared__ float sa[kLruSeg][16], sb[kLruSeg][16];
  const int tid = threadIdx.x, ch = tid & 15, seg = tid >> 4, c = blockIdx.x * 16 + ch, cc = min(c, a.channels - 1);
  const int len = (a.M + kLruSeg - 1) / kLruSeg, r0 = seg * len, r1 = min(a.M, r0 + len);
  const float2* ab = (const float2*)a.ab + cc;
  constexpr int U = 8;
  float pa = 1.0f, pb = 0.0f;
  for (int r = r0; r < r1; r += U) {
    float2 v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) v[u] = ab[(size_t)min(r + u, a.M - 1) * a.channels];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (r + u < r1) {
        pa *= v[u].x;
        pb = fmaf(v[u].x, pb, v[u].y);
      }
  }
  sa[seg][ch] = pa;
  sb[seg][ch] = pb;
  __syncthreads();
  float* st = a.state + (size_t)a.slot0 * a.channels + cc;
  if (seg == 0) {   // sb becomes every segment's start value
    float s = a.pos[0] > 0 ? *st : 0.0f;
    for (int k = 0; k < kLruSeg; ++k) {
      const float x = sa[k][ch], y = sb[k][ch];
      sb[k][ch] = s;
      s = fmaf(x, s, y);
    }
    if (c < a.channels) *st = s;
  }
  __syncthreads();
  if (c >= a.channels) return;
  float s = sb[seg][ch];
  const T* y = (const T*)a.y + c;
  T* out = (T*)a.out + c;
  for (int r = r0; r < r1; r += U) {
    float2 v[U];
    T yv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      v[u] = ab[(size_t)min(r + u, a.M - 1) * a.channels];
      yv[u] = y[(size_t)min(r + u, a.M - 1) * a.ldy];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (r + u < r1) {
        s = fmaf(v[u].x, s, v[u].y);
        out[(size_t)(r + u) * a.ldo] = (T)(s * (float)yv[u]);
      }
  }
  const int back = seg;   // the last taps - 1 rows' inputs enter the ring
  if (back < a.taps - 1 && a.M - 1 - back >= 0) {
    const int m = a.M - 1 - back;
    ((T*)a.ring)[((size_t)a.slot0 * a.taps + a.pos[m] % a.taps) * a.channels + c] = ((const T*)a.x)[(size_t)m * a.ldy + c];
  }
}

// ------------------------------------------------------------------ launchers
template <class T>
int launch_conv(const ti_conv_args& a, hipStream_t s) {
  const int sections = a.c0 < a.channels ? (a.channels - a.c0) / a.bw : 0, places = sections ? a.o0 + sections * a.bwp : a.channels;
  const int rb = (a.M + kConvRows - 1) / kConvRows;
  const bool vec = ((a.channels | a.ldx | a.ldo | a.c0) & 3) == 0 && (!sections || ((a.o0 | a.bw | a.bwp) & 3) == 0);
  if (vec && sizeof(T) * 4 <= 16)
    hipLaunchKernelGGL((conv_kernel<T, 4>), dim3((places / 4 + 255) / 256, rb), dim3(256), 0, s, a, places);
  else
    hipLaunchKernelGGL((conv_kernel<T, 1>), dim3((places + 255) / 256, rb), dim3(256), 0, s, a, places);
  TI_LAUNCH_CHECK("conv_kernel");
  return TI_OK;
}

template <class T>
int launch_ssd_step(const ti_ssd_args& a, hipStream_t s) {
  const int np = (a.state_n + 3) / 4 * 4, n4 = np / 4;
  // few rows: slices of 16 fill the chip; many: whole heads (the slices repeat the convolution of B and C)
  const int ps = (long)a.M * a.heads >= 1024 ? std::min(a.vdim, 128) : 16;
  const dim3 grid((a.vdim + ps - 1) / ps, a.heads, a.M), blk(256);
  const size_t lds = (size_t)((ps + 3) / 4 * 4 + 2 * np) * 4;
  if (n4 <= 4) hipLaunchKernelGGL((ssd_step_kernel<T, 4>), grid, blk, lds, s, a, ps);
  else if (n4 <= 8) hipLaunchKernelGGL((ssd_step_kernel<T, 8>), grid, blk, lds, s, a, ps);
  else if (n4 <= 16) hipLaunchKernelGGL((ssd_step_kernel<T, 16>), grid, blk, lds, s, a, ps);
  else if (n4 <= 32) hipLaunchKernelGGL((ssd_step_kernel<T, 32>), grid, blk, lds, s, a, ps);
  else hipLaunchKernelGGL((ssd_step_kernel<T, 64>), grid, blk, lds, s, a, ps);
  TI_LAUNCH_CHECK("ssd_step_kernel");
  return TI_OK;
}

template <class T>
size_t ssd_scan_lds(int N) {
  const int kt = El<T>::KT, nk = (N + kt - 1) / kt * kt;
  return (size_t)2 * kSsdTok * (nk * sizeof(T) + 16) + 16 * (kSsdTok + 4) * 4 + 16 * 64 * 16 + kSsdTok * 8 + 3 * kSsdTok * 4;
}

template <class T>
int launch_ssd_scan(const ti_ssd_args& a, hipStream_t s) {
  const dim3 grid((a.vdim + 15) / 16, a.heads), blk(256);
  const size_t lds = ssd_scan_lds<T>(a.state_n);
  const int nt = (a.state_n + 15) / 16;
  if (nt <= 4) hipLaunchKernelGGL((ssd_scan_kernel<T, 1>), grid, blk, lds, s, a);
  else if (nt <= 8) hipLaunchKernelGGL((ssd_scan_kernel<T, 2>), grid, blk, lds, s, a);
  else hipLaunchKernelGGL((ssd_scan_kernel<T, 4>), grid, blk, lds, s, a);
  TI_LAUNCH_CHECK("ssd_scan_kernel");
  return TI_OK;
}

template <class T>
int recurrent_prepare() {
  const void* k[] = {(const void*)ssd_scan_kernel<T, 1>, (const void*)ssd_scan_kernel<T, 2>, (const void*)ssd_scan_kernel<T, 4>,
                     (const void*)ssd_norm_kernel<T>};
  for (const void* f : k)
    TI_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 163840 - 1024), "recurrent kernels' LDS");
  return TI_OK;
}

int gqa_prepare_all();   // gqa_attn.hip

inline bool rec_dtype(int dt) { return dt == TI_DT_BF16 || dt == TI_DT_F32; }

}  // namespace ti

extern "C" int ti_recurrent_prepare(void) {
  int rc = ti::gqa_prepare_all();
  if (!rc) rc = ti::recurrent_prepare<ti::bf16>();
  return rc ? rc : ti::recurrent_prepare<float>();
}

extern "C" int ti_conv(const ti_conv_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->x || !a->ring || !a->w || !a->b || !a->out || !a->pos || a->M < 1 || a->channels < 1 || a->taps < 1 ||
      a->c0 < 0 || a->c0 > a->channels || !rec_dtype(a->dtype) || a->ldx < a->channels ||
      (a->act != TI_CONV_LINEAR && a->act != TI_CONV_SILU))
    return ti_set_error(TI_ERR_ARG, "ti_conv: bad arguments");
  const int rest = a->channels - a->c0;
  if (rest && (a->bw < 1 || a->bwp < a->bw || rest % a->bw || a->o0 < a->c0))
    return ti_set_error(TI_ERR_ARG, "ti_conv: sections of %d in %d at %d", a->bw, a->bwp, a->o0);
  if (a->ldo < (rest ? a->o0 + rest / a->bw * a->bwp : a->channels) || (a->M + kConvRows - 1) / kConvRows > 65535)
    return ti_set_error(TI_ERR_ARG, "ti_conv: ldo %d, M %d", a->ldo, a->M);
  return a->dtype == TI_DT_BF16 ? launch_conv<bf16>(*a, (hipStream_t)stream) : launch_conv<float>(*a, (hipStream_t)stream);
}

static int ssd_check(const ti_ssd_args* a, const char* what) {
  using namespace ti;
  if (!a || !a->a || !a->dt || !a->dt_bias || !a->a_log || !a->d || !a->state || !a->y || !a->pos || a->M < 1 || a->heads < 1 ||
      a->heads > 65535 || a->vdim < 1 || a->state_n < 1 || a->groups < 1 || a->heads % a->groups || !rec_dtype(a->dtype) ||
      a->ldy < a->heads * a->vdim)
    return ti_set_error(TI_ERR_ARG, "%s: bad arguments", what);
  return TI_OK;
}

extern "C" int ti_ssd_step(const ti_ssd_args* a, ti_stream_t stream) {
  using namespace ti;
  const int rc = ssd_check(a, "ti_ssd_step");
  if (rc) return rc;
  if (!a->conv_w || !a->conv_b || !a->ring || a->taps < 1 || a->M > 65535 || a->state_n > 4096 ||
      a->lda < 2 * a->heads * a->vdim + 2 * a->groups * a->state_n)
    return ti_set_error(TI_ERR_ARG, "ti_ssd_step: bad arguments");
  return a->dtype == TI_DT_BF16 ? launch_ssd_step<bf16>(*a, (hipStream_t)stream) : launch_ssd_step<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_ssd_scan(const ti_ssd_args* a, ti_stream_t stream) {
  using namespace ti;
  const int rc = ssd_check(a, "ti_ssd_scan");
  if (rc) return rc;
  if (a->state_n > 256) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_ssd_scan: state %d (at most 256)", a->state_n);
  const int vec = a->dtype == TI_DT_BF16 ? 8 : 4, nk = (a->state_n + 4 * vec - 1) / (4 * vec) * (4 * vec);
  if (a->lda % vec || a->o0 % vec || a->o0 < a->heads * a->vdim || a->lda < a->o0 + 2 * a->groups * nk || a->slot0 < 0)
    return ti_set_error(TI_ERR_ARG, "ti_ssd_scan: lda %d, o0 %d", a->lda, a->o0);
  return a->dtype == TI_DT_BF16 ? launch_ssd_scan<bf16>(*a, (hipStream_t)stream) : launch_ssd_scan<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_ssd_norm(const ti_ssd_norm_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->y || !a->raw || !a->w || !a->out || a->M < 1 || a->inner < 1 || a->groups < 1 || a->inner % a->groups ||
      a->ldy < a->inner || a->ldo < a->inner || a->lda < a->inner + (a->ring ? a->channels : 0) || (a->ring && !a->pos) ||
      !rec_dtype(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_ssd_norm: bad arguments");
  if (a->inner > 32768) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_ssd_norm: %d values (at most 32768)", a->inner);
  const size_t lds = (size_t)a->inner * 4;
  if (a->dtype == TI_DT_BF16)
    hipLaunchKernelGGL(ssd_norm_kernel<bf16>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  else
    hipLaunchKernelGGL(ssd_norm_kernel<float>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  TI_LAUNCH_CHECK("ssd_norm_kernel");
  return TI_OK;
}

extern "C" int ti_lru_scan(const ti_lru_scan_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->ab || !a->y || !a->x || !a->out || !a->state || !a->ring || !a->pos || a->M < 1 || a->channels < 1 || a->taps < 1 ||
      a->taps > kLruSeg || a->ldy < a->channels || a->ldo < a->channels || !rec_dtype(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_lru_scan: bad arguments");
  const dim3 grid((a->channels + 15) / 16), blk(1024);
  if (a->dtype == TI_DT_BF16)
    hipLaunchKernelGGL(lru_scan_kernel<bf16>, grid, blk, 0, (hipStream_t)stream, *a);
  else
    hipLaunchKernelGGL(lru_scan_kernel<float>, grid, blk, 0, (hipStream_t)stream, *a);
  TI_LAUNCH_CHECK("lru_scan_kernel");
  return TI_OK;
}
