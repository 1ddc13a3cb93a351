// recurrent.hip -- recurrent mixers of the layer-stack models (ti_stack.h): short causal convolutions, the
// state-space recurrence (SSD) and the gated linear recurrence over prompt chunks and single tokens.
//
//   * conv_kernel: convolution over a prompt chunk and the slot's ring of earlier inputs.
//   * ssd_step_kernel: one token per row: convolution, step size, state update and output of a slice of
//     one head; the state is streamed once (read, update, write).
//   * ssd_scan_kernel: a prompt chunk in blocks of 64 tokens: scores C B^T under the decay mask, the state
//     carried in MFMA accumulators; products that involve decays or the state are fp32 MFMA.
//   * ssd_norm_kernel: SiLU gate and grouped RMS norm.
//   * lru_scan_kernel: S = a S + b per channel, the chunk cut into 64 segments scanned side by side.
//   * lru_step_kernel: one token per row: convolution, gate products, state update.
// Step sizes, decays, states and sums are fp32 (cumulated log decays fp64).
#include <algorithm>

#include "elem.hpp"

namespace ti {

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
      const T* ring = (const T*)a.ring + (size_t)a.slot0 * a.taps * a.channels + c0;
      float acc[VQ];
#pragma unroll
      for (int e = 0; e < VQ; ++e) acc[e] = a.b[c0 + e];
      for (int back = a.taps - 1; back >= 0; --back) {
        const int p = pos - back;
        if (p < 0) continue;
        const T* src = m >= back ? (const T*)a.x + (size_t)(m - back) * a.ldx + c0
                                 : ring + (size_t)(p % a.taps) * a.channels;
        const TV cur = *(const TV*)src;
#pragma unroll
        for (int e = 0; e < VQ; ++e) acc[e] = fmaf(a.w[(size_t)(a.taps - 1 - back) * a.channels + c0 + e], (float)cur[e], acc[e]);
      }
#pragma unroll
      for (int e = 0; e < VQ; ++e) o[e] = (T)(a.act == TI_CONV_SILU ? acc[e] * fast_sigmoid(acc[e]) : acc[e]);
    }
    *(TV*)((T*)a.out + (size_t)m * a.ldo + i0) = o;
  }
}

// The same for TAPS known and 16-byte places (VEC channels): a thread slides over R rows with all their inputs
// in flight.
template <class T, int TAPS>
__global__ __launch_bounds__(256) void conv_vec_kernel(const ti_conv_args a, int places) {
  typedef typename El<T>::V V;
  constexpr int VEC = El<T>::VEC, R = 8, NX = R + TAPS - 1;
  const int i0 = ((int)blockIdx.x * 64 + (int)(threadIdx.x & 63)) * VEC, m0 = ((int)blockIdx.y * 4 + (int)(threadIdx.x >> 6)) * R;
  if (i0 >= places || m0 >= a.M) return;
  int c0 = i0;
  if (i0 >= a.c0) {
    const int s = i0 - a.o0, r = s % a.bwp;
    c0 = s >= 0 && r < a.bw ? a.c0 + s / a.bwp * a.bw + r : -1;
    if (s < 0 && i0 < a.o0) return;
  }
  T* out = (T*)a.out + (size_t)m0 * a.ldo + i0;
  if (c0 < 0) {
    const V z = {};
    for (int r = 0; r < R && m0 + r < a.M; ++r) *(V*)(out + (size_t)r * a.ldo) = z;
    return;
  }
  const int pos = a.pos[m0];
  const T* ring = (const T*)a.ring + (size_t)a.slot0 * TAPS * a.channels + c0;
  V x[NX];   // x[i]: the input i - (TAPS - 1) rows after m0
#pragma unroll
  for (int i = 0; i < NX; ++i) {
    const int d = i - (TAPS - 1);
    const T* src = m0 + d >= 0 ? (const T*)a.x + (size_t)min(m0 + d, a.M - 1) * a.ldx + c0
                               : ring + (size_t)(max(pos + d, 0) % TAPS) * a.channels;
    x[i] = *(const V*)src;
  }
  typedef float FV __attribute__((ext_vector_type(VEC), aligned(16)));
  const FV b = *(const FV*)(a.b + c0);
  FV w[TAPS];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) w[j] = *(const FV*)(a.w + (size_t)j * a.channels + c0);
  const V z = {};
#pragma unroll
  for (int i = 0; i < TAPS - 1; ++i)
    if (pos + i - (TAPS - 1) < 0) x[i] = z;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    if (m0 + r >= a.M) return;
    V o;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      float acc = b[e];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) acc = fmaf(w[j][e], (float)x[r + j][e], acc);
      o[e] = (T)(a.act == TI_CONV_SILU ? acc * fast_sigmoid(acc) : acc);
    }
    *(V*)(out + (size_t)r * a.ldo) = o;
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
          v = fmaf(a.conv_w[(size_t)(a.taps - 1 - back) * channels + c], (float)ring[(size_t)((pos - back) % a.taps) * channels + c], v);
      v = fmaf(a.conv_w[(size_t)(a.taps - 1) * channels + c], (float)cur, v);
      // (the place written is read by no one: it held position pos - taps)
      if (own) ring[(size_t)(pos % a.taps) * channels + c] = cur;
      v = (float)(T)(v * fast_sigmoid(v));
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
// Running sums over the lanes of a wave (inclusive): within rows of 16 by lane shifts, then the rows' totals.
template <int N>
__device__ __forceinline__ double row_shift(double v) {   // lane l - N of the row; 0 before its start
  const uint64_t u = __builtin_bit_cast(uint64_t, v);
  const uint32_t lo = __builtin_amdgcn_update_dpp(0u, (uint32_t)u, 0x110 + N, 0xf, 0xf, true);
  const uint32_t hi = __builtin_amdgcn_update_dpp(0u, (uint32_t)(u >> 32), 0x110 + N, 0xf, 0xf, true);
  return __builtin_bit_cast(double, (uint64_t)hi << 32 | lo);
}
template <int L>
__device__ __forceinline__ double lane_value(double v) {
  const uint64_t u = __builtin_bit_cast(uint64_t, v);
  const uint32_t lo = __builtin_amdgcn_readlane((uint32_t)u, L), hi = __builtin_amdgcn_readlane((uint32_t)(u >> 32), L);
  return __builtin_bit_cast(double, (uint64_t)hi << 32 | lo);
}
__device__ __forceinline__ double wave_prefix(double v) {
  v += row_shift<1>(v);
  v += row_shift<2>(v);
  v += row_shift<4>(v);
  v += row_shift<8>(v);
  const double a = lane_value<15>(v), b = a + lane_value<31>(v), c = b + lane_value<47>(v);
  const int row = (int)(threadIdx.x & 63) >> 4;
  return v + (row == 0 ? 0.0 : row == 1 ? a : row == 2 ? b : c);
}

constexpr int kSsdTok = 64;

// Grid (slices of 16 value dimensions, heads).  Blocks of 64 tokens one after another; per block, with
// L(t, s) = exp(cum_t - cum_s):
//   y_t = sum_{s <= t} (C_t . B_s) L(t, s) dt_s x_s + exp(cum_t) S^T C_t + D x_t
//   S  <- exp(cum_last) S + sum_t L(last, t) dt_t B_t x_t^T
// Waves 0..3 carry the state, 16 * NTW of its rows each, tile i holding every NTW-th from the i-th (a lane's
// rows are 4 * NTW consecutive ones, its operands of all tiles come in one read): its share of every token's output, then
// its update.  Waves 4..7 own 16 tokens each: their scores within the block and the output.  Accumulators
// are the operand fragments of the next product (scores, state).  Waves 4..7 also load the next block and
// stage it at the end of this one (DB: into the other buffer); wave 4, which has the fewest scores, prepares
// its step sizes and decays.
template <class T, int NTW, bool DB>
__global__ __launch_bounds__(512, 1) void ssd_scan_kernel(const ti_ssd_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, PF = NTW * 16 / VEC < 4 ? NTW * 16 / VEC : 4, XLD = kSsdTok + 4, TH = 256;
  extern __shared__ char lds[];
  const int N = a.state_n, nk = (N + KT - 1) / KT * KT, np = (N + 3) & ~3;
  constexpr int LN = 64 * NTW, ld = LN + 16 / (int)sizeof(T);   // (places past nk stay 0)
  T* bc = (T*)lds;                       // [DB ? 2 : 1][B, C][64][ld]
  float* xts = (float*)(bc + (DB ? 4 : 2) * kSsdTok * ld);   // [2][16][XLD] values, transposed
  f32x4* reds = (f32x4*)(xts + 2 * 16 * XLD);                // [DB ? 2 : 1][4][4][64] the state's output shares
  // [2][5][64]: cum_t / ln 2 in two floats, dt, L(last, t) dt_t, exp(cum_t)
  float* coef = (float*)(reds + (DB ? 2 : 1) * 16 * 64);
  const int h = blockIdx.y, p0 = blockIdx.x * 16, tid = threadIdx.x, lane = tid & 63, col = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), grp = h / (a.heads / a.groups);
  const bool sw = wave < 4;
  const int w4 = wave & 3;
  const T* src = (const T*)a.a;
  const T* bsrc = src + a.o0 + (size_t)grp * nk;
  const size_t c_off = (size_t)a.groups * nk;
  const int ppr = nk / VEC, pieces = kSsdTok * ppr;   // 16-byte pieces per row, per block
  const float A = -expf(a.a_log[h]), bias = a.dt_bias[h], D = a.d[h];
  float* state = a.state + (((size_t)a.slot0 * a.heads + h) * a.vdim + p0) * np;
  const bool prow = p0 + col < a.vdim;
  const int n0 = 16 * NTW * (wave & 3);   // this wave's state rows
  f32x4 S[NTW];   // S[i][r]: state row n0 + NTW (4 g + r) + i, value dimension col
#pragma unroll
  for (int q = 0; q < NTW; ++q) {
    const int n = n0 + 4 * NTW * g + 4 * q;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (sw && a.pos[0] > 0 && prow && n < np) v = *(const f32x4*)(state + (size_t)col * np + n);
#pragma unroll
    for (int e = 0; e < 4; ++e) S[(4 * q + e) % NTW][(4 * q + e) / NTW] = v[e];
  }
  for (int i = tid; i < (DB ? 4 : 2) * kSsdTok * (LN - nk); i += 512)
    bc[i / (LN - nk) * ld + nk + i % (LN - nk)] = (T)0.0f;
  // Rows past the end repeat the last one: their step size is 0, so nothing of them is kept.  (The values
  // past a head's last dimension are its row's next elements; their results are not stored.)
  struct Regs {   // a block on its way
    V b[PF], c[PF];
    T x[4];
  } reg;
  int prow_[PF], pcol_[PF];
#pragma unroll
  for (int u = 0; u < PF; ++u) {
    prow_[u] = ((tid & 255) + u * TH) / ppr;
    pcol_[u] = ((tid & 255) + u * TH - prow_[u] * ppr) * VEC;
  }
  const T* xsrc = src + h * a.vdim + p0 + (tid & 3) * 4;
  auto load = [&](Regs& d, int m0) {
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      const T* s = bsrc + (size_t)min(m0 + prow_[u], a.M - 1) * a.lda + pcol_[u];
      d.b[u] = *(const V*)s;
      d.c[u] = *(const V*)(s + c_off);
    }
    const T* x = xsrc + (size_t)min(m0 + ((tid & 255) >> 2), a.M - 1) * a.lda;
#pragma unroll
    for (int e = 0; e < 4; ++e) d.x[e] = x[e];
  };
  auto stage = [&](const Regs& d, int buf, int m0) {
    T* B = bc + (DB ? buf : 0) * 2 * kSsdTok * ld;
    T* C = B + kSsdTok * ld;
#pragma unroll
    for (int u = 0; u < PF; ++u)
      if (prow_[u] < kSsdTok) {
        *(V*)(B + prow_[u] * ld + pcol_[u]) = d.b[u];
        *(V*)(C + prow_[u] * ld + pcol_[u]) = d.c[u];
      }
    for (int i = (tid & 255) + PF * TH; i < pieces; i += TH) {   // (long states)
      const int t = i / ppr, c = (i - t * ppr) * VEC;
      const T* s = bsrc + (size_t)min(m0 + t, a.M - 1) * a.lda + c;
      *(V*)(B + t * ld + c) = *(const V*)s;
      *(V*)(C + t * ld + c) = *(const V*)(s + c_off);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) xts[buf * 16 * XLD + ((tid & 3) * 4 + e) * XLD + ((tid & 255) >> 2)] = (float)d.x[e];
  };
  auto steps = [&](int buf, int m0, float raw) {   // one wave: step sizes, cumulated log decays
    const float dt = m0 + lane < a.M ? softplusf(raw + bias) : 0.0f;   // (past the end: no decay, no input)
    const double c = wave_prefix((double)(A * dt) * 1.4426950408889634), last = lane_value<63>(c);
    float* k = coef + buf * 5 * kSsdTok;
    const float hi = (float)c;
    k[lane] = hi;
    k[kSsdTok + lane] = (float)(c - hi);
    k[2 * kSsdTok + lane] = dt;
    k[3 * kSsdTok + lane] = __builtin_amdgcn_exp2f((float)(last - c)) * dt;
    k[4 * kSsdTok + lane] = __builtin_amdgcn_exp2f(hi);
  };
  auto raw_dt = [&](int m0) { return a.dt[(size_t)min(m0 + lane, a.M - 1) * a.heads + h]; };
  if (!sw) {
    load(reg, 0);
    stage(reg, 0, 0);
  }
  if (wave == 4) steps(0, 0, raw_dt(0));
  lds_sync();
  for (int m0 = 0, buf = 0; m0 < a.M; m0 += kSsdTok, buf ^= 1) {
    const T* Bs = bc + (DB ? buf : 0) * 2 * kSsdTok * ld;
    const T* Cs = Bs + kSsdTok * ld;
    const float *xt = xts + buf * 16 * XLD, *ch = coef + buf * 5 * kSsdTok, *cl = ch + kSsdTok, *dts = cl + kSsdTok, *wl = dts + kSsdTok,
                *ec = wl + kSsdTok;
    f32x4* red = reds + (DB ? buf : 0) * 16 * 64;
    const bool more = m0 + kSsdTok < a.M;
    float rdt = 0.0f;
    if (more && !sw) load(reg, m0 + kSsdTok);
    if (more && wave == 4) rdt = raw_dt(m0 + kSsdTok);
    const int tok = w4 * 16 + col;
    f32x4 y = {0.f, 0.f, 0.f, 0.f};
    float et = 0.0f;
    if (sw) {
      // the carried state's share of every token, over this wave's state rows
      f32x4 yi[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) yi[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
      typedef T TN __attribute__((ext_vector_type(4 * NTW), aligned(4 * NTW * sizeof(T) < 16 ? 4 * NTW * sizeof(T) : 16)));
      TN c[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) c[t] = *(const TN*)(Cs + (t * 16 + col) * ld + n0 + 4 * NTW * g);
#pragma unroll
      for (int k = 0; k < 4 * NTW; ++k)
#pragma unroll
        for (int t = 0; t < 4; ++t)
          yi[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(S[k % NTW][k / NTW], (float)c[t][k], yi[t], 0, 0, 0);
#pragma unroll
      for (int t = 0; t < 4; ++t) red[(w4 * 4 + t) * 64 + lane] = yi[t];
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
      for (int i = 0; i < NTW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][r] *= last;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        typedef T TB __attribute__((ext_vector_type(NTW)));
        TB b[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) b[r] = *(const TB*)(Bs + (t * 16 + 4 * g + r) * ld + n0 + NTW * col);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int i = 0; i < NTW; ++i) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32((float)b[r][i], wx[t][r], S[i], 0, 0, 0);
      }
    } else {
      // scores of this wave's tokens with the block's earlier ones, decayed, times their inputs
      et = ec[tok];
      // (two or all four tiles of earlier tokens side by side; those past the wave's own tokens are masked)
      const float th = ch[tok], tl = cl[tok];
      f32x4 y2 = {0.f, 0.f, 0.f, 0.f};
      auto scores = [&]<int NS>() {
        f32x4 sc[NS];
#pragma unroll
        for (int i = 0; i < NS; ++i) sc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const T *crow = Cs + tok * ld + g * VEC, *brow = Bs + col * ld + g * VEC;
        constexpr int UF = 2;
        for (int k = 0; k < nk; k += UF * KT) {
          V cf[UF], bf[UF][NS];
#pragma unroll
          for (int f = 0; f < UF; ++f) {
            const int kf = min(k + f * KT, LN - KT);   // (past nk: zeros)
            cf[f] = *(const V*)(crow + kf);
#pragma unroll
            for (int i = 0; i < NS; ++i) bf[f][i] = *(const V*)(brow + i * 16 * ld + kf);
          }
#pragma unroll
          for (int f = 0; f < UF; ++f)
#pragma unroll
            for (int i = 0; i < NS; ++i) sc[i] = mma(bf[f][i], cf[f], sc[i]);
        }
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          const int s0 = i * 16 + 4 * g;
          const f32x4 sh = *(const f32x4*)(ch + s0), sl = *(const f32x4*)(cl + s0), d = *(const f32x4*)(dts + s0);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float e = __builtin_amdgcn_exp2f((th - sh[r]) + (tl - sl[r]));
            sc[i][r] = s0 + r <= tok ? sc[i][r] * (e * d[r]) : 0.0f;
          }
        }
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          const f32x4 x = *(const f32x4*)(xt + col * XLD + i * 16 + 4 * g);
          if (i & 1) y2 = mma(x, sc[i], y2);
          else y = mma(x, sc[i], y);
        }
      };
      if (w4 < 2) scores.template operator()<2>();
      else scores.template operator()<4>();
      y += y2;
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = fmaf(D, xt[(4 * g + r) * XLD + tok], y[r]);
      if (wave == 4 && more) steps(buf ^ 1, m0 + kSsdTok, rdt);
    }
    if (DB && more && !sw) stage(reg, buf ^ 1, m0 + kSsdTok);
    lds_sync();
    if (!sw && m0 + tok < a.M) {   // out: this wave's tokens, dimensions 4 g + r
      f32x4 z = red[w4 * 64 + lane];
#pragma unroll
      for (int w = 1; w < 4; ++w) z += red[(w * 4 + w4) * 64 + lane];
      float* o = a.y + (size_t)(m0 + tok) * a.ldy + h * a.vdim + p0 + 4 * g;
      f32x4 v;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = fmaf(et, z[r], y[r]);
      if (p0 + 4 * g + 4 <= a.vdim && ((a.ldy | a.vdim) & 3) == 0) {
        *(f32x4*)o = v;
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (p0 + 4 * g + r < a.vdim) o[r] = v[r];
      }
    }
    if (!DB && more) {
      if (!sw) stage(reg, buf ^ 1, m0 + kSsdTok);
      lds_sync();
    }
  }
  if (!sw) return;
#pragma unroll
  for (int q = 0; q < NTW; ++q) {
    const int n = n0 + 4 * NTW * g + 4 * q;
    f32x4 v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = S[(4 * q + e) % NTW][(4 * q + e) / NTW];
    if (prow && n < np) *(f32x4*)(state + (size_t)col * np + n) = v;
  }
}

// ------------------------------------------------------------------ gate and norm
// Grid (groups, rows).
__device__ __forceinline__ float gated(float y, float z) { return y * z * fast_sigmoid(z); }
template <class T>
__device__ __forceinline__ void ssd_ring(const ti_ssd_norm_args& a, int m, const T* raw) {
  if (!a.ring || blockIdx.x || m < a.M - (a.taps - 1)) return;
  T* ring = (T*)a.ring + ((size_t)a.slot0 * a.taps + a.pos[m] % a.taps) * a.channels;
  for (int i = threadIdx.x; i < a.channels; i += blockDim.x) ring[i] = raw[a.inner + i];
}
template <class T>
__global__ __launch_bounds__(512) void ssd_norm_kernel(const ti_ssd_norm_args a) {
  extern __shared__ float v[];
  __shared__ float red[8];
  const int m = blockIdx.y, tid = threadIdx.x, per = a.inner / a.groups, i0 = blockIdx.x * per;
  const float* y = a.y + (size_t)m * a.ldy + i0;
  const T* raw = (const T*)a.raw + (size_t)m * a.lda;
  T* out = (T*)a.out + (size_t)m * a.ldo + i0;
  float q = 0.0f;
  for (int i = tid; i < per; i += 512) {
    v[i] = gated(y[i], (float)raw[i0 + i]);
    q = fmaf(v[i], v[i], q);
  }
  const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)per + a.eps);
  for (int i = tid; i < per; i += 512) out[i] = (T)(v[i] * inv * a.w[i0 + i]);
  ssd_ring<T>(a, m, raw);
}
// Groups of a multiple of 4 values, at most 4 * TH * NC: held in registers, every load in flight at once.
template <class T, int TH, int NC>
__global__ __launch_bounds__(TH) void ssd_norm_vec_kernel(const ti_ssd_norm_args a) {
  typedef typename El<T>::Q Q;
  __shared__ float red[TH / 64];
  const int m = blockIdx.y, tid = threadIdx.x, per = a.inner / a.groups, i0 = blockIdx.x * per, n4 = per >> 2;
  const T* raw = (const T*)a.raw + (size_t)m * a.lda;
  const f32x4 *y = (const f32x4*)(a.y + (size_t)m * a.ldy + i0), *w = (const f32x4*)(a.w + i0);
  f32x4 v[NC], wv[NC];
  Q z[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = min(tid + c * TH, n4 - 1);
    v[c] = y[i];
    z[c] = *(const Q*)(raw + i0 + 4 * i);
    wv[c] = w[i];
  }
  float q = 0.0f;
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[c][e] = gated(v[c][e], (float)z[c][e]);
      if (tid + c * TH < n4) q = fmaf(v[c][e], v[c][e], q);
    }
  const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)per + a.eps);
#pragma unroll
  for (int c = 0; c < NC; ++c) {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[c][e] *= inv * wv[c][e];
    if (tid + c * TH < n4) *(Q*)((T*)a.out + (size_t)m * a.ldo + i0 + 4 * (tid + c * TH)) = quad<T>(v[c]);
  }
  ssd_ring<T>(a, m, raw);
}

// ------------------------------------------------------------------ gated linear recurrence over a chunk
// 16 channels x 64 segments of at most LEN rows, held in registers: every segment's product and end value
// from zero, one scan over the segments, then the segments again from their start values.
constexpr int kLruSeg = 64;
template <class T, int LEN>
__global__ __launch_bounds__(1024) void lru_scan_kernel(const ti_lru_scan_args a, int row0, int rows) {
  __shared__ float sa[kLruSeg][16], sb[kLruSeg][16];
  const int tid = threadIdx.x, ch = tid & 15, seg = tid >> 4, c = blockIdx.x * 16 + ch, cc = min(c, a.channels - 1);
  const int len = (rows + kLruSeg - 1) / kLruSeg, end = row0 + rows, r0 = row0 + seg * len, n = min(end - r0, len);
  const float2* ab = (const float2*)a.ab + cc;
  const T* y = (const T*)a.y + cc;
  float2 v[LEN];
  T yv[LEN];
#pragma unroll
  for (int u = 0; u < LEN; ++u) v[u] = ab[(size_t)min(r0 + u, end - 1) * a.channels];
#pragma unroll
  for (int u = 0; u < LEN; ++u) yv[u] = y[(size_t)min(r0 + u, end - 1) * a.ldy];
  float pa = 1.0f, pb = 0.0f;
#pragma unroll
  for (int u = 0; u < LEN; ++u)
    if (u < n) {
      pa *= v[u].x;
      pb = fmaf(v[u].x, pb, v[u].y);
    }
  sa[seg][ch] = pa;
  sb[seg][ch] = pb;
  lds_sync();
  float* st = a.state + (size_t)a.slot0 * a.channels + cc;
  if (seg == 0) {   // sb becomes every segment's start value
    float s = a.pos[row0] > 0 ? *st : 0.0f;
#pragma unroll 16
    for (int k = 0; k < kLruSeg; ++k) {
      const float x = sa[k][ch], e = sb[k][ch];
      sb[k][ch] = s;
      s = fmaf(x, s, e);
    }
    if (c < a.channels) *st = s;
  }
  lds_sync();
  if (c >= a.channels) return;
  float s = sb[seg][ch];
  T* out = (T*)a.out + c;
#pragma unroll
  for (int u = 0; u < LEN; ++u)
    if (u < n) {
      s = fmaf(v[u].x, s, v[u].y);
      out[(size_t)(r0 + u) * a.ldo] = (T)(s * (float)yv[u]);
    }
  const int back = seg;   // the last taps - 1 rows' inputs enter the ring
  if (back < a.taps - 1 && rows - 1 - back >= 0) {
    const int m = end - 1 - back;
    ((T*)a.ring)[((size_t)a.slot0 * a.taps + a.pos[m] % a.taps) * a.channels + c] = ((const T*)a.x)[(size_t)m * a.ldy + c];
  }
}

// ------------------------------------------------------------------ gated linear recurrence, one token per row
// Grid (groups of 4 tiles of 16 gate columns = 8 channels, blocks, tiles of 16 rows).  Every workgroup makes
// its rows' convolution of the whole block in LDS, while the first weight fragments, the states and the
// epilogue's operands are in flight; each wave multiplies its tile and steps its channels' states.  VQ:
// channels a thread convolves at a time.
template <class T, int VQ>
__global__ __launch_bounds__(256) void lru_step_kernel(const ti_lru_step_args a) {
  typedef typename El<T>::V V;
  typedef T TV __attribute__((ext_vector_type(VQ)));
  typedef float FV __attribute__((ext_vector_type(VQ), aligned(VQ > 1 ? 16 : 4)));
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, PF = 8;
  extern __shared__ char lds[];
  const int blk = blockIdx.y, m0 = blockIdx.z * 16, rows = min(16, a.M - m0), bw = a.channels / a.blocks, tiles = (2 * bw + 15) >> 4;
  const int kp = ti_kpad<T>(bw), nk = kp / KT, ld = kp + VEC, c0 = blk * bw;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nt = blockIdx.x * 4 + wave;
  T* us = (T*)lds;   // [16][ld]
  const V* wp = (const V*)a.gates + ((size_t)blk * tiles + min(nt, tiles - 1)) * nk * 64 + lane;
  V wf[PF];
#pragma unroll
  for (int u = 0; u < PF; ++u) wf[u] = wp[(size_t)min(u, nk - 1) * 64];
  // this lane's results: row r, channels j0 and j0 + 1 of the block
  const int r = min(lane & 15, rows - 1), m = m0 + r, j0 = nt * 8 + 2 * (lane >> 4);
  const int rpos = a.pos[m], rslot = a.slot ? a.slot[m] : m;
  float rb[2], ib[2], rate[2], st[2];
  T y[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int c = c0 + min(j0 + i, bw - 1);
    rb[i] = a.gate_b[2 * c];
    ib[i] = a.gate_b[2 * c + 1];
    rate[i] = a.lru_rate[c];
    st[i] = a.state[(size_t)rslot * a.channels + c];
    y[i] = ((const T*)a.y)[(size_t)m * a.ldx + c];
  }
  for (int i = tid; i < rows * (kp / VQ); i += 256) {
    const int q = i / (kp / VQ), c = (i - q * (kp / VQ)) * VQ, mq = m0 + q;
    TV o;
#pragma unroll
    for (int e = 0; e < VQ; ++e) o[e] = (T)0.0f;
    if (c < bw) {   // (bw is a multiple of VQ)
      const int pos = a.pos[mq], ch = c0 + c;
      T* ring = (T*)a.ring + (size_t)(a.slot ? a.slot[mq] : mq) * a.taps * a.channels + ch;
      const TV cur = *(const TV*)((const T*)a.x + (size_t)mq * a.ldx + ch);
      FV acc = *(const FV*)(a.conv_b + ch);
      for (int b0 = a.taps - 1; b0 >= 0; b0 -= 4) {   // four taps' loads in flight
        TV v[4];
        FV w[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int back = max(b0 - u, 0);
          v[u] = cur;
          if (back && pos >= back) v[u] = *(const TV*)(ring + (size_t)((pos - back) % a.taps) * a.channels);
          w[u] = *(const FV*)(a.conv_w + (size_t)(a.taps - 1 - back) * a.channels + ch);
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (b0 - u >= 0 && pos >= b0 - u)
#pragma unroll
            for (int e = 0; e < VQ; ++e) acc[e] = fmaf(w[u][e], (float)v[u][e], acc[e]);
      }
      // (the place written is read by no one: it held position pos - taps)
      if (blockIdx.x == 0) *(TV*)(ring + (size_t)(pos % a.taps) * a.channels) = cur;
#pragma unroll
      for (int e = 0; e < VQ; ++e) o[e] = (T)acc[e];
    }
    *(TV*)(us + q * ld + c) = o;
  }
  lds_sync();
  const V* up = (const V*)(us + r * ld + (lane >> 4) * VEC);
  f32x4 g = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int u = 0; u < PF; ++u)
    if (u < nk) g = mma(wf[u], up[u * (KT / VEC)], g);
  for (int kt = PF; kt < nk; ++kt) g = mma(wp[(size_t)kt * 64], up[kt * (KT / VEC)], g);
  if ((lane & 15) >= rows || nt >= tiles) return;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int j = j0 + i, c = c0 + j;
    if (j >= bw) return;
    const float2 k = lru_coef(g[2 * i] + rb[i], g[2 * i + 1] + ib[i], rate[i], (float)us[r * ld + j]);
    const float s = rpos > 0 ? fmaf(k.x, st[i], k.y) : k.y;
    a.state[(size_t)rslot * a.channels + c] = s;
    ((T*)a.out)[(size_t)m * a.ldo + c] = (T)(s * (float)y[i]);
  }
}

// ------------------------------------------------------------------ launchers
template <class T>
int launch_conv(const ti_conv_args& a, hipStream_t s) {
  const int sections = a.c0 < a.channels ? (a.channels - a.c0) / a.bw : 0, places = sections ? a.o0 + sections * a.bwp : a.channels;
  const int rb = (a.M + kConvRows - 1) / kConvRows;
  const int all = a.channels | a.ldx | a.ldo | a.c0 | (sections ? a.o0 | a.bw | a.bwp : 0);
  constexpr int VEC = El<T>::VEC;
  if (all % VEC == 0 && a.taps >= 2 && a.taps <= 4) {
    const dim3 grid((places / VEC + 63) / 64, (a.M + 31) / 32), blk(256);
    if (a.taps == 2) hipLaunchKernelGGL((conv_vec_kernel<T, 2>), grid, blk, 0, s, a, places);
    else if (a.taps == 3) hipLaunchKernelGGL((conv_vec_kernel<T, 3>), grid, blk, 0, s, a, places);
    else hipLaunchKernelGGL((conv_vec_kernel<T, 4>), grid, blk, 0, s, a, places);
    TI_LAUNCH_CHECK("conv_vec_kernel");
    return TI_OK;
  }
  if (all % 4 == 0)
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

constexpr size_t kSsdLds = 163840 - 1024;

template <class T>
size_t ssd_scan_lds(int ntw, bool db) {
  return (size_t)(db ? 4 : 2) * kSsdTok * (64 * ntw * sizeof(T) + 16) + 2 * 16 * (kSsdTok + 4) * 4 + (db ? 2 : 1) * 16 * 64 * 16 +
         2 * 5 * kSsdTok * 4;
}

template <class T>
int launch_ssd_scan(const ti_ssd_args& a, hipStream_t s) {
  const dim3 grid((a.vdim + 15) / 16, a.heads), blk(512);
  const int ntw = a.state_n <= 64 ? 1 : a.state_n <= 128 ? 2 : 4;
  const bool db = ssd_scan_lds<T>(ntw, true) <= kSsdLds;
  const size_t lds = ssd_scan_lds<T>(ntw, db);
#define TI_SS(NTW)                                                                       \
  if (db) hipLaunchKernelGGL((ssd_scan_kernel<T, NTW, true>), grid, blk, lds, s, a);     \
  else hipLaunchKernelGGL((ssd_scan_kernel<T, NTW, false>), grid, blk, lds, s, a)
  if (ntw == 1) TI_SS(1);
  else if (ntw == 2) TI_SS(2);
  else TI_SS(4);
#undef TI_SS
  TI_LAUNCH_CHECK("ssd_scan_kernel");
  return TI_OK;
}

template <class T>
int recurrent_prepare() {
  const void* k[] = {(const void*)ssd_scan_kernel<T, 1, true>,  (const void*)ssd_scan_kernel<T, 2, true>,
                     (const void*)ssd_scan_kernel<T, 4, true>,  (const void*)ssd_scan_kernel<T, 1, false>,
                     (const void*)ssd_scan_kernel<T, 2, false>, (const void*)ssd_scan_kernel<T, 4, false>,
                     (const void*)ssd_norm_kernel<T>};
  const void* step[] = {(const void*)lru_step_kernel<T, 1>, (const void*)lru_step_kernel<T, El<T>::VEC>};
  for (const void* f : k)
    TI_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSsdLds), "recurrent kernels' LDS");
  for (const void* f : step)   // (16 rows of ti_lru_step_max_block inputs; the kernel's own LDS beside them)
    TI_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 16 * (4096 + 8) * 2), "recurrent kernels' LDS");
  return TI_OK;
}

template <class T>
int launch_ssd_norm(const ti_ssd_norm_args& a, hipStream_t s) {
  const int per = a.inner / a.groups;
  const dim3 grid(a.groups, a.M);
  const bool vec = ((per | a.ldy | a.lda | a.ldo) & 3) == 0 && per <= 8192;
  if (vec && per <= 1024) hipLaunchKernelGGL((ssd_norm_vec_kernel<T, 256, 1>), grid, dim3(256), 0, s, a);
  else if (vec && per <= 4096) hipLaunchKernelGGL((ssd_norm_vec_kernel<T, 512, 2>), grid, dim3(512), 0, s, a);
  else if (vec) hipLaunchKernelGGL((ssd_norm_vec_kernel<T, 1024, 2>), grid, dim3(1024), 0, s, a);
  else hipLaunchKernelGGL(ssd_norm_kernel<T>, grid, dim3(512), (size_t)per * 4, s, a);
  TI_LAUNCH_CHECK("ssd_norm_kernel");
  return TI_OK;
}

template <class T>
int launch_lru_scan(const ti_lru_scan_args& a, hipStream_t s) {
  const dim3 grid((a.channels + 15) / 16), blk(1024);
  for (int r = 0; r < a.M; r += 32 * kLruSeg) {
    const int rows = std::min(a.M - r, 32 * kLruSeg), len = (rows + kLruSeg - 1) / kLruSeg;
    if (len <= 4) hipLaunchKernelGGL((lru_scan_kernel<T, 4>), grid, blk, 0, s, a, r, rows);
    else if (len <= 8) hipLaunchKernelGGL((lru_scan_kernel<T, 8>), grid, blk, 0, s, a, r, rows);
    else if (len <= 16) hipLaunchKernelGGL((lru_scan_kernel<T, 16>), grid, blk, 0, s, a, r, rows);
    else hipLaunchKernelGGL((lru_scan_kernel<T, 32>), grid, blk, 0, s, a, r, rows);
  }
  TI_LAUNCH_CHECK("lru_scan_kernel");
  return TI_OK;
}

template <class T>
int launch_lru_step(const ti_lru_step_args& a, hipStream_t s) {
  constexpr int VEC = El<T>::VEC;
  const int bw = a.channels / a.blocks;
  const dim3 grid((2 * bw + 63) / 64, a.blocks, (a.M + 15) / 16), blk(256);
  const size_t lds = (size_t)16 * (ti_kpad<T>(bw) + VEC) * sizeof(T);
  if ((bw | a.ldx) % VEC == 0) hipLaunchKernelGGL((lru_step_kernel<T, VEC>), grid, blk, lds, s, a);
  else hipLaunchKernelGGL((lru_step_kernel<T, 1>), grid, blk, lds, s, a);
  TI_LAUNCH_CHECK("lru_step_kernel");
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

extern "C" int ti_lru_step_max_block(int dtype) { return dtype == TI_DT_BF16 ? 4096 : 2048; }

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
  if (!a || !a->y || !a->raw || !a->w || !a->out || a->M < 1 || a->M > 65535 || a->inner < 1 || a->groups < 1 || a->inner % a->groups ||
      a->ldy < a->inner || a->ldo < a->inner || a->lda < a->inner + (a->ring ? a->channels : 0) || (a->ring && !a->pos) ||
      !rec_dtype(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_ssd_norm: bad arguments");
  if (a->inner > 32768) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_ssd_norm: %d values (at most 32768)", a->inner);
  return a->dtype == TI_DT_BF16 ? launch_ssd_norm<bf16>(*a, (hipStream_t)stream) : launch_ssd_norm<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_lru_scan(const ti_lru_scan_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->ab || !a->y || !a->x || !a->out || !a->state || !a->ring || !a->pos || a->M < 1 || a->channels < 1 || a->taps < 1 ||
      a->taps > kLruSeg || a->ldy < a->channels || a->ldo < a->channels || !rec_dtype(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_lru_scan: bad arguments");
  return a->dtype == TI_DT_BF16 ? launch_lru_scan<bf16>(*a, (hipStream_t)stream) : launch_lru_scan<float>(*a, (hipStream_t)stream);
}

extern "C" int ti_lru_step(const ti_lru_step_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->x || !a->y || !a->ring || !a->conv_w || !a->conv_b || !a->gates || !a->gate_b || !a->lru_rate || !a->state || !a->out ||
      !a->pos || a->M < 1 || a->channels < 1 || a->blocks < 1 || a->blocks > 65535 || a->channels % a->blocks || a->taps < 1 ||
      a->ldx < a->channels || a->ldo < a->channels || !rec_dtype(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_lru_step: bad arguments");
  if (a->channels / a->blocks > ti_lru_step_max_block(a->dtype))
    return ti_set_error(TI_ERR_UNSUPPORTED, "ti_lru_step: blocks of %d channels", a->channels / a->blocks);
  return a->dtype == TI_DT_BF16 ? launch_lru_step<bf16>(*a, (hipStream_t)stream) : launch_lru_step<float>(*a, (hipStream_t)stream);
}
