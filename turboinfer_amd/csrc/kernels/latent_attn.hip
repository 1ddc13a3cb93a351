// latent_attn.hip -- attention over a shared low-rank latent (ti_stack.h): keys and values of every
// head are linear images of one cached latent row per position, plus one rotated key part all heads
// share.
//
//   * latent_prep_kernel: RMS norms of the query latent and the cached latent, rotary of the shared
//     key part, cache append, sigmoid of the head gates -- one launch per layer.
//   * latent_decode_kernel: the up-projections are carried over to the query and output side, so 16
//     heads share every cached row: scores are one MFMA chain over [latent | rotated] with the heads as
//     the MFMA columns, the weighted sum a second one over the latent part.  Keys are split over
//     workgroups (splits) and over the waves of each.
//   * latent_prefill_kernel: prompt chunks, keys and values expanded per head into MFMA fragments
//     (dense.hip TI_DE_KFRAG / TI_DE_VFRAG); a workgroup owns 16 or 32 query rows of one head, its waves
//     split the keys.
// Scores, softmax and sums are fp32; the softmax denominator holds exp(sink) of the head once.
#include <algorithm>

#include "elem.hpp"

namespace ti {

template <class T>
__global__ __launch_bounds__(512) void latent_prep_kernel(const ti_latent_prep_args a) {
  extern __shared__ float r[];   // the fused projection's row
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x, pos = a.pos[m], n4 = (a.gate_off + a.heads + 3) >> 2;
  const f32x4* src = (const f32x4*)(a.a32 + (size_t)m * a.lda);
  for (int i = tid; i < n4; i += 512) ((f32x4*)r)[i] = src[i];
  __syncthreads();
  float q2 = 0.0f, c2 = 0.0f;
  for (int i = tid; i < a.q_rank; i += 512) q2 = fmaf(r[i], r[i], q2);
  for (int i = tid; i < a.kv_rank; i += 512) c2 = fmaf(r[a.lat_off + i], r[a.lat_off + i], c2);
  const float qi = 1.0f / sqrtf(block_sum(q2, red) / (float)a.q_rank + a.eps);
  const float ci = 1.0f / sqrtf(block_sum(c2, red) / (float)a.kv_rank + a.eps);
  T* cq = (T*)a.cq + (size_t)m * a.ldq;
  for (int i = tid; i < a.q_rank; i += 512) cq[i] = (T)(r[i] * qi * a.q_w[i]);
  T* row = (T*)a.cache + (size_t)(a.slot ? a.slot[m] : m) * a.slot_stride + (size_t)pos * (a.lat_p + a.rot_p);
  for (int i = tid; i < a.lat_p; i += 512) row[i] = i < a.kv_rank ? (T)(r[a.lat_off + i] * ci * a.c_w[i]) : (T)0.0f;
  for (int i = tid; i < a.rot_p / 2; i += 512) {
    float u = 0.0f, v = 0.0f;
    if (2 * i < a.rot_dim) u = r[a.rot_off + 2 * i];
    if (2 * i + 1 < a.rot_dim) v = r[a.rot_off + 2 * i + 1];
    const float2 cs = *(const float2*)(a.rope_cs + ((size_t)pos * (a.rot_p / 2) + i) * 2);
    row[a.lat_p + 2 * i] = (T)(u * cs.x - v * cs.y);
    row[a.lat_p + 2 * i + 1] = (T)(v * cs.x + u * cs.y);
  }
  for (int i = tid; i < a.heads; i += 512) a.gate[(size_t)m * a.heads + i] = sigmoidf(r[a.gate_off + i]);
}

// The VEC x VEC transpose a value fragment needs: in[j] = VEC consecutive value dims of key j of this
// lane group; out(c) = dim c of the VEC keys.
__device__ __forceinline__ bf16x8 gather_dim(const bf16x8* in, int c) {
  const u32x4* d = (const u32x4*)in;
  const uint32_t sel = (c & 1) ? 0x07060302u : 0x05040100u;   // the high or low halves of two dwords
  u32x4 o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = __builtin_amdgcn_perm(d[2 * j + 1][c >> 1], d[2 * j][c >> 1], sel);
  return __builtin_bit_cast(bf16x8, o);
}

// acc[c] += (value dims i * VEC + c, i = a-row) x (weights p of VEC-per-lane-group keys)
__device__ __forceinline__ void mma_values(f32x4* acc, const bf16x8* vin, bf16x8 p) {
#pragma unroll
  for (int c = 0; c < 8; ++c) acc[c] = mma(gather_dim(vin, c), p, acc[c]);
}
__device__ __forceinline__ void mma_values(f32x4* acc, const f32x4* vin, f32x4 p) {
#pragma unroll
  for (int s = 0; s < 4; ++s)
#pragma unroll
    for (int c = 0; c < 4; ++c) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(vin[s][c], p[s], acc[c], 0, 0, 0);
}

// Grid (splits, head tiles of 16, rows).  A block is 64 keys: wave w scores keys [16 w, +16), then sums
// value dims of its groups (wave, wave + 4, ...; a group is 16 * VEC dims) over all 64.  A wave's key
// fragments of a block (NKU k-tiles at a time) and, with one group per wave, its value rows -- the same
// cache lines -- are all in flight before the first product.
template <class T, int GPW>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(const ti_latent_attn_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, KB = 64, NVB = KB / KT, PLD = KB + 16 / (int)sizeof(T), NKU = 18, NQ = 5;
  extern __shared__ char lds[];
  const int split = blockIdx.x, ht = blockIdx.y, m = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int cw = a.lat_p + a.rot_p, nkt = cw / KT, lkt = a.lat_p / KT, G = a.lat_p / (16 * VEC) + (a.lat_p % (16 * VEC) != 0);
  V* qf = (V*)lds;                                  // [nkt][64]
  T* pb = (T*)(lds + (size_t)nkt * 1024);           // [16][PLD]
  float* sm = (float*)(pb + 16 * PLD);              // [4][16] wave maxima, then [4][16] wave sums
  const int pos = a.pos[m], head = ht * 16 + col;
  const T* cache = (const T*)a.cache + (size_t)(a.slot ? a.slot[m] : m) * a.slot_stride;
  auto load_q = [&](int kt) -> V {
    V v = {};
    if (head < a.heads && kt < nkt)
      v = kt < lkt ? *(const V*)((const T*)a.qa + ((size_t)m * a.heads + head) * a.lat_p + kt * KT + g * VEC)
                   : *(const V*)((const T*)a.q + ((size_t)m * a.heads + head) * a.ldqr + a.qr_off + (kt - lkt) * KT + g * VEC);
    return v;
  };
  f32x4 o[GPW][VEC];
#pragma unroll
  for (int i = 0; i < GPW; ++i)
#pragma unroll
    for (int c = 0; c < VEC; ++c) o[i][c] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float mr = -INFINITY, lr = 0.0f;
  const int nb = (pos + KB) / KB, bps = (nb + a.splits - 1) / a.splits, b0 = split * bps, b1 = min(nb, b0 + bps);
  V k[NKU], vin[GPW == 1 ? NVB : 1][VEC];
  auto load_k = [&](int b, int kt0) {
    const V* kp = (const V*)(cache + (size_t)(b * KB + wave * 16 + col) * cw) + g;
#pragma unroll
    for (int u = 0; u < NKU; ++u) k[u] = kp[min(kt0 + u, nkt - 1) * 4];
  };
  auto load_v = [&](int b) {   // (dims past the latent: clamped, not stored)
    if constexpr (GPW == 1) {
      const T* vd = cache + (size_t)(b * KB + g * VEC) * cw + min(wave * 16 * VEC + col * VEC, a.lat_p - VEC);
#pragma unroll
      for (int kb = 0; kb < NVB; ++kb)
#pragma unroll
        for (int j = 0; j < VEC; ++j) vin[kb][j] = *(const V*)(vd + (size_t)(kb * KT + j) * cw);
    }
  };
  {
    V q0[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) q0[i] = load_q(wave + 4 * i);
    if (b0 < b1) {
      load_k(b0, 0);
      load_v(b0);
    }
#pragma unroll
    for (int i = 0; i < NQ; ++i)
      if (wave + 4 * i < nkt) qf[(wave + 4 * i) * 64 + lane] = q0[i];
    for (int kt = wave + 4 * NQ; kt < nkt; kt += 4) qf[kt * 64 + lane] = load_q(kt);
  }
  lds_sync();
  for (int b = b0; b < b1; ++b) {
    const int k0 = b * KB + wave * 16;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    const T* vp = cache + (size_t)(b * KB + g * VEC) * cw;
    for (int kt0 = 0; kt0 < nkt; kt0 += NKU) {
      if (kt0) load_k(b, kt0);
#pragma unroll
      for (int u = 0; u < NKU; ++u)
        if (kt0 + u < nkt) s = mma(k[u], qf[(kt0 + u) * 64 + lane], s);
    }
    if (b + 1 < b1) load_k(b + 1, 0);   // the next block's keys fly through the softmax and the sums
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = k0 + 4 * g + r <= pos ? s[r] * a.scale : -INFINITY;
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
#pragma unroll
    for (int i = 0; i < GPW; ++i) {
      const int gi = wave + 4 * i;
      if (gi >= G) continue;
#pragma unroll
      for (int c = 0; c < VEC; ++c) o[i][c] *= alpha;
      const T* vd = vp + min(gi * 16 * VEC + col * VEC, a.lat_p - VEC);
#pragma unroll
      for (int kb = 0; kb < NVB; ++kb) {
        const V p = *(const V*)(pb + col * PLD + kb * KT + g * VEC);
        if constexpr (GPW == 1) {
          mma_values(o[i], vin[kb], p);
        } else {
          V v[VEC];
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[j] = *(const V*)(vd + (size_t)(kb * KT + j) * cw);
          mma_values(o[i], v, p);
        }
      }
    }
    if (b + 1 < b1) load_v(b + 1);
  }
  lr = lane_xor<16>(lr) + lr;
  lr = lane_xor<32>(lr) + lr;
  __syncthreads();
  if (lane < 16) sm[wave * 16 + col] = lr;
  __syncthreads();
  float l = sm[col] + sm[16 + col] + sm[32 + col] + sm[48 + col];
  if (head >= a.heads) return;
  const size_t row = a.splits > 1 ? (((size_t)m * a.splits + split) * a.heads + head) : (size_t)m * a.heads + head;
  if (a.splits > 1) {
    if (wave == 0 && lane < 16) {
      a.part_ml[row * 2] = mr;
      a.part_ml[row * 2 + 1] = l;
    }
    if (b0 >= b1) return;
  } else {   // the whole row: the sink joins the denominator here
    l += expf(a.sink[head] - mr);   // (a huge sink gives inf: weights 0)
  }
  const float inv = 1.0f / l;
  T* out = (T*)(a.splits > 1 ? a.part_o : a.out) + row * a.lat_p;
#pragma unroll
  for (int i = 0; i < GPW; ++i) {
    const int gi = wave + 4 * i;
    if (gi >= G) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = gi * 16 * VEC + (4 * g + r) * VEC;
      if (d >= a.lat_p) continue;
      V v;
#pragma unroll
      for (int c = 0; c < VEC; ++c) v[c] = (T)(o[i][c][r] * inv);
      *(V*)(out + d) = v;
    }
  }
}

// The splits' rows merged and carried through the value up-projection in one launch: grid (groups of
// NTW 16-dim value tiles, heads, tiles of 4 rows).  The merged rows go to LDS in operand fragments: a
// thread sums one 16-byte piece over a share of the splits (SG threads share a piece when there are
// few); then the 8 waves split the value tiles and k.
constexpr int kMaxSplits = 64, kOutRows = 4;
template <class T, int NTW>
__global__ __launch_bounds__(512) void latent_out_kernel(const ti_latent_out_args a) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, KP = 8 / NTW;
  extern __shared__ char lds[];
  __shared__ float wt[kOutRows][kMaxSplits];
  __shared__ f32x4 red[8][64];
  const int h = blockIdx.y, m0 = blockIdx.z * kOutRows, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int rows = min(kOutRows, a.M - m0), S = a.splits, nk = a.lat_p / KT, NT = (a.vdim + 15) >> 4;
  const int nt = blockIdx.x * NTW + wave % NTW, kpart = wave / NTW;
  const int C = a.lat_p / VEC;   // pieces per row
  V* xf = (V*)lds;               // [nk][64]
  float* part = (float*)(lds + (size_t)nk * 1024);   // [512][VEC] partial pieces
  if (wave < rows) {
    float mx = -INFINITY, l = 0.0f;
    if (lane < S) {
      const float2 ml = *(const float2*)(a.part_ml + (((size_t)(m0 + wave) * S + lane) * a.heads + h) * 2);
      mx = ml.x;
      l = ml.y;
    }
    const float sink = a.sink[h], mm = fmaxf(wave_max(mx), sink), e = l > 0.0f ? l * expf(mx - mm) : 0.0f;
    wt[wave][lane] = e / (group_sum<64>(e) + expf(sink - mm));
  }
  __syncthreads();
  const size_t sstride = (size_t)a.heads * a.lat_p;
  int SG = 1;
  while (SG < 8 && rows * C * SG * 2 <= 512 && SG * 2 <= S) SG *= 2;
  const int per = 512 / SG, ss = (S + SG - 1) / SG, sg = tid / per;
  for (int p0 = 0; p0 < rows * C; p0 += per) {
    const int p = p0 + tid % per;
    const bool live = p < rows * C;
    const int m = live ? p / C : 0, c = live ? p - m * C : 0;
    const T* po = (const T*)a.part_o + ((size_t)(m0 + m) * S * a.heads + h) * a.lat_p + c * VEC;
    float x[VEC] = {};
    const int s1 = min(S, (sg + 1) * ss);
    for (int s0 = sg * ss; s0 < s1; s0 += 8) {
      V v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = *(const V*)(po + (size_t)min(s0 + u, S - 1) * sstride);
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float f = s0 + u < s1 ? wt[m][s0 + u] : 0.0f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[e] = f != 0.0f ? fmaf(f, (float)v[u][e], x[e]) : x[e];   // (empty split: no row)
      }
    }
    if (SG > 1) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) part[tid * VEC + e] = x[e];
      __syncthreads();
      if (sg == 0)
        for (int g = 1; g < SG; ++g)
#pragma unroll
          for (int e = 0; e < VEC; ++e) x[e] += part[(g * per + tid) * VEC + e];
    }
    if (live && sg == 0) {
      V o;
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = (T)x[e];
      xf[(c >> 2) * 64 + (c & 3) * 16 + m] = o;
    }
  }
  const V* wp = (const V*)a.w + (size_t)h * (a.w_batch / VEC) + (size_t)min(nt, NT - 1) * nk * 64 + lane;
  __syncthreads();
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const int slot = (lane & 48) + min(lane & 15, rows - 1);
  for (int kt = kpart; kt < nk; kt += 4 * KP) {
    V w[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) w[u] = wp[(size_t)min(kt + u * KP, nk - 1) * 64];
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (kt + u * KP < nk) acc = mma(w[u], xf[(kt + u * KP) * 64 + slot], acc);
  }
  red[wave][lane] = acc;
  __syncthreads();
  if (kpart == 0 && (lane & 15) < rows && nt < NT) {
    const int m = lane & 15;
    f32x4 v = acc;
#pragma unroll
    for (int k = 1; k < KP; ++k) v += red[k * NTW + wave][lane];
    const float gt = a.gate[(size_t)(m0 + m) * a.heads + h];
    const int n0 = nt * 16 + 4 * (lane >> 4);
    T* o = (T*)a.out + (size_t)(m0 + m) * a.ldo + (size_t)h * a.vdim + n0;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n0 + i < a.vdim) o[i] = (T)(v[i] * gt);
  }
}

template <class T>
__global__ __launch_bounds__(128) void latent_merge_kernel(const ti_latent_attn_args a) {
  typedef typename El<T>::V V;
  constexpr int VEC = El<T>::VEC;
  const int h = blockIdx.x, m = blockIdx.y;
  const size_t row0 = (size_t)m * a.splits * a.heads + h;
  float mx = a.sink[h];
  for (int s = 0; s < a.splits; ++s) mx = fmaxf(mx, a.part_ml[(row0 + (size_t)s * a.heads) * 2]);
  float den = expf(a.sink[h] - mx);
  for (int s = 0; s < a.splits; ++s) {
    const float* ml = a.part_ml + (row0 + (size_t)s * a.heads) * 2;
    den += ml[1] * expf(ml[0] - mx);
  }
  for (int d = threadIdx.x * VEC; d < a.lat_p; d += 128 * VEC) {
    float acc[VEC] = {};
    for (int s = 0; s < a.splits; ++s) {
      const size_t r = row0 + (size_t)s * a.heads;
      const float w = a.part_ml[r * 2 + 1] * expf(a.part_ml[r * 2] - mx) / den;
      if (w == 0.0f) continue;   // (a split without keys holds no partial)
      const V v = *(const V*)((const T*)a.part_o + r * a.lat_p + d);
#pragma unroll
      for (int c = 0; c < VEC; ++c) acc[c] = fmaf(w, (float)v[c], acc[c]);
    }
    V o;
#pragma unroll
    for (int c = 0; c < VEC; ++c) o[c] = (T)acc[c];
    *(V*)((T*)a.out + ((size_t)m * a.heads + h) * a.lat_p + d) = o;
  }
}

// ------------------------------------------------------------------ prompt chunks
// Weights of 64 keys (4 key tiles, lane: query column, keys t * 16 + 4 g + r) x value fragments.
__device__ __forceinline__ void pv_block(f32x4& acc, const bf16x8* vf, const f32x4* p) {
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
__device__ __forceinline__ void pv_block(f32x4& acc, const f32x4* vf, const f32x4* p) {
#pragma unroll
  for (int t = 0; t < 4; ++t) acc = mma(vf[t], p[t], acc);
}

// A workgroup owns 16 * MQ rows of one head; its 4 waves take the 64-key blocks in turn and merge their
// sums at the end.  Each XCD gets a contiguous run of the (head, row block) list, so a head's keys and
// values stay in one L2; a head's last row blocks (most keys) start first.
template <class T, int MQ, int NV>
__global__ __launch_bounds__(256, NV > 8 ? 2 : 3) void latent_prefill_kernel(const ti_latent_prefill_args a, int row_blocks) {
  typedef typename El<T>::V V;
  constexpr int KT = El<T>::KT, VEC = El<T>::VEC, VB = 64 / KT;
  extern __shared__ char lds[];
  __shared__ float ml[2][4][MQ * 16];   // the waves' maxima, sums
  const int list = row_blocks * a.heads, per = (list + 7) >> 3;
  const int id = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per || id >= list) return;
  const int h = id / row_blocks, row0 = (row_blocks - 1 - id % row_blocks) * 16 * MQ;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int dkt = a.dim_p / KT, rkt = a.rot_p / KT, nkt = dkt + rkt, cw = a.lat_p + a.rot_p, nv = a.vdim_p >> 4;
  V* qf = (V*)lds;
  for (int i = wave; i < nkt * MQ; i += 4) {
    const int m = min(row0 + i % MQ * 16 + col, a.M - 1);
    qf[i * 64 + lane] = *(const V*)((const T*)a.q + ((size_t)m * a.heads + h) * (a.dim_p + a.rot_p) + i / MQ * KT + g * VEC);
  }
  __syncthreads();
  const V* kf = (const V*)a.kfrag + (size_t)h * a.key_blocks * dkt * 64 + lane;
  const V* vf = (const V*)a.vfrag + (size_t)h * nv * (a.key_blocks * 16 / KT) * 64 + lane;
  const V* rp = (const V*)((const T*)a.cache + a.lat_p + (size_t)col * cw) + g;
  f32x4 o[MQ][NV];
  float mr[MQ], lr[MQ];
#pragma unroll
  for (int q = 0; q < MQ; ++q) {
    mr[q] = a.sink[h];   // the sink: weight exp(sink - max), no value; counted by one wave
    lr[q] = wave == 0 && g == 0 ? 1.0f : 0.0f;
#pragma unroll
    for (int v = 0; v < NV; ++v) o[q][v] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  const int last = a.pos0 + min(row0 + 16 * MQ, a.M) - 1;   // the rows' last position
  for (int k0 = wave * 64; k0 <= last; k0 += 256) {
    f32x4 s[MQ][4];
#pragma unroll
    for (int q = 0; q < MQ; ++q)
#pragma unroll
      for (int t = 0; t < 4; ++t) s[q][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int kt = 0; kt < dkt; ++kt) {
      V k[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) k[t] = kf[((size_t)((k0 >> 4) + t) * dkt + kt) * 64];
#pragma unroll
      for (int q = 0; q < MQ; ++q) {
        const V qv = qf[(kt * MQ + q) * 64 + lane];
#pragma unroll
        for (int t = 0; t < 4; ++t) s[q][t] = mma(k[t], qv, s[q][t]);
      }
    }
    for (int kt = 0; kt < rkt; ++kt) {
      V k[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) k[t] = rp[(size_t)(k0 + t * 16) * cw / VEC + kt * 4];
#pragma unroll
      for (int q = 0; q < MQ; ++q) {
        const V qv = qf[((dkt + kt) * MQ + q) * 64 + lane];
#pragma unroll
        for (int t = 0; t < 4; ++t) s[q][t] = mma(k[t], qv, s[q][t]);
      }
    }
#pragma unroll
    for (int q = 0; q < MQ; ++q) {
      const int p = a.pos0 + row0 + q * 16 + col;
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
    const int nkb = a.key_blocks * 16 / KT;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      if (v < nv) {
        V vv[VB];
#pragma unroll
        for (int b = 0; b < VB; ++b) vv[b] = vf[((size_t)v * nkb + k0 / KT + b) * 64];
#pragma unroll
        for (int q = 0; q < MQ; ++q) pv_block(o[q][v], vv, s[q]);
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
    const int m = row0 + q * 16 + col;
    float mx = ml[0][0][q * 16 + col], l = 0.0f;
#pragma unroll
    for (int w = 1; w < 4; ++w) mx = fmaxf(mx, ml[0][w][q * 16 + col]);
#pragma unroll
    for (int w = 0; w < 4; ++w) l += ml[1][w][q * 16 + col] * expf(ml[0][w][q * 16 + col] - mx);
    const float f = expf(mr[q] - mx);
#pragma unroll
    for (int v = 0; v < NV; ++v) ob[(wave * NV + v) * 64 + lane] = o[q][v] * f;
    __syncthreads();
    if (m < a.M) {
      const float sc = a.gate[(size_t)m * a.heads + h] / l;
      T* out = (T*)a.out + (size_t)m * a.ldo + (size_t)h * a.vdim;
#pragma unroll
      for (int v0 = 0; v0 < NV; v0 += 4) {
        const int v = v0 + wave, d = v * 16 + 4 * g;
        if (d >= a.vdim) continue;
        f32x4 x = ob[v * 64 + lane];
#pragma unroll
        for (int w = 1; w < 4; ++w) x += ob[(w * NV + v) * 64 + lane];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (d + r < a.vdim) out[d + r] = (T)(x[r] * sc);
      }
    }
    if (q + 1 < MQ) __syncthreads();
  }
}

template <class T>
int launch_decode(const ti_latent_attn_args& a, hipStream_t s) {
  constexpr int VEC = El<T>::VEC;
  const int G = (a.lat_p + 16 * VEC - 1) / (16 * VEC), gpw = (G + 3) / 4;
  const size_t lds = (size_t)(a.lat_p + a.rot_p) / El<T>::KT * 1024 + (size_t)16 * (64 + 16 / sizeof(T)) * sizeof(T) + 64 * 4;
  const dim3 grid(a.splits, (a.heads + 15) / 16, a.M), blk(256);
  if (gpw == 1) hipLaunchKernelGGL((latent_decode_kernel<T, 1>), grid, blk, lds, s, a);
  else if (gpw == 2) hipLaunchKernelGGL((latent_decode_kernel<T, 2>), grid, blk, lds, s, a);
  else hipLaunchKernelGGL((latent_decode_kernel<T, 4>), grid, blk, lds, s, a);
  TI_LAUNCH_CHECK("latent_decode_kernel");
  if (a.splits > 1 && a.out) {
    hipLaunchKernelGGL(latent_merge_kernel<T>, dim3(a.heads, a.M), dim3(128), 0, s, a);
    TI_LAUNCH_CHECK("latent_merge_kernel");
  }
  return TI_OK;
}

template <class T>
int launch_prefill(const ti_latent_prefill_args& a, hipStream_t s) {
  const int nkt = (a.dim_p + a.rot_p) / El<T>::KT, nv = a.vdim_p / 16;
  // 32-row blocks where they still give every CU two workgroups
  const bool two = nkt <= 32 && nv <= 8 && (long)((a.M + 31) / 32) * a.heads >= 512;
  const int mq = two ? 2 : 1, rb = (a.M + 16 * mq - 1) / (16 * mq), nvp = nv <= 4 ? 4 : nv <= 8 ? 8 : 16;
  const size_t lds = (size_t)std::max(nkt * mq, 4 * nvp) * 1024;
  if (lds > 131072) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_latent_attn_prefill: head of %d + %d dims", a.dim_p, a.rot_p);
  const dim3 grid((unsigned)(((long)rb * a.heads + 7) / 8 * 8)), blk(256);
#define TI_LP(MQ, NV) hipLaunchKernelGGL((latent_prefill_kernel<T, MQ, NV>), grid, blk, lds, s, a, rb)
  if (two && nv <= 4) TI_LP(2, 4);
  else if (two) TI_LP(2, 8);
  else if (nv <= 4) TI_LP(1, 4);
  else if (nv <= 8) TI_LP(1, 8);
  else TI_LP(1, 16);
#undef TI_LP
  TI_LAUNCH_CHECK("latent_prefill_kernel");
  return TI_OK;
}

// Kernels whose dynamic LDS can pass 64 KiB (before any graph capture); at most 128 KiB is used.
template <class T>
int prepare() {
  const void* k[] = {(const void*)latent_decode_kernel<T, 1>, (const void*)latent_decode_kernel<T, 2>,
                     (const void*)latent_decode_kernel<T, 4>, (const void*)latent_prefill_kernel<T, 2, 4>,
                     (const void*)latent_prefill_kernel<T, 2, 8>, (const void*)latent_prefill_kernel<T, 1, 4>,
                     (const void*)latent_prefill_kernel<T, 1, 8>, (const void*)latent_out_kernel<T, 2>,
                     (const void*)latent_out_kernel<T, 4>, (const void*)latent_out_kernel<T, 8>, (const void*)latent_prefill_kernel<T, 1, 16>};
  for (const void* f : k)
    TI_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 131072), "latent attention LDS");
  return TI_OK;
}

bool dtype_ok(int dt) { return dt == TI_DT_BF16 || dt == TI_DT_F32; }

}  // namespace ti

extern "C" int ti_latent_prepare(void) {
  const int rc = ti::prepare<ti::bf16>();
  return rc ? rc : ti::prepare<float>();
}

extern "C" int ti_latent_prep(const ti_latent_prep_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->a32 || !a->q_w || !a->c_w || !a->rope_cs || !a->pos || !a->cq || !a->cache || !a->gate || a->M < 1 ||
      a->q_rank < 1 || a->kv_rank < 1 || a->rot_dim < 2 || a->rot_dim > a->rot_p || a->kv_rank > a->lat_p || a->ldq < a->q_rank ||
      a->heads < 1 || a->lda % 4 || a->lda < a->gate_off + a->heads || a->lda > 16000 || !dtype_ok(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_latent_prep: bad arguments");
  const size_t lds = (size_t)a->lda * 4;
  if (a->dtype == TI_DT_BF16)
    hipLaunchKernelGGL(latent_prep_kernel<bf16>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  else
    hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(a->M), dim3(512), lds, (hipStream_t)stream, *a);
  TI_LAUNCH_CHECK("latent_prep_kernel");
  return TI_OK;
}

extern "C" int ti_latent_attn_splits(int M, int heads, int max_seq) {
  // one or two workgroups per CU (splits cost a merge), none with less than one 64-key block
  const int wgs = M * ((heads + 15) / 16), cap = std::max(1, (max_seq + 63) / 64);
  return std::max(1, std::min({cap, ti::kMaxSplits, ((M == 1 ? 512 : 256) + wgs - 1) / std::max(1, wgs)}));
}

extern "C" int ti_latent_attn_decode(const ti_latent_attn_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->qa || !a->q || !a->cache || !a->pos || !a->sink || (!a->out && a->splits < 2) || a->M < 1 || a->M > 65535 ||
      a->heads < 1 || a->splits < 1 || a->splits > kMaxSplits || !dtype_ok(a->dtype) || (a->splits > 1 && (!a->part_o || !a->part_ml)))
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_decode: bad arguments");
  const int kt = a->dtype == TI_DT_BF16 ? 32 : 16, lim = a->dtype == TI_DT_BF16 ? 2048 : 1024;
  if (a->lat_p < kt || a->lat_p % kt || a->rot_p < kt || a->rot_p % kt || a->seq_p % 128 || a->ldqr % (kt / 4) || a->qr_off % (kt / 4))
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_decode: lat_p %d rot_p %d seq_p %d", a->lat_p, a->rot_p, a->seq_p);
  if (a->lat_p > lim || (a->lat_p + a->rot_p) / kt * 1024 > 122880)
    return ti_set_error(TI_ERR_UNSUPPORTED, "ti_latent_attn_decode: latent size %d (at most %d)", a->lat_p, lim);
  hipStream_t s = (hipStream_t)stream;
  if (a->dtype == TI_DT_BF16) return launch_decode<bf16>(*a, s);
  return launch_decode<float>(*a, s);
}

extern "C" int ti_latent_attn_out(const ti_latent_out_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->part_o || !a->part_ml || !a->sink || !a->w || !a->gate || !a->out || a->M < 1 || a->heads < 1 || a->heads > 65535 ||
      a->splits < 1 || a->splits > kMaxSplits || a->vdim < 1 || !dtype_ok(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_out: bad arguments");
  const int kt = a->dtype == TI_DT_BF16 ? 32 : 16;
  if (a->lat_p < kt || a->lat_p % kt || a->w_batch % (kt / 4) || a->ldo < a->heads * a->vdim)
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_out: lat_p %d ldo %d", a->lat_p, a->ldo);
  const size_t lds = (size_t)a->lat_p / kt * 1024 + (size_t)512 * (kt / 4) * 4;
  const int nt = (a->vdim + 15) / 16, z = (a->M + kOutRows - 1) / kOutRows;
  hipStream_t s = (hipStream_t)stream;
  // fewer value tiles per workgroup (the merge repeated) only while the chip is not filled
  auto launch = [&]<int NTW>() {
    const dim3 grid((nt + NTW - 1) / NTW, a->heads, z);
    if (a->dtype == TI_DT_BF16) hipLaunchKernelGGL((latent_out_kernel<bf16, NTW>), grid, dim3(512), lds, s, *a);
    else hipLaunchKernelGGL((latent_out_kernel<float, NTW>), grid, dim3(512), lds, s, *a);
  };
  if ((long)a->heads * z * nt <= 512) launch.template operator()<2>();
  else if ((long)a->heads * z * nt <= 1024) launch.template operator()<4>();
  else launch.template operator()<8>();
  TI_LAUNCH_CHECK("latent_out_kernel");
  return TI_OK;
}

extern "C" int ti_latent_attn_prefill(const ti_latent_prefill_args* a, ti_stream_t stream) {
  using namespace ti;
  if (!a || !a->q || !a->kfrag || !a->vfrag || !a->cache || !a->sink || !a->gate || !a->out || a->M < 1 || a->pos0 < 0 ||
      a->heads < 1 || a->heads > 65535 || !dtype_ok(a->dtype))
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_prefill: bad arguments");
  const int kt = a->dtype == TI_DT_BF16 ? 32 : 16;
  if (a->dim_p < kt || a->dim_p % kt || a->rot_p < kt || a->rot_p % kt || a->lat_p % kt || a->vdim_p % 16 || a->vdim > a->vdim_p ||
      a->ldo < a->heads * a->vdim || a->key_blocks % 8 || (long)a->key_blocks * 16 < (long)a->pos0 + a->M)
    return ti_set_error(TI_ERR_ARG, "ti_latent_attn_prefill: sizes");
  if (a->vdim_p > 256) return ti_set_error(TI_ERR_UNSUPPORTED, "ti_latent_attn_prefill: value size %d (at most 256)", a->vdim_p);
  hipStream_t s = (hipStream_t)stream;
  return a->dtype == TI_DT_BF16 ? launch_prefill<bf16>(*a, s) : launch_prefill<float>(*a, s);
}
