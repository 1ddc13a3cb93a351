// elem.hpp -- element types of the layer-stack kernels: bf16 and fp32 behind one fragment shape.
//
// A fragment is 64 lanes x 16 bytes (ti_stack.h): lane l holds row (l & 15) and VEC consecutive k
// starting at VEC * (l >> 4) of a k-tile of KT.  bf16: one v_mfma_f32_16x16x32_bf16 per fragment
// pair; fp32: four v_mfma_f32_16x16x4_f32, the i-th taking k = VEC * (l >> 4) + i from every lane
// group (both operands use the same k order, so the sum is the same set of products).
// Result of mma(a, b): lane l, register i = a-row 4 * (l >> 4) + i, b-row (l & 15).
#pragma once

#include "common.hpp"
#include "ti_stack.h"

namespace ti {

typedef __bf16 bf16;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));

template <class T>
struct El;
template <>
struct El<bf16> {
  static constexpr int VEC = 8, KT = 32;
  typedef bf16x8 V;
  typedef bf16x4 Q;   // 4 consecutive elements
};
template <>
struct El<float> {
  static constexpr int VEC = 4, KT = 16;
  typedef f32x4 V;
  typedef f32x4 Q;
};

__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}

// ti_stack_kpad of the element type
template <class T>
__host__ __device__ __forceinline__ int ti_kpad(int K) {
  constexpr int u = 2 * El<T>::KT;
  return (K + u - 1) / u * u;
}

template <class T>
__device__ __forceinline__ typename El<T>::Q quad(f32x4 v) {
  typename El<T>::Q q;
#pragma unroll
  for (int i = 0; i < 4; ++i) q[i] = (T)v[i];
  return q;
}

// LDS hand-off between the waves of a workgroup that leaves their global loads in flight (a plain
// __syncthreads() may wait for them).
__device__ __forceinline__ void lds_sync() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// block-wide sum of one float per thread; every thread gets it.  red: one float per wave.
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = group_sum<64>(v);
  const int wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  lds_sync();   // red may still be read from the previous sum
  if ((threadIdx.x & 63) == 0) red[wave] = v;
  lds_sync();
  float s = 0.0f;
  for (int i = 0; i < nw; ++i) s += red[i];
  return s;
}

// All-reduce maximum over the wave (group_sum's lane exchanges).
__device__ __forceinline__ float wave_max(float v) {
  v = fmaxf(v, lane_xor<1>(v));
  v = fmaxf(v, lane_xor<2>(v));
  v = fmaxf(v, dpp_f<0x141>(v));
  v = fmaxf(v, dpp_f<0x140>(v));
  return xor32_max(xor16_max(v));
}

// Routing of one row over E <= 64 experts by one wave, lane l holding expert l's logit v: softmax over
// the experts, the `top` largest scores (lowest index first among equals) to idx / wgt.  NaN logits:
// expert 0.
__device__ __forceinline__ void route_top64(float v, int E, int top, int32_t* idx, float* wgt) {
  const int lane = threadIdx.x & 63;
  const float mx = wave_max(lane < E ? v : -INFINITY);
  float p = lane < E ? expf(v - mx) : -1.0f;
  const float score = p / group_sum<64>(lane < E ? p : 0.0f);
  for (int k = 0; k < top; ++k) {
    const unsigned long long best = __ballot(p == wave_max(p) && p >= 0.0f);
    const int e = best ? __builtin_ctzll(best) : 0;
    if (lane == e) {
      idx[k] = e;
      wgt[k] = score;
      p = -1.0f;
    }
  }
}

// exp and the logistic function through the hardware exponential and reciprocal (about an ulp each; the
// exponential's argument rounding adds |z| * 2^-24 relative).
__device__ __forceinline__ float fast_exp(float z) { return __builtin_amdgcn_exp2f(z * 1.44269504088896340736f); }
__device__ __forceinline__ float fast_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + fast_exp(-z)); }

// 1 - exp(y), y <= 0: its series near 0, where the difference would cancel.
__device__ __forceinline__ float one_minus_exp(float y) {
  float s = fmaf(y, 1.0f / 40320.0f, 1.0f / 5040.0f);
  s = fmaf(y, s, 1.0f / 720.0f);
  s = fmaf(y, s, 1.0f / 120.0f);
  s = fmaf(y, s, 1.0f / 24.0f);
  s = fmaf(y, s, 1.0f / 6.0f);
  s = fmaf(y, s, 0.5f);
  s = fmaf(y, s, 1.0f);
  return y > -0.5f ? -y * s : 1.0f - fast_exp(y);
}

// A gated linear recurrence's coefficients (a, b) from its gates' logits r and i, rate and input u.
__device__ __forceinline__ float2 lru_coef(float r, float i, float rate, float u) {
  const float la = -fast_sigmoid(r) * rate;
  return make_float2(fast_exp(la), __builtin_amdgcn_sqrtf(one_minus_exp(2.0f * la)) * fast_sigmoid(i) * u);
}

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }

}  // namespace ti
