// Shared helpers of the sequence-mixer kernels (seq_*.hip): activation-type
// generic loads/stores (bf16 or fp32 activations, fp32 math) and accurate
// fp32 transcendental wrappers.  gfx950 only, wave size 64.
#pragma once

#include "common.h"

template <typename T>
DEV_INLINE float ldf(const T* p);
template <>
DEV_INLINE float ldf<float>(const float* p) { return *p; }
template <>
DEV_INLINE float ldf<bf16_t>(const bf16_t* p) { return bf2f(*p); }

template <typename T>
DEV_INLINE void stf(T* p, float v);
template <>
DEV_INLINE void stf<float>(float* p, float v) { *p = v; }
template <>
DEV_INLINE void stf<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }

DEV_INLINE float sigmoidf_acc(float x) { return 1.f / (1.f + expf(-x)); }
DEV_INLINE float siluf_acc(float x) { return x / (1.f + expf(-x)); }
DEV_INLINE float softplusf_acc(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}
// The same through the hardware exponential and reciprocal (each good to an
// ulp), for kernels whose lanes spend most of their time in them.
DEV_INLINE float sigmoidf_fast(float x) {
  return __builtin_amdgcn_rcpf(
      1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}
// log(1 + e) for e = exp(-|x|) in [0, 1] as 2 atanh(s), s = e / (2 + e) <=
// 1/3, by the odd power series of atanh: relative error below 3e-7 for every
// e, also where 1 + e rounds to one
DEV_INLINE float softplusf_fast(float x) {
  const float e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(x));
  const float s = e * __builtin_amdgcn_rcpf(2.f + e);
  const float w = s * s;
  float p = 1.f / 13.f;
  p = p * w + 1.f / 11.f;
  p = p * w + 1.f / 9.f;
  p = p * w + 1.f / 7.f;
  p = p * w + 1.f / 5.f;
  p = p * w + 1.f / 3.f;
  p = p * w + 1.f;
  return fmaxf(x, 0.f) + 2.f * s * p;
}
DEV_INLINE float gelu_tanhf_acc(float z) {
  const float c = 0.7978845608028654f;  // sqrt(2/pi)
  return 0.5f * z * (1.f + tanhf(c * (z + 0.044715f * z * z * z)));
}

DEV_INLINE float gelu_erff_acc(float z) {
  return 0.5f * z * (1.f + erff(z * 0.70710678118654752f));
}

// sum over the 2^k lanes l, l^1, ..., l^(G-1) (G a power of two <= 64)
template <int G>
DEV_INLINE float lanegroup_sum(float x) {
#pragma unroll
  for (int off = G / 2; off > 0; off >>= 1) x += __shfl_xor(x, off, WAVE_SIZE);
  return x;
}

// sum over the four lanes 4j .. 4j+3 by two
// quad permutes in the VALU data path: partner lane^2, then lane^1
DEV_INLINE float quad_sum(float x) {
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
      0, __builtin_bit_cast(int, x), 0x4E, 0xF, 0xF, false));  // [2,3,0,1]
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
      0, __builtin_bit_cast(int, x), 0xB1, 0xF, 0xF, false));  // [1,0,3,2]
  return x;
}

// sum over the eight lanes 8j .. 8j+7: the quads, then the mirrored half row
DEV_INLINE float oct_sum(float x) {
  x = quad_sum(x);
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
      0, __builtin_bit_cast(int, x), 0x141, 0xF, 0xF, false));
  return x;
}

// Four consecutive activations as they lie in memory: fetched ahead of their
// use, turned into fp32 where they are used (a conversion next to the load
// would wait for it there).
template <typename T>
struct Raw4;
template <>
struct Raw4<bf16_t> {
  uint2 r;
  template <bool VEC>
  DEV_INLINE void load(const bf16_t* p, int valid) {
    if (VEC) {
      r = *reinterpret_cast<const uint2*>(p);
    } else {
      unsigned short h[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        h[e] = e < valid ? reinterpret_cast<const unsigned short*>(p)[e] : 0;
      r.x = h[0] | (unsigned)h[1] << 16;
      r.y = h[2] | (unsigned)h[3] << 16;
    }
  }
  DEV_INLINE f32x4v get() const {
    f32x4v o;
    o.v[0] = __builtin_bit_cast(float, r.x << 16);
    o.v[1] = __builtin_bit_cast(float, r.x & 0xffff0000u);
    o.v[2] = __builtin_bit_cast(float, r.y << 16);
    o.v[3] = __builtin_bit_cast(float, r.y & 0xffff0000u);
    return o;
  }
};
template <>
struct Raw4<float> {
  f32x4v r;
  template <bool VEC>
  DEV_INLINE void load(const float* p, int valid) {
    if (VEC) {
      r = *reinterpret_cast<const f32x4v*>(p);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) r.v[e] = e < valid ? p[e] : 0.f;
    }
  }
  DEV_INLINE f32x4v get() const { return r; }
};

// four consecutive numbers as fp32: one 8- or 16-byte load when ``vec`` (the
// caller has checked the alignment and that all four exist), else the first
// ``valid`` of them and zeros
template <typename T>
DEV_INLINE f32x4v load4(const T* p, int valid, bool vec) {
  f32x4v o;
  if (vec) {
    if constexpr (sizeof(T) == 2) {
      const uint2 r = *reinterpret_cast<const uint2*>(p);
      o.v[0] = __builtin_bit_cast(float, r.x << 16);
      o.v[1] = __builtin_bit_cast(float, r.x & 0xffff0000u);
      o.v[2] = __builtin_bit_cast(float, r.y << 16);
      o.v[3] = __builtin_bit_cast(float, r.y & 0xffff0000u);
    } else {
      o = *reinterpret_cast<const f32x4v*>(p);
    }
    return o;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) o.v[e] = e < valid ? ldf(p + e) : 0.f;
  return o;
}

template <typename T>
DEV_INLINE void store4(T* p, const f32x4v& x, int valid, bool vec) {
  if (vec) {
    if constexpr (sizeof(T) == 2) {
      T q[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) stf(q + e, x.v[e]);
      uint2 r;
      __builtin_memcpy(&r, q, 8);
      *reinterpret_cast<uint2*>(p) = r;
    } else {
      *reinterpret_cast<f32x4v*>(p) = x;
    }
    return;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (e < valid) stf(p + e, x.v[e]);
}

// host check for load4 / store4's vector form: the view's base, row stride
// and a column offset are multiples of four elements and aligned to them
template <typename T>
static bool rows_by4(const torch::Tensor& t, long cols) {
  return (uintptr_t)t.data_ptr() % (4 * sizeof(T)) == 0 &&
         t.stride(0) % 4 == 0 && cols % 4 == 0;
}

// activation-type dispatch on a torch dtype
#define SEQ_DISPATCH_T(dtype, ...)                                   \
  do {                                                               \
    if ((dtype) == torch::kBFloat16) {                               \
      using T = bf16_t;                                              \
      __VA_ARGS__;                                                   \
    } else if ((dtype) == torch::kFloat32) {                         \
      using T = float;                                               \
      __VA_ARGS__;                                                   \
    } else {                                                         \
      TORCH_CHECK(false, "activations must be bf16 or fp32");        \
    }                                                                \
  } while (0)

#define CHECK_I32(t) TORCH_CHECK((t).is_cuda() && (t).dtype() == torch::kInt32 && (t).is_contiguous(), #t " must be a contiguous int32 device tensor")
#define CHECK_F32(t) TORCH_CHECK((t).is_cuda() && (t).dtype() == torch::kFloat32 && (t).is_contiguous(), #t " must be a contiguous fp32 device tensor")
#define CHECK_ROWS(t) TORCH_CHECK((t).is_cuda() && (t).dim() == 2 && (t).stride(1) == 1, #t " must be 2-D with unit inner stride")
