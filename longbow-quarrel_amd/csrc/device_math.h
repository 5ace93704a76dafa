// Device functions that the recurrent mixers' kernels share: activations, stores in the run's dtype, sums over the lanes
// of a column.
#pragma once

#include "common.h"

namespace {

__device__ inline float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ inline float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ inline float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
__device__ inline float gelu_tanh_f(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

__device__ inline float gelu_erf_f(float z) { return 0.5f * z * (1.f + erff(z * 0.70710678118654752f)); }

enum { ACT_NONE = 0, ACT_SILU = 1, ACT_RELU = 2, ACT_GELU_TANH = 3, ACT_GELU_ERF = 4, ACT_RELU2 = 5 };

__device__ inline float activate(float z, int act) {
  switch (act) {
    case ACT_SILU: return silu_f(z);
    case ACT_RELU: return fmaxf(z, 0.f);
    case ACT_GELU_TANH: return gelu_tanh_f(z);
    case ACT_GELU_ERF: return gelu_erf_f(z);
    case ACT_RELU2: { const float r = fmaxf(z, 0.f); return r * r; }
    default: return z;
  }
}

template <typename T>
__device__ inline void store_as(T* p, float v);
template <>
__device__ inline void store_as<float>(float* p, float v) { *p = v; }
template <>
__device__ inline void store_as<bf16_t>(bf16_t* p, float v) { *p = f32_to_bf16(v); }

template <int CTRL>
__device__ inline float dpp_swap(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}

// the sum over the LN lanes of a column; every lane gets it
template <int LN>
__device__ inline float group_sum(float v) {
  if (LN >= 2) v += dpp_swap<0xB1>(v);    // lanes 1 apart (quad_perm [1,0,3,2])
  if (LN >= 4) v += dpp_swap<0x4E>(v);    // 2 apart (quad_perm [2,3,0,1])
  if (LN >= 8) v += dpp_swap<0x141>(v);   // the other quad of eight lanes (row_half_mirror)
  if (LN >= 16) v += dpp_swap<0x140>(v);  // the other half of sixteen (row_mirror)
  if (LN >= 32) v += __shfl_xor(v, 16, LQ_WAVE);
  if (LN >= 64) v += __shfl_xor(v, 32, LQ_WAVE);
  return v;
}

}  // namespace
