// Shared helpers of libnvl_seq.so (gfx950 only: 64-wide wavefronts are assumed throughout).
#pragma once
#include <hip/hip_runtime.h>
#include <stdarg.h>
#include <stdint.h>
#include <stdio.h>
#include "../../../include/nvl_seq.h"

typedef __bf16 bf16_t;

void nvs_set_error(const char* fmt, ...);
int nvs_check_launch(const char* what);

#define NVS_REQUIRE(cond, ...)       \
  do {                               \
    if (!(cond)) {                   \
      nvs_set_error(__VA_ARGS__);    \
      return NVS_EINVAL;             \
    }                                \
  } while (0)

// element access in 32-bit whatever the storage type
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ float ldf(const bf16_t* p) { return (float)*p; }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }
__device__ __forceinline__ void stf(bf16_t* p, float v) { *p = (bf16_t)v; }   // round to nearest even

// VEC consecutive elements at once (16 / 8 bytes for VEC 4; the address is aligned to VEC elements)
template <int VEC>
__device__ __forceinline__ void ldv(const float* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const float4 f = *(const float4*)p;
    v[0] = f.x, v[1] = f.y, v[2] = f.z, v[3] = f.w;
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = p[i];
  }
}
template <int VEC>
__device__ __forceinline__ void ldv(const bf16_t* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    typedef __attribute__((ext_vector_type(4))) __bf16 b4_t;
    const b4_t b = *(const b4_t*)p;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (float)b[i];
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = (float)p[i];
  }
}
template <int VEC>
__device__ __forceinline__ void stv(float* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
  else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = v[i];
  }
}
template <int VEC>
__device__ __forceinline__ void stv(bf16_t* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    typedef __attribute__((ext_vector_type(4))) __bf16 b4_t;
    b4_t b;
#pragma unroll
    for (int i = 0; i < 4; ++i) b[i] = (bf16_t)v[i];
    *(b4_t*)p = b;
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = (bf16_t)v[i];
  }
}

// N (a power of two up to 8) consecutive elements in one piece (the address is aligned to the piece)
template <int N, typename T>
__device__ __forceinline__ void ldp(const T* p, float (&v)[N]) {
  typedef __attribute__((ext_vector_type(N))) T vec_t;
  const vec_t f = *(const vec_t*)p;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = (float)f[i];
}
template <int N, typename T>
__device__ __forceinline__ void stp(T* p, const float (&v)[N]) {
  typedef __attribute__((ext_vector_type(N))) T vec_t;
  vec_t f;
#pragma unroll
  for (int i = 0; i < N; ++i) f[i] = (T)v[i];
  *(vec_t*)p = f;
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}
// sum over a workgroup of up to 1024 threads; `red` is LDS for 16 floats; every thread gets the result
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();                       // `red` may still be read from a previous call
  if ((threadIdx.x & 63) == 0) red[w] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; ++i) s += red[i];
  return s;
}

__device__ __forceinline__ float sigmoidf_(float x) { return 1.f / (1.f + __expf(-x)); }
__device__ __forceinline__ float softplusf_(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float siluf_(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float gelu_tanhf_(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

#define NVS_DISPATCH(dtype, ...)                       \
  do {                                                 \
    if ((dtype) == NVS_BF16) {                         \
      typedef bf16_t T;                                \
      __VA_ARGS__;                                     \
    } else {                                           \
      typedef float T;                                 \
      __VA_ARGS__;                                     \
    }                                                  \
  } while (0)
