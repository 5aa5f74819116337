// elem.h — element access shared by the layered-model kernels. Activations
// are T = short (bf16 bits) or float; arithmetic is always 32-bit.
#pragma once
#include "../hip_common.h"

__device__ __forceinline__ float ld(const short* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ float ld(const float* p) { return *p; }
__device__ __forceinline__ void st(short* p, float f) { *p = f32_to_bf16(f); }
__device__ __forceinline__ void st(float* p, float f) { *p = f; }

// N consecutive elements; N > 1 is 8 and needs 16-byte aligned pointers
template <int N>
__device__ __forceinline__ void ldn(const short* p, float* f) {
  if constexpr (N == 8) {
    short8 v = *(const short8*)p;
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = bf16_to_f32(v[j]);
  } else {
    f[0] = ld(p);
  }
}
template <int N>
__device__ __forceinline__ void ldn(const float* p, float* f) {
  if constexpr (N == 8) {
    float4v a = ((const float4v*)p)[0], b = ((const float4v*)p)[1];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = a[j];
      f[4 + j] = b[j];
    }
  } else {
    f[0] = *p;
  }
}
template <int N>
__device__ __forceinline__ void stn(short* p, const float* f) {
  if constexpr (N == 8) {
    short8 v;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = f32_to_bf16(f[j]);
    *(short8*)p = v;
  } else {
    st(p, f[0]);
  }
}
template <int N>
__device__ __forceinline__ void stn(float* p, const float* f) {
  if constexpr (N == 8) {
    ((float4v*)p)[0] = (float4v){f[0], f[1], f[2], f[3]};
    ((float4v*)p)[1] = (float4v){f[4], f[5], f[6], f[7]};
  } else {
    p[0] = f[0];
  }
}

// 1 / x to an ulp or so
__device__ __forceinline__ float rcp_f(float x) {
  return __builtin_amdgcn_rcpf(x);
}
__device__ __forceinline__ float sigmoid_f(float x) {
  return rcp_f(1.f + __expf(-x));
}
enum Act { ACT_GELU_TANH, ACT_SILU, ACT_RELU_SQUARED, ACTS };
__device__ __forceinline__ float activate(int act, float z) {
  if (act == ACT_RELU_SQUARED) return z > 0.f ? z * z : 0.f;
  // 0.5 (1 + tanh(a)) = 1 / (1 + exp(-2a))
  const float a = act == ACT_SILU
                      ? z
                      : 2.f * 0.7978845608028654f *
                            (z + 0.044715f * z * z * z);
  return z / (1.f + expf(-a));
}
// log(1 + e^x) = max(x, 0) + log(1 + e^-|x|); with e = e^-|x| in (0, 1],
// log(1 + e) = 2 artanh(s), s = e / (2 + e) <= 1/3: the odd series to s^15
// leaves less than 1e-8 of the first term, also for small e
__device__ __forceinline__ float softplus_f(float x) {
  const float e = __expf(-fabsf(x));
  const float s = e * rcp_f(2.f + e), z = s * s;
  float p = 1.f / 15.f;
  p = fmaf(p, z, 1.f / 13.f);
  p = fmaf(p, z, 1.f / 11.f);
  p = fmaf(p, z, 1.f / 9.f);
  p = fmaf(p, z, 1.f / 7.f);
  p = fmaf(p, z, 1.f / 5.f);
  p = fmaf(p, z, 1.f / 3.f);
  p = fmaf(p, z, 1.f);
  return fmaf(2.f * s, p, fmaxf(x, 0.f));
}

// Workgroup barrier that orders LDS accesses only: global loads issued before
// it stay in flight across it (__syncthreads waits for them)
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// sum over a block of NW waves; every thread gets it. Two calls in a row
// need different scratch (NW floats each).
template <int NW>
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  v = wave_reduce_sum(v);
  if (threadIdx.x % WAVE == 0) scratch[threadIdx.x / WAVE] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) t += scratch[w];
  return t;
}

// Sequences of a batch: [n_seqs, 4] = first row, rows, tokens before, slot
struct Seq {
  int row0, n, prior, slot;
};
__device__ __forceinline__ Seq load_seq(const int32_t* meta, int s) {
  const int4 m = ((const int4*)meta)[s];
  return {m.x, m.y, m.z, m.w};
}
