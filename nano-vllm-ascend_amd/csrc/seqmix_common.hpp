// Device helpers shared by the sequence-mixer kernels (seqmix.hip, stream_delta.hip).
#pragma once
#include "mi_common.hpp"

namespace mi {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

template <typename T>
__device__ __forceinline__ float ld_f(const T* p);
template <>
__device__ __forceinline__ float ld_f<float>(const float* p) { return *p; }
template <>
__device__ __forceinline__ float ld_f<uint16_t>(const uint16_t* p) { return bf2f(*p); }
template <typename T>
__device__ __forceinline__ void st_f(T* p, float v);
template <>
__device__ __forceinline__ void st_f<float>(float* p, float v) { *p = v; }
template <>
__device__ __forceinline__ void st_f<uint16_t>(uint16_t* p, float v) { *p = f2bf(v); }

// sum over a 256-thread workgroup; every thread gets the result.  red: 4 floats of LDS per concurrent reduction.
__device__ __forceinline__ float block_sum256(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();  // (red may still be read from the previous reduction)
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// the sequence a step row belongs to (n_seqs is small: a linear walk, identical on every lane)
__device__ __forceinline__ int seq_of_row(const int32_t* cu_q, int n_seqs, int row) {
  int s = 0;
  while (s + 1 < n_seqs && row >= cu_q[s + 1]) ++s;
  return s;
}

}  // namespace mi
