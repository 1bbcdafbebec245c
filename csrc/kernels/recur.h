// Parts that element-wise linear recurrences S_t = a_t S_(t-1) + b_t share: prompt portions run in chunks in parallel, each
// chunk leaving the product of its a and what it adds to a state of zero; carry_kernel takes the states through them.
#pragma once
#include "rows.h"

namespace {

// ACT decides the exponential and the reciprocal: the hardware's for bf16 activations, the library's on the 32-bit path
template <typename ACT> __device__ __forceinline__ float exp_of(float x);
template <> __device__ __forceinline__ float exp_of<uint16_t>(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
template <> __device__ __forceinline__ float exp_of<float>(float x) { return expf(x); }
template <typename ACT> __device__ __forceinline__ float over1(float x);              // 1 / (1 + x)
template <> __device__ __forceinline__ float over1<uint16_t>(float x) { return __builtin_amdgcn_rcpf(1.f + x); }
template <> __device__ __forceinline__ float over1<float>(float x) { return 1.f / (1.f + x); }

constexpr int CARRY_FLIGHT = 8;      // chunks requested ahead of their use

// sums [chunks][2][W]; sums[chunk][0] becomes the state ahead of the chunk
template <int V>
__global__ void __launch_bounds__(64) carry_kernel(const int32_t* __restrict__ chunk_cu, const int32_t* __restrict__ cu_q,
                                                      const int32_t* __restrict__ ctx_lens, const int32_t* __restrict__ slots,
                                                      int W, float* __restrict__ sums, float* __restrict__ state) {
  const int s = blockIdx.x, c = (blockIdx.y * 64 + threadIdx.x) * V;
  if (c >= W) return;
  const int i0 = chunk_cu[s], i1 = chunk_cu[s + 1];
  float* sp = state + (size_t)slots[s] * W + c;
  Vec<V> S = ctx_lens[s] > cu_q[s + 1] - cu_q[s] ? ldv<V>(sp) : zerov<V>();
  for (int i = i0; i < i1; i += CARRY_FLIGHT) {
    Vec<V> A[CARRY_FLIGHT], B[CARRY_FLIGHT];
#pragma unroll
    for (int k = 0; k < CARRY_FLIGHT; ++k) {
      const float* p = sums + (size_t)min(i + k, i1 - 1) * 2 * W + c;
      A[k] = ldv<V>(p);
      B[k] = ldv<V>(p + W);
    }
#pragma unroll
    for (int k = 0; k < CARRY_FLIGHT; ++k)
      if (i + k < i1) {
        stv<V>(sums + (size_t)(i + k) * 2 * W + c, S);
#pragma unroll
        for (int e = 0; e < V; ++e) S.v[e] = A[k].v[e] * S.v[e] + B[k].v[e];
      }
  }
  stv<V>(sp, S);
}

}  // namespace
