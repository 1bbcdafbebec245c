// Merge of an attention row's key slices: unnormalised outputs part_o [rows][P][RS] with each slice's running maximum
// (log2 domain) and sum part_ml [rows][P][2]; exp(sink) of the row's head joins the denominator once.
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ void merge_st(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void merge_st(float* p, float v) { *p = v; }

// one workgroup of 128 threads per (token, head) row; slices of RS columns, of which RV leave; P <= MERGE_MAXP
constexpr int MERGE_MAXP = 256;
template <typename ACT>
__global__ void __launch_bounds__(128) slice_merge_kernel(const float* __restrict__ part_o,
                                                            const float* __restrict__ part_ml, int P, int RS, int RV,
                                                         const float* __restrict__ sink, int H, ACT* __restrict__ out) {
  __shared__ float wt[MERGE_MAXP];
  const size_t row = blockIdx.x;
  const float* ml = part_ml + row * P * 2;
  // every wave computes the weights (at most four slices per lane), the first stores them
  const int lane = threadIdx.x & 63;
  float m[MERGE_MAXP / 64], l[MERGE_MAXP / 64], mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < MERGE_MAXP / 64; ++i) {
    const int p = lane + 64 * i;
    m[i] = p < P ? ml[2 * p] : -INFINITY;
    l[i] = p < P ? ml[2 * p + 1] : 0.f;
    mx = fmaxf(mx, m[i]);
  }
  mx = wave_max(mx);
  const float sk = sink ? sink[row % H] * 1.4426950408889634f : -INFINITY;
  mx = fmaxf(mx, sk);
  const float ref = mx == -INFINITY ? 0.f : mx;
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < MERGE_MAXP / 64; ++i) {
    m[i] = exp2f(m[i] - ref);
    sum += m[i] * l[i];
  }
  sum = wave_sum(sum) + exp2f(sk - ref);          // no sink: 0
  const float inv = sum > 0.f ? 1.f / sum : 0.f;
  if (threadIdx.x < 64) {
#pragma unroll
    for (int i = 0; i < MERGE_MAXP / 64; ++i)
      if (lane + 64 * i < P) wt[lane + 64 * i] = m[i] * inv;
  }
  __syncthreads();
  for (int c = threadIdx.x * 4; c < RS; c += 512) {
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int p0 = 0; p0 < P; p0 += 8) {          // eight slices in flight (past the last: re-read, weight 0)
      float4 v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = *reinterpret_cast<const float4*>(part_o + (row * P + min(p0 + u, P - 1)) * RS + c);
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float e = p0 + u < P ? wt[p0 + u] : 0.f;
        s.x += e * v[u].x; s.y += e * v[u].y; s.z += e * v[u].z; s.w += e * v[u].w;
      }
    }
    ACT* o = out + row * RV + c;
    if (c + 3 < RV) {
      merge_st(o, s.x); merge_st(o + 1, s.y); merge_st(o + 2, s.z); merge_st(o + 3, s.w);
    } else {
      if (c < RV) merge_st(o, s.x);
      if (c + 1 < RV) merge_st(o + 1, s.y);
      if (c + 2 < RV) merge_st(o + 2, s.z);
    }
  }
}

}  // namespace
