// Merge of an attention row's key slices: unnormalised outputs part_o [rows][P][RS] with each slice's running maximum
// (log2 domain) and sum part_ml [rows][P][2]; exp(sink) of the row's head joins the denominator once.  What leaves may
// pass a gate per element (OutGate).
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ void merge_st(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void merge_st(float* p, float v) { *p = v; }

// An attention row's way out: token rows of stride ld; with p, times scale sigmoid(gate), the gate's columns one per output
// column, in activations (split 0) or fp32 slabs
struct OutGate {
  const void* p = nullptr;
  int split = 0;
  int64_t pld = 0, plane = 0;
  float scale = 1.f;
  int64_t ld = 0;
  int vec = 0;                 // rows of both allow vectors of four
};

__device__ __forceinline__ float gate_ld(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float gate_ld(const float* p) { return *p; }
template <typename ACT> __device__ __forceinline__ float gate_sigmoid(float x);
template <> __device__ __forceinline__ float gate_sigmoid<uint16_t>(float x) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}
template <> __device__ __forceinline__ float gate_sigmoid<float>(float x) { return 1.f / (1.f + expf(-x)); }

template <typename ACT>
__device__ __forceinline__ float out_gate(const OutGate& g, int64_t token, int col) {
  if (!g.p) return g.scale;
  const int64_t o = token * g.pld + col;
  float x = 0.f;
  if (g.split == 0) x = gate_ld(reinterpret_cast<const ACT*>(g.p) + o);
  else for (int i = 0; i < g.split; ++i) x += reinterpret_cast<const float*>(g.p)[o + i * g.plane];
  return g.scale * gate_sigmoid<ACT>(x);
}

// the factors of four neighbouring columns (g.vec)
template <typename ACT>
__device__ __forceinline__ f32x4_t out_gate4(const OutGate& g, int64_t token, int col) {
  if (!g.p) return f32x4_t{g.scale, g.scale, g.scale, g.scale};
  const int64_t o = token * g.pld + col;
  f32x4_t x{0.f, 0.f, 0.f, 0.f};
  if (g.split == 0) {
    if constexpr (sizeof(ACT) == 2) {
      const uint2 u = *reinterpret_cast<const uint2*>(reinterpret_cast<const ACT*>(g.p) + o);
      x = f32x4_t{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                  __uint_as_float(u.y & 0xffff0000u)};
    } else {
      x = *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const ACT*>(g.p) + o);
    }
  } else {
    const float* p = reinterpret_cast<const float*>(g.p) + o;
    for (int i0 = 0; i0 < g.split; i0 += 4) {           // four slabs in flight (past the last: re-read, not added)
      f32x4_t v[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) v[u] = *reinterpret_cast<const f32x4_t*>(p + (int64_t)min(i0 + u, g.split - 1) * g.plane);
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (i0 + u < g.split)
#pragma unroll
          for (int e = 0; e < 4; ++e) x[e] += v[u][e];
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) x[e] = g.scale * gate_sigmoid<ACT>(x[e]);
  return x;
}

// one workgroup of 128 threads per (token, head) row; slices of RS columns, of which RV leave; P <= MERGE_MAXP
constexpr int MERGE_MAXP = 256;
template <typename ACT>
__global__ void __launch_bounds__(128) slice_merge_kernel(const float* __restrict__ part_o,
                                                            const float* __restrict__ part_ml, int P, int RS, int RV,
                                                         const float* __restrict__ sink, int H, OutGate g, ACT* __restrict__ out) {
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
    const size_t token = row / H;
    const int col = (int)(row - token * H) * RV + c;
    ACT* o = out + token * g.ld + col;
    if (g.p) {
      if (c < RV) s.x *= out_gate<ACT>(g, token, col);
      if (c + 1 < RV) s.y *= out_gate<ACT>(g, token, col + 1);
      if (c + 2 < RV) s.z *= out_gate<ACT>(g, token, col + 2);
      if (c + 3 < RV) s.w *= out_gate<ACT>(g, token, col + 3);
    }
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
