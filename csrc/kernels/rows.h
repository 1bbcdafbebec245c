// Row kernels' shared parts (one workgroup per row of a 32-bit stream, channels in vectors of V per thread): vector
// loads and stores of activations (bf16 bits or float), sums of fp32 k-slice slabs, launch shapes.
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ld1(const float* p) { return *p; }

template <int V> struct Vec { float v[V]; };

template <int V>
__device__ __forceinline__ Vec<V> ldv(const float* p) {
  Vec<V> r;
  if constexpr (V == 4) {
    const float4 f = *reinterpret_cast<const float4*>(p);
    r.v[0] = f.x; r.v[1] = f.y; r.v[2] = f.z; r.v[3] = f.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V>
__device__ __forceinline__ Vec<V> ldv(const uint16_t* p) {
  Vec<V> r;
  if constexpr (V == 4) {
    const uint2 u = *reinterpret_cast<const uint2*>(p);
    r.v[0] = __uint_as_float(u.x << 16); r.v[1] = __uint_as_float(u.x & 0xffff0000u);
    r.v[2] = __uint_as_float(u.y << 16); r.v[3] = __uint_as_float(u.y & 0xffff0000u);
  } else {
    r.v[0] = bf2f(*p);
  }
  return r;
}
template <int V>
__device__ __forceinline__ void stv(float* p, const Vec<V>& r) {
  if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else *p = r.v[0];
}
template <int V>
__device__ __forceinline__ void stv(uint16_t* p, const Vec<V>& r) {
  if constexpr (V == 4) *reinterpret_cast<uint2*>(p) = make_uint2(pack2bf(r.v[0], r.v[1]), pack2bf(r.v[2], r.v[3]));
  else *p = f2bf(r.v[0]);
}
template <int V>
__device__ __forceinline__ Vec<V> zerov() {
  Vec<V> r;
#pragma unroll
  for (int e = 0; e < V; ++e) r.v[e] = 0.f;
  return r;
}

// y += slabs of row offset `off`, eight in flight (past the last: re-read, not added)
template <int V>
__device__ __forceinline__ void add_slabs(Vec<V>& y, const float* p, int split, int64_t plane, size_t off) {
  if (split == 1) {
    const Vec<V> a = ldv<V>(p + off);
#pragma unroll
    for (int e = 0; e < V; ++e) y.v[e] += a.v[e];
    return;
  }
  for (int p0 = 0; p0 < split; p0 += 8) {
    Vec<V> a[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) a[u] = ldv<V>(p + (size_t)min(p0 + u, split - 1) * plane + off);
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (p0 + u < split)
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += a[u].v[e];
  }
}

}  // namespace

// NV, BT for rows of W channels in vectors of V
#define ROW_SHAPES(GO, vecs)           \
  if (vecs <= 64) GO(1, 64);           \
  else if (vecs <= 256) GO(1, 256);    \
  else if (vecs <= 512) GO(1, 512);    \
  else if (vecs <= 1024) GO(1, 1024);  \
  else if (vecs <= 4096) GO(4, 1024);  \
  else if (vecs <= 16384) GO(16, 1024); \
  else return -4
