// Routed experts (mixture of experts):
//   * moe_route   sigmoid or softmax scores of the router logits; experts chosen by score + correction among the
//                 best groups; weights from the scores alone, over their sum or as they are.  One wave per token
//   * moe_rows    the (token, choice) pairs sorted by expert, each expert's rows padded to whole tiles: what the
//                 grouped products (dgemm.hip, pgemm.hip) and the gather of their results go by.  Nothing
//                 comes back to the host, so a captured decode step routes anew on every replay.  Choices past
//                 the last expert (outputs of the router without matrices) take no row
//   * moe_any     grouped products of any shape and both activation types (the 32-bit path, odd widths)
#include "common.h"

namespace {

__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ld1(const float* p) { return *p; }
__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

constexpr int MR_MAXE = 1024;

// logits: fp32 slabs [split] of row stride ld; E = groups * size experts
template <int NE>
__global__ void __launch_bounds__(256) moe_route_kernel(const float* __restrict__ logits, int split, int64_t ld, int64_t plane,
                                                       const float* __restrict__ correction, int T, int E, int groups, int keep,
                                                       int top, float scale, int softmax, int renorm, int32_t* __restrict__ ids,
                                                       float* __restrict__ weights) {
  __shared__ float choice[4][64 * NE], gscore[4][MR_MAXE];
  __shared__ int kept[4][MR_MAXE];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, t = blockIdx.x * 4 + w;
  const int size = E / groups;
  float s[NE], c[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    float z = 0.f;
    if (e < E && t < T)
      for (int p0 = 0; p0 < split; p0 += 16) {         // sixteen slabs in flight (past the last: re-read, not added)
        float v[16];
#pragma unroll
        for (int u = 0; u < 16; ++u) v[u] = logits[(int64_t)min(p0 + u, split - 1) * plane + (int64_t)t * ld + e];
#pragma unroll
        for (int u = 0; u < 16; ++u) z += p0 + u < split ? v[u] : 0.f;
      }
    s[i] = softmax ? (e < E ? z : -INFINITY) : 1.f / (1.f + expf(-z));
  }
  if (softmax) {
    float mx = -INFINITY, all = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) mx = fmaxf(mx, s[i]);
    mx = wave_max(mx);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      s[i] = expf(s[i] - mx);
      all += s[i];
    }
    all = wave_sum(all);
#pragma unroll
    for (int i = 0; i < NE; ++i) s[i] /= all;
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    c[i] = e < E ? s[i] + correction[min(e, E - 1)] : -INFINITY;
    choice[w][e] = c[i];
  }
  __syncthreads();
  for (int g = keep < groups ? lane : groups; g < groups; g += 64) {
    float a = -INFINITY, b = -INFINITY;           // the two largest
    for (int i = 0; i < size; ++i) {
      const float v = choice[w][g * size + i];
      if (v > a) { b = a; a = v; }
      else b = fmaxf(b, v);
    }
    gscore[w][g] = size > 1 ? a + b : a;
  }
  __syncthreads();
  for (int g = keep < groups ? lane : groups; g < groups; g += 64) {
    const float v = gscore[w][g];
    int better = 0;
    for (int o = 0; o < groups; ++o) better += gscore[w][o] > v || (gscore[w][o] == v && o < g);
    kept[w][g] = better < keep;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    if (keep < groups && e < E && !kept[w][e / size]) c[i] = -INFINITY;
  }
  float mine = 0.f, sum = 0.f;
  int mine_id = 0;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY, bs = 0.f;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (c[i] > best) { best = c[i]; bi = lane + 64 * i; bs = s[i]; }
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) {
      const float ov = __shfl_xor(best, m, 64), os = __shfl_xor(bs, m, 64);
      const int oi = __shfl_xor(bi, m, 64);
      if (ov > best || (ov == best && oi < bi)) { best = ov; bi = oi; bs = os; }
    }
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (bi == lane + 64 * i) c[i] = -INFINITY;
    if (lane == k) { mine = bs; mine_id = min(bi, E - 1); }
    sum += bs;
  }
  if (t < T && lane < top) {
    ids[(size_t)t * top + lane] = mine_id;
    weights[(size_t)t * top + lane] = (renorm ? mine / (sum + 1e-20f) : mine) * scale;
  }
}

// one workgroup per expert: counts of all, then the places of its own pairs in pair order
__global__ void __launch_bounds__(1024) moe_rows_kernel(const int32_t* __restrict__ ids, int pairs, int top, int E, int tile,
                                                       int max_tiles, int32_t* __restrict__ rows, int32_t* __restrict__ pos,
                                                       int32_t* __restrict__ tile_expert) {
  __shared__ int count[MR_MAXE], wsum[16], base_s;
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  for (int i = tid; i < E; i += 1024) count[i] = 0;
  if (tid == 0) base_s = 0;
  __syncthreads();
  for (int p = tid; p < pairs; p += 1024) {
    const int i = ids[p];
    if (i < E) atomicAdd(&count[i], 1);
    else if (e == 0) pos[p] = 0;               // no row of its own: a place that exists
  }
  __syncthreads();
  for (int i = tid; i < e; i += 1024) atomicAdd(&base_s, (count[i] + tile - 1) / tile);
  __syncthreads();
  const int t0 = base_s, n = count[e], nt = (n + tile - 1) / tile;
  int at = t0 * tile;
  for (int p0 = 0; p0 < pairs; p0 += 1024) {
    const int p = p0 + tid;
    const bool mine = p < pairs && ids[p] == e;
    const unsigned long long b = __ballot(mine);
    if (lane == 0) wsum[w] = __popcll(b);
    __syncthreads();
    int before = 0, all = 0;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      before += i < w ? wsum[i] : 0;
      all += wsum[i];
    }
    if (mine) {
      const int r = at + before + __popcll(b & ((1ull << lane) - 1));
      rows[r] = p / top;
      pos[p] = r;
    }
    at += all;
    __syncthreads();
  }
  for (int r = t0 * tile + n + tid; r < (t0 + nt) * tile; r += 1024) rows[r] = 0;
  for (int i = tid; i < nt; i += 1024) tile_expert[t0 + i] = e;
  if (e == E - 1)
    for (int i = t0 + nt + tid; i < max_tiles; i += 1024) {
      tile_expert[i] = -1;
      for (int r = 0; r < tile; ++r) rows[i * tile + r] = 0;
    }
}

// Row-major W [experts][GLU ? 2 N : N][K]; 32 rows x 64 columns per workgroup, K in steps of 16 through LDS.
// GLU: columns n of the gate rows 0 .. N - 1 and of the up rows N .. 2 N - 1, g = min(gate, limit):
// g sigmoid(alpha g) (clamp(up, +-limit) + beta); else the product
template <typename ACT, bool GLU>
__global__ void __launch_bounds__(256) moe_any_kernel(const ACT* __restrict__ x, const ACT* __restrict__ W, int N, int K,
                                                     const int32_t* __restrict__ rows, const int32_t* __restrict__ tile_expert,
                                                     int tile, void* __restrict__ out, int ldo, float limit, float alpha,
                                                     float beta) {
  constexpr int NM = GLU ? 2 : 1;
  __shared__ float xs[16][33], wsm[NM][16][65];
  const int m0 = blockIdx.y * 32, n0 = blockIdx.x * 64, e = tile_expert[m0 / tile], tid = threadIdx.x;
  if (e < 0) return;
  const ACT* w = W + (size_t)e * NM * N * K;
  const int tn = tid & 15, tm = tid >> 4;        // 2 rows x 4 columns
  float acc[NM][2][4] = {};
  for (int k0 = 0; k0 < K; k0 += 16) {
    for (int i = tid; i < 32 * 16; i += 256) {
      const int m = m0 + (i >> 4), k = k0 + (i & 15);
      xs[i & 15][i >> 4] = k < K ? ld1(x + (size_t)(rows ? rows[m] : m) * K + k) : 0.f;
    }
#pragma unroll
    for (int g = 0; g < NM; ++g)
      for (int i = tid; i < 64 * 16; i += 256) {
        const int n = n0 + (i >> 4), k = k0 + (i & 15);
        wsm[g][i & 15][i >> 4] = k < K && n < N ? ld1(w + ((size_t)g * N + n) * K + k) : 0.f;
      }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k)
#pragma unroll
      for (int g = 0; g < NM; ++g)
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
          for (int b = 0; b < 4; ++b) acc[g][a][b] += xs[k][2 * tm + a] * wsm[g][k][tn + 16 * b];
    __syncthreads();
  }
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int m = m0 + 2 * tm + a, n = n0 + tn + 16 * b;
      if (n >= N) continue;
      if constexpr (GLU) {
        const float g = fminf(acc[0][a][b], limit), u = fminf(fmaxf(acc[NM - 1][a][b], -limit), limit);
        st1(reinterpret_cast<ACT*>(out) + (size_t)m * ldo + n, g / (1.f + expf(-alpha * g)) * (u + beta));
      } else {
        st1(reinterpret_cast<ACT*>(out) + (size_t)m * ldo + n, acc[0][a][b]);
      }
    }
}

}  // namespace

CFC_API int cfc_moe_route(const float* logits, int split, int64_t ld, int64_t plane, const float* correction, int T, int E,
                          int groups, int keep, int top, float scale, int softmax, int renorm, int32_t* ids, float* weights,
                          hipStream_t stream) {
  if (T <= 0) return 0;
  if (E < 1 || E > MR_MAXE || groups < 1 || E % groups || keep < 1 || keep > groups || top < 1 || top > 64 ||
      top > keep * (E / groups) || split < 1)
    return -1;
#define MO(NE) \
  moe_route_kernel<NE><<<(T + 3) / 4, 256, 0, stream>>>(logits, split, ld, plane, correction, T, E, groups, keep, top, scale, softmax, renorm, ids, weights)
  if (E <= 64) MO(1);
  else if (E <= 128) MO(2);
  else if (E <= 256) MO(4);
  else MO(16);
#undef MO
  return CFC_CHECK_LAUNCH();
}

// rows [max_tiles tile], pos [pairs], tile_expert [max_tiles]; max_tiles >= pairs / tile + min(E, pairs)
CFC_API int cfc_moe_rows(const int32_t* ids, int pairs, int top, int E, int tile, int max_tiles, int32_t* rows, int32_t* pos,
                         int32_t* tile_expert, hipStream_t stream) {
  if (pairs <= 0) return 0;
  const int most = pairs / tile + (E < pairs ? E : pairs);
  if (E < 1 || E > MR_MAXE || top < 1 || tile < 1 || max_tiles < (most < pairs ? most : pairs)) return -1;
  moe_rows_kernel<<<E, 1024, 0, stream>>>(ids, pairs, top, E, tile, max_tiles, rows, pos, tile_expert);
  return CFC_CHECK_LAUNCH();
}

// M sorted rows in tiles of `tile` (a multiple of 32), activations [M][N] of row stride ldo
CFC_API int cfc_moe_any(int f32, int glu, const void* x, const void* w, int M, int N, int K, const int32_t* rows,
                        const int32_t* tile_expert, int tile, void* out, int ldo, float limit, float alpha, float beta, hipStream_t stream) {
  if (M == 0) return 0;
  if (M < 0 || N < 1 || K < 1 || tile < 32 || tile % 32 || M % tile || ldo < N || M / 32 > 65535 || !tile_expert) return -1;
  const dim3 grid((N + 63) / 64, M / 32);
#define MA(ACT, G) moe_any_kernel<ACT, G><<<grid, 256, 0, stream>>>((const ACT*)x, (const ACT*)w, N, K, rows, tile_expert, tile, out, ldo, limit, alpha, beta)
  if (f32) { if (glu) MA(float, true); else MA(float, false); }
  else if (glu) MA(uint16_t, true);
  else MA(uint16_t, false);
#undef MA
  return CFC_CHECK_LAUNCH();
}
