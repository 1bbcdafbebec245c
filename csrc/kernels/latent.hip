// Latent attention for gfx950: every head's keys and values are products of ONE cached latent row per
// token, so the paged cache holds [blocks][32][RS] latents (RS = rank rounded up to 32, zero-filled)
// and attention runs in the latent space: with q' = W_uk^T q per head, score = q' . c and the head's
// output is W_uv (sum p c).  All heads of a token then read the same rows (a multi-query attention
// whose key and value are the same bytes, loaded once).
//
//   * latent_norm     RMS norms of the query latent and the cached latent from the fp32 slabs of the
//                     joint down projection; the latter goes straight into the cache slot
//   * latent_rope     the same for designs with rotary positions: the normed latent and, behind it in the
//                     row, the rotated key part all heads share; the heads' rotated query parts
//   * head_linear     out[t][h] = W[h] in[t][h], the per-head products on both sides of the attention
//   * latent_attn     flash-style attention over the paged latents.  A work item is 16 MR rows of the
//                     flattened (token, head) rows of one sequence -- one decoded token's heads and a
//                     prompt portion's rows are the same thing to it -- and a slice of its keys
//   * slice_merge     merges the slices (split_merge.h)
//   * latent_gather   the latents of whole sequences as dense rows, in token order and in the slot order
//                     of the prefill attention's V^T: two products turn them into per-head keys and
//                     values for long portions, where that costs fewer flops (attention.hip, EXP)
#include "split_merge.h"

namespace {

typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));     // arrays of these stay in registers
typedef short i16x4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) i16x4_t lds_i16x4_t;

__device__ __forceinline__ float ldf(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// ---------------------------------------------------------------------------------- latent_norm
// part: fp32 slabs [split][T][NQ + NC] of the joint projection (query latent | cached latent).  One
// workgroup per row, a thread holds up to NV vectors of V columns (V divides NQ).
template <typename ACT, int V>
__device__ __forceinline__ void st_vec(ACT* p, const float* v) {
  if constexpr (V == 1) stf(p, v[0]);
  else if constexpr (sizeof(ACT) == 2) *reinterpret_cast<uint2*>(p) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
  else *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

template <typename ACT, int V, int NV, int BT>
__global__ void __launch_bounds__(BT) latent_norm_kernel(const float* __restrict__ part, int split, int T, int NQ, int NC,
                                                        const float* __restrict__ wq, const float* __restrict__ wc,
                                                        float eps, const int32_t* __restrict__ slots,
                                                        ACT* __restrict__ q_out, int ldq, ACT* __restrict__ cache, int RS) {
  __shared__ float red[16];
  const int t = blockIdx.x, N = NQ + NC;
  const size_t plane = (size_t)T * N;
  const float* src = part + (size_t)t * N;
  const int slot = slots[t];
  float x[NV][V], sq = 0.f, sc = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) x[k][e] = 0.f;
    if (c >= N) continue;
    if (split == 1) {
      if constexpr (V == 4) {
        const float4 f = *reinterpret_cast<const float4*>(src + c);
        x[k][0] = f.x; x[k][1] = f.y; x[k][2] = f.z; x[k][3] = f.w;
      } else {
        x[k][0] = src[c];
      }
    } else for (int p0 = 0; p0 < split; p0 += 8) {       // eight slabs in flight (past the last: re-read, not added)
      float y[8][V];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float* s = src + (size_t)min(p0 + u, split - 1) * plane + c;
        if constexpr (V == 4) {
          const float4 f = *reinterpret_cast<const float4*>(s);
          y[u][0] = f.x; y[u][1] = f.y; y[u][2] = f.z; y[u][3] = f.w;
        } else {
          y[u][0] = *s;
        }
      }
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (p0 + u < split)
#pragma unroll
          for (int e = 0; e < V; ++e) x[k][e] += y[u][e];
    }
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < V; ++e) ss += x[k][e] * x[k][e];
    if (c < NQ) sq += ss;
    else sc += ss;
  }
  sq = block_sum(sq, red);
  sc = block_sum(sc, red);
  const float rq = 1.f / sqrtf(sq / (float)NQ + eps), rc = 1.f / sqrtf(sc / (float)NC + eps);
  ACT* dst = cache + (size_t)slot * RS;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= N) continue;
    const bool isq = c < NQ;
    const float* w = isq ? wq + c : wc + (c - NQ);
    const float r = isq ? rq : rc;
    float v[V];
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = x[k][e] * r * w[e];
    st_vec<ACT, V>(isq ? q_out + (size_t)t * ldq + c : dst + (c - NQ), v);
  }
}

template <typename ACT, int V>
int latent_norm_go(hipStream_t st, const float* part, int split, int T, int NQ, int NC, const float* wq, const float* wc,
                   float eps, const int32_t* slots, void* q_out, int ldq, void* cache, int RS) {
  const int vecs = (NQ + NC + V - 1) / V;
#define LN_GO(NV, BT) \
  latent_norm_kernel<ACT, V, NV, BT><<<T, BT, 0, st>>>(part, split, T, NQ, NC, wq, wc, eps, slots, (ACT*)q_out, ldq, (ACT*)cache, RS)
  if (vecs <= 256) LN_GO(1, 256);
  else if (vecs <= 512) LN_GO(1, 512);
  else if (vecs <= 1024) LN_GO(1, 1024);
  else if (vecs <= 4096) LN_GO(4, 1024);
  else if (vecs <= 16384) LN_GO(16, 1024);
  else return -4;
#undef LN_GO
  return CFC_CHECK_LAUNCH();
}

// ---------------------------------------------------------------------------------- latent_rope
// Columns of a product: activations (split 0) or fp32 slabs.
struct LatCols { const void* p; int split; int64_t ld, plane; };

template <typename ACT>
__device__ __forceinline__ float ldcol(const LatCols& a, int64_t t, int c) {
  const int64_t o = t * a.ld + c;
  if (a.split == 0) return ldf(reinterpret_cast<const ACT*>(a.p) + o);
  const float* p = reinterpret_cast<const float*>(a.p) + o;
  if (a.split == 1) return *p;
  float s = 0.f;
  for (int i0 = 0; i0 < a.split; i0 += 8) {
    float v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = p[(int64_t)min(i0 + u, a.split - 1) * a.plane];
#pragma unroll
    for (int u = 0; u < 8; ++u) s += i0 + u < a.split ? v[u] : 0.f;
  }
  return s;
}

struct RopeArgs {
  const float* freq;          // [rot / 2]
  float mag;                  // on cos and sin
  const int32_t* positions;
  int rot;
};

constexpr int ROPE_MAX = 1024;

// grid (rows, 1 + NB).  y = 0: RMS norm of the NC latent columns, the rotated key part behind them
// (from column RV of the cache row).  y > 0: a run of heads' rotated query parts, PQ columns (the pad zeroed) at
// qr + (t H + h) qs; where q comes as slabs its unrotated part goes to qn [T][H][dim] as activations, and the
// output gate's columns to gate [T][H vdim].
template <typename ACT>
__global__ void __launch_bounds__(256) latent_rope_kernel(LatCols kv, int NC, const float* __restrict__ wc, float eps,
                                                         const int32_t* __restrict__ slots, ACT* __restrict__ cache, int RS,
                                                         int RV, LatCols q, int H, int dim, ACT* __restrict__ qr, int qs,
                                                         int PQ, ACT* __restrict__ qn, LatCols g, int vdim, ACT* __restrict__ gate,
                                                         RopeArgs r) {
  __shared__ float red[16];
  __shared__ float2 cs[ROPE_MAX / 2];
  const int t = blockIdx.x, tid = threadIdx.x, pos = r.positions[t];
  for (int i = tid; i < r.rot / 2; i += 256) {
    float sn, co;
    sincosf((float)pos * r.freq[i], &sn, &co);
    cs[i] = make_float2(co * r.mag, sn * r.mag);
  }
  __syncthreads();
  auto rotate = [&](int i, float& u, float& v) {
    const float2 c = cs[i];
    const float a = u * c.x - v * c.y, b = v * c.x + u * c.y;
    u = a;
    v = b;
  };
  if (blockIdx.y == 0) {
    ACT* dst = cache + (size_t)slots[t] * RS;
    float x[4], s = 0.f;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int c = k * 256 + tid;
      x[k] = c < NC ? ldcol<ACT>(kv, t, c) : 0.f;
      s += x[k] * x[k];
    }
    for (int c = 1024 + tid; c < NC; c += 256) {
      const float v = ldcol<ACT>(kv, t, c);
      s += v * v;
    }
    const float rs = 1.f / sqrtf(block_sum(s, red) / (float)NC + eps);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int c = k * 256 + tid;
      if (c < NC) stf(dst + c, x[k] * rs * wc[c]);
    }
    for (int c = 1024 + tid; c < NC; c += 256) stf(dst + c, ldcol<ACT>(kv, t, c) * rs * wc[c]);
    for (int i = tid; i < r.rot / 2; i += 256) {
      float u = ldcol<ACT>(kv, t, NC + 2 * i), v = ldcol<ACT>(kv, t, NC + 2 * i + 1);
      rotate(i, u, v);
      stf(dst + RV + 2 * i, u);
      stf(dst + RV + 2 * i + 1, v);
    }
    return;
  }
  // bf16 pairs as one word
  const bool pairs = sizeof(ACT) == 2 && q.split == 0 && dim % 2 == 0 && q.ld % 2 == 0 && ((uintptr_t)q.p & 3) == 0 &&
                     qs % 2 == 0 && ((uintptr_t)qr & 3) == 0;
  const int NB = gridDim.y - 1, h0 = H * (blockIdx.y - 1) / NB, h1 = H * blockIdx.y / NB, hp = PQ / 2;
  for (int e = tid; e < (h1 - h0) * hp; e += 256) {
    const int h = h0 + e / hp, i = e % hp;
    float u = 0.f, v = 0.f;
    if (i < r.rot / 2) {
      const int c = h * (dim + r.rot) + dim + 2 * i;
      if (pairs) {
        const uint32_t w = *reinterpret_cast<const uint32_t*>(reinterpret_cast<const uint16_t*>(q.p) + t * q.ld + c);
        u = __uint_as_float(w << 16);
        v = __uint_as_float(w & 0xffff0000u);
      } else {
        u = ldcol<ACT>(q, t, c);
        v = ldcol<ACT>(q, t, c + 1);
      }
      rotate(i, u, v);
    }
    ACT* row = qr + ((size_t)t * H + h) * qs + 2 * i;
    if (pairs) {
      *reinterpret_cast<uint32_t*>(row) = pack2bf(u, v);
    } else {
      stf(row, u);
      stf(row + 1, v);
    }
  }
  if (qn)
    for (int e = h0 * dim + tid; e < h1 * dim; e += 256)
      stf(qn + (size_t)t * H * dim + e, ldcol<ACT>(q, t, e / dim * (dim + r.rot) + e % dim));
  if (gate)
    for (int e = h0 * vdim + tid; e < h1 * vdim; e += 256) stf(gate + (size_t)t * H * vdim + e, ldcol<ACT>(g, t, e));
}

// Prompt rows (q as activations): a wave per row, everything it reads requested before its first wait.  NK x 64
// latent columns; rot <= 128
template <typename ACT, int NK>
__global__ void __launch_bounds__(256) latent_rope_rows_kernel(LatCols kv, int T, int NC, const float* __restrict__ wc, float eps,
                                                              const int32_t* __restrict__ slots, ACT* __restrict__ cache,
                                                              int RS, int RV, LatCols q, int H, int dim,
                                                              ACT* __restrict__ qr, int qs, int PQ, RopeArgs r) {
  __shared__ float2 cs[4][64];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, hr = r.rot / 2;
  const int t = min((int)blockIdx.x * 4 + w, T - 1);        // rows past the last: the last one again
  const int pos = r.positions[t];
  ACT* dst = cache + (size_t)slots[t] * RS;
  float x[NK];
#pragma unroll
  for (int k = 0; k < NK; ++k) x[k] = ldcol<ACT>(kv, t, min(64 * k + lane, NC - 1));
  const int pr = min(lane, max(hr - 1, 0));
  float ku = ldcol<ACT>(kv, t, NC + 2 * pr), kw = ldcol<ACT>(kv, t, NC + 2 * pr + 1);
  float sn, co;
  sincosf((float)pos * r.freq[pr], &sn, &co);
  const float2 mine = make_float2(co * r.mag, sn * r.mag);
  cs[w][lane] = mine;
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  float s = 0.f;
#pragma unroll
  for (int k = 0; k < NK; ++k) s += 64 * k + lane < NC ? x[k] * x[k] : 0.f;
  const float rs = 1.f / sqrtf(wave_sum(s) / (float)NC + eps);
#pragma unroll
  for (int k = 0; k < NK; ++k)
    if (64 * k + lane < NC) stf(dst + 64 * k + lane, x[k] * rs * wc[64 * k + lane]);
  if (lane < hr) {
    stf(dst + RV + 2 * lane, ku * mine.x - kw * mine.y);
    stf(dst + RV + 2 * lane + 1, kw * mine.x + ku * mine.y);
  }
  const int hp = PQ / 2, n = H * hp, step = dim + r.rot;
  const ACT* qrow = reinterpret_cast<const ACT*>(q.p) + (int64_t)t * q.ld + dim;
  ACT* orow = qr + (size_t)t * H * qs;
  for (int e0 = 0; e0 < n; e0 += 512) {
    float u[8], v[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int e = min(e0 + 64 * k + lane, n - 1), h = e / hp, i = min(e % hp, hr - 1);
      const ACT* p = qrow + h * step + 2 * i;
      if constexpr (sizeof(ACT) == 2) {
        const uint32_t b = *reinterpret_cast<const uint32_t*>(p);
        u[k] = __uint_as_float(b << 16);
        v[k] = __uint_as_float(b & 0xffff0000u);
      } else {
        u[k] = ldf(p);
        v[k] = ldf(p + 1);
      }
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int e = e0 + 64 * k + lane, h = min(e, n - 1) / hp, i = min(e, n - 1) % hp;
      if (e >= n) continue;
      const float2 c = cs[w][min(i, 63)];
      const float a = i < hr ? u[k] * c.x - v[k] * c.y : 0.f, b = i < hr ? v[k] * c.x + u[k] * c.y : 0.f;
      ACT* o = orow + h * qs + 2 * i;
      if constexpr (sizeof(ACT) == 2) *reinterpret_cast<uint32_t*>(o) = pack2bf(a, b);
      else { stf(o, a); stf(o + 1, b); }
    }
  }
}

// ---------------------------------------------------------------------------------- head_linear
// W [H][NP][KP] zero-padded (NP % 64 == 0, KP % 32 == 0).  Operands: A = W rows, B = token rows, so a
// lane ends with four consecutive outputs of one token.  grid (token tiles, NP / (16 NT 4), H), four
// waves side by side over the outputs, each with TT x NT 16 x 16 tiles.
__device__ __forceinline__ f32x4_t mfma16(uint4 a, uint4 b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0,
                                                 0, 0);
}

__device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + __expf(-z)); }

// four consecutive outputs times the sigmoid of their gates
__device__ __forceinline__ void gate4(float (&v)[4], const uint16_t* g) {
  const uint2 u = *reinterpret_cast<const uint2*>(g);
  v[0] *= sigmoid(__uint_as_float(u.x << 16));
  v[1] *= sigmoid(__uint_as_float(u.x & 0xffff0000u));
  v[2] *= sigmoid(__uint_as_float(u.y << 16));
  v[3] *= sigmoid(__uint_as_float(u.y & 0xffff0000u));
}

template <bool VEC>
__device__ __forceinline__ uint4 ld_frag(const uint16_t* p, int k, int K) {
  if constexpr (VEC) {
    return k < K ? *reinterpret_cast<const uint4*>(p + k) : make_uint4(0, 0, 0, 0);
  } else {
    uint32_t w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const uint32_t lo = k + 2 * i < K ? p[k + 2 * i] : 0, hi = k + 2 * i + 1 < K ? p[k + 2 * i + 1] : 0;
      w[i] = lo | (hi << 16);
    }
    return make_uint4(w[0], w[1], w[2], w[3]);
  }
}

template <int TT, int NT, bool VEC>
__global__ void __launch_bounds__(256) head_linear_kernel(const uint16_t* __restrict__ x, int64_t ldx, int64_t hsx,
                                                         const uint16_t* __restrict__ w, int NP, int KP, int T, int N,
                                                         int K, uint16_t* __restrict__ out, int64_t ldo, int64_t hso,
                                                         const uint16_t* __restrict__ gate, int64_t ldg) {
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, col = lane & 15, kq = lane >> 4;
  const int h = blockIdx.z, t0 = blockIdx.x * 16 * TT, n0 = (blockIdx.y * 4 + wv) * 16 * NT;
  if (n0 >= NP) return;
  const uint16_t* wp = w + ((size_t)h * NP + n0 + col) * KP + 8 * kq;
  const uint16_t* xp[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) xp[i] = x + (int64_t)min(t0 + 16 * i + col, T - 1) * ldx + h * hsx;
  f32x4_t acc[NT][TT];
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int i = 0; i < TT; ++i) acc[j][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  // RK steps of K a round, all their loads requested before the first product
  constexpr int RK = VEC ? 4 : 1;
  for (int k = 0; k < KP; k += 32 * RK) {
    uint4 a[RK][NT], b[RK][TT];
#pragma unroll
    for (int u = 0; u < RK; ++u) {
      const int kk = min(k + 32 * u, KP - 32);
#pragma unroll
      for (int j = 0; j < NT; ++j) a[u][j] = *reinterpret_cast<const uint4*>(wp + (size_t)16 * j * KP + kk);
#pragma unroll
      for (int i = 0; i < TT; ++i) b[u][i] = ld_frag<VEC>(xp[i], kk + 8 * kq, K);
    }
#pragma unroll
    for (int u = 0; u < RK; ++u)
      if (k + 32 * u < KP)
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
          for (int i = 0; i < TT; ++i) acc[j][i] = mfma16(a[u][j], b[u][i], acc[j][i]);
  }
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int t = t0 + 16 * i + col;
    if (t >= T) continue;
    uint16_t* o = out + (int64_t)t * ldo + h * hso;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int n = n0 + 16 * j + 4 * kq;
      if constexpr (VEC) {
        if (n < N) {
          float v[4] = {acc[j][i][0], acc[j][i][1], acc[j][i][2], acc[j][i][3]};
          if (gate) gate4(v, gate + (int64_t)t * ldg + (size_t)h * N + n);
          *reinterpret_cast<uint2*>(o + n) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
        }
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float v = acc[j][i][e];
          if (n + e < N) o[n + e] = f2bf(gate ? v * sigmoid(bf2f(gate[(int64_t)t * ldg + (size_t)h * N + n + e])) : v);
        }
      }
    }
  }
}

// few tokens: the four waves of a workgroup share 16 outputs of 16 TT tokens, each a quarter of K with
// all its loads in flight in rounds of four steps, and their sums meet in LDS
template <int TT>
__global__ void __launch_bounds__(256) head_linear_ks_kernel(const uint16_t* __restrict__ x, int64_t ldx, int64_t hsx,
                                                            const uint16_t* __restrict__ w, int NP, int KP, int T, int N,
                                                            int K, uint16_t* __restrict__ out, int64_t ldo, int64_t hso,
                                                         const uint16_t* __restrict__ gate, int64_t ldg) {
  __shared__ float4 red[3][TT][64];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, col = lane & 15, kq = lane >> 4;
  const int h = blockIdx.z, t0 = blockIdx.x * 16 * TT, n0 = blockIdx.y * 16;
  const int ks = KP / 32, k0 = ks * wv / 4, k1 = ks * (wv + 1) / 4;
  const uint16_t* wp = w + ((size_t)h * NP + n0 + col) * KP + 8 * kq;
  const uint16_t* xp[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) xp[i] = x + (int64_t)min(t0 + 16 * i + col, T - 1) * ldx + h * hsx;
  f32x4_t acc[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k = k0; k < k1; k += 4) {
    uint4 a[4], b[4][TT];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int kk = 32 * min(k + u, k1 - 1);
      a[u] = *reinterpret_cast<const uint4*>(wp + kk);
#pragma unroll
      for (int i = 0; i < TT; ++i) b[u][i] = ld_frag<true>(xp[i], kk + 8 * kq, K);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (k + u < k1)
#pragma unroll
        for (int i = 0; i < TT; ++i) acc[i] = mfma16(a[u], b[u][i], acc[i]);
  }
  if (wv) {
#pragma unroll
    for (int i = 0; i < TT; ++i) red[wv - 1][i][lane] = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
  }
  __syncthreads();
  if (wv) return;
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    float v[4] = {acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
#pragma unroll
    for (int u = 0; u < 3; ++u) {
      const float4 r = red[u][i][lane];
      v[0] += r.x; v[1] += r.y; v[2] += r.z; v[3] += r.w;
    }
    const int t = t0 + 16 * i + col, n = n0 + 4 * kq;
    if (t < T && n < N) {
      if (gate) gate4(v, gate + (int64_t)t * ldg + (size_t)h * N + n);
      *reinterpret_cast<uint2*>(out + (int64_t)t * ldo + h * hso + n) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
    }
  }
}

__global__ void __launch_bounds__(256) head_linear_f32_kernel(const float* __restrict__ x, int64_t ldx, int64_t hsx,
                                                             const float* __restrict__ w, int NP, int KP, int N, int K,
                                                             float* __restrict__ out, int64_t ldo, int64_t hso,
                                                             const float* __restrict__ gate, int64_t ldg) {
  const int n = blockIdx.y * 256 + threadIdx.x, t = blockIdx.x, h = blockIdx.z;
  if (n >= N) return;
  const float* xr = x + t * ldx + h * hsx;
  const float* wr = w + ((size_t)h * NP + n) * KP;
  float s = 0.f;
  for (int k = 0; k < K; ++k) s += xr[k] * wr[k];
  if (gate) s *= sigmoid(gate[t * ldg + (size_t)h * N + n]);
  out[t * ldo + h * hso + n] = s;
}

// ---------------------------------------------------------------------------------- latent_attn
struct LatArgs {
  const int32_t* block_tables;
  const int32_t* cu_q;        // null: one token per sequence
  const int32_t* ctx_lens;    // cached + new tokens
  const int32_t* tile_seq;    // null: tile b is rows 16 MR (b % tiles_per_seq) of sequence b / tiles_per_seq
  const int32_t* tile_m0;
  int tiles_per_seq, H, RS, RV, max_blocks, P;   // RS: columns of a key, RV: of them the value
  float scale;
  int window;                 // keys a row sees, itself included (0: all before it)
  const float* sink;          // [H] or null: exp(sink) joins the denominator once
  float* part_o;              // [rows][P][RV], unnormalised
  float* part_ml;             // [rows][P][2]: running maximum (log2 domain), sum
};

struct LatTile { int m0, rows, q_row, pos_base, kt0, kt1, kend; const int32_t* bt; };

// first key a row with ``limit`` keys before its end sees
__device__ __forceinline__ int lat_low(const LatArgs& a, int limit) { return a.window > 0 ? max(limit - a.window, 0) : 0; }

// running maximum m (log2 domain) and sum l with the row's sink: what to scale the output by
__device__ __forceinline__ float lat_inv(const LatArgs& a, int row, float m, float l) {
  if (!a.sink) return l > 0.f ? 1.f / l : 0.f;
  const float sk = a.sink[row % a.H] * 1.4426950408889634f, M = fmaxf(m, sk), f = exp2f(m - M);
  return f / (l * f + exp2f(sk - M));
}

// the tile's rows and its slice of 64-key tiles
__device__ __forceinline__ LatTile lat_tile(const LatArgs& a, int tile, int p, int rows_per_tile) {
  LatTile r;
  const int s = a.tile_seq ? a.tile_seq[tile] : tile / a.tiles_per_seq;
  r.m0 = a.tile_m0 ? a.tile_m0[tile] : (tile % a.tiles_per_seq) * rows_per_tile;
  const int q0 = a.cu_q ? a.cu_q[s] : s, n = a.cu_q ? a.cu_q[s + 1] - q0 : 1;
  r.rows = n * a.H;
  r.q_row = q0 * a.H;
  r.pos_base = a.ctx_lens[s] - n;
  r.kend = r.pos_base + (min(r.m0 + rows_per_tile, r.rows) - 1) / a.H + 1;
  const int t0 = lat_low(a, r.pos_base + r.m0 / a.H + 1) / 64, nt = (r.kend + 63) / 64 - t0;
  r.kt0 = t0 + (int)((int64_t)nt * p / a.P);
  r.kt1 = t0 + (int)((int64_t)nt * (p + 1) / a.P);
  r.bt = a.block_tables + (size_t)s * a.max_blocks;
  return r;
}

// workgroup barrier that orders LDS only (__syncthreads also waits for every global load issued before it)
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

constexpr int LP = 72;      // P row stride in LDS, elements (64 keys + 8 against bank conflicts)

// Eight waves, a 64-key x R64 tile of latents double-buffered in LDS (row-major, 16-byte chunks
// XOR-swizzled by the key).
//   scores   S^T = C q'^T: wave (row group rg, key group) multiplies 16-key A fragments from LDS with
//            its 16 rows' q' held in registers; a lane owns one row's scores for 4 (or 8) keys
//   softmax  per row across the lane groups by lane swaps, across the waves of a row group through LDS
//   output   O^T += C^T P^T: wave w owns latent columns 16 (w + 8 j) of every row; the C^T fragments
//            are transposing LDS reads (ds_read_b64_tr_b16) of the same tile, P^T comes from LDS
// Two phases per tile, a barrier after each: [scores of tile t + 1 | output of tile t], independent of each
// other, then [softmax of t + 1, tile t + 2 from registers into the buffer t leaves, loads of t + 3].  The
// barriers order LDS only, so the loads stay in flight across a whole tile.
template <int R64, int V64, int MR>
__global__ void __launch_bounds__(512, 1) latent_attn_kernel(const uint16_t* __restrict__ q,
                                                            const uint16_t* __restrict__ cache, LatArgs a,
                                                            uint16_t* __restrict__ out) {
  constexpr int CH = R64 / 8;                     // 16-byte chunks per key
  // chunk swizzle by key.  Rows of a multiple of 256 bytes: both the 16-row score fragments and the
  // transposing reads (two chunks of keys 0-3, 8-11 or 4-7, 12-15 together) touch every bank once
  auto swz = [](int key) {
    if constexpr (R64 % 128 == 0) {
      const int i = key & 3, q4 = (key >> 2) & 3;
      return 2 * i | (q4 & 1) | (((q4 ^ (q4 >> 1)) & 1) << 3);
    } else {
      return key & 7;
    }
  };
  constexpr int KS = R64 / 32;                    // MFMA steps over the rank
  constexpr int NL = CH / 8;                      // chunks per thread of a 64-key tile
  constexpr int KG = MR == 4 ? 2 : 1;             // 16-key groups per wave
  constexpr int SL = 4 / KG;                      // waves per row group
  constexpr int RT = V64 / 16;                    // 16-column output tiles
  constexpr int NO = (RT + 7) / 8;                // per wave
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* kbuf = smem;                                            // [2][64][R64] bf16
  uint16_t* sp = reinterpret_cast<uint16_t*>(smem + 2 * 64 * R64 * 2);   // [16 MR][LP]
  float* smax = reinterpret_cast<float*>(sp + 16 * MR * LP);    // [MR][4][16]
  float* salpha = smax + MR * 64;                               // [16 MR]

  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 15, kq = lane >> 4;
  // one XCD takes neighbouring tiles: a sequence's tiles read the same latents through one L2
  const LatTile tl = lat_tile(a, a.P == 1 ? xcd_remap(blockIdx.x, gridDim.x) : blockIdx.x, blockIdx.y, 16 * MR);
  const int RS = a.RS;

  // score role: row group and key groups of this wave (MR = 1: waves 4-7 have none)
  const int rg = MR == 1 ? 0 : w % MR, slot = MR == 1 ? w : w / MR;
  const bool scorer = slot < SL;
  const int gm = min(tl.m0 + 16 * rg + col, tl.rows - 1);
  const int limit = tl.pos_base + gm / a.H + 1;   // keys this row sees: low .. limit - 1
  const int low = lat_low(a, limit);
  u32x4_t qf[KS];
  if (scorer) {
    const uint16_t* qr = q + (size_t)(tl.q_row + gm) * RS + 8 * kq;
#pragma unroll
    for (int k = 0; k < KS; ++k)
      qf[k] = *reinterpret_cast<const u32x4_t*>(qr + min(32 * k, RS - 32));
#pragma unroll
    for (int k = 0; k < KS; ++k) qf[k] &= 32 * k < RS ? ~0u : 0u;
  }

  const int nb = (tl.kend + CFC_KV_BS - 1) / CFC_KV_BS;
  u32x4_t st[NL];
  int b0 = 0, b1 = 0;
  // the block ids of a tile's keys, asked for a phase before its latents
  auto ids = [&](int kt) {
    b0 = tl.bt[min(2 * kt, nb - 1)];
    b1 = tl.bt[min(2 * kt + 1, nb - 1)];
  };
  // unconditional (a branch per load would wait at every join): columns past the stride re-read the last
  // chunk -- q' is zero there and such outputs are not stored
  auto gload = [&]() {
    const uint16_t* p0 = cache + (size_t)b0 * 32 * RS;
    const uint16_t* p1 = cache + (size_t)b1 * 32 * RS;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = tid + 512 * i, key = e / CH, c = e % CH;
      const int off = (key & 31) * RS + min(8 * c, RS - 8);
      st[i] = *reinterpret_cast<const u32x4_t*>((key < 32 ? p0 : p1) + off);
    }
  };
  auto lwrite = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = tid + 512 * i, key = e / CH, c = e % CH;
      *reinterpret_cast<u32x4_t*>(kbuf + buf * (64 * R64 * 2) + key * (R64 * 2) + ((c ^ swz(key)) << 4)) = st[i];
    }
  };

  f32x4_t o[NO][MR];
#pragma unroll
  for (int j = 0; j < NO; ++j)
#pragma unroll
    for (int r = 0; r < MR; ++r) o[j][r] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  f32x4_t s[KG];

  auto scores = [&](int kt, int buf) {
    if (!scorer) return;
    const char* kb = kbuf + buf * (64 * R64 * 2);
    float mx = -INFINITY;
#pragma unroll
    for (int g = 0; g < KG; ++g) {
      const int key = 16 * (slot * KG + g) + col;
      const char* kr = kb + key * (R64 * 2);
      f32x4_t s0{0.f, 0.f, 0.f, 0.f}, s1{0.f, 0.f, 0.f, 0.f};
      // fragments in batches: one LDS round trip per batch, not per product
      constexpr int KB = MR == 4 && KS > 8 ? 2 : KS < 8 ? KS : (KS % 8 == 0 ? 8 : 6);
#pragma unroll
      for (int kb0 = 0; kb0 < KS; kb0 += KB) {
        uint4 kf[KB];
#pragma unroll
        for (int k = 0; k < KB; ++k)
          kf[k] = *reinterpret_cast<const uint4*>(kr + (((4 * (kb0 + k) + kq) ^ swz(key)) << 4));
        if constexpr (MR == 1) __builtin_amdgcn_sched_barrier(0);      // left alone, the reads go out two at a time
#pragma unroll
        for (int k = 0; k < KB; ++k) {
          if (k & 1) s1 = mfma16(kf[k], __builtin_bit_cast(uint4, qf[kb0 + k]), s1);
          else s0 = mfma16(kf[k], __builtin_bit_cast(uint4, qf[kb0 + k]), s0);
        }
      }
      const int k0 = kt * 64 + 16 * (slot * KG + g) + 4 * kq;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[g][i] = (unsigned)(k0 + i - low) < (unsigned)(limit - low) ? (s0[i] + s1[i]) * a.scale : -INFINITY;
        mx = fmaxf(mx, s[g][i]);
      }
    }
    mx = xor32_max(xor16_max(mx));
    if (lane < 16) smax[(rg * 4 + slot) * 16 + lane] = mx;
  };

  auto softmax = [&]() {
    if (!scorer) return;
    float mn = m;
#pragma unroll
    for (int u = 0; u < SL; ++u) mn = fmaxf(mn, smax[(rg * 4 + u) * 16 + col]);
    const float ref = mn == -INFINITY ? 0.f : mn;
    const float alpha = __builtin_amdgcn_exp2f(m - ref);      // m = -inf: 0
    m = mn;
    l *= alpha;
#pragma unroll
    for (int g = 0; g < KG; ++g) {
      float e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        e[i] = __builtin_amdgcn_exp2f(s[g][i] - ref);
        l += e[i];
      }
      *reinterpret_cast<uint2*>(sp + (16 * rg + col) * LP + 16 * (slot * KG + g) + 4 * kq) =
          make_uint2(cvt_pk_bf16_f32(e[0], e[1]), cvt_pk_bf16_f32(e[2], e[3]));
    }
    if (slot == 0 && lane < 16) salpha[16 * rg + lane] = alpha;
  };

  auto output = [&](int buf) {
    const char* kb = kbuf + buf * (64 * R64 * 2);
    uint4 pf[2][MR];
#pragma unroll
    for (int r = 0; r < MR; ++r) {
      const float al = salpha[16 * r + col];
      if (!__all(al == 1.f)) {
#pragma unroll
        for (int j = 0; j < NO; ++j) o[j][r] *= al;
      }
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        pf[kk][r] = *reinterpret_cast<const uint4*>(sp + (16 * r + col) * LP + 32 * kk + 8 * kq);
    }
    // lane i of a 16-lane group addresses 4 latent columns of key 8 kq + i / 4 and receives one column's 4
    // keys; the fragments of OB column tiles are requested before their products
    constexpr int OB = NO < 2 || (MR == 4 && KS > 8) ? 1 : 2;
#pragma unroll
    for (int j0 = 0; j0 < NO; j0 += OB) {
      uint4 cf[OB][2];
#pragma unroll
      for (int jj = 0; jj < OB; ++jj)
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
          const int rt = min(w + 8 * (j0 + jj), RT - 1);      // a tile past the last: computed, not stored
          uint32_t f[4];
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            const int key = 32 * kk + 8 * kq + 4 * u + (col >> 2), c = 2 * rt + ((col & 3) >> 1);
            const char* p = kb + key * (R64 * 2) + ((c ^ swz(key)) << 4) + 8 * (col & 1);
            const i16x4_t v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (lds_i16x4_t*)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) const char*)p);
            const uint2 vv = __builtin_bit_cast(uint2, v);
            f[2 * u] = vv.x;
            f[2 * u + 1] = vv.y;
          }
          cf[jj][kk] = make_uint4(f[0], f[1], f[2], f[3]);
        }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int jj = 0; jj < OB; ++jj)
        if (j0 + jj < NO)
#pragma unroll
          for (int kk = 0; kk < 2; ++kk)
#pragma unroll
            for (int r = 0; r < MR; ++r) o[min(j0 + jj, NO - 1)][r] = mfma16(cf[jj][kk], pf[kk][r], o[min(j0 + jj, NO - 1)][r]);
    }
  };

  // tile t + 1 into LDS from the registers, the loads of t + 2 (past the last tile: re-read, not used), the
  // block ids of t + 3
  auto advance = [&](int t, int buf) {
    if (t + 1 >= tl.kt1) return;
    lwrite(buf);
    gload();
    ids(t + 3);
  };

  if (tl.kt0 < tl.kt1) {
    const int k0 = tl.kt0;
    ids(k0);
    gload();
    ids(k0 + 1);
    advance(k0 - 1, 0);
    __syncthreads();
    scores(k0, 0);
    lds_barrier();
    softmax();
    advance(k0, 1);
    lds_barrier();
    int cur = 0;
    for (int kt = k0;; ++kt, cur ^= 1) {
      if (kt + 1 < tl.kt1) scores(kt + 1, cur ^ 1);
      output(cur);
      if (kt + 1 >= tl.kt1) break;
      lds_barrier();
      softmax();
      advance(kt + 1, cur);
      lds_barrier();
    }
  }
  // row sums over the lane groups and the row group's waves
  __syncthreads();
  if (scorer) {
    l = xor32_sum(xor16_sum(l));
    if (lane < 16) {
      smax[(rg * 4 + slot) * 16 + lane] = l;
      if (slot == 0) salpha[16 * rg + lane] = m;
    }
  }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < MR; ++r) {
    const int mrow = tl.m0 + 16 * r + col;
    if (mrow >= tl.rows) continue;
    float lt = 0.f;
#pragma unroll
    for (int u = 0; u < SL; ++u) lt += smax[(r * 4 + u) * 16 + col];
    const size_t grow = (size_t)tl.q_row + mrow;
    if (a.P > 1) {
      float* po = a.part_o + (grow * a.P + blockIdx.y) * a.RV;
#pragma unroll
      for (int j = 0; j < NO; ++j) {
        const int n = 16 * (w + 8 * j) + 4 * kq;
        if (w + 8 * j < RT && n < a.RV) *reinterpret_cast<float4*>(po + n) = make_float4(o[j][r][0], o[j][r][1], o[j][r][2], o[j][r][3]);
      }
      if (w == 0 && kq == 0) {
        float* ml = a.part_ml + (grow * a.P + blockIdx.y) * 2;
        ml[0] = salpha[16 * r + col];
        ml[1] = lt;
      }
    } else {
      const float inv = lat_inv(a, mrow, salpha[16 * r + col], lt);
      uint16_t* po = out + grow * a.RV;
#pragma unroll
      for (int j = 0; j < NO; ++j) {
        const int n = 16 * (w + 8 * j) + 4 * kq;
        if (w + 8 * j < RT && n < a.RV)
          *reinterpret_cast<uint2*>(po + n) = make_uint2(cvt_pk_bf16_f32(o[j][r][0] * inv, o[j][r][1] * inv),
                                                         cvt_pk_bf16_f32(o[j][r][2] * inv, o[j][r][3] * inv));
      }
    }
  }
}

// Any rank up to 3776 and both activation types, one wave per (token, head) row and key slice: a lane
// scores one key of 64, then owns every 64th latent column of the output.  The 32-bit path.
template <typename ACT, int LG_C>      // LG_C columns per lane
__global__ void __launch_bounds__(256) latent_attn_any_kernel(const ACT* __restrict__ q, const ACT* __restrict__ cache,
                                                             LatArgs a, ACT* __restrict__ out) {
  extern __shared__ float sq[];                 // [4][RS] q' rows, then [4][64] weights
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, RS = a.RS;
  const LatTile tl = lat_tile(a, blockIdx.x, blockIdx.y, 4);
  float* myq = sq + w * RS;
  float* pw = sq + 4 * RS + 64 * w;
  const int mrow = tl.m0 + w;
  const bool live = mrow < tl.rows;             // the other waves of the tile go on: barriers below are the tile's
  const size_t grow = (size_t)tl.q_row + (live ? mrow : tl.rows - 1);
  for (int c = lane; c < RS; c += 64) myq[c] = ldf(q + grow * RS + c);
  __syncthreads();
  const int limit = tl.pos_base + (live ? mrow : tl.rows - 1) / a.H + 1, low = lat_low(a, limit);
  float o[LG_C];
#pragma unroll
  for (int j = 0; j < LG_C; ++j) o[j] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int kt = tl.kt0; kt < tl.kt1; ++kt) {
    const int key = kt * 64 + lane;
    float s = -INFINITY;
    if (key < limit && key >= low) {
      const ACT* c = cache + ((size_t)tl.bt[key / CFC_KV_BS] * CFC_KV_BS + key % CFC_KV_BS) * RS;
      float s4[4] = {0.f, 0.f, 0.f, 0.f};
      for (int r = 0; r < RS; r += 4)
#pragma unroll
        for (int u = 0; u < 4; ++u) s4[u] += myq[r + u] * ldf(c + r + u);
      s = ((s4[0] + s4[1]) + (s4[2] + s4[3])) * a.scale;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float ref = mn == -INFINITY ? 0.f : mn;
    const float alpha = exp2f(m - ref), p = exp2f(s - ref);
    m = mn;
    l = l * alpha + wave_sum(p);
    pw[lane] = p;
    __syncthreads();
#pragma unroll
    for (int j = 0; j < LG_C; ++j) o[j] *= alpha;
    const int nk = min(64, limit - kt * 64);
    for (int k = max(0, low - kt * 64); k < nk; ++k) {
      const int kk = kt * 64 + k;
      const ACT* c = cache + ((size_t)tl.bt[kk / CFC_KV_BS] * CFC_KV_BS + kk % CFC_KV_BS) * RS;
      const float pk = pw[k];
#pragma unroll
      for (int j = 0; j < LG_C; ++j)
        if (lane + 64 * j < a.RV) o[j] += pk * ldf(c + lane + 64 * j);
    }
    __syncthreads();
  }
  if (!live) return;
  const float inv = lat_inv(a, mrow, m, l);
#pragma unroll
  for (int j = 0; j < LG_C; ++j) {
    const int c = lane + 64 * j;
    if (c >= a.RV) continue;
    if (a.P > 1) a.part_o[(grow * a.P + blockIdx.y) * a.RV + c] = o[j];
    else stf(out + grow * a.RV + c, o[j] * inv);
  }
  if (a.P > 1 && lane == 0) {
    a.part_ml[(grow * a.P + blockIdx.y) * 2] = m;
    a.part_ml[(grow * a.P + blockIdx.y) * 2 + 1] = l;
  }
}

// tiles [n][2]: {sequence, first position} of 64 tokens each, at dense rows 64 blockIdx.x ..; positions past
// the context are zero rows.  The slot-ordered copy is a product's W operand in the fragment-packed layout
// of cfc_dgemm_pack for 64-row workgroups ([rows / 64][RS / 32][4][64 lanes][8])
__global__ void __launch_bounds__(256) latent_gather_kernel(const uint16_t* __restrict__ cache,
                                                           const int32_t* __restrict__ block_tables, int max_blocks,
                                                           const int32_t* __restrict__ ctx_lens,
                                                           const int32_t* __restrict__ tiles, int RS, int RV,
                                                           uint16_t* __restrict__ rows, uint16_t* __restrict__ slot_rows,
                                                           uint16_t* __restrict__ k2) {
  const int s = tiles[2 * blockIdx.x], p0 = tiles[2 * blockIdx.x + 1], ctx = ctx_lens[s], ch = RV / 8;
  const int32_t* bt = block_tables + (size_t)s * max_blocks;
  for (int e = threadIdx.x; e < 64 * ch; e += 256) {
    const int r = e / ch, c = e % ch, p = p0 + r;
    const uint4 v = p < ctx ? *reinterpret_cast<const uint4*>(
                                  cache + ((size_t)bt[p / CFC_KV_BS] * CFC_KV_BS + p % CFC_KV_BS) * RS + 8 * c)
                            : make_uint4(0, 0, 0, 0);
    const size_t base = (size_t)blockIdx.x * 64;
    reinterpret_cast<uint4*>(rows + (base + r) * RV)[c] = v;
    const int sr = (r & 32) + kv_v_slot(r & 31);
    reinterpret_cast<uint4*>(slot_rows)[(((size_t)blockIdx.x * (RV / 32) + (c >> 2)) * 4 + (sr >> 4)) * 64 + (sr & 15) +
                                        16 * (c & 3)] = v;
  }
  if (k2)
    for (int e = threadIdx.x; e < 64 * 8; e += 256) {      // the rest of the row, padded to 64 columns
      const int r = e >> 3, c = e & 7, p = p0 + r;
      const uint4 v = p < ctx && RV + 8 * c < RS
                          ? *reinterpret_cast<const uint4*>(cache + ((size_t)bt[p / CFC_KV_BS] * CFC_KV_BS + p % CFC_KV_BS) * RS + RV + 8 * c)
                          : make_uint4(0, 0, 0, 0);
      reinterpret_cast<uint4*>(k2 + ((size_t)blockIdx.x * 64 + r) * 64)[c] = v;
    }
}

template <int R64, int V64, int MR>
int lat_go(dim3 grid, hipStream_t s, const void* q, const void* cache, const LatArgs& a, void* out) {
  constexpr int lds = 2 * 64 * R64 * 2 + 16 * MR * LP * 2 + (MR * 64 + 16 * MR) * 4;
  static bool raised = false;
  if (lds > 65536 && !raised) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attn_kernel<R64, V64, MR>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    raised = true;
  }
  latent_attn_kernel<R64, V64, MR><<<grid, 512, lds, s>>>((const uint16_t*)q, (const uint16_t*)cache, a, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

template <int R64, int V64>
int lat_mr(int mr, dim3 grid, hipStream_t s, const void* q, const void* cache, const LatArgs& a, void* out) {
  switch (mr) {
    case 1: return lat_go<R64, V64, 1>(grid, s, q, cache, a, out);
    case 2: return lat_go<R64, V64, 2>(grid, s, q, cache, a, out);
    case 4:
      if constexpr (R64 <= 512) return lat_go<R64, V64, 4>(grid, s, q, cache, a, out);      // past that the registers spill
  }
  return -3;
}

}  // namespace

CFC_API int cfc_latent_norm(int f32, const float* part, int split, int T, int NQ, int NC, const float* wq, const float* wc,
                            float eps, const int32_t* slots, void* q_out, int ldq, void* cache, int RS,
                            hipStream_t stream) {
  if (T <= 0) return 0;
  if (split < 1 || NQ < 1 || NC < 1 || NC > RS || ldq < NQ) return -1;
  const bool v4 = NQ % 4 == 0 && NC % 4 == 0 && ldq % 4 == 0;
#define LN_ARGS stream, part, split, T, NQ, NC, wq, wc, eps, slots, q_out, ldq, cache, RS
  if (f32) return v4 ? latent_norm_go<float, 4>(LN_ARGS) : latent_norm_go<float, 1>(LN_ARGS);
  return v4 ? latent_norm_go<uint16_t, 4>(LN_ARGS) : latent_norm_go<uint16_t, 1>(LN_ARGS);
#undef LN_ARGS
}

// kv columns [NC latent | rot key part], q columns per head [dim | rot]; each operand: pointer, split (0:
// activations, else fp32 slabs), row stride, slab stride.  Rotated queries: PQ columns of row t H + h at qr (row stride
// qs); qn, gate may be null
CFC_API int cfc_latent_rope(int f32, const void* kv, int kv_split, int64_t kv_ld, int64_t kv_plane, int T, int NC,
                            const float* wc, float eps, const int32_t* slots, void* cache, int RS, int RV, const void* q,
                            int q_split, int64_t q_ld, int64_t q_plane, int H, int dim, void* qr, int qs, int PQ, void* qn, const void* g,
                            int g_split, int64_t g_ld, int64_t g_plane, int vdim, void* gate, const float* freq, int rot,
                            float mag, const int32_t* positions, hipStream_t stream) {
  if (T <= 0) return 0;
  if (NC < 1 || NC > RV || RV % 2 || rot < 0 || rot % 2 || rot > ROPE_MAX || RV + rot > RS || PQ < rot || PQ % 2 || qs < PQ ||
      H < 1 || dim < 1)
    return -1;
  // few rows: up to one workgroup per head, so their slab sums do not follow one another; no more than run at once
  const int fit = T >= 512 ? 1 : max(2, 1024 / T), NB = H < fit ? H : fit < 64 ? fit : 64;
  const LatCols ckv{kv, kv_split, kv_ld, kv_plane}, cq{q, q_split, q_ld, q_plane}, cg{g, g_split, g_ld, g_plane};
  const RopeArgs r{freq, mag, positions, rot};
  // prompt rows whose pairs are words
  if (T >= 512 && q_split == 0 && rot >= 2 && rot <= 128 && NC <= 1024 && !qn && !gate && dim % 2 == 0 && q_ld % 2 == 0 &&
      qs % 2 == 0 && (((uintptr_t)q | (uintptr_t)qr) & 3) == 0) {
#define LRR(ACT, NK)                                                                                                 \
  latent_rope_rows_kernel<ACT, NK><<<(T + 3) / 4, 256, 0, stream>>>(ckv, T, NC, wc, eps, slots, (ACT*)cache, RS, RV, cq, H, \
                                                                   dim, (ACT*)qr, qs, PQ, r)
    if (NC <= 512) { if (f32) LRR(float, 8); else LRR(uint16_t, 8); }
    else if (f32) LRR(float, 16);
    else LRR(uint16_t, 16);
#undef LRR
    return CFC_CHECK_LAUNCH();
  }
#define LR(ACT)                                                                                                         \
  latent_rope_kernel<ACT><<<dim3(T, 1 + NB), 256, 0, stream>>>(ckv, NC, wc, eps, slots, (ACT*)cache, RS, RV, cq, H, dim, \
                                                              (ACT*)qr, qs, PQ, (ACT*)qn, cg, vdim, (ACT*)gate, r)
  if (f32) LR(float);
  else LR(uint16_t);
#undef LR
  return CFC_CHECK_LAUNCH();
}

// x row (t, h) at t ldx + h hsx (K values), out at t ldo + h hso (N values); W [H][NP][KP] zero-padded.
// gate (may be null): output n of head h is multiplied by the sigmoid of gate[t ldg + h N + n]
CFC_API int cfc_head_linear(int f32, const void* x, int64_t ldx, int64_t hsx, const void* w, int NP, int KP, int T, int H,
                            int N, int K, void* out, int64_t ldo, int64_t hso, const void* gate, int64_t ldg,
                            hipStream_t stream) {
  if (T <= 0) return 0;
  if (H < 1 || H > 65535 || N < 1 || K < 1 || N > NP || K > KP || NP % 64 || KP % 32) return -1;
  if (f32) {
    const dim3 grid(T, (N + 255) / 256, H);
    head_linear_f32_kernel<<<grid, 256, 0, stream>>>((const float*)x, ldx, hsx, (const float*)w, NP, KP, N, K, (float*)out,
                                                     ldo, hso, (const float*)gate, ldg);
    return CFC_CHECK_LAUNCH();
  }
  const bool vec = K % 8 == 0 && ldx % 8 == 0 && hsx % 8 == 0 && ((uintptr_t)x & 15) == 0 && N % 4 == 0 && ldo % 4 == 0 &&
                   hso % 4 == 0 && ((uintptr_t)out & 7) == 0 && ldg % 4 == 0 && ((uintptr_t)gate & 7) == 0;
#define HL(TT, NT, V)                                                                                                 \
  head_linear_kernel<TT, NT, V><<<dim3((T + 16 * TT - 1) / (16 * TT), (NP + 64 * NT - 1) / (64 * NT), H), 256, 0, stream>>>( \
      (const uint16_t*)x, ldx, hsx, (const uint16_t*)w, NP, KP, T, N, K, (uint16_t*)out, ldo, hso, (const uint16_t*)gate, ldg)
#define HK(TT)                                                                                                   \
  head_linear_ks_kernel<TT><<<dim3((T + 16 * TT - 1) / (16 * TT), (N + 15) / 16, H), 256, 0, stream>>>(          \
      (const uint16_t*)x, ldx, hsx, (const uint16_t*)w, NP, KP, T, N, K, (uint16_t*)out, ldo, hso, (const uint16_t*)gate, ldg)
  if (!vec) HL(4, 1, false);
  else if (T <= 256 && KP >= 256 && T <= 16) HK(1);
  else if (T <= 64 && KP >= 256) HK(2);
  else if (T <= 256 && KP >= 256) HK(4);
  else if (T <= 16) HL(1, 1, true);
  else if (T <= 256) HL(4, 1, true);
  else HL(4, 2, true);
#undef HL
#undef HK
  return CFC_CHECK_LAUNCH();
}

// rows_per_tile: 16 / 32 / 64 on the MFMA kernel (bf16, RS <= 512; 16 / 32 for RS <= 576 with RV <= 512), 4 on the
// general one.  A cached row's RS columns are the key, its first RV the value; out [rows][RV]
CFC_API int cfc_latent_attention(int f32, const void* q, const void* cache, const int32_t* block_tables,
                                 const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* tile_seq,
                                 const int32_t* tile_m0, int n_tiles, int tiles_per_seq, int rows_per_tile, int H, int RS,
                                 int RV, int max_blocks, float scale, int window, const float* sink, int P, int total_rows, float* part_o, float* part_ml,
                                 void* out, hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (H < 1 || RS < 32 || RS % 32 || RV < 32 || RV % 32 || RV > RS || P < 1 || P > MERGE_MAXP || max_blocks < 1 || window < 0)
    return -1;
  if ((tile_seq == nullptr) != (tile_m0 == nullptr) || (!tile_seq && tiles_per_seq < 1)) return -1;
  if (P > 1 && (!part_o || !part_ml)) return -2;
  LatArgs a{block_tables, cu_q, ctx_lens, tile_seq, tile_m0, tiles_per_seq, H, RS, RV, max_blocks, P,
            scale * 1.4426950408889634f, window, sink, part_o, part_ml};
  const dim3 grid(n_tiles, P);
  int rc = -3;
  if (rows_per_tile == 4) {
    if (RS > 3776) return -4;                   // 4 query rows + the weights in 64 KB of LDS
    const size_t lds = (size_t)(4 * RS + 256) * 4;
#define LA_ANY(T, C) latent_attn_any_kernel<T, C><<<grid, 256, lds, stream>>>((const T*)q, (const T*)cache, a, (T*)out)
    if (RS <= 1024) { if (f32) LA_ANY(float, 16); else LA_ANY(uint16_t, 16); }
    else if (f32) LA_ANY(float, 64);
    else LA_ANY(uint16_t, 64);
#undef LA_ANY
    rc = CFC_CHECK_LAUNCH();
  } else {
    if (f32 || RV > 512 || RS > 576) return -4;
    const int mr = rows_per_tile / 16, rv = (RV + 63) / 64;
#define LAT(R, V) rc = lat_mr<R, V>(mr, grid, stream, q, cache, a, out); break
    switch ((RS + 63) / 64) {
      case 1: LAT(64, 64);
      case 2: if (rv == 1) { LAT(128, 64); } else { LAT(128, 128); }
      case 3: if (rv <= 2) { LAT(192, 128); } else { LAT(192, 192); }
      case 4: if (rv <= 2) { LAT(256, 128); } else { LAT(256, 256); }
      case 5: case 6: if (rv <= 4) { LAT(384, 256); } else { LAT(384, 384); }
      case 7: case 8: if (rv <= 6) { LAT(512, 384); } else { LAT(512, 512); }
      default: LAT(576, 512);
    }
#undef LAT
  }
  if (rc || P == 1) return rc;
  OutGate g;
  g.ld = (int64_t)H * RV;
  if (f32) slice_merge_kernel<float><<<total_rows, 128, 0, stream>>>(part_o, part_ml, P, RV, RV, sink, H, g, (float*)out);
  else slice_merge_kernel<uint16_t><<<total_rows, 128, 0, stream>>>(part_o, part_ml, P, RV, RV, sink, H, g, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

CFC_API int cfc_latent_gather(const void* cache, const int32_t* block_tables, int max_blocks, const int32_t* ctx_lens,
                              const int32_t* tiles, int n_tiles, int RS, int RV, void* rows, void* slot_rows, void* k2,
                              hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (RV < 32 || RV % 32 || RS < RV || RS % 8 || (k2 && RS - RV > 64) || max_blocks < 1) return -1;
  latent_gather_kernel<<<n_tiles, 256, 0, stream>>>((const uint16_t*)cache, block_tables, max_blocks, ctx_lens, tiles, RS,
                                                    RV, (uint16_t*)rows, (uint16_t*)slot_rows, (uint16_t*)k2);
  return CFC_CHECK_LAUNCH();
}
