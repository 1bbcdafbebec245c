// Real-gated linear recurrence with block-diagonal gates, behind a short convolution, element by element
//   u = conv(x + bx) + cb over time,   r = sigmoid(R u + br),   i = sigmoid(I u + bi)   (R, I: one square matrix per block)
//   a = exp(rate r)   (rate <= 0 per channel),   S_t = a S_(t-1) + sqrt(1 - a^2) i u
// and out = S_t gelu(y + by), gelu in its tanh form.  States are fp32, a row per sequence slot; a sequence's first token
// starts from zero whatever the slot holds.  The convolution's earlier inputs x lie in the sequence's slot too, as the
// projection leaves them: [slots][taps][W] fp32, position p at p % taps (one row more than is read, so that the row being
// stored is not one that another workgroup still reads).
//   * short_conv   prompt rows: u as rows [T][blocks][KP], a block's columns padded with zeros to whole operands
//   * rglru_scan   segments of prompt portions on the matrix cores: a wave keeps the gate matrices of its 16 channels in
//                  registers and takes 16 tokens at a time; a lane holds four neighbouring tokens of one channel, the four
//                  lane groups are composed with shuffles.  Once for what each segment does to the state, then (behind
//                  carry, recur.h) again from the states, for the outputs: cheaper than keeping 32-bit gates
//   * rglru_step   one token per sequence, straight from a joint product's slabs: convolution, gates, state, output
//   * rglru_any    any block size and the 32-bit path, prompt rows and decoded ones: gates a workgroup per (row, block),
//                  then a thread per channel
#include "recur.h"

#include <type_traits>

namespace {

typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));

struct LruCols { const void* p; int split; int64_t ld, plane; };      // split 0: activations, else fp32 slabs

struct LruArgs {
  LruCols x, y;
  const float* bx; const float* conv; const float* cb; int taps;      // conv [taps][W]
  const float* br; const float* bi; const float* rate; const float* by;
  const void* wg;              // bf16: [2][blocks][NP][KP] rows of R, then I; fp32: [2][blocks][k][n]
  int blocks, bs, KP, NP, W;   // bs columns per block, W = blocks bs
  float* tail;
  float* state;                // [slots][W]
  const int32_t* slots;
};

template <typename ACT, int V>
__device__ __forceinline__ Vec<V> lru_ld(const LruCols& a, int64_t t, int c) {
  const int64_t o = t * a.ld + c;
  if (a.split == 0) return ldv<V>(reinterpret_cast<const ACT*>(a.p) + o);
  Vec<V> y = zerov<V>();
  add_slabs<V>(y, reinterpret_cast<const float*>(a.p), a.split, a.plane, (size_t)o);
  return y;
}

__device__ __forceinline__ f32x4_t mfma16(u32x4_t a, u32x4_t b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// -expm1(z) for z <= 0: 1 - e^z keeps its digits near zero
template <typename ACT> __device__ __forceinline__ float one_minus_exp(float z);
template <> __device__ __forceinline__ float one_minus_exp<float>(float z) { return -expm1f(z); }
template <> __device__ __forceinline__ float one_minus_exp<uint16_t>(float z) {
  const float s = -z * (1.f + z * (0.5f + z * (1.f / 6.f + z * (1.f / 24.f))));       // next term z^4 / 120
  return z > -0.125f ? s : 1.f - exp_of<uint16_t>(z);
}
template <typename ACT> __device__ __forceinline__ float root(float x);
template <> __device__ __forceinline__ float root<float>(float x) { return sqrtf(x); }
template <> __device__ __forceinline__ float root<uint16_t>(float x) { return __builtin_amdgcn_sqrtf(x); }

template <typename ACT>
__device__ __forceinline__ float sigm(float x) { return over1<ACT>(exp_of<ACT>(fminf(-x, 80.f))); }

// decay a and contribution of one token from the gates' pre-activations
template <typename ACT>
__device__ __forceinline__ void lru_gates(float pr, float pi, float u, float rate, float& a, float& b) {
  const float la = rate * sigm<ACT>(pr);
  a = exp_of<ACT>(la);
  b = root<ACT>(fmaxf(one_minus_exp<ACT>(2.f * la), 0.f)) * sigm<ACT>(pi) * u;
}

// z / 2 (1 + tanh(k (z + 0.044715 z^3))) = z sigmoid(2 k (..)), k = sqrt(2 / pi)
template <typename ACT>
__device__ __forceinline__ float gelu_tanh(float z) { return z * sigm<ACT>(1.5957691216057308f * z * (1.f + 0.044715f * z * z)); }

__device__ __forceinline__ float round_act(float v, const uint16_t*) { return bf2f(f2bf(v)); }
__device__ __forceinline__ float round_act(float v, const float*) { return v; }

// ------------------------------------------------------------------------------------------ convolution, prompt rows
// tiles [2][n][4] {first row, rows, first position, sequence}, {portion rows before the tile, the portion's rows, 0, 0}; a
// portion's tiles but the last hold at least taps - 1 rows, so only its first tile reads the state, and then stores it.
// grid (tiles, vectors).  TAPS 0: any number
template <typename ACT, int V, int TAPS>
__global__ void __launch_bounds__(256) short_conv_kernel(LruArgs a, const int32_t* __restrict__ tiles, ACT* __restrict__ u) {
  const int taps = TAPS ? TAPS : a.taps, W = a.W, UW = a.blocks * a.KP;
  const int row0 = tiles[4 * blockIdx.x], n = tiles[4 * blockIdx.x + 1], pos0 = tiles[4 * blockIdx.x + 2];
  const int seq = tiles[4 * blockIdx.x + 3], lead = tiles[4 * (gridDim.x + blockIdx.x)];
  const int uc = (blockIdx.y * 256 + threadIdx.x) * V;
  if (uc >= UW) return;
  const int blk = uc / a.KP, k = uc - blk * a.KP;
  if (k >= a.bs) {                                     // the pad
    const Vec<V> z = zerov<V>();
    for (int r = 0; r < n; ++r) stv<V>(u + (size_t)(row0 + r) * UW + uc, z);
    return;
  }
  const int c = blk * a.bs + k;
  const Vec<V> bx = ldv<V>(a.bx + c), cb = ldv<V>(a.cb + c);
  float* st = a.tail + (size_t)a.slots[seq] * taps * W + c;
  auto raw = [&](int r) {                              // the projection of row row0 + r
    return r >= -lead ? ldv<V>(reinterpret_cast<const ACT*>(a.x.p) + (row0 + r) * a.x.ld + c)
                      : ldv<V>(st + (size_t)((pos0 + r) % taps) * W);
  };
  auto input = [&](int r) {
    if (pos0 + r < 0) return zerov<V>();
    Vec<V> v = raw(r);
#pragma unroll
    for (int e = 0; e < V; ++e) v.v[e] += bx.v[e];
    return v;
  };
  if constexpr (TAPS > 0) {
    Vec<V> w[TAPS], win[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = ldv<V>(a.conv + (size_t)j * W + c);
#pragma unroll
    for (int j = 0; j + 1 < TAPS; ++j) win[j + 1] = input(j - (TAPS - 1));
    Vec<V> next = input(0);
    for (int r = 0; r < n; ++r) {
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j) win[j] = win[j + 1];
      win[TAPS - 1] = next;
      next = input(min(r + 1, n - 1));
      Vec<V> y = cb;
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += w[j].v[e] * win[j].v[e];
      stv<V>(u + (size_t)(row0 + r) * UW + uc, y);
    }
  } else {
    for (int r = 0; r < n; ++r) {
      Vec<V> y = cb;
      for (int j = 0; j < taps; ++j) {
        const Vec<V> s = input(r - taps + 1 + j), w = ldv<V>(a.conv + (size_t)j * W + c);
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += w.v[e] * s.v[e];
      }
      stv<V>(u + (size_t)(row0 + r) * UW + uc, y);
    }
  }
  if (lead == 0) {
    const int N = tiles[4 * (gridDim.x + blockIdx.x) + 1];
    for (int r = max(0, N - (taps - 1)); r < N; ++r) stv<V>(st + (size_t)((pos0 + r) % taps) * W, raw(r));
  }
}

// ------------------------------------------------------------------------------------------ gates and scan, prompt rows
// the segment's steps of 16 tokens; a lane's four tokens are 4 kq .. of one channel.  grid (segments, blocks * NP / 64
// rounded up); chunks [n][2] {first row, rows}; sums [n][2][W]: decay and contribution, or (APPLY) the state ahead
template <int KS, bool APPLY>
__global__ void __launch_bounds__(256, KS <= 8 ? 2 : 1) rglru_scan_kernel(LruArgs a, const uint16_t* __restrict__ u,
                                                                         const int32_t* __restrict__ chunks,
                                                                         float* __restrict__ sums, uint16_t* __restrict__ out) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, col = lane & 15, kq = lane >> 4;
  const int groups = (a.NP + 63) / 64, blk = blockIdx.y / groups, n0 = (blockIdx.y - blk * groups) * 64 + 16 * w;
  if (n0 >= a.NP) return;
  const int row0 = chunks[2 * blockIdx.x], n = chunks[2 * blockIdx.x + 1], UW = a.blocks * a.KP, W = a.W;
  const bool live = n0 + col < a.bs;
  const int c = blk * a.bs + min(n0 + col, a.bs - 1);
  u32x4_t wr[KS], wi[KS];
  {
    const uint16_t* p = reinterpret_cast<const uint16_t*>(a.wg) + ((size_t)blk * a.NP + n0 + col) * a.KP + 8 * kq;
    const size_t second = (size_t)a.blocks * a.NP * a.KP;
#pragma unroll
    for (int k = 0; k < KS; ++k) {                     // steps past the block's: the last again, against zeros
      const int o = 32 * min(k, a.KP / 32 - 1);
      wr[k] = *reinterpret_cast<const u32x4_t*>(p + o);
      wi[k] = *reinterpret_cast<const u32x4_t*>(p + second + o);
    }
  }
  const float br = a.br[c], bi = a.bi[c], rate = a.rate[c], by = APPLY ? a.by[c] : 0.f;
  const uint16_t* ub = u + (size_t)row0 * UW + (size_t)blk * a.KP;
  const uint16_t* yb = reinterpret_cast<const uint16_t*>(a.y.p) + (APPLY ? (int64_t)row0 * a.y.ld + c : 0);
  const int ku = min(n0 + col, a.bs - 1);
  float* sp = sums + (size_t)blockIdx.x * 2 * W + c;
  float S = APPLY ? sp[0] : 0.f, A = 1.f;
  u32x4_t uf[KS], un[KS];
  uint16_t uo[4], uon[4], yo[4], yon[4];
  auto load = [&](int t, u32x4_t* f, uint16_t* o, uint16_t* yv) {      // rows past the segment: its last
    const uint16_t* p = ub + (size_t)min(t + col, n - 1) * UW + 8 * kq;
#pragma unroll
    for (int k = 0; k < KS; ++k) f[k] = *reinterpret_cast<const u32x4_t*>(p + 32 * min(k, a.KP / 32 - 1));
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = min(t + 4 * kq + e, n - 1);
      o[e] = ub[(size_t)r * UW + ku];
      if (APPLY) yv[e] = yb[r * a.y.ld];
    }
  };
  load(0, uf, uo, yo);
  for (int t = 0; t < n; t += 16) {
    load(t + 16, un, uon, yon);
    f32x4_t pr{0.f, 0.f, 0.f, 0.f}, pi{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      if (32 * k < a.KP) {
        pr = mfma16(uf[k], wr[k], pr);
        pi = mfma16(uf[k], wi[k], pi);
      }
    }
    float ta[4], tb[4], ga = 1.f, gb = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      lru_gates<uint16_t>(pr[e] + br, pi[e] + bi, bf2f(uo[e]), rate, ta[e], tb[e]);
      if (t + 4 * kq + e >= n) {
        ta[e] = 1.f;
        tb[e] = 0.f;
      }
      ga *= ta[e];
      gb = ta[e] * gb + tb[e];
    }
    // composition over the four lane groups, up to and with the own one
#pragma unroll
    for (int d = 16; d <= 32; d *= 2) {
      const float pa = __shfl(ga, lane - d, 64), pb = __shfl(gb, lane - d, 64);
      if (lane >= d) {
        gb = ga * pb + gb;
        ga = ga * pa;
      }
    }
    const float la = __shfl(ga, 48 + col, 64), lb = __shfl(gb, 48 + col, 64);
    if constexpr (APPLY) {
      float ea = __shfl(ga, lane - 16, 64), eb = __shfl(gb, lane - 16, 64);
      if (kq == 0) {
        ea = 1.f;
        eb = 0.f;
      }
      float s = ea * S + eb;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s = ta[e] * s + tb[e];
        const int r = t + 4 * kq + e;
        if (r < n && live) out[(size_t)(row0 + r) * W + c] = f2bf(s * gelu_tanh<uint16_t>(bf2f(yo[e]) + by));
      }
      S = la * S + lb;
    } else {
      S = la * S + lb;
      A *= la;
    }
#pragma unroll
    for (int k = 0; k < KS; ++k) uf[k] = un[k];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      uo[e] = uon[e];
      if (APPLY) yo[e] = yon[e];
    }
  }
  if (!APPLY && kq == 0 && live) {
    sp[0] = A;
    sp[W] = S;
  }
}

// ------------------------------------------------------------------------------------------ one token per sequence
// u of 16 rows x a block's columns into LDS (row stride ldu), the block's raw inputs into the state by the workgroup whose
// channels n0 .. n1 they are
template <typename ACT, typename LT, int V>
__device__ __forceinline__ void step_conv(const LruArgs& a, int b0, int nb, int rows, int blk, int n0, int n1,
                                          const int32_t* positions, LT* ul, int ldu) {
  const int nv = a.KP / V, back = a.taps - 1;
  for (int i = threadIdx.x; i < rows * nv; i += blockDim.x) {
    const int r = i / nv, k = (i - r * nv) * V;
    Vec<V> y = zerov<V>();
    if (r < nb && k < a.bs) {
      const int b = b0 + r, c = blk * a.bs + k, pos = positions[b];
      float* st = a.tail + (size_t)a.slots[b] * a.taps * a.W + c;
      const Vec<V> x = lru_ld<ACT, V>(a.x, b, c), bx = ldv<V>(a.bx + c), w0 = ldv<V>(a.conv + (size_t)back * a.W + c);
      y = ldv<V>(a.cb + c);
      Vec<V> o[3], w[3];                               // three rows back asked for together
#pragma unroll
      for (int d = 1; d <= 3; ++d) {
        const bool on = d <= back && d <= pos;
        o[d - 1] = on ? ldv<V>(st + (size_t)((pos - d) % a.taps) * a.W) : zerov<V>();
        w[d - 1] = on ? ldv<V>(a.conv + (size_t)(back - d) * a.W + c) : zerov<V>();
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
        y.v[e] += w0.v[e] * (x.v[e] + bx.v[e]);
#pragma unroll
        for (int d = 0; d < 3; ++d) y.v[e] += w[d].v[e] * (o[d].v[e] + bx.v[e]);
      }
      for (int d = 4; d <= back && d <= pos; ++d) {
        const Vec<V> od = ldv<V>(st + (size_t)((pos - d) % a.taps) * a.W), wd = ldv<V>(a.conv + (size_t)(back - d) * a.W + c);
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += wd.v[e] * (od.v[e] + bx.v[e]);
      }
      if (back > 0 && k >= n0 && k < n1) stv<V>(st + (size_t)(pos % a.taps) * a.W, x);
    }
    stv<V>(ul + r * ldu + k, y);
  }
}

// grid (rows / 16, blocks * NP / 64 rounded up); four waves of 16 channels.  V: vectors of channels (4 or 1)
template <int V>
__global__ void __launch_bounds__(256) rglru_step_kernel(LruArgs a, const int32_t* __restrict__ positions,
                                                        const int32_t* __restrict__ ctx_lens, int B, uint16_t* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* ul = reinterpret_cast<uint16_t*>(smem);
  const int ldu = a.KP + 8, W = a.W;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, col = lane & 15, kq = lane >> 4;
  const int groups = (a.NP + 63) / 64, blk = blockIdx.y / groups, g0 = (blockIdx.y - blk * groups) * 64, n0 = g0 + 16 * w;
  const int b0 = 16 * blockIdx.x, nb = min(16, B - b0), b = b0 + min(col, nb - 1);
  // this lane's row and channels 4 kq .. of the wave's: what the end needs, asked for first
  const int k0 = n0 + 4 * kq;
  const bool on = col < nb && k0 < a.bs;
  const int c = blk * a.bs + min(k0, a.bs - 1);
  float* sp = a.state + (size_t)a.slots[b] * W + c;
  Vec<4> S = zerov<4>(), y = zerov<4>(), br, bi, rate;
  auto get = [&](auto ld) {
    Vec<4> r;
    if constexpr (V == 4) {
      r = ld(0, std::integral_constant<int, 4>{});
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) r.v[e] = ld(k0 + e < a.bs ? e : 0, std::integral_constant<int, 1>{}).v[0];
    }
    return r;
  };
  if (on) {
    if (ctx_lens[b] > 1) S = get([&](int e, auto n) { return ldv<decltype(n)::value>(sp + e); });
    y = get([&](int e, auto n) { return lru_ld<uint16_t, decltype(n)::value>(a.y, b, c + e); });
    const Vec<4> by = get([&](int e, auto n) { return ldv<decltype(n)::value>(a.by + c + e); });
    br = get([&](int e, auto n) { return ldv<decltype(n)::value>(a.br + c + e); });
    bi = get([&](int e, auto n) { return ldv<decltype(n)::value>(a.bi + c + e); });
    rate = get([&](int e, auto n) { return ldv<decltype(n)::value>(a.rate + c + e); });
#pragma unroll
    for (int e = 0; e < 4; ++e) y.v[e] += by.v[e];
  }
  step_conv<uint16_t, uint16_t, V>(a, b0, nb, 16, blk, g0, g0 + 64, positions, ul, ldu);
  __syncthreads();
  if (n0 >= a.NP) return;
  f32x4_t pr{0.f, 0.f, 0.f, 0.f}, pi{0.f, 0.f, 0.f, 0.f};
  const uint16_t* p = reinterpret_cast<const uint16_t*>(a.wg) + ((size_t)blk * a.NP + n0 + col) * a.KP + 8 * kq;
  const size_t second = (size_t)a.blocks * a.NP * a.KP;
  const int KS = a.KP / 32;
  for (int s0 = 0; s0 < KS; s0 += 4) {                 // four steps' matrices in flight (past the last: again, not used)
    u32x4_t wr[4], wi[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int o = 32 * min(s0 + j, KS - 1);
      wr[j] = *reinterpret_cast<const u32x4_t*>(p + o);
      wi[j] = *reinterpret_cast<const u32x4_t*>(p + second + o);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (s0 + j < KS) {
        const u32x4_t uf = *reinterpret_cast<const u32x4_t*>(ul + col * ldu + 32 * (s0 + j) + 8 * kq);
        pr = mfma16(wr[j], uf, pr);
        pi = mfma16(wi[j], uf, pi);
      }
  }
  if (!on) return;
  Vec<4> o;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    float ga, gb;
    lru_gates<uint16_t>(pr[e] + br.v[e], pi[e] + bi.v[e], bf2f(ul[col * ldu + min(k0 + e, a.bs - 1)]), rate.v[e], ga, gb);
    S.v[e] = ga * S.v[e] + gb;
    o.v[e] = S.v[e] * gelu_tanh<uint16_t>(y.v[e]);
  }
  uint16_t* dst = out + (size_t)b * W + c;
  if constexpr (V == 4) {
    stv<4>(sp, S);
    stv<4>(dst, o);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (k0 + e < a.bs) {
        sp[e] = S.v[e];
        dst[e] = f2bf(o.v[e]);
      }
  }
}

// ------------------------------------------------------------------------------------------ any size, 32 bits
// element (row n, column k) of block blk's matrix `which`
__device__ __forceinline__ float gate_w(const LruArgs& a, const uint16_t*, int which, int blk, int k, int n) {
  return bf2f(reinterpret_cast<const uint16_t*>(a.wg)[(((size_t)which * a.blocks + blk) * a.NP + n) * a.KP + k]);
}
__device__ __forceinline__ float gate_w(const LruArgs& a, const float*, int which, int blk, int k, int n) {
  return reinterpret_cast<const float*>(a.wg)[(((size_t)which * a.blocks + blk) * a.bs + k) * a.bs + n];
}

// grid (rows, blocks), dynamic LDS: the row's u of the block in fp32.  u null: one token per sequence, its convolution here
// and its state and output at once; else ab [T][2][W] gets decay and contribution
template <typename ACT>
__global__ void __launch_bounds__(256) rglru_any_kernel(LruArgs a, const ACT* __restrict__ u, const int32_t* __restrict__ positions,
                                                       const int32_t* __restrict__ ctx_lens, float* __restrict__ ab,
                                                       ACT* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* ul = reinterpret_cast<float*>(smem);
  const int t = blockIdx.x, blk = blockIdx.y, W = a.W;
  if (u) {
    for (int k = threadIdx.x; k < a.bs; k += 256) ul[k] = ld1(u + (size_t)t * a.blocks * a.KP + blk * a.KP + k);
  } else {
    step_conv<ACT, float, 1>(a, t, 1, 1, blk, 0, a.bs, positions, ul, a.KP);
    __syncthreads();
    for (int k = threadIdx.x; k < a.bs; k += 256) ul[k] = round_act(ul[k], (const ACT*)nullptr);
  }
  __syncthreads();
  for (int n = threadIdx.x; n < a.bs; n += 256) {
    float pr = 0.f, pi = 0.f;
    for (int k = 0; k < a.bs; ++k) {
      pr += gate_w(a, (const ACT*)nullptr, 0, blk, k, n) * ul[k];
      pi += gate_w(a, (const ACT*)nullptr, 1, blk, k, n) * ul[k];
    }
    const int c = blk * a.bs + n;
    float ga, gb;
    lru_gates<ACT>(pr + a.br[c], pi + a.bi[c], ul[n], a.rate[c], ga, gb);
    if (u) {
      ab[(size_t)t * 2 * W + c] = ga;
      ab[(size_t)t * 2 * W + W + c] = gb;
      continue;
    }
    float* sp = a.state + (size_t)a.slots[t] * W + c;
    const float S = ga * (ctx_lens[t] > 1 ? *sp : 0.f) + gb;
    *sp = S;
    const Vec<1> o{{S * gelu_tanh<ACT>(lru_ld<ACT, 1>(a.y, t, c).v[0] + a.by[c])}};
    stv<1>(out + (size_t)t * W + c, o);
  }
}

// grid (portions, channels / 64): a portion's rows in turn
template <typename ACT>
__global__ void __launch_bounds__(64) rglru_rows_kernel(LruArgs a, const float* __restrict__ ab, const int32_t* __restrict__ cu_q,
                                                       const int32_t* __restrict__ ctx_lens, ACT* __restrict__ out) {
  const int s = blockIdx.x, c = blockIdx.y * 64 + threadIdx.x, W = a.W;
  if (c >= W) return;
  const int r0 = cu_q[s], r1 = cu_q[s + 1];
  float* sp = a.state + (size_t)a.slots[s] * W + c;
  float S = ctx_lens[s] > r1 - r0 ? *sp : 0.f;
  const float by = a.by[c];
  for (int r = r0; r < r1; r += 8) {
    float ga[8], gb[8], y[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int t = min(r + k, r1 - 1);
      ga[k] = ab[(size_t)t * 2 * W + c];
      gb[k] = ab[(size_t)t * 2 * W + W + c];
      y[k] = ld1(reinterpret_cast<const ACT*>(a.y.p) + t * a.y.ld + c);
    }
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (r + k < r1) {
        S = ga[k] * S + gb[k];
        const Vec<1> o{{S * gelu_tanh<ACT>(y[k] + by)}};
        stv<1>(out + (size_t)(r + k) * W + c, o);
      }
  }
  *sp = S;
}

template <typename ACT, int V>
int conv_go(hipStream_t s, int n, const LruArgs& a, const int32_t* tiles, void* u) {
  const dim3 grid(n, (a.blocks * a.KP + 256 * V - 1) / (256 * V));
#define SC(T) short_conv_kernel<ACT, V, T><<<grid, 256, 0, s>>>(a, tiles, (ACT*)u)
  switch (a.taps) {
    case 1: SC(1); break;
    case 2: SC(2); break;
    case 3: SC(3); break;
    case 4: SC(4); break;
    default: SC(0); break;
  }
#undef SC
  return CFC_CHECK_LAUNCH();
}

bool lru_cols_vec(const LruCols& a, int f32) {
  return a.ld % 4 == 0 && a.plane % 4 == 0 && ((uintptr_t)a.p & (a.split == 0 && !f32 ? 7 : 15)) == 0;
}

constexpr int LRU_ANY_MAX = 12288;       // block columns of the general kernel (its LDS)

}  // namespace

// tokens per segment of the prompt kernels; widest block they take
CFC_API int cfc_rglru_segment() { return 128; }
CFC_API int cfc_rglru_max_block() { return 512; }

// x, y: columns of products (pointer, split (0: activations, else fp32 slabs), row stride, slab stride).  wg: bf16
// [2][blocks][NP][KP] (zero pad; KP a multiple of 32, NP of 16) or fp32 [2][blocks][k][n] with KP a multiple of 4
CFC_API int cfc_rglru_step(int f32, const void* x, int x_split, int64_t x_ld, int64_t x_plane, const void* y, int y_split,
                           int64_t y_ld, int64_t y_plane, const float* bx, const float* conv, const float* cb, int taps,
                           const float* br, const float* bi, const float* rate, const float* by, const void* wg, int blocks, int bs,
                           int KP, int NP, float* tail, float* state, const int32_t* slots, const int32_t* positions,
                           const int32_t* ctx_lens, int B, void* out, hipStream_t stream) {
  if (B <= 0) return 0;
  if (blocks < 1 || bs < 1 || KP < bs || KP % 4 || taps < 1 || !wg || !tail || !state || !slots || !positions || !ctx_lens) return -1;
  if (!f32 && (KP % 32 || NP < bs || NP % 16)) return -2;
  const LruArgs a{{x, x_split, x_ld, x_plane}, {y, y_split, y_ld, y_plane}, bx, conv, cb, taps, br, bi, rate, by, wg, blocks, bs, KP,
                  NP, blocks * bs, tail, state, slots};
  if (!f32 && KP <= 1024) {
    const dim3 grid((B + 15) / 16, blocks * ((NP + 63) / 64));
    const size_t lds = (size_t)16 * (KP + 8) * 2;
    const bool v4 = bs % 4 == 0 && lru_cols_vec(a.x, 0) && lru_cols_vec(a.y, 0) && ((uintptr_t)out & 7) == 0;
    if (v4) rglru_step_kernel<4><<<grid, 256, lds, stream>>>(a, positions, ctx_lens, B, (uint16_t*)out);
    else rglru_step_kernel<1><<<grid, 256, lds, stream>>>(a, positions, ctx_lens, B, (uint16_t*)out);
    return CFC_CHECK_LAUNCH();
  }
  if (KP > LRU_ANY_MAX) return -3;
  const dim3 grid(B, blocks);
  if (f32) rglru_any_kernel<float><<<grid, 256, (size_t)KP * 4, stream>>>(a, nullptr, positions, ctx_lens, nullptr, (float*)out);
  else rglru_any_kernel<uint16_t><<<grid, 256, (size_t)KP * 4, stream>>>(a, nullptr, positions, ctx_lens, nullptr, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

// packed portions, x and y activations.  tiles as in short_conv; chunks [n][2] {first row, rows} (segments), chunk_cu
// [portions + 1]; u scratch [T][blocks KP] activations; sums scratch, n or (general path) T times 2 W floats
CFC_API int cfc_rglru_prefill(int f32, const void* x, int64_t x_ld, const void* y, int64_t y_ld, const float* bx, const float* conv,
                              const float* cb, int taps, const float* br, const float* bi, const float* rate, const float* by,
                              const void* wg, int blocks, int bs, int KP, int NP, float* tail, float* state, const int32_t* slots,
                              const int32_t* tiles, int n_tiles, const int32_t* chunks, int n_chunks, const int32_t* chunk_cu,
                              const int32_t* cu_q, const int32_t* ctx_lens, int portions, int T, void* u, float* sums, void* out,
                              hipStream_t stream) {
  if (T <= 0 || portions <= 0) return 0;
  if (blocks < 1 || bs < 1 || KP < bs || KP % 4 || taps < 1 || !wg || !tail || !state || !slots || !tiles || !chunks || !chunk_cu || !cu_q ||
      !ctx_lens || !u || !sums || n_tiles < 1 || n_chunks < 1)
    return -1;
  if (!f32 && (KP % 32 || NP < bs || NP % 16)) return -2;
  const LruArgs a{{x, 0, x_ld, 0}, {y, 0, y_ld, 0}, bx, conv, cb, taps, br, bi, rate, by, wg, blocks, bs, KP, NP, blocks * bs, tail,
                  state, slots};
  const bool v4 = bs % 4 == 0 && lru_cols_vec(a.x, f32);
  int rc;
  if (f32) rc = v4 ? conv_go<float, 4>(stream, n_tiles, a, tiles, u) : conv_go<float, 1>(stream, n_tiles, a, tiles, u);
  else rc = v4 ? conv_go<uint16_t, 4>(stream, n_tiles, a, tiles, u) : conv_go<uint16_t, 1>(stream, n_tiles, a, tiles, u);
  if (rc) return rc;
  if (!f32 && KP <= cfc_rglru_max_block()) {
    const dim3 grid(n_chunks, blocks * ((NP + 63) / 64));
    const uint16_t* up = (const uint16_t*)u;
#define RS(KS, AP) rglru_scan_kernel<KS, AP><<<grid, 256, 0, stream>>>(a, up, chunks, sums, (uint16_t*)out)
#define RP(AP)                \
  if (KP <= 64) RS(2, AP);    \
  else if (KP <= 128) RS(4, AP); \
  else if (KP <= 256) RS(8, AP); \
  else RS(16, AP)
    RP(false);
    if (const int e = CFC_CHECK_LAUNCH()) return e;
    if (a.W % 4) carry_kernel<1><<<dim3(portions, (a.W + 63) / 64), 64, 0, stream>>>(chunk_cu, cu_q, ctx_lens, slots, a.W, sums, state);
    else carry_kernel<4><<<dim3(portions, (a.W + 255) / 256), 64, 0, stream>>>(chunk_cu, cu_q, ctx_lens, slots, a.W, sums, state);
    RP(true);
#undef RP
#undef RS
    return CFC_CHECK_LAUNCH();
  }
  if (KP > LRU_ANY_MAX) return -3;
  const dim3 rows(portions, (a.W + 63) / 64);
  if (f32) {
    rglru_any_kernel<float><<<dim3(T, blocks), 256, (size_t)KP * 4, stream>>>(a, (const float*)u, nullptr, nullptr, sums, nullptr);
    rglru_rows_kernel<float><<<rows, 64, 0, stream>>>(a, sums, cu_q, ctx_lens, (float*)out);
  } else {
    rglru_any_kernel<uint16_t><<<dim3(T, blocks), 256, (size_t)KP * 4, stream>>>(a, (const uint16_t*)u, nullptr, nullptr, sums, nullptr);
    rglru_rows_kernel<uint16_t><<<rows, 64, 0, stream>>>(a, sums, cu_q, ctx_lens, (uint16_t*)out);
  }
  return CFC_CHECK_LAUNCH();
}
