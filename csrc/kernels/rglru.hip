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
//                  lane groups are composed with lane swaps.  Once for what each segment does to the state, then (behind
//                  carry, recur.h) again from the states, for the outputs: cheaper than keeping 32-bit gates.  Where the
//                  portions alone fill the chip each is one segment, and the second pass does it all
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
  const float* p = reinterpret_cast<const float*>(a.p) + o;
  for (int p0 = 0; p0 < a.split; p0 += 4) {            // four slabs in flight (past the last: re-read, not added)
    Vec<V> v[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) v[s] = ldv<V>(p + min(p0 + s, a.split - 1) * a.plane);
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int e = 0; e < V; ++e) y.v[e] += p0 + s < a.split ? v[s].v[e] : 0.f;
  }
  return y;
}

__device__ __forceinline__ f32x4_t mfma16(u32x4_t a, u32x4_t b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// 1 - a^2 for a = e^la, la <= 0: near 1 by the series of -expm1(2 la), whose next term is la^3 / 3 of it
template <typename ACT> __device__ __forceinline__ float one_minus_sq(float la, float a);
template <> __device__ __forceinline__ float one_minus_sq<float>(float la, float) { return -expm1f(2.f * la); }
template <> __device__ __forceinline__ float one_minus_sq<uint16_t>(float la, float a) {
  const float s = la * (-2.f + la * (-2.f - la * (4.f / 3.f)));
  return la > -0.015f ? s : 1.f - a * a;
}
template <typename ACT> __device__ __forceinline__ float root(float x);
template <> __device__ __forceinline__ float root<float>(float x) { return sqrtf(x); }
template <> __device__ __forceinline__ float root<uint16_t>(float x) { return __builtin_amdgcn_sqrtf(x); }

// far below zero e^-x is infinite and 1 / (1 + e^-x) zero
template <typename ACT>
__device__ __forceinline__ float sigm(float x) { return over1<ACT>(exp_of<ACT>(-x)); }

// decay a and contribution of one token from the gates' pre-activations
template <typename ACT>
__device__ __forceinline__ void lru_gates(float pr, float pi, float u, float rate, float& a, float& b) {
  const float la = rate * sigm<ACT>(pr);
  a = exp_of<ACT>(la);
  b = root<ACT>(one_minus_sq<ACT>(la, a)) * sigm<ACT>(pi) * u;
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
// grid (segments, blocks * NP / 64 rounded up); chunks [n][2] {first row, rows}.  Tiles of 32 tokens of u in LDS, double
// buffered, in two steps of 16; a lane's four tokens of a step are 4 kq .. of one channel.
//   SCAN_SUMS   sums [n][2][W]: what each segment does to the state
//   SCAN_APPLY  outputs, from the state ahead of each segment in sums
//   SCAN_WHOLE  a segment is a portion (chunks null: cu_q): outputs, from the sequence's state, which is updated
enum { SCAN_SUMS = 0, SCAN_APPLY = 1, SCAN_WHOLE = 2 };
constexpr int SCAN_TILE = 32;

template <int KS, int MODE>
__global__ void __launch_bounds__(256, KS <= 4 ? 4 : KS <= 8 ? 3 : 2) rglru_scan_kernel(LruArgs a, const uint16_t* __restrict__ u,
                                                                         const int32_t* __restrict__ chunks,
                                                                         const int32_t* __restrict__ cu_q,
                                                                         const int32_t* __restrict__ ctx_lens,
                                                                         float* __restrict__ sums, uint16_t* __restrict__ out) {
  constexpr int LDU = 32 * KS + 8, NL = SCAN_TILE * 4 * KS / 256 > 0 ? SCAN_TILE * 4 * KS / 256 : 1;      // 16-byte pieces per thread
  __shared__ __attribute__((aligned(16))) uint16_t tile[2][SCAN_TILE][LDU];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, col = lane & 15, kq = lane >> 4;
  const int groups = (a.NP + 63) / 64, blk = blockIdx.y / groups, n0 = min((blockIdx.y - blk * groups) * 64 + 16 * w, a.NP - 16);
  const bool mine = (blockIdx.y - blk * groups) * 64 + 16 * w < a.NP;      // else a wave that only loads
  const int row0 = MODE == SCAN_WHOLE ? cu_q[blockIdx.x] : chunks[2 * blockIdx.x];
  const int n = MODE == SCAN_WHOLE ? cu_q[blockIdx.x + 1] - row0 : chunks[2 * blockIdx.x + 1];
  const int UW = a.blocks * a.KP, W = a.W, kb = a.KP / 32;
  const bool live = mine && n0 + col < a.bs;
  const int ku = min(n0 + col, a.bs - 1), c = blk * a.bs + ku;
  u32x4_t wr[KS], wi[KS];
  {
    const uint16_t* p = reinterpret_cast<const uint16_t*>(a.wg) + ((size_t)blk * a.NP + n0 + col) * a.KP + 8 * kq;
    const size_t second = (size_t)a.blocks * a.NP * a.KP;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int o = 32 * min(k, kb - 1);
      wr[k] = *reinterpret_cast<const u32x4_t*>(p + o);
      wi[k] = *reinterpret_cast<const u32x4_t*>(p + second + o);
      if (k >= kb) wr[k] = wi[k] = u32x4_t{0, 0, 0, 0};        // steps past the block's: its last columns against zeros
    }
  }
  const float br = a.br[c], bi = a.bi[c], rate = a.rate[c], by = MODE ? a.by[c] : 0.f;
  const uint16_t* ub = u + (size_t)row0 * UW + (size_t)blk * a.KP;
  const uint16_t* yb = MODE ? reinterpret_cast<const uint16_t*>(a.y.p) + (int64_t)row0 * a.y.ld + c : nullptr;
  float* sp = MODE == SCAN_WHOLE ? a.state + (size_t)a.slots[blockIdx.x] * W + c : sums + (size_t)blockIdx.x * 2 * W + c;
  float S = 0.f, A = 1.f;
  if (MODE == SCAN_APPLY || (MODE == SCAN_WHOLE && ctx_lens[blockIdx.x] > n)) S = sp[0];

  u32x4_t pre[NL];
  uint16_t yv[2][4], yn[2][4];
  const int pieces = SCAN_TILE * 4 * kb;
  int prow[NL], pk[NL];                                 // row and columns of this thread's pieces
#pragma unroll
  for (int i = 0; i < NL; ++i) {
    const int e = min(tid + 256 * i, pieces - 1);      // past the last: it again
    prow[i] = e / (4 * kb);
    pk[i] = 8 * (e - prow[i] * 4 * kb);
  }
  auto fetch = [&](int t) {                            // rows past the segment: its last
#pragma unroll
    for (int i = 0; i < NL; ++i) pre[i] = *reinterpret_cast<const u32x4_t*>(ub + (size_t)min(t + prow[i], n - 1) * UW + pk[i]);
    if constexpr (MODE != SCAN_SUMS)
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int e = 0; e < 4; ++e) yn[h][e] = yb[min(t + 16 * h + 4 * kq + e, n - 1) * a.y.ld];
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NL; ++i) *reinterpret_cast<u32x4_t*>(&tile[buf][prow[i]][pk[i]]) = pre[i];
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int e = 0; e < 4; ++e) yv[h][e] = yn[h][e];
  };
  fetch(0);
  put(0);
  __syncthreads();
  for (int t = 0, buf = 0; t < n; t += SCAN_TILE, buf ^= 1) {
    if (t + SCAN_TILE < n) fetch(t + SCAN_TILE);
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      f32x4_t pr{br, br, br, br}, pi{bi, bi, bi, bi};
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const u32x4_t uf = *reinterpret_cast<const u32x4_t*>(&tile[buf][16 * h + col][32 * min(k, kb - 1) + 8 * kq]);
        pr = mfma16(uf, wr[k], pr);
        pi = mfma16(uf, wi[k], pi);
      }
      float ta[4], tb[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        lru_gates<uint16_t>(pr[e], pi[e], bf2f(tile[buf][16 * h + 4 * kq + e][ku]), rate, ta[e], tb[e]);
      if (t + 16 * h + 16 > n)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (t + 16 * h + 4 * kq + e >= n) {
            ta[e] = 1.f;
            tb[e] = 0.f;
          }
      float ga = ta[0], gb = tb[0];
#pragma unroll
      for (int e = 1; e < 4; ++e) {
        ga *= ta[e];
        gb = ta[e] * gb + tb[e];
      }
      // composition over the four lane groups: swaps leave every lane with both values of its pair of groups, then of the
      // two pairs, in their order
      float ea = ga, eb = gb, oa = ga, ob = gb;
      swap16(ea, oa);
      swap16(eb, ob);
      float fa = ea * oa, fb = oa * eb + ob, la = fa, lb = fb;
      swap32(fa, la);
      swap32(fb, lb);
      if constexpr (MODE != SCAN_SUMS) {
        float s = kq & 2 ? fa * S + fb : S;
        s = kq & 1 ? ea * s + eb : s;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s = ta[e] * s + tb[e];
          const int r = t + 16 * h + 4 * kq + e;
          if (r < n && live) out[(size_t)(row0 + r) * W + c] = f2bf(s * gelu_tanh<uint16_t>(bf2f(yv[h][e]) + by));
        }
      } else {
        A *= fa * la;
      }
      S = la * (fa * S + fb) + lb;
    }
    if (t + SCAN_TILE < n) put(buf ^ 1);
    __syncthreads();
  }
  if (kq == 0 && live) {
    if (MODE == SCAN_SUMS) {
      sp[0] = A;
      sp[W] = S;
    } else if (MODE == SCAN_WHOLE) {
      sp[0] = S;
    }
  }
}

// ------------------------------------------------------------------------------------------ one token per sequence
// u of up to 16 rows x a block's columns into LDS (row stride ldu), the block's raw inputs into the state by the workgroup
// whose channels n0 .. n1 they are
template <typename ACT, typename LT, int V>
__device__ __forceinline__ void step_conv(const LruArgs& a, int b0, int nb, int blk, int n0, int n1, const int32_t* positions, LT* ul,
                                          int ldu) {
  constexpr int IN = 2;                                // vectors a thread asks for together
  const int nv = a.KP / V, back = a.taps - 1, items = nb * nv;
  const bool same = blockDim.x % nv == 0;              // a thread's vectors are of the same channels
  for (int i0 = threadIdx.x; i0 < items; i0 += IN * blockDim.x) {
    Vec<V> x[IN], o[IN][3], y[IN], bx[IN], w[IN][4];
    int64_t at[IN];
    int ps[IN];
#pragma unroll
    for (int j = 0; j < IN; ++j) {                     // past the last or in the pad: another's, not stored
      const int i = min(i0 + j * (int)blockDim.x, items - 1), r = i / nv, k = (i - r * nv) * V, b = b0 + r;
      const int c = blk * a.bs + min(k, a.bs - V);
      ps[j] = positions[b];
      at[j] = (int64_t)a.slots[b] * a.taps * a.W + c;
      x[j] = lru_ld<ACT, V>(a.x, b, c);
      if (j && same) {
        bx[j] = bx[0];
        y[j] = y[0];
#pragma unroll
        for (int d = 0; d < 4; ++d) w[j][d] = w[0][d];
      } else {
        bx[j] = ldv<V>(a.bx + c);
        y[j] = ldv<V>(a.cb + c);
#pragma unroll
        for (int d = 0; d < 4; ++d) w[j][d] = ldv<V>(a.conv + (size_t)max(back - d, 0) * a.W + c);
      }
#pragma unroll
      for (int d = 1; d <= 3; ++d) o[j][d - 1] = ldv<V>(a.tail + at[j] + (size_t)(max(ps[j] - d, 0) % a.taps) * a.W);
    }
#pragma unroll
    for (int j = 0; j < IN; ++j) {
      const int i = i0 + j * (int)blockDim.x, r = i / nv, k = (i - r * nv) * V, pos = ps[j];
      if (i >= items) break;
      if (k >= a.bs) {
        stv<V>(ul + r * ldu + k, zerov<V>());
        continue;
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
        y[j].v[e] += w[j][0].v[e] * (x[j].v[e] + bx[j].v[e]);
#pragma unroll
        for (int d = 1; d <= 3; ++d) y[j].v[e] += d <= back && d <= pos ? w[j][d].v[e] * (o[j][d - 1].v[e] + bx[j].v[e]) : 0.f;
      }
      for (int d = 4; d <= back && d <= pos; ++d) {
        const int c = blk * a.bs + k;
        const Vec<V> od = ldv<V>(a.tail + at[j] + (size_t)((pos - d) % a.taps) * a.W), wd = ldv<V>(a.conv + (size_t)(back - d) * a.W + c);
#pragma unroll
        for (int e = 0; e < V; ++e) y[j].v[e] += wd.v[e] * (od.v[e] + bx[j].v[e]);
      }
      if (back > 0 && k >= n0 && k < n1) stv<V>(a.tail + at[j] + (size_t)(pos % a.taps) * a.W, x[j]);
      stv<V>(ul + r * ldu + k, y[j]);
    }
  }
}

// 1-D grid of rows / 16 x blocks x NP / 16 NW, rounded up each; where eight divides the blocks, an XCD takes all of a block's,
// so that its matrices and inputs come into one L2.  NW waves of 16 channels.  V: vectors of channels (4 or 1)
template <int V, int NW>
__global__ void __launch_bounds__(64 * NW) rglru_step_kernel(LruArgs a, const int32_t* __restrict__ positions,
                                                        const int32_t* __restrict__ ctx_lens, int B, uint16_t* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* ul = reinterpret_cast<uint16_t*>(smem);
  const int ldu = a.KP + 8, W = a.W;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, col = lane & 15, kq = lane >> 4;
  const int groups = (a.NP + 16 * NW - 1) / (16 * NW), per = groups * ((B + 15) / 16);
  int blk = blockIdx.x / per, rest = blockIdx.x - blk * per;
  if (a.blocks % 8 == 0) {
    const int i = blockIdx.x / 8;
    blk = blockIdx.x % 8 + 8 * (i / per);
    rest = i % per;
  }
  const int g0 = rest % groups * (16 * NW), n0 = g0 + 16 * w, b0 = 16 * (rest / groups), nb = min(16, B - b0);
  const int b = b0 + min(col, nb - 1);
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
  const uint16_t* p = reinterpret_cast<const uint16_t*>(a.wg) + ((size_t)blk * a.NP + min(n0, a.NP - 16) + col) * a.KP + 8 * kq;
  const size_t second = (size_t)a.blocks * a.NP * a.KP;
  const int KS = a.KP / 32;
  u32x4_t wr[4], wi[4];                                // four steps' matrices in flight (past the last: again, not used)
  auto matrices = [&](int s0) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int o = 32 * min(s0 + j, KS - 1);
      wr[j] = *reinterpret_cast<const u32x4_t*>(p + o);
      wi[j] = *reinterpret_cast<const u32x4_t*>(p + second + o);
    }
  };
  matrices(0);
  step_conv<uint16_t, uint16_t, V>(a, b0, nb, blk, g0, g0 + 16 * NW, positions, ul, ldu);
  __syncthreads();
  if (n0 >= a.NP) return;
  f32x4_t pr{0.f, 0.f, 0.f, 0.f}, pi{0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < KS; s0 += 4) {
    if (s0) matrices(s0);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (s0 + j < KS) {                               // columns past the rows there are: not looked at
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
    step_conv<ACT, float, 1>(a, t, 1, blk, 0, a.bs, positions, ul, a.KP);
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
    // many rows: more channels per workgroup, so that fewer repeat a row's convolution
    const int nw = B >= 32 && NP > 64 ? 8 : 4, grid = (B + 15) / 16 * blocks * ((NP + 16 * nw - 1) / (16 * nw));
    const size_t lds = (size_t)16 * (KP + 8) * 2;
    const bool v4 = bs % 4 == 0 && lru_cols_vec(a.x, 0) && lru_cols_vec(a.y, 0) && ((uintptr_t)out & 7) == 0;
#define ST(V, NW) rglru_step_kernel<V, NW><<<grid, 64 * NW, lds, stream>>>(a, positions, ctx_lens, B, (uint16_t*)out)
    if (nw == 8) { if (v4) ST(4, 8); else ST(1, 8); }
    else if (v4) ST(4, 4);
    else ST(1, 4);
#undef ST
    return CFC_CHECK_LAUNCH();
  }
  if (KP > LRU_ANY_MAX) return -3;
  const dim3 grid(B, blocks);
  if (f32) rglru_any_kernel<float><<<grid, 256, (size_t)KP * 4, stream>>>(a, nullptr, positions, ctx_lens, nullptr, (float*)out);
  else rglru_any_kernel<uint16_t><<<grid, 256, (size_t)KP * 4, stream>>>(a, nullptr, positions, ctx_lens, nullptr, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

// packed portions, x and y activations.  tiles as in short_conv; chunks [n][2] {first row, rows} (segments), chunk_cu
// [portions + 1], or whole: every portion one segment (both unused); u scratch [T][blocks KP] activations; sums scratch, n or (general path) T times 2 W floats
CFC_API int cfc_rglru_prefill(int f32, const void* x, int64_t x_ld, const void* y, int64_t y_ld, const float* bx, const float* conv,
                              const float* cb, int taps, const float* br, const float* bi, const float* rate, const float* by,
                              const void* wg, int blocks, int bs, int KP, int NP, float* tail, float* state, const int32_t* slots,
                              const int32_t* tiles, int n_tiles, int whole, const int32_t* chunks, int n_chunks, const int32_t* chunk_cu,
                              const int32_t* cu_q, const int32_t* ctx_lens, int portions, int T, void* u, float* sums, void* out,
                              hipStream_t stream) {
  if (T <= 0 || portions <= 0) return 0;
  if (blocks < 1 || bs < 1 || KP < bs || KP % 4 || taps < 1 || !wg || !tail || !state || !slots || !tiles || !cu_q ||
      !ctx_lens || !u || n_tiles < 1)
    return -1;
  const bool mfma = !f32 && KP <= cfc_rglru_max_block();
  if ((mfma && !whole && (!chunks || !chunk_cu || n_chunks < 1)) || (!(mfma && whole) && !sums)) return -1;
  if (!f32 && (KP % 32 || NP < bs || NP % 16)) return -2;
  const LruArgs a{{x, 0, x_ld, 0}, {y, 0, y_ld, 0}, bx, conv, cb, taps, br, bi, rate, by, wg, blocks, bs, KP, NP, blocks * bs, tail,
                  state, slots};
  const bool v4 = bs % 4 == 0 && lru_cols_vec(a.x, f32);
  int rc;
  if (f32) rc = v4 ? conv_go<float, 4>(stream, n_tiles, a, tiles, u) : conv_go<float, 1>(stream, n_tiles, a, tiles, u);
  else rc = v4 ? conv_go<uint16_t, 4>(stream, n_tiles, a, tiles, u) : conv_go<uint16_t, 1>(stream, n_tiles, a, tiles, u);
  if (rc) return rc;
  if (mfma) {
    const dim3 grid(whole ? portions : n_chunks, blocks * ((NP + 63) / 64));
    const uint16_t* up = (const uint16_t*)u;
#define RS(KS, M) rglru_scan_kernel<KS, M><<<grid, 256, 0, stream>>>(a, up, chunks, cu_q, ctx_lens, sums, (uint16_t*)out)
#define RP(M)                    \
  if (KP <= 64) RS(2, M);        \
  else if (KP <= 128) RS(4, M);  \
  else if (KP <= 256) RS(8, M);  \
  else RS(16, M)
    if (whole) {
      RP(SCAN_WHOLE);
      return CFC_CHECK_LAUNCH();
    }
    RP(SCAN_SUMS);
    if (const int e = CFC_CHECK_LAUNCH()) return e;
    if (a.W % 4) carry_kernel<1><<<dim3(portions, (a.W + 63) / 64), 64, 0, stream>>>(chunk_cu, cu_q, ctx_lens, slots, a.W, sums, state);
    else carry_kernel<4><<<dim3(portions, (a.W + 255) / 256), 64, 0, stream>>>(chunk_cu, cu_q, ctx_lens, slots, a.W, sums, state);
    RP(SCAN_APPLY);
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
