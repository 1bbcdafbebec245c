// Residual-stream kernels for decoders that keep a 32-bit stream and look back in depth and in time:
//
//   * embed_f32          token rows of a bf16 / fp32 table as the fp32 stream, scaled, with the positions' sinusoids if asked
//   * depth_norm         X_new = x + sublayer outputs (fp32 split-K slabs, bias), x' = sum_j a_j X_j over
//                        the results of every earlier layer, and the RMS norm that follows, one row per
//                        workgroup.  Three endings: the norm's 1 / rms only (a prompt's rows, before
//                        input_conv), the normed row (the model's last norm), or the normed row run
//                        through both sublayers' input convolutions with the cached tail (decode)
//   * depth_pre          the older results' share of the next few layers' averages, in one pass over them
//   * input_conv         h + conv(h) over time on each channel, for both sublayers at once, over a packed
//                        batch of prompt portions
//   * clamped_glu        min(g, limit) sigmoid(alpha g (1 + cubic g^2)) (clamp(u, +-limit) + beta), optional biases
//   * softcap            cap * tanh(x / cap), in place on fp32
//
// The tail of a sequence's convolution inputs lives in the paged cache, beside the KV block that holds
// the position: tail[block][slot][width] fp32, slot = position % slots.  A block therefore carries what
// a sequence that continues (or shares) it needs, and freeing the block frees the tail.  slots is
// taps + 1 (at most one block's 32 positions): taps - 1 inputs are live, and two spare rows keep a
// position that is run again (a decode graph's warm-up) from overwriting what it reads.
// Or it lives in a slot per sequence (max_blocks 0: block_tables holds each sequence's slot): then the tile that a portion
// starts with also stores the portion's last inputs, after it has read the old ones.
//
// ACT is the activation type the matrix products read: uint16_t (bf16 bits) or float.
#include "rows.h"

#include <type_traits>

namespace {

__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

template <typename TAB>
__global__ void __launch_bounds__(256) embed_f32_kernel(float* __restrict__ out, const TAB* __restrict__ table,
                                                       const int32_t* __restrict__ ids, int W, int vocab, float scale,
                                                       const int32_t* __restrict__ positions, const double* __restrict__ turns) {
  const int t = blockIdx.x;
  const int id = min(max(ids[t], 0), vocab - 1);
  const double pos = positions ? positions[t] : 0;
  const TAB* row = table + (size_t)id * W;
  float* o = out + (size_t)t * W;
  if (!positions) {
    for (int c = threadIdx.x; c < W; c += 256) o[c] = scale * ld1(row + c);
    return;
  }
  for (int c = 2 * threadIdx.x; c < W; c += 512) {
    // turns per position in 64 bits: the angle's fraction of a turn keeps its digits however far the position
    const double n = pos * turns[c >> 1];
    float sn, co;
    sincospif(2.f * (float)(n - floor(n)), &sn, &co);
    o[c] = scale * ld1(row + c) + sn;
    if (c + 1 < W) o[c + 1] = scale * ld1(row + c + 1) + co;
  }
}

// What a convolution input of an earlier step is read from.
struct TailArg {
  float* tail;                    // [blocks][slots][W]
  const int32_t* block_tables;    // [sequences][max_blocks], or [sequences] slots
  int max_blocks, slots;
};

__device__ __forceinline__ float* tail_row(const TailArg& a, int seq, int pos, int W) {
  const int blk = a.block_tables[a.max_blocks ? (size_t)seq * a.max_blocks + pos / CFC_KV_BS : (size_t)seq];
  return a.tail + ((size_t)blk * a.slots + pos % a.slots) * W;
}

enum { DN_RSTD = 0, DN_NORM = 1, DN_CONV = 2 };

struct DepthArgs {
  const float* x_in;      // current stream [T][W]
  float* hist;            // [layers + 1][T][W]: X_0 .. X_n-1 filled, X_n written when part is given
  const float* part;      // fp32 slabs [split][T][W] of the sublayers' sum, or null (no update)
  const float* bias;      // [W] fp32 or null
  const float* dwa;       // [n + 1]
  const float* pre;       // [T][W] sum of the first j0 terms of the average (null: j0 = 0)
  int j0;
  const float* norm_w;    // [W] fp32: the multiplier itself (1 + stored weight where the design stores it so)
  float* x_out;           // [T][W] (may be x_in), not written when null
  float* rstd;            // DN_RSTD: [T]
  const int32_t* rows;    // row of the b-th workgroup (null: b); normed outputs are at b
  int T, W, split, n;
  float eps;
  // DN_CONV
  const float* w1; const float* w2;   // [taps][W]; w2 null: one sublayer
  const int32_t* positions;
  TailArg tail;
  int taps, ld1_, ld2_;
};

// one workgroup of BT threads per row; a thread holds NV vectors of V channels, NV * V * BT >= W
template <typename ACT, int V, int NV, int MODE, int BT>
__global__ void __launch_bounds__(BT) depth_norm_kernel(DepthArgs a, ACT* __restrict__ h1, ACT* __restrict__ h2) {
  __shared__ float red[16];
  const int b = blockIdx.x, t = a.rows ? a.rows[b] : b;
  const size_t row = (size_t)t * a.W, plane = (size_t)a.T * a.W;
  Vec<V> x[NV];
  float ss = 0.f;
  // the last row's convolution past and every weight, requested ahead of the stream they wait for
  constexpr int PRE = MODE == DN_CONV && NV == 1 ? 4 : 0;
  Vec<V> past[PRE ? PRE : 1], k1[PRE ? PRE : 1], k2[PRE ? PRE : 1], gw;
  const int pos = MODE == DN_CONV ? a.positions[b] : 0;
  const bool pre_ok = PRE > 0 && a.taps <= PRE;
  if constexpr (PRE > 0) {
    const int c = min((int)threadIdx.x * V, a.W - V);
    gw = ldv<V>(a.norm_w + c);
#pragma unroll
    for (int u = 0; u < PRE; ++u) {          // tap taps - 1 - u: u positions back
      const int j = max(a.taps - 1 - u, 0);
      k1[u] = ldv<V>(a.w1 + (size_t)j * a.W + c);
      k2[u] = ldv<V>((a.w2 ? a.w2 : a.w1) + (size_t)j * a.W + c);
      if (u && a.taps > 1) past[u] = ldv<V>(tail_row(a.tail, b, max(pos - u, 0), a.W) + c);
    }
  }
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) x[k].v[e] = 0.f;
    if (c >= a.W) continue;
    Vec<V> cur = ldv<V>(a.x_in + row + c);
    if (a.part) {
      Vec<V> pre;
      if (a.pre) pre = ldv<V>(a.pre + row + c);
      constexpr int SU = NV == 1 ? 8 : 4;             // slabs in flight (past the last: re-read, not added)
      if (a.split == 1) {
        const Vec<V> y = ldv<V>(a.part + row + c);
#pragma unroll
        for (int e = 0; e < V; ++e) cur.v[e] += y.v[e];
      } else for (int p0 = 0; p0 < a.split; p0 += SU) {
        Vec<V> y[SU];
#pragma unroll
        for (int u = 0; u < SU; ++u) y[u] = ldv<V>(a.part + (size_t)min(p0 + u, a.split - 1) * plane + row + c);
#pragma unroll
        for (int u = 0; u < SU; ++u)
          if (p0 + u < a.split)
#pragma unroll
            for (int e = 0; e < V; ++e) cur.v[e] += y[u].v[e];
      }
      if (a.bias) {
        const Vec<V> y = ldv<V>(a.bias + c);
#pragma unroll
        for (int e = 0; e < V; ++e) cur.v[e] += y.v[e];
      }
      if (MODE != DN_NORM) stv<V>(a.hist + (size_t)a.n * plane + row + c, cur);   // DN_NORM: nothing reads it again
      Vec<V> acc;
      const float an = a.dwa[a.n];
#pragma unroll
      for (int e = 0; e < V; ++e) acc.v[e] = an * cur.v[e];
      for (int j = a.j0; j < a.n; j += 4) {      // four rows of the history in flight
        Vec<V> y[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) y[u] = ldv<V>(a.hist + (size_t)min(j + u, a.n - 1) * plane + row + c);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const float wj = j + u < a.n ? a.dwa[j + u] : 0.f;
#pragma unroll
          for (int e = 0; e < V; ++e) acc.v[e] += wj * y[u].v[e];
        }
      }
      if (a.pre) {
#pragma unroll
        for (int e = 0; e < V; ++e) acc.v[e] += pre.v[e];
      }
      cur = acc;
    }
    x[k] = cur;
    if (a.x_out) stv<V>(a.x_out + row + c, cur);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += cur.v[e] * cur.v[e];
  }
  ss = block_sum(ss, red);
  const float rstd = 1.f / sqrtf(ss / (float)a.W + a.eps);
  if constexpr (MODE == DN_RSTD) {
    if (threadIdx.x == 0) a.rstd[t] = rstd;
  } else {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      if (c >= a.W) continue;
      const Vec<V> g = PRE > 0 ? gw : ldv<V>(a.norm_w + c);
      Vec<V> h;
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] = x[k].v[e] * rstd * g.v[e];
      if constexpr (MODE == DN_NORM) {
        stv<V>(h1 + (size_t)b * a.ld1_ + c, h);
      } else {
        Vec<V> y1 = h, y2 = h;
        if (pre_ok) {
          if constexpr (PRE > 0) {
#pragma unroll
            for (int u = PRE - 1; u >= 0; --u) {
              if (u >= a.taps || pos - u < 0) continue;
#pragma unroll
              for (int e = 0; e < V; ++e) {
                const float s = u ? past[u].v[e] : h.v[e];
                y1.v[e] += k1[u].v[e] * s;
                y2.v[e] += k2[u].v[e] * s;
              }
            }
          }
        } else {
          for (int j = 0; j < a.taps; ++j) {
            const int q = pos - a.taps + 1 + j;
            if (q < 0) continue;
            const Vec<V> s = j == a.taps - 1 ? h : ldv<V>(tail_row(a.tail, b, q, a.W) + c);
            const Vec<V> c1 = ldv<V>(a.w1 + (size_t)j * a.W + c);
#pragma unroll
            for (int e = 0; e < V; ++e) y1.v[e] += c1.v[e] * s.v[e];
            if (a.w2) {
              const Vec<V> c2 = ldv<V>(a.w2 + (size_t)j * a.W + c);
#pragma unroll
              for (int e = 0; e < V; ++e) y2.v[e] += c2.v[e] * s.v[e];
            }
          }
        }
        if (a.taps > 1) stv<V>(tail_row(a.tail, b, pos, a.W) + c, h);
        stv<V>(h1 + (size_t)b * a.ld1_ + c, y1);
        if (a.w2) stv<V>(h2 + (size_t)b * a.ld2_ + c, y2);
      }
    }
  }
}

// The oldest n results' share of the averages after up to DP_MAX consecutive layers, in one pass over the
// history: pre[l] = sum_{j < n} dwa_l[j] X_j.  The averages of a run of layers then read only what that run
// has added, instead of the whole history each.
constexpr int DP_MAX = 4;
struct PreArgs { const float* dwa[DP_MAX]; };

template <int V, int CNT>
__global__ void __launch_bounds__(256) depth_pre_kernel(const float* __restrict__ hist, size_t plane, int n, PreArgs w,
                                                       float* __restrict__ pre) {
  const size_t c = ((size_t)blockIdx.x * 256 + threadIdx.x) * V;
  if (c >= plane) return;
  Vec<V> acc[CNT];
#pragma unroll
  for (int l = 0; l < CNT; ++l)
#pragma unroll
    for (int e = 0; e < V; ++e) acc[l].v[e] = 0.f;
  int j = 0;
  auto step = [&](auto nu) {
    constexpr int U = decltype(nu)::value;
    Vec<V> y[U];
#pragma unroll
    for (int u = 0; u < U; ++u) y[u] = ldv<V>(hist + (size_t)(j + u) * plane + c);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int l = 0; l < CNT; ++l)
#pragma unroll
        for (int e = 0; e < V; ++e) acc[l].v[e] += w.dwa[l][j + u] * y[u].v[e];
    j += U;
  };
  while (j + 8 <= n) step(std::integral_constant<int, 8>{});
  if (j + 4 <= n) step(std::integral_constant<int, 4>{});
  while (j < n) step(std::integral_constant<int, 1>{});
#pragma unroll
  for (int l = 0; l < CNT; ++l) stv<V>(pre + (size_t)l * plane + c, acc[l]);
}

// Packed prompt portions.  A tile is the rows of one portion inside ONE cache block: {first row, rows,
// first position, sequence}; a thread walks its V channels down the tile.  Rows before the portion come
// from the tail: of this tile's own block they are read here before the tile's last rows replace them
// (same thread, same channels), and an earlier block's are not written in this launch unless another
// sequence owns it, which the engine rules out by sharing blocks only after they are computed.
// TAPS 0: any number of taps, the inputs recomputed per tap instead of kept in a register window.
template <typename ACT, int V, int TAPS>
__global__ void __launch_bounds__(256) input_conv_kernel(const float* __restrict__ x, const float* __restrict__ rstd,
                                                        const float* __restrict__ norm_w, const float* __restrict__ w1,
                                                        const float* __restrict__ w2, const int32_t* __restrict__ tiles,
                                                        TailArg ta, int W, int taps_rt, ACT* __restrict__ h1, int ld_1,
                                                        ACT* __restrict__ h2, int ld_2) {
  const int taps = TAPS ? TAPS : taps_rt;
  const int row0 = tiles[4 * blockIdx.x], n = tiles[4 * blockIdx.x + 1];
  const int pos0 = tiles[4 * blockIdx.x + 2], seq = tiles[4 * blockIdx.x + 3];
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= W) return;
  const Vec<V> g = ldv<V>(norm_w + c);
  // rows of this portion that precede the tile: tile_lead rows are in x, the rest in the tail
  const int lead = tiles[4 * (gridDim.x + blockIdx.x)];
  const bool paged = ta.max_blocks != 0;
  auto input = [&](int r) -> Vec<V> {        // convolution input of row row0 + r (r may be negative)
    Vec<V> h;
    if (pos0 + r < 0) {
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] = 0.f;
    } else if (r >= -lead) {
      h = ldv<V>(x + (size_t)(row0 + r) * W + c);
      const float s = rstd[row0 + r];
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] *= s * g.v[e];
    } else {
      h = ldv<V>(tail_row(ta, seq, pos0 + r, W) + c);
    }
    return h;
  };
  auto put = [&](int r, const Vec<V>& h, const Vec<V>& y1, const Vec<V>& y2) {
    stv<V>(h1 + (size_t)(row0 + r) * ld_1 + c, y1);
    if (w2) stv<V>(h2 + (size_t)(row0 + r) * ld_2 + c, y2);
    if (paged && r >= n - (taps - 1)) stv<V>(tail_row(ta, seq, pos0 + r, W) + c, h);
  };
  if constexpr (TAPS > 0) {
    float k1[TAPS][V], k2[TAPS][V];
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int e = 0; e < V; ++e) {
        k1[j][e] = w1[(size_t)j * W + c + e];
        k2[j][e] = w2 ? w2[(size_t)j * W + c + e] : 0.f;
      }
    Vec<V> win[TAPS];
#pragma unroll
    for (int j = 0; j + 1 < TAPS; ++j) win[j + 1] = input(j - (TAPS - 1));
    for (int r = 0; r < n; ++r) {
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j) win[j] = win[j + 1];
      win[TAPS - 1] = input(r);
      Vec<V> y1 = win[TAPS - 1], y2 = y1;
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          y1.v[e] += k1[j][e] * win[j].v[e];
          y2.v[e] += k2[j][e] * win[j].v[e];
        }
      put(r, win[TAPS - 1], y1, y2);
    }
  } else {
    for (int r = 0; r < n; ++r) {
      const Vec<V> h = input(r);
      Vec<V> y1 = h, y2 = h;
      for (int j = 0; j < taps; ++j) {
        const Vec<V> s = j == taps - 1 ? h : input(r - taps + 1 + j);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          y1.v[e] += w1[(size_t)j * W + c + e] * s.v[e];
          if (w2) y2.v[e] += w2[(size_t)j * W + c + e] * s.v[e];
        }
      }
      put(r, h, y1, y2);
    }
  }
  if (!paged && lead == 0) {
    const int N = tiles[4 * (gridDim.x + blockIdx.x) + 1];
    for (int r = max(0, N - (taps - 1)); r < N; ++r) stv<V>(tail_row(ta, seq, pos0 + r, W) + c, input(r));
  }
}

template <typename ACT>
__device__ __forceinline__ float glu(float g, float u, float limit, float alpha, float beta, float cubic) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + __expf(-alpha * g * (1.f + cubic * g * g))) * (u + beta);
}
template <>
__device__ __forceinline__ float glu<float>(float g, float u, float limit, float alpha, float beta, float cubic) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-alpha * g * (1.f + cubic * g * g))) * (u + beta);
}

// gu [split][T][2F] (ACT, or fp32 slabs whose sum is the product): gate | up halves, or 8-column
// interleaved groups
template <typename ACT, typename IN>
__global__ void __launch_bounds__(256) clamped_glu_kernel(ACT* __restrict__ out, int ldo, const IN* __restrict__ gu,
                                                         const float* __restrict__ gb, const float* __restrict__ ub,
                                                         int F, int interleaved, float limit, float alpha, float beta, float cubic, int split,
                                                         size_t slab) {
  const int t = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= F) return;
  const IN* r = gu + (size_t)t * 2 * F;
  const int gc = interleaved ? 16 * (c >> 3) + (c & 7) : c, uc = interleaved ? gc + 8 : F + c;
  float g = gb ? gb[c] : 0.f, u = ub ? ub[c] : 0.f;
  for (int p = 0; p < split; ++p) {
    g += ld1(r + p * slab + gc);
    u += ld1(r + p * slab + uc);
  }
  st1(out + (size_t)t * ldo + c, glu<ACT>(g, u, limit, alpha, beta, cubic));
}

// relu(sum of slabs)^2 of n values (a multiple of V)
template <typename ACT, int V>
__global__ void __launch_bounds__(256) relu_sq_kernel(ACT* __restrict__ out, const float* __restrict__ x, int split, size_t n) {
  for (size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * V; i < n; i += (size_t)gridDim.x * 256 * V) {
    Vec<V> v = zerov<V>();
    add_slabs<V>(v, x, split, (int64_t)n, i);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      v.v[e] = fmaxf(v.v[e], 0.f);
      v.v[e] *= v.v[e];
    }
    stv<V>(out + i, v);
  }
}

__global__ void __launch_bounds__(256) softcap_kernel(float* __restrict__ x, size_t n, float cap) {
  const float inv = 1.f / cap;
  for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) x[i] = cap * tanhf(x[i] * inv);
}

// few rows (a decode step): the widest workgroup the row fills, one vector per thread
template <typename ACT, int V, int MODE>
int depth_nv(int W, dim3 grid, hipStream_t s, const DepthArgs& a, void* h1, void* h2) {
#define DN_GO(NV, BT) depth_norm_kernel<ACT, V, NV, MODE, BT><<<grid, BT, 0, s>>>(a, (ACT*)h1, (ACT*)h2)
  const int vecs = (W + V - 1) / V;
  const bool few = grid.x <= 512 && vecs > 256;
  if (vecs <= 256) DN_GO(1, 256);
  else if (few && vecs <= 1024) DN_GO(1, 1024);
  else if (few && vecs <= 2048) DN_GO(2, 1024);
  else if (vecs <= 512) DN_GO(2, 256);
  else if (vecs <= 1024) DN_GO(4, 256);
  else if (vecs <= 4096) DN_GO(4, 1024);
  else if (vecs <= 8192) DN_GO(8, 1024);
  else return -4;
#undef DN_GO
  return CFC_CHECK_LAUNCH();
}

template <typename ACT>
int depth_launch(int mode, int nrows, hipStream_t s, const DepthArgs& a, void* h1, void* h2) {
  const bool v4 = a.W % 4 == 0 && (mode == DN_RSTD || (a.ld1_ % 4 == 0 && (!a.w2 || a.ld2_ % 4 == 0)));
  const dim3 grid(nrows);
#define DN_MODE(M)                                                                             \
  return v4 ? depth_nv<ACT, 4, M>(a.W, grid, s, a, h1, h2) : depth_nv<ACT, 1, M>(a.W, grid, s, a, h1, h2)
  switch (mode) {
    case DN_RSTD: DN_MODE(DN_RSTD);
    case DN_NORM: DN_MODE(DN_NORM);
    case DN_CONV: DN_MODE(DN_CONV);
  }
#undef DN_MODE
  return -3;
}

template <typename ACT, int V>
int conv_launch(dim3 grid, hipStream_t s, const float* x, const float* rstd, const float* nw, const float* w1,
                const float* w2, const int32_t* tiles, const TailArg& ta, int W, int taps, void* h1, int ld_1, void* h2,
                int ld_2) {
#define IC(T) input_conv_kernel<ACT, V, T><<<grid, 256, 0, s>>>(x, rstd, nw, w1, w2, tiles, ta, W, taps, (ACT*)h1, ld_1, (ACT*)h2, ld_2)
  switch (taps) {
    case 1: IC(1); break;
    case 2: IC(2); break;
    case 3: IC(3); break;
    case 4: IC(4); break;
    default: IC(0); break;
  }
#undef IC
  return CFC_CHECK_LAUNCH();
}

}  // namespace

// table: bf16 (f32 = 0) or fp32 rows; ids outside [0, vocab) are clamped
// positions (null: none): entries 2i and 2i + 1 get the sine and the cosine of positions * turns[i] turns
CFC_API int cfc_embed_f32(float* out, const void* table, const int32_t* ids, int T, int W, int vocab, int f32, float scale,
                          const int32_t* positions, const double* turns, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W <= 0 || vocab <= 0 || (positions && !turns)) return -1;
  if (f32) embed_f32_kernel<float><<<T, 256, 0, stream>>>(out, (const float*)table, ids, W, vocab, scale, positions, turns);
  else embed_f32_kernel<uint16_t><<<T, 256, 0, stream>>>(out, (const uint16_t*)table, ids, W, vocab, scale, positions, turns);
  return CFC_CHECK_LAUNCH();
}

// mode: 0 x' and 1 / rms; 1 normed rows into h1 (row stride ld1); 2 normed rows through the input
// convolutions w1 / w2 into h1 / h2 (row strides ld1 / ld2), their tails read and written.  f32: the
// normed outputs are fp32 (else bf16).  nrows workgroups; rows null: row b of T.
CFC_API int cfc_depth_norm(int mode, int f32, int nrows, const int32_t* rows, const float* x_in, float* hist,
                           const float* part, int split, const float* bias, const float* dwa, int n,
                           const float* pre, int j0,
                           const float* norm_w, float eps, float* x_out, float* rstd, int T, int W, void* h1, int ld1,
                           void* h2, int ld2, const float* w1, const float* w2, int taps, const int32_t* positions,
                           float* tail, int slots, const int32_t* block_tables, int max_blocks, hipStream_t stream) {
  if (nrows <= 0) return 0;
  if (W <= 0 || T <= 0 || n < 0 || (pre && (j0 < 0 || j0 > n)) || (part && (split < 1 || !hist || !dwa))) return -1;
  if (mode == DN_RSTD && !rstd) return -2;
  if (mode != DN_RSTD && (!h1 || !norm_w)) return -2;
  if (mode == DN_CONV && (!w1 || taps < 1 || !positions || (w2 && !h2) || rows ||
                          (taps > 1 && (!tail || slots < (taps - 1 < CFC_KV_BS ? taps - 1 : CFC_KV_BS) || !block_tables))))
    return -2;
  DepthArgs a{x_in, hist, part, bias, dwa, pre, pre ? j0 : 0, norm_w, x_out, rstd, rows, T, W, split, n, eps, w1, w2, positions,
              TailArg{tail, block_tables, max_blocks, slots > 0 ? slots : 1}, taps, ld1, ld2};
  return f32 ? depth_launch<float>(mode, nrows, stream, a, h1, h2) : depth_launch<uint16_t>(mode, nrows, stream, a, h1, h2);
}

// pre [count][T][W] (count <= 4): sums of the first n planes of hist [.][T][W] weighted by dwa0 .. dwa3
CFC_API int cfc_depth_pre(const float* hist, int64_t plane, int n, int count, const float* dwa0, const float* dwa1,
                          const float* dwa2, const float* dwa3, float* pre, hipStream_t stream) {
  if (plane <= 0) return 0;
  if (n < 1 || count < 1 || count > DP_MAX || !pre || !hist) return -1;
  const PreArgs w{{dwa0, dwa1, dwa2, dwa3}};
  const bool v4 = plane % 4 == 0 && ((uintptr_t)hist & 15) == 0 && ((uintptr_t)pre & 15) == 0;
  const unsigned grid = (unsigned)((plane + (v4 ? 1023 : 255)) / (v4 ? 1024 : 256));
#define DP_GO(V, C) depth_pre_kernel<V, C><<<grid, 256, 0, stream>>>(hist, (size_t)plane, n, w, pre); break
  if (v4) switch (count) { case 1: DP_GO(4, 1); case 2: DP_GO(4, 2); case 3: DP_GO(4, 3); default: DP_GO(4, 4); }
  else switch (count) { case 1: DP_GO(1, 1); case 2: DP_GO(1, 2); case 3: DP_GO(1, 3); default: DP_GO(1, 4); }
#undef DP_GO
  return CFC_CHECK_LAUNCH();
}

// tiles [2][n_tiles][4]: {first row, rows, first position, sequence}, then {portion rows before the tile, the portion's rows,
// 0, 0}.  max_blocks 0: block_tables holds each sequence's slot, tail [slots][tail slots][W]
CFC_API int cfc_input_conv(int f32, int n_tiles, const int32_t* tiles, const float* x, const float* rstd,
                           const float* norm_w, const float* w1, const float* w2, int taps, float* tail, int slots,
                           const int32_t* block_tables, int max_blocks, int W, void* h1, int ld1, void* h2, int ld2,
                           hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (W <= 0 || taps < 1 || !w1 || (w2 && !h2)) return -1;
  if (taps > 1 && (!tail || slots < (taps - 1 < CFC_KV_BS ? taps - 1 : CFC_KV_BS) || !block_tables)) return -2;
  const TailArg ta{tail, block_tables, max_blocks, slots > 0 ? slots : 1};
  const bool v4 = W % 4 == 0 && ld1 % 4 == 0 && (!w2 || ld2 % 4 == 0);
  const dim3 grid(n_tiles, (W + (v4 ? 1023 : 255)) / (v4 ? 1024 : 256));
#define IC_GO(A, V) return conv_launch<A, V>(grid, stream, x, rstd, norm_w, w1, w2, tiles, ta, W, taps, h1, ld1, h2, ld2)
  if (f32) { if (v4) IC_GO(float, 4); IC_GO(float, 1); }
  if (v4) IC_GO(uint16_t, 4);
  IC_GO(uint16_t, 1);
#undef IC_GO
}

// in_f32: gu is fp32 (else the activation type)
CFC_API int cfc_clamped_glu(int f32, int in_f32, void* out, int ldo, const void* gu, int split, const float* gb,
                            const float* ub, int T, int F, int interleaved, float limit, float alpha, float beta, float cubic,
                            hipStream_t stream) {
  if (T <= 0) return 0;
  if (F <= 0 || (interleaved && F % 8) || split < 1 || (split > 1 && !f32 && !in_f32) || T > 65535 * 16) return -1;
  const int rows = T > 65535 ? 65535 : T;
  for (int t0 = 0; t0 < T; t0 += rows) {
    const int n = T - t0 < rows ? T - t0 : rows;
    const dim3 grid((F + 255) / 256, n);
    const size_t slab = (size_t)T * 2 * F, go = (size_t)t0 * 2 * F, oo = (size_t)t0 * ldo;
    if (f32)
      clamped_glu_kernel<float, float><<<grid, 256, 0, stream>>>((float*)out + oo, ldo, (const float*)gu + go, gb, ub, F,
                                                                 interleaved, limit, alpha, beta, cubic, split, slab);
    else if (in_f32)
      clamped_glu_kernel<uint16_t, float><<<grid, 256, 0, stream>>>((uint16_t*)out + oo, ldo, (const float*)gu + go, gb, ub,
                                                                    F, interleaved, limit, alpha, beta, cubic, split, slab);
    else
      clamped_glu_kernel<uint16_t, uint16_t><<<grid, 256, 0, stream>>>((uint16_t*)out + oo, ldo, (const uint16_t*)gu + go,
                                                                       gb, ub, F, interleaved, limit, alpha, beta, cubic, split, slab);
  }
  return CFC_CHECK_LAUNCH();
}

CFC_API int cfc_softcap(float* x, int64_t n, float cap, hipStream_t stream) {
  if (n <= 0) return 0;
  if (!(cap > 0.f)) return -1;
  const int64_t blocks = (n + 255) / 256;
  softcap_kernel<<<(unsigned)(blocks < 4096 ? blocks : 4096), 256, 0, stream>>>(x, (size_t)n, cap);
  return CFC_CHECK_LAUNCH();
}

// x: fp32 slabs [split][n]; out n activations
CFC_API int cfc_relu_sq(int f32, void* out, const float* x, int split, int64_t n, hipStream_t stream) {
  if (n <= 0) return 0;
  if (split < 1) return -1;
  const bool v4 = n % 4 == 0;
  const int64_t blocks = (n / (v4 ? 4 : 1) + 255) / 256;
  const unsigned g = (unsigned)(blocks < 16384 ? blocks : 16384);
#define RS(A, V) relu_sq_kernel<A, V><<<g, 256, 0, stream>>>((A*)out, x, split, (size_t)n)
  if (f32) { if (v4) RS(float, 4); else RS(float, 1); }
  else if (v4) RS(uint16_t, 4);
  else RS(uint16_t, 1);
#undef RS
  return CFC_CHECK_LAUNCH();
}
