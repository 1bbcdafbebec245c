// Residual branches that are gated and normed on their way into a 32-bit stream, and the token shift ahead
// of the next sublayer:
//
//   * shift_mix     prompt rows: h = x + (x' - x) shift with x' the token before, then up to eight mixes
//                   h + (h' - h) mu_s of the shifted row with the one before it (h' needs x two tokens back)
//   * gated_norm    y = (sum of the branch's fp32 slabs [+ a second product's] [+ routed experts' rows])
//                   * sigmoid(gate + bias); x += LayerNorm(y) w.  One row per workgroup.  The row leaves as
//                   the next products' input as well
//   * gated_shift   the same for decoded rows, running on into the next layer's shift_mix: its rows before
//                   come from the sequence's state and the new row goes there
//   * final_norm    LayerNorm of chosen rows
//
// State: prev[slot][2][W] fp32 per layer, the layer's input rows of the last two tokens at position % 2.
// Rows of positions before the first token count as zeros, so a slot needs no clearing.  A prompt portion's
// last rows are stored by gated_norm (the shift_mix of the same layer, an earlier launch, has read the old
// ones by then); a decoded row's thread reads what it overwrites.
//
// ACT is the activation type the matrix products read: uint16_t (bf16 bits) or float.
#include "rows.h"

namespace {

constexpr int META_TAIL = 4, META_SLOT = 3;
constexpr int MAX_MIX = 8;

struct ShiftArgs {
  const float* shift;     // [W]
  const float* mus;       // [n_mix][W] or null: the shifted row itself is the output
  int n_mix;
  float* prev;            // [slots][2][W]
  const int32_t* positions;
};

// the row's outputs at p, p + stride, ..: x itself, then the shifted row or its mixes.  NM: their number, the mixes'
// weights given in registers (0: read as they come)
template <typename ACT, int V, int NM = 0>
__device__ __forceinline__ void shift_row(const ShiftArgs& a, const Vec<V>& x, const Vec<V>& xp, const Vec<V>& xpp, bool any,
                                          const Vec<V>& sh, int W, int c, ACT* p, size_t stride, const Vec<V>* mu_r = nullptr) {
  stv<V>(p, x);
  Vec<V> h, hp;
#pragma unroll
  for (int e = 0; e < V; ++e) {
    h.v[e] = x.v[e] + (xp.v[e] - x.v[e]) * sh.v[e];
    hp.v[e] = any ? xp.v[e] + (xpp.v[e] - xp.v[e]) * sh.v[e] : 0.f;
  }
  if (!a.mus) {
    stv<V>(p + stride, h);
    return;
  }
  if constexpr (NM > 0) {
#pragma unroll
    for (int s = 0; s < NM; ++s) {
      Vec<V> m;
#pragma unroll
      for (int e = 0; e < V; ++e) m.v[e] = h.v[e] + (hp.v[e] - h.v[e]) * mu_r[s].v[e];
      stv<V>(p + (size_t)(1 + s) * stride, m);
    }
    return;
  }
  for (int s = 0; s < a.n_mix; ++s) {
    const Vec<V> mu = ldv<V>(a.mus + (size_t)s * W + c);
    Vec<V> m;
#pragma unroll
    for (int e = 0; e < V; ++e) m.v[e] = h.v[e] + (hp.v[e] - h.v[e]) * mu.v[e];
    stv<V>(p + (size_t)(1 + s) * stride, m);
  }
}

// prompt rows: ROWS consecutive rows of 256 V channels per workgroup; acts [1 + outputs][T][W]
constexpr int SM_ROWS = 8;
template <typename ACT, int V, int NM>
__global__ void __launch_bounds__(256) shift_mix_kernel(const float* __restrict__ x, const int32_t* __restrict__ meta,
                                                       ShiftArgs a, int T, int W, ACT* __restrict__ acts) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * V, t0 = blockIdx.x * SM_ROWS;
  if (c >= W) return;
  const Vec<V> sh = ldv<V>(a.shift + c);
  Vec<V> xp = zerov<V>(), xpp = zerov<V>(), mu[NM ? NM : 1];
#pragma unroll
  for (int s = 0; s < NM; ++s) mu[s] = ldv<V>(a.mus + (size_t)s * W + c);
  for (int t = t0; t < min(t0 + SM_ROWS, T); ++t) {
    const int m = meta[t], lead = m & 3, pos = a.positions[t];
    const size_t row = (size_t)t * W + c;
    if (t == t0 || lead == 0) {          // later rows of a portion carry on in registers
      const float* st = a.prev + (size_t)(m >> META_SLOT) * 2 * W + c;
      xp = pos < 1 ? zerov<V>() : ldv<V>(lead >= 1 ? x + row - W : st + (size_t)((pos - 1) & 1) * W);
      xpp = pos < 2 ? zerov<V>() : ldv<V>(lead >= 2 ? x + row - 2 * (size_t)W : st + (size_t)(pos & 1) * W);
    }
    const Vec<V> xt = ldv<V>(x + row);
    shift_row<ACT, V, NM>(a, xt, xp, xpp, pos >= 1, sh, W, c, acts + row, (size_t)T * W, mu);
    xpp = xp;
    xp = xt;
  }
}

struct BranchArgs {
  const float* y;  int ysplit;            // slabs [ysplit][T][W] (null: none)
  const float* y2; int y2split;           // a second product's
  const void* ym; const int32_t* mrow; const float* mwt; int top;   // routed rows [*][W] (activations), row and weight per (token, choice)
  const void* gate; int gate_act, gsplit; int64_t gld, gplane;       // pre-sigmoid: slabs, or activations (gate_act)
  const float* gbias;                     // [W]
  const float* norm_w;                    // [W]
  float eps;
  int T, W;
};

// MODE 0: prompt rows; 1: decoded rows (shift_mix of the next layer follows); 2: decoded rows, shift only
// (b.y == null, b.y2 == null, b.ym == null: no branch, the first layer's).  x is updated in place.
enum { GN_PROMPT = 0, GN_SHIFT = 1 };
template <typename ACT, int V, int NV, int BT, int MODE>
__global__ void __launch_bounds__(BT) gated_norm_kernel(BranchArgs b, float* __restrict__ x, ACT* __restrict__ h,
                                                       float* __restrict__ prev, const int32_t* __restrict__ meta,
                                                       const int32_t* __restrict__ positions, ShiftArgs a,
                                                       const int32_t* __restrict__ slots, ACT* __restrict__ acts) {
  __shared__ float red[16];
  const int t = blockIdx.x, W = b.W;
  const size_t row = (size_t)t * W;
  const bool branch = MODE == GN_PROMPT || b.norm_w != nullptr;
  int pos = 0;
  float* st = nullptr;
  Vec<V> xv[NV], xp[MODE == GN_SHIFT ? NV : 1], xpp[MODE == GN_SHIFT ? NV : 1];
  if constexpr (MODE == GN_SHIFT) {
    if (acts) {
      pos = a.positions[t];
      st = a.prev + (size_t)slots[t] * 2 * W;
    }
  }
#pragma unroll
  for (int k = 0; k < NV; ++k) {          // asked for ahead of the branch they wait for
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= W) continue;
    xv[k] = ldv<V>(x + row + c);
    if constexpr (MODE == GN_SHIFT) {
      xp[k] = xpp[k] = zerov<V>();
      if (acts && pos >= 1) xp[k] = ldv<V>(st + (size_t)((pos - 1) & 1) * W + c);
      if (acts && pos >= 2) xpp[k] = ldv<V>(st + (size_t)(pos & 1) * W + c);
    }
  }
  if (branch) {
    Vec<V> y[NV];
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      y[k] = zerov<V>();
      if (c >= W) continue;
      if (b.y) add_slabs<V>(y[k], b.y, b.ysplit, (int64_t)b.T * W, row + c);
      if (b.y2) add_slabs<V>(y[k], b.y2, b.y2split, (int64_t)b.T * W, row + c);
      if (b.ym)
        for (int i = 0; i < b.top; ++i) {
          const float wt = b.mwt[(size_t)t * b.top + i];
          const Vec<V> r = ldv<V>(reinterpret_cast<const ACT*>(b.ym) + (size_t)b.mrow[(size_t)t * b.top + i] * W + c);
#pragma unroll
          for (int e = 0; e < V; ++e) y[k].v[e] += wt * r.v[e];
        }
      Vec<V> g = zerov<V>();
      if (b.gate_act) g = ldv<V>(reinterpret_cast<const ACT*>(b.gate) + (size_t)t * b.gld + c);
      else add_slabs<V>(g, reinterpret_cast<const float*>(b.gate), b.gsplit, b.gplane, (size_t)t * b.gld + c);
      const Vec<V> gb = ldv<V>(b.gbias + c);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        y[k].v[e] *= 1.f / (1.f + expf(-(g.v[e] + gb.v[e])));
        s += y[k].v[e];
      }
    }
    const float mean = block_sum(s, red) / (float)W;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k)
      if ((k * BT + (int)threadIdx.x) * V < W)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          y[k].v[e] -= mean;
          ss += y[k].v[e] * y[k].v[e];
        }
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + b.eps);
    int m = 0;
    if constexpr (MODE == GN_PROMPT) {
      if (prev) {
        m = meta[t];
        pos = positions[t];
      }
    }
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      if (c >= W) continue;
      if constexpr (MODE == GN_PROMPT) {
        if (prev && (m & META_TAIL)) stv<V>(prev + ((size_t)(m >> META_SLOT) * 2 + (pos & 1)) * W + c, xv[k]);
      }
      const Vec<V> w = ldv<V>(b.norm_w + c);
#pragma unroll
      for (int e = 0; e < V; ++e) xv[k].v[e] += y[k].v[e] * r * w.v[e];
      stv<V>(x + row + c, xv[k]);
      if (h) stv<V>(h + row + c, xv[k]);
    }
  }
  if constexpr (MODE == GN_SHIFT) {
    if (!acts) return;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      if (c >= W) continue;
      shift_row<ACT, V>(a, xv[k], xp[k], xpp[k], pos >= 1, ldv<V>(a.shift + c), W, c, acts + row + c, (size_t)b.T * W);
      stv<V>(st + (size_t)(pos & 1) * W + c, xv[k]);
    }
  }
}

template <typename ACT, int V, int NV, int BT>
__global__ void __launch_bounds__(BT) final_norm_kernel(const float* __restrict__ x, const int32_t* __restrict__ rows,
                                                       const float* __restrict__ w, float eps, int W, ACT* __restrict__ out) {
  __shared__ float red[16];
  const size_t row = (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * W;
  Vec<V> y[NV];
  float s = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= W) continue;
    y[k] = ldv<V>(x + row + c);
#pragma unroll
    for (int e = 0; e < V; ++e) s += y[k].v[e];
  }
  const float mean = block_sum(s, red) / (float)W;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k)
    if ((k * BT + (int)threadIdx.x) * V < W)
#pragma unroll
      for (int e = 0; e < V; ++e) {
        y[k].v[e] -= mean;
        ss += y[k].v[e] * y[k].v[e];
      }
  const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= W) continue;
    const Vec<V> wv = ldv<V>(w + c);
#pragma unroll
    for (int e = 0; e < V; ++e) y[k].v[e] *= r * wv.v[e];
    stv<V>(out + (size_t)blockIdx.x * W + c, y[k]);
  }
}

template <typename ACT, int V, int MODE>
int gated_go(hipStream_t s, int n, const BranchArgs& b, float* x, void* h, float* prev, const int32_t* meta,
             const int32_t* positions, const ShiftArgs& a, const int32_t* slots, void* acts) {
  const int vecs = (b.W + V - 1) / V;
#define GO(NV, BT) \
  gated_norm_kernel<ACT, V, NV, BT, MODE><<<n, BT, 0, s>>>(b, x, (ACT*)h, prev, meta, positions, a, slots, (ACT*)acts)
  ROW_SHAPES(GO, vecs);
#undef GO
  return CFC_CHECK_LAUNCH();
}

template <typename ACT, int V>
int final_go(hipStream_t s, int n, const float* x, const int32_t* rows, const float* w, float eps, int W, void* out) {
  const int vecs = (W + V - 1) / V;
#define GO(NV, BT) final_norm_kernel<ACT, V, NV, BT><<<n, BT, 0, s>>>(x, rows, w, eps, W, (ACT*)out)
  ROW_SHAPES(GO, vecs);
#undef GO
  return CFC_CHECK_LAUNCH();
}

}  // namespace

// acts [1 + max(1, n_mix)][T][W]: the row, then the shifted row (mus null) or its mixes
CFC_API int cfc_shift_mix(int f32, const float* x, const int32_t* meta, const int32_t* positions, const float* shift,
                          const float* mus, int n_mix, float* prev, int T, int W, void* acts, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W < 1 || (mus ? n_mix < 1 || n_mix > MAX_MIX : n_mix != 0) || !prev || !meta || !positions) return -1;
  const ShiftArgs a{shift, mus, n_mix, prev, positions};
  const int V = W % 4 == 0 ? 4 : 1;
  const dim3 grid((T + SM_ROWS - 1) / SM_ROWS, (W + 256 * V - 1) / (256 * V));
#define SM(ACT, VV)                                                                               \
  do {                                                                                            \
    if (n_mix == 5) shift_mix_kernel<ACT, VV, 5><<<grid, 256, 0, stream>>>(x, meta, a, T, W, (ACT*)acts); \
    else shift_mix_kernel<ACT, VV, 0><<<grid, 256, 0, stream>>>(x, meta, a, T, W, (ACT*)acts);    \
  } while (0)
  if (f32) { if (V == 4) SM(float, 4); else SM(float, 1); }
  else if (V == 4) SM(uint16_t, 4);
  else SM(uint16_t, 1);
#undef SM
  return CFC_CHECK_LAUNCH();
}

// mode 0: prompt rows (h: the updated row as an activation, prev: store the portion's last rows of x as they
// were); mode 1: decoded rows (acts null: no shift follows; norm_w null: no branch comes first)
CFC_API int cfc_gated_norm(int mode, int f32, const float* y, int ysplit, const float* y2, int y2split, const void* ym,
                           const int32_t* mrow, const float* mwt, int top, const void* gate, int gate_act, int gsplit,
                           int64_t gld, int64_t gplane, const float* gbias, const float* norm_w, float eps, float* x, int T,
                           int W, void* h, float* prev, const int32_t* meta, const int32_t* positions, const float* shift,
                           const float* mus, int n_mix, const int32_t* slots, void* acts, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W < 1 || (mode != 0 && mode != 1)) return -1;
  if ((mode == 0 || norm_w) && (!gate || !gbias || !norm_w || (!y && !y2 && !ym))) return -2;
  if ((y && ysplit < 1) || (y2 && y2split < 1) || (ym && (top < 1 || !mrow || !mwt)) || (!gate_act && gate && gsplit < 1)) return -2;
  if (mode == 0 && prev && (!meta || !positions)) return -2;
  if (mode == 1 && acts && (!prev || !positions || !slots || !shift || (mus && (n_mix < 1 || n_mix > MAX_MIX)))) return -2;
  const BranchArgs b{y, ysplit, y2, y2split, ym, mrow, mwt, top, gate, gate_act, gsplit, gld, gplane, gbias, norm_w, eps, T, W};
  const ShiftArgs a{shift, mus, n_mix, prev, positions};
  const bool v4 = W % 4 == 0 && gld % 4 == 0 && gplane % 4 == 0 && ((uintptr_t)gate & (gate_act && !f32 ? 7 : 15)) == 0;
#define GN_ARGS stream, T, b, x, h, mode == 0 ? prev : nullptr, meta, positions, a, slots, acts
#define GN(ACT, MODE) (v4 ? gated_go<ACT, 4, MODE>(GN_ARGS) : gated_go<ACT, 1, MODE>(GN_ARGS))
  if (mode == 0) return f32 ? GN(float, GN_PROMPT) : GN(uint16_t, GN_PROMPT);
  return f32 ? GN(float, GN_SHIFT) : GN(uint16_t, GN_SHIFT);
#undef GN
#undef GN_ARGS
}

CFC_API int cfc_final_norm(int f32, const float* x, const int32_t* rows, int n, const float* w, float eps, int W, void* out,
                           hipStream_t stream) {
  if (n <= 0) return 0;
  if (W < 1) return -1;
  if (f32) return W % 4 ? final_go<float, 1>(stream, n, x, rows, w, eps, W, out) : final_go<float, 4>(stream, n, x, rows, w, eps, W, out);
  return W % 4 ? final_go<uint16_t, 1>(stream, n, x, rows, w, eps, W, out) : final_go<uint16_t, 4>(stream, n, x, rows, w, eps, W, out);
}
