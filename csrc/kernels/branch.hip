// Residual branches between two RMS norms (one ahead of the sublayer, one on its way back into the stream), on a
// 32-bit stream.  One kernel stands between two sublayers, one row per workgroup:
//
//   y   the finished sublayer's result: the sum of a product's fp32 slabs; or two products' (mixers side by side),
//       each over its root mean square, times its weight, and factor times their sum; or routed experts' rows,
//       where a choice past the last expert counts the sublayer's own input instead
//   x  += y / rms(y) gain
//   h   = x / rms(x) next gain: the next sublayer's input, as an activation
//
// Without a branch (the first layer) only h.  Gains are one number or a vector.
#include "rows.h"

namespace {

struct Gain {
  const float* p;
  int vec;                     // 0: one number for all channels
};

struct BranchIn {
  const float* y;  int ysplit;  const float* wy;      // slabs [ysplit][T][W]; wy [W]: the branch's own norm weight (two products)
  const float* y2; int y2split; const float* wy2;
  float factor;
  const void* rows; const int32_t* mrow; const float* mwt; const int32_t* ids; int top, experts;   // routed rows
  const void* own;                                    // [T][W] the sublayer's input (choices >= experts)
  Gain g;
  float eps;
  int T, W;
};

template <int V>
__device__ __forceinline__ Vec<V> ldgain(const Gain& g, int c) {
  if (g.vec) return ldv<V>(g.p + c);
  Vec<V> r;
  const float v = *g.p;
#pragma unroll
  for (int e = 0; e < V; ++e) r.v[e] = v;
  return r;
}

template <typename ACT, int V, int NV, int BT>
__global__ void __launch_bounds__(BT) branch_norm_kernel(BranchIn b, int branch, float* __restrict__ x, Gain next,
                                                        ACT* __restrict__ h) {
  __shared__ float red[16], red2[16];
  const int t = blockIdx.x, W = b.W;
  const size_t row = (size_t)t * W;
  const float inv_w = 1.f / (float)W;
  Vec<V> xv[NV];
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    xv[k] = c < W ? ldv<V>(x + row + c) : zerov<V>();
  }
  if (branch) {
    Vec<V> y[NV];
    float s = 0.f;
    if (b.wy) {
      Vec<V> z[NV];
      float s2 = 0.f;
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = (k * BT + threadIdx.x) * V;
        y[k] = z[k] = zerov<V>();
        if (c >= W) continue;
        add_slabs<V>(y[k], b.y, b.ysplit, (int64_t)b.T * W, row + c);
        add_slabs<V>(z[k], b.y2, b.y2split, (int64_t)b.T * W, row + c);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          s += y[k].v[e] * y[k].v[e];
          s2 += z[k].v[e] * z[k].v[e];
        }
      }
      const float r1 = b.factor / sqrtf(block_sum(s, red) * inv_w + b.eps);
      const float r2 = b.factor / sqrtf(block_sum(s2, red2) * inv_w + b.eps);
      s = 0.f;
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = (k * BT + threadIdx.x) * V;
        if (c >= W) continue;
        const Vec<V> w1 = ldv<V>(b.wy + c), w2 = ldv<V>(b.wy2 + c);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          y[k].v[e] = y[k].v[e] * r1 * w1.v[e] + z[k].v[e] * r2 * w2.v[e];
          s += y[k].v[e] * y[k].v[e];
        }
      }
    } else {
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = (k * BT + threadIdx.x) * V;
        y[k] = zerov<V>();
        if (c >= W) continue;
        if (b.y) add_slabs<V>(y[k], b.y, b.ysplit, (int64_t)b.T * W, row + c);
        if (b.mrow)
          for (int i0 = 0; i0 < b.top; i0 += 4) {         // four choices in flight (past the last: weight 0)
            Vec<V> r[4];
            float wt[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
              const int64_t i = (int64_t)t * b.top + min(i0 + u, b.top - 1);
              const bool own = b.ids[i] >= b.experts;
              const ACT* src = own ? reinterpret_cast<const ACT*>(b.own) + row
                                   : reinterpret_cast<const ACT*>(b.rows) + (size_t)b.mrow[i] * W;
              wt[u] = i0 + u < b.top ? b.mwt[i] : 0.f;
              r[u] = ldv<V>(src + c);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
              for (int e = 0; e < V; ++e) y[k].v[e] += wt[u] * r[u].v[e];
          }
#pragma unroll
        for (int e = 0; e < V; ++e) s += y[k].v[e] * y[k].v[e];
      }
    }
    const float r = 1.f / sqrtf(block_sum(s, red) * inv_w + b.eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      if (c >= W) continue;
      const Vec<V> g = ldgain<V>(b.g, c);
#pragma unroll
      for (int e = 0; e < V; ++e) xv[k].v[e] += y[k].v[e] * r * g.v[e];
      stv<V>(x + row + c, xv[k]);
    }
  }
  if (!h) return;
  float s = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k)
#pragma unroll
    for (int e = 0; e < V; ++e) s += xv[k].v[e] * xv[k].v[e];
  const float r = 1.f / sqrtf(block_sum(s, red2) * inv_w + b.eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= W) continue;
    const Vec<V> g = ldgain<V>(next, c);
    Vec<V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.v[e] = xv[k].v[e] * r * g.v[e];
    stv<V>(h + row + c, o);
  }
}

template <typename ACT, int V>
int branch_go(hipStream_t s, const BranchIn& b, int branch, float* x, Gain next, void* h) {
  const int vecs = (b.W + V - 1) / V;
#define GO(NV, BT) branch_norm_kernel<ACT, V, NV, BT><<<b.T, BT, 0, s>>>(b, branch, x, next, (ACT*)h)
  ROW_SHAPES(GO, vecs);
#undef GO
  return CFC_CHECK_LAUNCH();
}

}  // namespace

// branch 0: x is only normed into h.  wy, wy2 (both or none): two products side by side.  h may be null
CFC_API int cfc_branch_norm(int f32, int branch, const float* y, int ysplit, const float* wy, const float* y2, int y2split,
                            const float* wy2, float factor, const void* rows, const int32_t* mrow, const float* mwt,
                            const int32_t* ids, int top, int experts, const void* own, const float* gain, int gain_vec, float eps,
                            float* x, int T, int W, const float* next, int next_vec, void* h, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W < 1 || !x || (h && !next)) return -1;
  if (branch) {
    if (!gain || (!y && !mrow) || (y && ysplit < 1)) return -2;
    if ((wy == nullptr) != (wy2 == nullptr) || (wy && (!y || !y2 || y2split < 1)) || (!wy && y2)) return -2;
    if (mrow && (!rows || !mwt || !ids || !own || top < 1 || experts < 1)) return -2;
  }
  const BranchIn b{y, ysplit, wy, y2, y2split, wy2, factor, rows, mrow, mwt, ids, top, experts, own, {gain, gain_vec}, eps, T, W};
  const Gain n{next, next_vec};
  if (f32) return W % 4 ? branch_go<float, 1>(stream, b, branch, x, n, h) : branch_go<float, 4>(stream, b, branch, x, n, h);
  return W % 4 ? branch_go<uint16_t, 1>(stream, b, branch, x, n, h) : branch_go<uint16_t, 4>(stream, b, branch, x, n, h);
}
