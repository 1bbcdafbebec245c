// Hyper-connections: a residual stream of several copies x_1 .. x_S per token, 32-bit, [T][S][W].  One kernel stands between
// two sublayers, one row per workgroup:
//
//   y    the finished sublayer's result, the sum of a product's fp32 slabs
//   x_t  = sum_s mix[s][t] x_s + out[t] y, all from the old ones
//   u    = sum_s in[s] x_s of the new ones: what the next sublayer reads (in null: the plain sum)
//
// and an ending: u and its 1 / rms (a prompt's rows, ahead of their convolution), the normed row u / rms(u) w as an
// activation, or (decode) the normed row h as h + conv(h) over time, its earlier inputs in a slot per sequence.  Without y
// (the first sublayer) the streams stay as they are; with a stream stride of 0 they are all the same row.
#include "rows.h"

namespace {

enum { HN_RSTD = 0, HN_NORM = 1, HN_CONV = 2 };

struct HyperArgs {
  const float* x;              // [T] rows of stride ldx, streams lds apart
  int64_t ldx, lds;
  float* x_out;                // [T][S][W], null: not stored (may be x)
  const float* y; int split;   // slabs [split][T][W] or null
  const float* mix; const float* out; const float* in;
  const float* w;              // [W] the norm's multiplier
  float eps;
  const int32_t* rows;         // row of the b-th workgroup (null: b); normed outputs are at b
  int T, W, S;
  float* u; float* rstd;       // HN_RSTD
  const float* cw; int taps;   // HN_CONV: [taps][W]
  const int32_t* positions; const int32_t* slots;
  float* tail; int ring;       // [slots][ring][W], position p at p % ring
};

// SM >= S copies in registers; a thread holds NV vectors of V channels
template <typename ACT, int V, int SM, int NV, int BT>
__global__ void __launch_bounds__(BT) hyper_norm_kernel(HyperArgs a, int mode, ACT* __restrict__ h) {
  __shared__ float red[16];
  __shared__ float mx[SM * SM + 2 * SM];       // mix [from][to], out, in
  const int b = blockIdx.x, t = a.rows ? a.rows[b] : b, W = a.W, S = a.S;
  const float* xr = a.x + t * a.ldx;
  for (int i = threadIdx.x; i < SM * SM + 2 * SM; i += BT) {
    const int s = i / SM, k = i % SM;          // past S: weight 0
    float v = 0.f;
    if (s < SM) v = s < S && k < S ? (a.y ? a.mix[s * S + k] : s == k ? 1.f : 0.f) : 0.f;
    else if (s == SM) v = k < S && a.y ? a.out[k] : 0.f;
    else v = k < S ? (a.in ? a.in[k] : 1.f) : 0.f;
    mx[i] = v;
  }
  // a decoded row's convolution past, asked for ahead of the stream
  constexpr int PRE = NV == 1 && V == 4 ? 3 : 0;
  const int pos = mode == HN_CONV ? a.positions[b] : 0, back = a.taps - 1;
  float* tail = mode == HN_CONV && back > 0 ? a.tail + (size_t)a.slots[b] * a.ring * W : nullptr;
  const bool ahead = PRE > 0 && back <= PRE;
  Vec<V> past[PRE ? PRE : 1], cw[PRE ? PRE + 1 : 1];
  if constexpr (PRE > 0)
    if (mode == HN_CONV && ahead) {
      const int c = min((int)threadIdx.x * V, W - V);
#pragma unroll
      for (int d = 0; d <= PRE; ++d) cw[d] = ldv<V>(a.cw + (size_t)max(back - d, 0) * W + c);
#pragma unroll
      for (int d = 1; d <= PRE; ++d) past[d - 1] = d <= back && d <= pos ? ldv<V>(tail + (size_t)((pos - d) % a.ring) * W + c) : zerov<V>();
    }
  Vec<V> u[NV], x[SM], y = zerov<V>();
  float ss = 0.f;
  auto load = [&](int c) {
#pragma unroll
    for (int s = 0; s < SM; ++s) x[s] = ldv<V>(xr + min(s, S - 1) * a.lds + c);
    if (a.y) {
      y = zerov<V>();
      add_slabs<V>(y, a.y, a.split, (int64_t)a.T * W, (size_t)t * W + c);
    }
  };
  load(min((int)threadIdx.x * V, W - V));
  __syncthreads();
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    u[k] = zerov<V>();
    if (c >= W) continue;
    if (k) load(c);
    if (a.y) {
#pragma unroll
      for (int q = 0; q < SM; ++q) {
        if (q >= S) break;
        Vec<V> n;
#pragma unroll
        for (int e = 0; e < V; ++e) n.v[e] = mx[SM * SM + q] * y.v[e];
#pragma unroll
        for (int s = 0; s < SM; ++s)
#pragma unroll
          for (int e = 0; e < V; ++e) n.v[e] += mx[s * SM + q] * x[s].v[e];
        if (a.x_out) stv<V>(a.x_out + ((size_t)t * S + q) * W + c, n);
#pragma unroll
        for (int e = 0; e < V; ++e) u[k].v[e] += mx[SM * SM + SM + q] * n.v[e];
      }
    } else {
#pragma unroll
      for (int s = 0; s < SM; ++s)
#pragma unroll
        for (int e = 0; e < V; ++e) u[k].v[e] += mx[SM * SM + SM + s] * x[s].v[e];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) ss += u[k].v[e] * u[k].v[e];
  }
  const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + a.eps);
  if (mode == HN_RSTD) {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + threadIdx.x) * V;
      if (c < W) stv<V>(a.u + (size_t)t * W + c, u[k]);
    }
    if (threadIdx.x == 0) a.rstd[t] = r;
    return;
  }
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + threadIdx.x) * V;
    if (c >= W) continue;
    const Vec<V> g = ldv<V>(a.w + c);
    Vec<V> n;
#pragma unroll
    for (int e = 0; e < V; ++e) n.v[e] = u[k].v[e] * r * g.v[e];
    if (mode == HN_CONV) {
      const Vec<V> own = n;
      if (ahead) {
        if constexpr (PRE > 0) {
#pragma unroll
          for (int e = 0; e < V; ++e) n.v[e] += cw[0].v[e] * own.v[e];
#pragma unroll
          for (int d = 1; d <= PRE; ++d)
            if (d <= back)
#pragma unroll
              for (int e = 0; e < V; ++e) n.v[e] += cw[d].v[e] * past[d - 1].v[e];
        }
      } else {
        for (int d = 0; d <= back && d <= pos; ++d) {
          const Vec<V> o = d ? ldv<V>(tail + (size_t)((pos - d) % a.ring) * W + c) : own;
          const Vec<V> wd = ldv<V>(a.cw + (size_t)(back - d) * W + c);
#pragma unroll
          for (int e = 0; e < V; ++e) n.v[e] += wd.v[e] * o.v[e];
        }
      }
      if (back > 0) stv<V>(tail + (size_t)(pos % a.ring) * W + c, own);
    }
    stv<V>(h + (size_t)b * W + c, n);
  }
}

template <typename ACT, int V, int SM>
int hyper_go(hipStream_t s, int n, const HyperArgs& a, int mode, void* h) {
  const int vecs = (a.W + V - 1) / V;
#define GO(NV, BT) hyper_norm_kernel<ACT, V, SM, NV, BT><<<n, BT, 0, s>>>(a, mode, (ACT*)h)
  if (vecs <= 64) GO(1, 64);
  else if (vecs <= 256) GO(1, 256);
  else if (vecs <= 512) GO(1, 512);
  else if (vecs <= 1024) GO(1, 1024);
  else if (vecs <= 4096) GO(4, 1024);
  else if (vecs <= 16384) GO(16, 1024);
  else return -4;
#undef GO
  return CFC_CHECK_LAUNCH();
}

constexpr int HYPER_MAX = 16;

}  // namespace

// mode 0: u and rstd; 1: normed rows into h [n][W]; 2: decoded rows, normed and convolved.  f32: h is fp32 (else bf16).
// y null: no update (mix, out unused); x_out null: streams not stored; rows null: row b of T (modes 1)
CFC_API int cfc_hyper_norm(int mode, int f32, int n, const int32_t* rows, const float* x, int64_t ldx, int64_t lds, float* x_out,
                           const float* y, int split, const float* mix, const float* out, const float* in, const float* w,
                           float eps, int T, int W, int S, float* u, float* rstd, const float* cw, int taps,
                           const int32_t* positions, const int32_t* slots, float* tail, int ring, void* h, hipStream_t stream) {
  if (n <= 0) return 0;
  if (T < 1 || W < 1 || S < 1 || S > HYPER_MAX || !x || (!rows && n > T)) return -1;
  if (y && (split < 1 || !mix || !out)) return -2;
  if (mode == HN_RSTD ? (!u || !rstd) : (!h || !w)) return -2;
  if (mode == HN_CONV && (rows || !cw || taps < 1 || !positions || (taps > 1 && (!slots || !tail || ring < taps - 1)))) return -3;
  if (mode < HN_RSTD || mode > HN_CONV || (mode != HN_NORM && rows)) return -3;
  const HyperArgs a{x, ldx, lds, x_out, y, split, mix, out, in, w, eps, rows, T, W, S, u, rstd, cw, taps, positions, slots, tail,
                    ring > 0 ? ring : 1};
  const bool v4 = W % 4 == 0 && ldx % 4 == 0 && lds % 4 == 0;
#define HG(ACT)                                                             \
  return !v4 ? hyper_go<ACT, 1, HYPER_MAX>(stream, n, a, mode, h)           \
             : S <= 4 ? hyper_go<ACT, 4, 4>(stream, n, a, mode, h) : hyper_go<ACT, 4, HYPER_MAX>(stream, n, a, mode, h)
  if (f32) HG(float);
  HG(uint16_t);
#undef HG
}
