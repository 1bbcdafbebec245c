// From the projections of an attention layer to its queries and its cache rows:
//   * qkv_rows    [short causal convolution over time per channel] -> [RMS norm, over the whole projection or per head]
//                 -> [rotation of neighbouring pairs] -> queries [T][H][D] (scaled into the exponent's base 2), keys
//                 and values into the paged cache [blocks][G][32][D].  A row's queries, keys and values take a
//                 workgroup each.  Decoded rows also store what the convolution remembers and, where a pooled block of
//                 tokens ends, the block's mean key and value
//   * conv_tail   the last inputs of prompt portions' convolutions into the sequences' state (a launch of its own:
//                 rows of the same portion read the old ones)
//   * pool_rows   mean keys and values of the blocks that prompt portions end, from the cache as it holds them
//
// Convolution state: [slots][taps - 1][channels] fp32, position p at row p % (taps - 1).  Pooled block b lies at entry
// b % E of page b / E (E a power of two, at least 32 / pool: the page of a block's mean exists when its tokens do).
// D: columns of a cached head, dim (or vdim) rounded up; the pad stays zero.
#include "rows.h"

namespace {

struct QkvArgs {
  const void* p; int split; int64_t ld, plane;      // columns [H dim | G dim | G vdim] of a product (split 0: activations)
  int H, G, dim, vdim, D, parts;                    // parts 1: queries only
  const float* qn; const float* kn;                 // norm weights: [H dim] / [G dim], or [dim] per head (null: no norm)
  int per_head;
  float eps;
  const float* freq; int rot;                       // rot dimensions of each head turn by position * freq[i]
  float qscale;
  const float* conv; int taps; float* tail;         // [taps][channels], null: none
  const int32_t* lead;                              // rows of the same portion before a row (null: decoded, none)
  const int32_t* slots; const int32_t* positions; const int32_t* cslots;
  void* q; void* kc; void* vc;
  void* pk; void* pv; int pool, le;                 // decoded rows: pooled cache (pool 0: none)
  const int32_t* bt; int max_blocks;
};

template <typename ACT, int V>
__device__ __forceinline__ Vec<V> qkv_ld(const QkvArgs& a, int64_t t, int c) {
  const int64_t o = t * a.ld + c;
  if (a.split == 0) return ldv<V>(reinterpret_cast<const ACT*>(a.p) + o);
  Vec<V> y = zerov<V>();
  add_slabs<V>(y, reinterpret_cast<const float*>(a.p), a.split, a.plane, (size_t)o);
  return y;
}

__device__ __forceinline__ float round_act(float v, const uint16_t*) { return bf2f(f2bf(v)); }
__device__ __forceinline__ float round_act(float v, const float*) { return v; }

constexpr int ROT_MAX = 1024;

// grid (rows, parts).  Dynamic LDS: per-vector sums, and for V = 1 the row
template <typename ACT, int V, int NV, int BT>
__global__ void __launch_bounds__(BT) qkv_rows_kernel(QkvArgs a) {
  __shared__ float red[16];
  __shared__ float2 cs[ROT_MAX / 2];
  extern __shared__ float dyn[];
  const int t = xcd_remap(blockIdx.x, gridDim.x), part = blockIdx.y, tid = threadIdx.x;
  const int pos = a.positions[t], heads = part == 0 ? a.H : a.G, hd = part == 2 ? a.vdim : a.dim, C = heads * hd;
  const int c0 = part == 0 ? 0 : part == 1 ? a.H * a.dim : (a.H + a.G) * a.dim;
  const int nvec = C / V, allc = a.H * a.dim + (a.parts > 1 ? a.G * (a.dim + a.vdim) : 0);
  const float* wn = part == 0 ? a.qn : part == 1 ? a.kn : nullptr;
  const int rot = part == 2 ? 0 : a.rot;
  Vec<V> x[NV];
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + tid) * V;
    x[k] = c < C ? qkv_ld<ACT, V>(a, t, c0 + c) : zerov<V>();
  }
  if (a.conv) {
    const int back = a.taps - 1, lead = a.lead ? a.lead[t] : 0;
    float* st = back ? a.tail + (size_t)a.slots[t] * back * allc + c0 : nullptr;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V;
      if (c >= C) continue;
      const Vec<V> u = x[k], w = ldv<V>(a.conv + (size_t)back * allc + c0 + c);
#pragma unroll
      for (int e = 0; e < V; ++e) x[k].v[e] *= w.v[e];
      for (int d = back; d > 0; --d) {               // d rows before
        if (pos < d) continue;
        const Vec<V> o = d <= lead ? qkv_ld<ACT, V>(a, t - d, c0 + c) : ldv<V>(st + (size_t)((pos - d) % back) * allc + c);
        const Vec<V> wd = ldv<V>(a.conv + (size_t)(back - d) * allc + c0 + c);
#pragma unroll
        for (int e = 0; e < V; ++e) x[k].v[e] += wd.v[e] * o.v[e];
      }
      if (!a.lead && back > 0) stv<V>(st + (size_t)(pos % back) * allc + c, u);
    }
  }
  for (int i = tid; i < rot / 2; i += BT) {
    float sn, co;
    sincosf((float)pos * a.freq[i], &sn, &co);
    cs[i] = make_float2(co, sn);
  }
  float r[NV];
#pragma unroll
  for (int k = 0; k < NV; ++k) r[k] = 1.f;
  if (wn) {
    float ss[NV], all = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      ss[k] = 0.f;
#pragma unroll
      for (int e = 0; e < V; ++e) ss[k] += x[k].v[e] * x[k].v[e];
      all += ss[k];
    }
    const int hv = hd / V;
    if (!a.per_head) {
      const float v = 1.f / sqrtf(block_sum(all, red) / (float)C + a.eps);
#pragma unroll
      for (int k = 0; k < NV; ++k) r[k] = v;
    } else if (hv <= 64 && (hv & (hv - 1)) == 0) {     // a head is a run of lanes
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        for (int m = hv / 2; m > 0; m >>= 1) ss[k] += __shfl_xor(ss[k], m, 64);
        r[k] = 1.f / sqrtf(ss[k] / (float)hd + a.eps);
      }
    } else {
#pragma unroll
      for (int k = 0; k < NV; ++k)
        if (k * BT + tid < nvec) dyn[k * BT + tid] = ss[k];
      __syncthreads();
      for (int h = tid; h < heads; h += BT) {
        float s = 0.f;
        for (int i = 0; i < hv; ++i) s += dyn[h * hv + i];
        dyn[nvec + h] = 1.f / sqrtf(s / (float)hd + a.eps);
      }
      __syncthreads();
#pragma unroll
      for (int k = 0; k < NV; ++k)
        if (k * BT + tid < nvec) r[k] = dyn[nvec + (k * BT + tid) / hv];
    }
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V;
      if (c >= C) continue;
      const Vec<V> w = ldv<V>(wn + (a.per_head ? c % hd : c));
#pragma unroll
      for (int e = 0; e < V; ++e) x[k].v[e] *= r[k] * w.v[e];
    }
  }
  __syncthreads();                                     // cs; and dyn, read above
  if constexpr (V == 1) {
    if (rot) {
#pragma unroll
      for (int k = 0; k < NV; ++k)
        if (k * BT + tid < C) dyn[k * BT + tid] = x[k].v[0];
      __syncthreads();
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = k * BT + tid, d = c % hd;
        if (c >= C || d >= rot) continue;
        const float2 f = cs[d >> 1];
        x[k].v[0] = d & 1 ? dyn[c] * f.x + dyn[c - 1] * f.y : dyn[c] * f.x - dyn[c + 1] * f.y;
      }
    }
  } else if (rot) {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V, d = c % hd;
      if (c >= C) continue;
#pragma unroll
      for (int e = 0; e < V; e += 2)
        if (d + e < rot) {
          const float2 f = cs[(d + e) >> 1];
          const float u = x[k].v[e], v = x[k].v[e + 1];
          x[k].v[e] = u * f.x - v * f.y;
          x[k].v[e + 1] = v * f.x + u * f.y;
        }
    }
  }
  if (part == 0) {
    ACT* q = reinterpret_cast<ACT*>(a.q) + (size_t)t * a.H * a.D;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V;
      if (c >= C) continue;
#pragma unroll
      for (int e = 0; e < V; ++e) x[k].v[e] *= a.qscale;
      stv<V>(q + c / hd * a.D + c % hd, x[k]);
    }
    return;
  }
  ACT* cache = reinterpret_cast<ACT*>(part == 1 ? a.kc : a.vc);
  const int slot = a.cslots[t];
  auto row = [&](int blk, int g, int off) { return (((size_t)blk * a.G + g) * CFC_KV_BS + off) * a.D; };
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + tid) * V;
    if (c < C) stv<V>(cache + row(slot / CFC_KV_BS, c / hd, slot % CFC_KV_BS) + c % hd, x[k]);
  }
  if (a.pool == 0 || (pos + 1) % a.pool) return;
  const int32_t* bt = a.bt + (size_t)t * a.max_blocks;
  const int b = pos / a.pool;
  ACT* pc = reinterpret_cast<ACT*>(part == 1 ? a.pk : a.pv) + (((size_t)bt[b >> a.le] * a.G) << a.le) * a.D;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + tid) * V, g = c / hd;
    if (c >= C) continue;
    Vec<V> m;
#pragma unroll
    for (int e = 0; e < V; ++e) m.v[e] = round_act(x[k].v[e], (const ACT*)nullptr);
    for (int j = 1; j < a.pool; ++j) {
      const int pj = pos - j;
      const Vec<V> o = ldv<V>(cache + row(bt[pj / CFC_KV_BS], g, pj % CFC_KV_BS) + c % hd);
#pragma unroll
      for (int e = 0; e < V; ++e) m.v[e] += o.v[e];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) m.v[e] /= (float)a.pool;
    stv<V>(pc + (((size_t)g << a.le) + (b & ((1 << a.le) - 1))) * a.D + c % hd, m);
  }
}

template <typename ACT, int V>
int qkv_go(hipStream_t s, int T, const QkvArgs& a) {
  int C = a.H * a.dim;
  if (a.parts > 1) C = max(C, a.G * max(a.dim, a.vdim));
  const int vecs = (C + V - 1) / V;
  const size_t lds = (size_t)(vecs + max(a.H, a.G)) * 4;
  if (lds > 49152) return -4;
#define GO(NV, BT) qkv_rows_kernel<ACT, V, NV, BT><<<dim3(T, a.parts), BT, lds, s>>>(a)
  if (vecs <= 64) GO(1, 64);
  else if (vecs <= 256) GO(1, 256);
  else if (vecs <= 512) GO(2, 256);
  else if (vecs <= 1024) GO(4, 256);
  else if (vecs <= 4096) GO(4, 1024);
  else if (vecs <= 16384) GO(16, 1024);
  else return -4;
#undef GO
  return CFC_CHECK_LAUNCH();
}

// grid (portions, taps - 1): the inputs of a portion's last rows
template <typename ACT>
__global__ void __launch_bounds__(256) conv_tail_kernel(const void* __restrict__ p, int split, int64_t ld, int64_t plane, int C,
                                                       const int32_t* __restrict__ cu_q, const int32_t* __restrict__ ctx_lens,
                                                       const int32_t* __restrict__ slots, int back, float* __restrict__ tail) {
  const int s = blockIdx.x, d = blockIdx.y, r1 = cu_q[s + 1], t = r1 - 1 - d;
  if (t < cu_q[s]) return;
  float* st = tail + ((size_t)slots[s] * back + (ctx_lens[s] - 1 - d) % back) * C;
  for (int c = threadIdx.x; c < C; c += 256) {
    float v = 0.f;
    if (split == 0) v = ld1(reinterpret_cast<const ACT*>(p) + t * ld + c);
    else for (int i = 0; i < split; ++i) v += reinterpret_cast<const float*>(p)[t * ld + i * plane + c];
    st[c] = v;
  }
}

// blocks [n][2]: {sequence, block}; grid (n, G)
template <typename ACT>
__global__ void __launch_bounds__(256) pool_rows_kernel(const int32_t* __restrict__ blocks, const int32_t* __restrict__ tables,
                                                       int max_blocks, const ACT* __restrict__ kc, const ACT* __restrict__ vc,
                                                       ACT* __restrict__ pk, ACT* __restrict__ pv, int G, int D, int pool, int le) {
  const int s = blocks[2 * blockIdx.x], b = blocks[2 * blockIdx.x + 1], g = blockIdx.y;
  const int32_t* bt = tables + (size_t)s * max_blocks;
  const size_t dst = ((((size_t)bt[b >> le] * G + g) << le) + (b & ((1 << le) - 1))) * D;
  for (int c = threadIdx.x; c < 2 * D; c += 256) {
    const ACT* src = c < D ? kc + c : vc + (c - D);
    float m = 0.f;
    for (int j0 = 0; j0 < pool; j0 += 8) {             // eight rows in flight (past the last: re-read, not added)
      float v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int p = b * pool + min(j0 + u, pool - 1);
        v[u] = ld1(src + (((size_t)bt[p / CFC_KV_BS] * G + g) * CFC_KV_BS + p % CFC_KV_BS) * D);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) m += j0 + u < pool ? v[u] : 0.f;
    }
    m /= (float)pool;
    if constexpr (sizeof(ACT) == 2) (c < D ? pk + dst + c : pv + dst + (c - D))[0] = f2bf(m);
    else (c < D ? pk + dst + c : pv + dst + (c - D))[0] = m;
  }
}

}  // namespace

// lead null: decoded rows (conv state and pooled blocks are written here).  parts 1: queries only (kc .. pv unused)
CFC_API int cfc_qkv_rows(int f32, const void* p, int split, int64_t ld, int64_t plane, int T, int H, int G, int dim, int vdim, int D,
                         int parts, const float* qn, const float* kn, int per_head, float eps, const float* freq, int rot,
                         float qscale, const float* conv, int taps, float* tail, const int32_t* lead, const int32_t* slots,
                         const int32_t* positions, const int32_t* cslots, void* q, void* kc, void* vc, void* pk, void* pv, int pool,
                         int le, const int32_t* bt, int max_blocks, hipStream_t stream) {
  if (T <= 0) return 0;
  if (H < 1 || G < 1 || dim < 1 || vdim < 1 || D < dim || D < vdim || rot < 0 || rot % 2 || rot > dim || rot > ROT_MAX ||
      (parts != 1 && parts != 3))
    return -1;
  if ((parts == 3 && (!kc || !vc || !cslots)) || (conv && (taps < 1 || (taps > 1 && (!tail || !slots)))) || (rot && !freq)) return -2;
  if (pool < 0 || (pool && parts == 3 && (!pk || !pv || !bt || le < 0 || le > 5 || (pool << le) < CFC_KV_BS))) return -3;
  const QkvArgs a{p, split, ld, plane, H, G, dim, vdim, D, parts, qn, kn, per_head, eps, freq, rot, qscale, conv, taps, tail,
                  lead, slots, positions, cslots, q, kc, vc, pk, pv, lead ? 0 : pool, le, bt, max_blocks};
  const bool v4 = dim % 4 == 0 && vdim % 4 == 0 && D % 4 == 0 && ld % 4 == 0 && plane % 4 == 0 &&
                  ((uintptr_t)p & (split == 0 && !f32 ? 7 : 15)) == 0;
  if (f32) return v4 ? qkv_go<float, 4>(stream, T, a) : qkv_go<float, 1>(stream, T, a);
  return v4 ? qkv_go<uint16_t, 4>(stream, T, a) : qkv_go<uint16_t, 1>(stream, T, a);
}

CFC_API int cfc_conv_tail(int f32, const void* p, int split, int64_t ld, int64_t plane, int C, const int32_t* cu_q,
                          const int32_t* ctx_lens, const int32_t* slots, int portions, int taps, float* tail, hipStream_t stream) {
  if (portions <= 0 || taps < 2) return 0;
  if (C < 1 || !cu_q || !ctx_lens || !slots || !tail) return -1;
  const dim3 grid(portions, taps - 1);
  if (f32) conv_tail_kernel<float><<<grid, 256, 0, stream>>>(p, split, ld, plane, C, cu_q, ctx_lens, slots, taps - 1, tail);
  else conv_tail_kernel<uint16_t><<<grid, 256, 0, stream>>>(p, split, ld, plane, C, cu_q, ctx_lens, slots, taps - 1, tail);
  return CFC_CHECK_LAUNCH();
}

CFC_API int cfc_pool_rows(int f32, const int32_t* blocks, int n, const int32_t* tables, int max_blocks, const void* kc, const void* vc,
                          void* pk, void* pv, int G, int D, int pool, int le, hipStream_t stream) {
  if (n <= 0) return 0;
  if (G < 1 || G > 65535 || D < 1 || pool < 1 || le < 0 || le > 5 || (pool << le) < CFC_KV_BS || max_blocks < 1) return -1;
  const dim3 grid(n, G);
  if (f32)
    pool_rows_kernel<float><<<grid, 256, 0, stream>>>(blocks, tables, max_blocks, (const float*)kc, (const float*)vc, (float*)pk,
                                                      (float*)pv, G, D, pool, le);
  else
    pool_rows_kernel<uint16_t><<<grid, 256, 0, stream>>>(blocks, tables, max_blocks, (const uint16_t*)kc, (const uint16_t*)vc,
                                                         (uint16_t*)pk, (uint16_t*)pv, G, D, pool, le);
  return CFC_CHECK_LAUNCH();
}
