// From the projections of an attention layer to its queries and its cache rows:
//   * qkv_rows    [short causal convolution over time per channel] -> [RMS norm, over the whole projection or per head]
//                 -> [rotation of neighbouring pairs] -> queries [T][H][D] (scaled into the exponent's base 2), keys
//                 and values into the paged cache [blocks][G][32][D].  A row's queries, keys and values take a
//                 workgroup each.  Decoded rows also store what the convolution remembers and, where a pooled block of
//                 tokens ends, the block's mean key and value
//   * qkv_prompt  the same for prompt rows of common shapes, many rows per workgroup
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
constexpr int MAX_BACK = 3;          // convolution rows before the own that a thread holds in registers

// grid (rows, parts).  Dynamic LDS: per-vector sums, and for V = 1 the row
template <typename ACT, int V, int NV, int BT>
__global__ void __launch_bounds__(BT) qkv_rows_kernel(QkvArgs a) {
  __shared__ float red[16];
  __shared__ float2 cs[ROT_MAX / 2];
  extern __shared__ float dyn[];
  const int t = xcd_remap(blockIdx.x, gridDim.x), part = blockIdx.y, tid = threadIdx.x;
  // gridDim.z > 1: each takes a run of the heads
  const int all_heads = part == 0 ? a.H : a.G, h0 = all_heads * blockIdx.z / gridDim.z, h1 = all_heads * (blockIdx.z + 1) / gridDim.z;
  const int pos = a.positions[t], heads = h1 - h0, hd = part == 2 ? a.vdim : a.dim, C = heads * hd;
  const int c0 = (part == 0 ? 0 : part == 1 ? a.H * a.dim : (a.H + a.G) * a.dim) + h0 * hd;
  if (heads == 0) return;
  const int nvec = C / V, allc = a.H * a.dim + (a.parts > 1 ? a.G * (a.dim + a.vdim) : 0);
  const float* wn = part == 0 ? a.qn : part == 1 ? a.kn : nullptr;
  const int rot = part == 2 ? 0 : a.rot;
  Vec<V> x[NV];
  if (!a.conv) {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V;
      x[k] = c < C ? qkv_ld<ACT, V>(a, t, c0 + c) : zerov<V>();
    }
  } else {
#pragma unroll
    for (int k = 0; k < NV; ++k) x[k] = zerov<V>();
    const int back = a.taps - 1, lead = a.lead ? a.lead[t] : 0;
    float* st = back ? a.tail + (size_t)a.slots[t] * back * allc + c0 : nullptr;
    if (!a.lead && back <= MAX_BACK) {
      // decoded rows: what a vector needs is asked for together
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = min((k * BT + tid) * V, C - V);
        Vec<V> o[MAX_BACK], w[MAX_BACK + 1];
#pragma unroll
        for (int d = 0; d <= MAX_BACK; ++d) w[d] = ldv<V>(a.conv + (size_t)max(back - d, 0) * allc + c0 + c);
#pragma unroll
        for (int d = 1; d <= MAX_BACK; ++d)
          o[d - 1] = d <= back && d <= pos ? ldv<V>(st + (size_t)((pos - d) % max(back, 1)) * allc + c) : zerov<V>();
        const Vec<V> u = qkv_ld<ACT, V>(a, t, c0 + c);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          x[k].v[e] = u.v[e] * w[0].v[e];
#pragma unroll
          for (int d = 1; d <= MAX_BACK; ++d) x[k].v[e] += d <= back ? o[d - 1].v[e] * w[d].v[e] : 0.f;
        }
        if ((k * BT + tid) * V >= C) x[k] = zerov<V>();
        else if (back > 0) stv<V>(st + (size_t)(pos % back) * allc + c, u);
      }
    } else
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * BT + tid) * V;
      if (c >= C) continue;
      x[k] = qkv_ld<ACT, V>(a, t, c0 + c);
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
    ACT* q = reinterpret_cast<ACT*>(a.q) + ((size_t)t * a.H + h0) * a.D;
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
    if (c < C) stv<V>(cache + row(slot / CFC_KV_BS, h0 + c / hd, slot % CFC_KV_BS) + c % hd, x[k]);
  }
  if (a.pool == 0 || (pos + 1) % a.pool) return;
  const int32_t* bt = a.bt + (size_t)t * a.max_blocks;
  const int b = pos / a.pool;
  ACT* pc = reinterpret_cast<ACT*>(part == 1 ? a.pk : a.pv) + (((size_t)bt[b >> a.le] * a.G) << a.le) * a.D;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BT + tid) * V, g = h0 + c / hd;
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

// Prompt rows from activations: PR_ROWS consecutive rows of one part (0: queries, 1: keys and values) per workgroup, two or four
// at a time, a vector of V channels per thread.  What the convolution reads back stays in registers, weights are read
// once, the rows of a time share one reduction.  Heads of a power of two of vectors (per-head norms) and, with a
// convolution, at most MAX_BACK + 1 taps.
constexpr int PR_ROWS = 16;
template <typename ACT, int V> struct Raw;
template <> struct Raw<uint16_t, 8> {
  uint4 u;
  __device__ __forceinline__ void get(const void* p) { u = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ void zero() { u = make_uint4(0, 0, 0, 0); }
  __device__ __forceinline__ Vec<8> val() const { Vec<8> r; unpack8(u, r.v); return r; }
};
template <> struct Raw<float, 4> {
  float4 f;
  __device__ __forceinline__ void get(const void* p) { f = *reinterpret_cast<const float4*>(p); }
  __device__ __forceinline__ void zero() { f = make_float4(0.f, 0.f, 0.f, 0.f); }
  __device__ __forceinline__ Vec<4> val() const { return Vec<4>{{f.x, f.y, f.z, f.w}}; }
};
template <int V>
__device__ __forceinline__ Vec<V> ldw(const float* p) {
  Vec<V> r;
#pragma unroll
  for (int e = 0; e < V; e += 4) {
    const float4 f = *reinterpret_cast<const float4*>(p + e);
    r.v[e] = f.x; r.v[e + 1] = f.y; r.v[e + 2] = f.z; r.v[e + 3] = f.w;
  }
  return r;
}
__device__ __forceinline__ void stw(uint16_t* p, const Vec<8>& r) { *reinterpret_cast<uint4*>(p) = pack8(r.v); }
__device__ __forceinline__ void stw(float* p, const Vec<4>& r) { *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]); }

template <typename ACT, int V, int BT, bool CONV>
__global__ void __launch_bounds__(BT, BT <= 512 ? 4 : 1) qkv_prompt_kernel(QkvArgs a, int T) {
  constexpr int RG = CONV ? 2 : 4, NW = BT / 64;
  __shared__ float red[2][RG][NW];
  __shared__ int4 meta[PR_ROWS];                       // position, rows before it in its portion, cache slot, state slot
  extern __shared__ float2 cs[];                       // [PR_ROWS][rot / 2]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, part = blockIdx.y;
  const int t0 = xcd_remap(blockIdx.x, gridDim.x) * PR_ROWS, t1 = min(t0 + PR_ROWS, T);
  const int allc = a.H * a.dim + (a.parts > 1 ? a.G * (a.dim + a.vdim) : 0), nk = a.G * a.dim, c = tid * V;
  const int C = part == 0 ? a.H * a.dim : nk, cp = part == 0 ? 0 : a.H * a.dim;
  const bool live = c < (part == 0 ? C : nk + a.G * a.vdim), isv = part == 1 && c >= nk;
  const int hd = isv ? a.vdim : a.dim, ch = isv ? c - nk : c, head = ch / hd, cd = ch - head * hd;
  const float* wn = isv || !live ? nullptr : part == 0 ? a.qn : a.kn;
  const int back = CONV ? a.taps - 1 : 0, half = a.rot / 2;
  const bool turn = !isv && live && cd < a.rot;
  for (int i = tid; i < PR_ROWS; i += BT) {
    const int t = min(t0 + i, T - 1);
    meta[i] = make_int4(a.positions[t], a.lead[t], a.cslots ? a.cslots[t] : 0, back ? a.slots[t] : 0);
  }
  const ACT* src = reinterpret_cast<const ACT*>(a.p) + cp + (live ? c : 0);
  Vec<V> nw, cw[MAX_BACK + 1];
#pragma unroll
  for (int e = 0; e < V; ++e) nw.v[e] = 1.f;
  if (wn) nw = ldw<V>(wn + (a.per_head ? cd : c));
  if (part == 0)
#pragma unroll
    for (int e = 0; e < V; ++e) nw.v[e] *= a.qscale;
  if constexpr (CONV) {
#pragma unroll
    for (int d = 0; d <= MAX_BACK; ++d) {
      cw[d] = ldw<V>(a.conv + (size_t)max(back - d, 0) * allc + cp + (live ? c : 0));
      if (d > back)
#pragma unroll
        for (int e = 0; e < V; ++e) cw[d].v[e] = 0.f;
    }
  }
  // win[MAX_BACK + r]: row r of the group
  Raw<ACT, V> win[MAX_BACK + RG], nxt[RG];
  if constexpr (CONV)
#pragma unroll
    for (int d = 1; d <= MAX_BACK; ++d) win[MAX_BACK - d].get(src + (int64_t)max(t0 - d, 0) * a.ld);
#pragma unroll
  for (int r = 0; r < RG; ++r) win[MAX_BACK + r].get(src + (int64_t)min(t0 + r, T - 1) * a.ld);
  __syncthreads();
  for (int i = tid; i < PR_ROWS * half; i += BT) {
    float sn, co;
    sincosf((float)meta[i / half].x * a.freq[i % half], &sn, &co);
    cs[i] = make_float2(co, sn);
  }
  __syncthreads();
  for (int g0 = t0, par = 0; g0 < t1; g0 += RG, par ^= 1) {
    int4 mt[RG];
    int least = MAX_BACK;
#pragma unroll
    for (int r = 0; r < RG; ++r) {
      mt[r] = meta[g0 - t0 + r];
      least = min(least, mt[r].y);
    }
    const bool inside = __builtin_amdgcn_readfirstlane(least) >= back;      // no row reads before its portion
#pragma unroll
    for (int r = 0; r < RG; ++r) nxt[r].get(src + (int64_t)min(g0 + RG + r, T - 1) * a.ld);
    Vec<V> y[RG];
    float ss[RG];
#pragma unroll
    for (int r = 0; r < RG; ++r) {
      y[r] = win[MAX_BACK + r].val();
      if constexpr (CONV) {
#pragma unroll
        for (int e = 0; e < V; ++e) y[r].v[e] *= cw[0].v[e];
        if (inside) {                          // weights past the taps are zero
#pragma unroll
          for (int d = 1; d <= MAX_BACK; ++d) {
            const Vec<V> o = win[MAX_BACK + r - d].val();
#pragma unroll
            for (int e = 0; e < V; ++e) y[r].v[e] += cw[d].v[e] * o.v[e];
          }
        } else {
          const int pos = __builtin_amdgcn_readfirstlane(mt[r].x), lead = __builtin_amdgcn_readfirstlane(mt[r].y);
#pragma unroll
          for (int d = 1; d <= MAX_BACK; ++d) {
            if (d > back || d > pos) break;
            const Vec<V> o = d <= lead ? win[MAX_BACK + r - d].val()
                                       : ldw<V>(a.tail + ((size_t)mt[r].w * back + (pos - d) % back) * allc + cp + (live ? c : 0));
#pragma unroll
            for (int e = 0; e < V; ++e) y[r].v[e] += cw[d].v[e] * o.v[e];
          }
        }
      }
      ss[r] = 0.f;
      if (wn)
#pragma unroll
        for (int e = 0; e < V; ++e) ss[r] += y[r].v[e] * y[r].v[e];
    }
    float inv[RG];
    if (a.per_head) {
      const int hv = a.dim / V;
#pragma unroll
      for (int r = 0; r < RG; ++r) {
        for (int m = hv / 2; m > 0; m >>= 1) ss[r] += __shfl_xor(ss[r], m, 64);
        inv[r] = 1.f / sqrtf(ss[r] / (float)a.dim + a.eps);
      }
    } else {
#pragma unroll
      for (int r = 0; r < RG; ++r) {
        ss[r] = wave_sum(ss[r]);
        if (lane == 0) red[par][r][w] = ss[r];
      }
      __syncthreads();
#pragma unroll
      for (int r = 0; r < RG; ++r) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < NW; ++i) s += red[par][r][i];
        inv[r] = 1.f / sqrtf(s / (float)C + a.eps);
      }
    }
#pragma unroll
    for (int r = 0; r < RG; ++r) {
      const int t = g0 + r;
      if (t >= t1 || !live) continue;
      const float f = wn ? inv[r] : 1.f;
#pragma unroll
      for (int e = 0; e < V; ++e) y[r].v[e] *= f * nw.v[e];
      if (turn) {
#pragma unroll
        for (int e = 0; e < V; e += 2)
          if (cd + e < a.rot) {
            const float2 k = cs[(t - t0) * half + ((cd + e) >> 1)];
            const float u = y[r].v[e], v = y[r].v[e + 1];
            y[r].v[e] = u * k.x - v * k.y;
            y[r].v[e + 1] = v * k.x + u * k.y;
          }
      }
      if (part == 0) {
        stw(reinterpret_cast<ACT*>(a.q) + ((size_t)t * a.H + head) * a.D + cd, y[r]);
      } else {
        const int slot = mt[r].z;
        stw(reinterpret_cast<ACT*>(isv ? a.vc : a.kc) +
                (((size_t)(slot / CFC_KV_BS) * a.G + head) * CFC_KV_BS + slot % CFC_KV_BS) * a.D + cd, y[r]);
      }
    }
#pragma unroll
    for (int d = 0; d < MAX_BACK; ++d) win[d] = win[d + RG];
#pragma unroll
    for (int r = 0; r < RG; ++r) win[MAX_BACK + r] = nxt[r];
  }
}

// whether the prompt kernel takes the layer; its threads
template <typename ACT, int V>
int prompt_threads(const QkvArgs& a) {
  if (!a.lead || a.split || a.dim % V || a.vdim % V || a.D % V || a.ld % V || ((uintptr_t)a.p & 15) || a.taps > MAX_BACK + 1 ||
      a.rot > 512)
    return 0;
  if (a.per_head && (a.dim / V > 64 || (a.dim / V & (a.dim / V - 1)) || (64 % (a.dim / V)))) return 0;
  const int vecs = max(a.H * a.dim, a.parts > 1 ? a.G * (a.dim + a.vdim) : 0) / V;
  return vecs <= 64 ? 64 : vecs <= 256 ? 256 : vecs <= 512 ? 512 : vecs <= 1024 ? 1024 : 0;
}

template <typename ACT, int V>
int qkv_prompt_go(hipStream_t s, int T, int threads, const QkvArgs& a) {
  const dim3 grid((T + PR_ROWS - 1) / PR_ROWS, a.parts > 1 ? 2 : 1);
  const size_t lds = (size_t)PR_ROWS * (a.rot / 2) * sizeof(float2) + 16;
#define GO(BT)                                                                             \
  if (a.conv) qkv_prompt_kernel<ACT, V, BT, true><<<grid, BT, lds, s>>>(a, T);             \
  else qkv_prompt_kernel<ACT, V, BT, false><<<grid, BT, lds, s>>>(a, T)
  if (threads == 64) { GO(64); }
  else if (threads == 256) { GO(256); }
  else if (threads == 512) { GO(512); }
  else { GO(1024); }
#undef GO
  return CFC_CHECK_LAUNCH();
}

template <typename ACT, int V>
int qkv_go(hipStream_t s, int T, const QkvArgs& a) {
  // few rows with norms per head: runs of heads beside each other, so their loads do not follow one another
  const int most = max(a.H, a.parts > 1 ? a.G : 0);
  const int z = a.per_head && T * a.parts < 512 ? max(1, min(min(most, 8), 512 / (T * a.parts))) : 1;
  int C = (a.H + z - 1) / z * a.dim;
  if (a.parts > 1) C = max(C, (a.G + z - 1) / z * max(a.dim, a.vdim));
  const int vecs = (C + V - 1) / V;
  const size_t lds = (size_t)(vecs + max(a.H, a.G)) * 4;
  if (lds > 49152) return -4;
#define GO(NV, BT) qkv_rows_kernel<ACT, V, NV, BT><<<dim3(T, a.parts, z), BT, lds, s>>>(a)
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
  if (const int th = f32 ? prompt_threads<float, 4>(a) : prompt_threads<uint16_t, 8>(a))
    return f32 ? qkv_prompt_go<float, 4>(stream, T, th, a) : qkv_prompt_go<uint16_t, 8>(stream, T, th, a);
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
