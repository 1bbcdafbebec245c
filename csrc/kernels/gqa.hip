// Grouped-query attention over a paged cache where a token sees two ranges of keys under one softmax:
//   * its window: the last `size` tokens (0: all), or with `chunk` those of its own run of `size` positions, and
//   * far keys: the first `keep` tokens, or one mean key and value per block of `pool` tokens that lies wholly ahead
//     of the window (pooled cache)
// and a learned sink per head joins the denominator.  Scores may be shaped ahead of the softmax: cap tanh(score / cap),
// then a bias per head and distance (a table, its last entry for all distances from there on).  Outputs may pass a gate
// (split_merge.h) and go to rows of any stride.  Keys and values lie row-major, [blocks][G][32][D]; pooled entries
// [blocks][G][E][D], entry b of a sequence in page b / E.  Queries [T][H][D] arrive scaled into the exponent's base 2,
// with a cap so that exp2 of the score is e^(2 score / cap).
// Heads h of G groups: R = H / G consecutive heads share a key / value head.
//
//   * gqa_decode   one token per sequence: a workgroup per (sequence, key head, slice of its keys), its four waves on
//                  32-key tiles of their own.  Keys go straight from memory into the score product's operand, values
//                  through a wave's own LDS tile, read back transposed (ds_read_b64_tr_b16); the score product's
//                  result is the output product's operand as it lies.  No barrier until the waves merge
//   * gqa_prompt   portions of prompts: 32 rows of the flattened (token, head of the group) rows per wave, 64-key tiles
//                  of both ranges double-buffered in LDS
//   * gqa_any      any head size and the 32-bit path: a wave per (token, head) row
//   * slices of a row's keys are merged by slice_merge (split_merge.h)
#include "split_merge.h"

namespace {

typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));     // arrays of these stay in registers
typedef short i16x4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) i16x4_t lds_i16x4_t;

constexpr float LOG2E = 1.4426950408889634f;
constexpr float RESCALE_AT = 8.f;             // log2: how far a row's maximum may run ahead of its reference

struct GqaArgs {
  const int32_t* block_tables;
  const int32_t* cu_q;        // null: one token per sequence
  const int32_t* ctx_lens;    // cached + new tokens
  const int32_t* tile_seq;    // prompt tiles: sequence, first row
  const int32_t* tile_m0;
  int n_tiles;
  int H, G, D, DV, max_blocks, P;      // DV: value columns that leave
  int size, keep, pool, le;            // window; first tokens; tokens per pooled block, log2 of entries per page
  int chunk;                           // size counts from multiples of it
  int capped; float cap2;              // 0: no cap, 1: any score, 2, 3: |score| <= 0.35, 0.25 cap; cap log2(e)
  float k0, k1, k2, k3;                // capped 2 and 3: s (k0 + t (k1 + t (k2 + t k3))), t = s^2
  const float* bias; int nb;           // [H][nb] by distance, times log2(e) (null: none)
  OutGate og;
  const float* sink;          // [H] or null
  float* part_o;              // [rows][P][D], unnormalised
  float* part_ml;             // [rows][P][2]
};

// pooled blocks the token at pos sees
__device__ __forceinline__ int pooled_seen(const GqaArgs& a, int pos) { return max(pos - a.size + 1, 0) / a.pool; }

// the window's first key for the row at pos (size > 0)
__device__ __forceinline__ int window_first(const GqaArgs& a, int pos) { return a.chunk ? pos - pos % a.size : max(0, pos - a.size + 1); }

constexpr float LN2 = 0.69314718055994531f;

// the capped score (base 2) of a score s = 2 log2(e) score / cap, plus b.  Near zero by the series of tanh in x = s ln(2) / 2
// (its next term, 62 / 2835 x^9, is below 4e-6 of x; without the one before it, nearer zero, 17 / 315 x^7 below 1.4e-5)
template <typename ACT>
__device__ __forceinline__ float cap_score(const GqaArgs& a, float s, float b) {
  if constexpr (sizeof(ACT) == 4) return a.cap2 * tanhf(s * (0.5f * LN2)) + b;
  if (a.capped >= 2) {
    const float t = s * s;
    return s * (a.k0 + t * (a.k1 + t * (a.k2 + t * a.k3))) + b;
  }
  return a.cap2 + b - 2.f * a.cap2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s));
}

// Tiles of KT keys for rows at positions pmin .. pmax: first `nat` of the far range (`na` keys), then the window's,
// from key `lo` on
struct KeyTiles { int na, nat, lo, nt; };
template <int KT>
__device__ __forceinline__ KeyTiles key_tiles(const GqaArgs& a, int pmin, int pmax) {
  KeyTiles r;
  r.lo = a.size > 0 ? window_first(a, pmin) / KT * KT : 0;
  r.na = a.size == 0 ? 0 : a.pool ? pooled_seen(a, pmax) : min(a.keep, r.lo);
  r.nat = (r.na + KT - 1) / KT;
  r.nt = r.nat + pmax / KT - r.lo / KT + 1;
  return r;
}

// a window tile's key j for the row at pos
__device__ __forceinline__ bool sees(const GqaArgs& a, int pos, int j) {
  return j <= pos && (a.size == 0 || j >= window_first(a, pos) || j < a.keep);
}

// where key e of a tile range lies: its table entry, then (with the page) its row of the [.][G][.] cache
__device__ __forceinline__ int key_page(const GqaArgs& a, bool pooled, int e) { return pooled ? e >> a.le : e >> 5; }
__device__ __forceinline__ int key_row(const GqaArgs& a, bool pooled, int page, int hk, int e) {
  const int l = pooled ? a.le : 5;
  return ((page * a.G + hk) << l) + (e & ((1 << l) - 1));
}

// running maximum m (log2 domain) and sum l with the head's sink: what to scale the output by
__device__ __forceinline__ float sink_inv(const GqaArgs& a, int head, float m, float l) {
  if (!a.sink) return l > 0.f ? 1.f / l : 0.f;
  const float sk = a.sink[head] * LOG2E, M = fmaxf(m, sk), f = exp2f(m - M);
  return f / (l * f + exp2f(sk - M));
}

__device__ __forceinline__ f32x4_t mfma16(u32x4_t a, u32x4_t b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}
__device__ __forceinline__ f32x16_t mfma32(u32x4_t a, u32x4_t b, f32x16_t c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// 16-byte chunk swizzles of D-column rows: keys are read 16 bytes per row by 16 neighbouring rows, values 64 bytes of
// four neighbouring rows at once; both then touch every bank once
template <int D>
__device__ __forceinline__ int kswz(int row) {
  constexpr int S = D / 32;
  return S % 4 == 0 ? row & 15 : S % 2 == 0 ? (row >> 1) & 7 : (row >> 2) & 3;
}
template <int D>
__device__ __forceinline__ int vswz(int row) {
  constexpr int S = D / 32;
  return S % 4 == 0 ? 4 * (row & 3) : S % 2 == 0 ? 4 * ((row >> 1) & 1) : 0;
}

// four keys of one value column: lane i of 16 addresses columns 4 (i & 3) .. of the run's key i / 4
__device__ __forceinline__ uint2 tr_read(const char* p) {
  const i16x4_t v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (lds_i16x4_t*)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) const char*)p);
  return __builtin_bit_cast(uint2, v);
}

__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// ------------------------------------------------------------------------------------------ decoded tokens
// grid (B * G * ceil(R / 16), P)
template <int D, bool SHAPED>
__global__ void __launch_bounds__(256, D <= 128 ? 2 : 1) gqa_decode_kernel(const uint16_t* __restrict__ q,
                                                                          const uint16_t* __restrict__ kc,
                                                                          const uint16_t* __restrict__ vc,
                                                                          const uint16_t* __restrict__ pk,
                                                                          const uint16_t* __restrict__ pv, GqaArgs a,
                                                                          uint16_t* __restrict__ out) {
  constexpr int KS = D / 32, NV = D / 16, CH = D / 8, DT = D / 16;
  __shared__ __attribute__((aligned(16))) char smem[4 * 64 * D];     // a wave's 32 x D values; then its 16 x D outputs
  __shared__ float ml[4][16][2];
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), col = lane & 15, kq = lane >> 4;
  const int R = a.H / a.G, RG = (R + 15) / 16;
  int item = blockIdx.x;
  const int rg = item % RG;
  item /= RG;
  const int hk = item % a.G, s = item / a.G, pos = a.ctx_lens[s] - 1;
  const int32_t* bt = a.block_tables + (size_t)s * a.max_blocks;
  const KeyTiles kt = key_tiles<32>(a, pos, pos);
  const int t0 = (int)((int64_t)kt.nt * blockIdx.y / a.P), t1 = (int)((int64_t)kt.nt * (blockIdx.y + 1) / a.P);
  const int r0 = 16 * rg, nr = min(16, R - r0);
  const size_t qrow = (size_t)s * a.H + hk * R + r0;

  u32x4_t qf[KS];
#pragma unroll
  for (int k = 0; k < KS; ++k)
    qf[k] = *reinterpret_cast<const u32x4_t*>(q + (qrow + min(col, nr - 1)) * D + 32 * k + 8 * kq);

  char* vbuf = smem + w * 64 * D;
  const float* bias = SHAPED && a.bias ? a.bias + (size_t)(hk * R + r0 + min(col, nr - 1)) * a.nb : nullptr;
  const float far_bias = bias ? bias[a.nb - 1] : 0.f;
  u32x4_t kf[2][KS], vf[NV];
  // row of this lane's key (lane & 31) in a tile; tiles past the slice: its last
  auto rows_of = [&](int t) {
    t = min(t, t1 - 1);
    const bool far = t < kt.nat, pooled = far && a.pool;
    const int e = far ? min(32 * t + (lane & 31), kt.na - 1) : kt.lo + 32 * (t - kt.nat) + (lane & 31);
    return key_row(a, pooled, bt[key_page(a, pooled, e)], hk, e);
  };
  auto load = [&](int t, int row) {
    const bool pooled = a.pool && min(t, t1 - 1) < kt.nat;
    const uint16_t *kb = pooled ? pk : kc, *vb = pooled ? pv : vc;
#pragma unroll
    for (int g = 0; g < 2; ++g) {
      const uint16_t* p = kb + (size_t)__shfl(row, 16 * g + col, 64) * D + 8 * kq;
#pragma unroll
      for (int k = 0; k < KS; ++k) kf[g][k] = *reinterpret_cast<const u32x4_t*>(p + 32 * k);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = lane + 64 * i;
      vf[i] = *reinterpret_cast<const u32x4_t*>(vb + (size_t)__shfl(row, e / CH, 64) * D + 8 * (e % CH));
    }
  };

  f32x4_t o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) o[d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  int t = t0 + w;
  if (t < t1) {
    int row = rows_of(t);
    load(t, row);
    row = rows_of(t + 4);
    for (; t < t1; t += 4) {
      wave_lds_fence();                      // the last tile's values have been read
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int e = lane + 64 * i, key = e / CH, c = e % CH;
        *reinterpret_cast<u32x4_t*>(vbuf + key * (2 * D) + ((c ^ vswz<D>(key)) << 4)) = vf[i];
      }
      f32x4_t sc[2];
#pragma unroll
      for (int g = 0; g < 2; ++g) {
        sc[g] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KS; ++k) sc[g] = mfma16(kf[g][k], qf[k], sc[g]);
      }
      load(t + 4, row);                      // past the slice: re-read, not used
      row = rows_of(t + 8);
      const bool far = t < kt.nat;
      if constexpr (SHAPED) {
        const int k0 = far ? 32 * t : kt.lo + 32 * (t - kt.nat);
        float bt8[2][4];
        if (bias && pos - k0 - 31 < a.nb - 1) {
#pragma unroll
          for (int g = 0; g < 2; ++g)
#pragma unroll
            for (int i = 0; i < 4; ++i) bt8[g][i] = bias[min(max(pos - k0 - (16 * g + 4 * kq + i), 0), a.nb - 1)];
        } else {
#pragma unroll
          for (int g = 0; g < 2; ++g)
#pragma unroll
            for (int i = 0; i < 4; ++i) bt8[g][i] = far_bias;
        }
#pragma unroll
        for (int g = 0; g < 2; ++g)
#pragma unroll
          for (int i = 0; i < 4; ++i) sc[g][i] = a.capped ? cap_score<uint16_t>(a, sc[g][i], bt8[g][i]) : sc[g][i] + bt8[g][i];
      }
      float mx = -INFINITY;
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = 16 * g + 4 * kq + i;
          const bool see = far ? 32 * t + key < kt.na : sees(a, pos, kt.lo + 32 * (t - kt.nat) + key);
          if (!see) sc[g][i] = -INFINITY;
          mx = fmaxf(mx, sc[g][i]);
        }
      mx = xor32_max(xor16_max(mx));
      const float mn = fmaxf(m, mx), ref = mn == -INFINITY ? 0.f : mn, alpha = __builtin_amdgcn_exp2f(m - ref);
      m = mn;
      l *= alpha;
      if (!__all(alpha == 1.f)) {
#pragma unroll
        for (int d = 0; d < DT; ++d) o[d] *= alpha;
      }
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          sc[g][i] = __builtin_amdgcn_exp2f(sc[g][i] - ref);
          l += sc[g][i];
        }
      // operand slots 8 kq + j: keys 4 kq + j of the first 16, then of the second
      u32x4_t pf;
      pf[0] = cvt_pk_bf16_f32(sc[0][0], sc[0][1]);
      pf[1] = cvt_pk_bf16_f32(sc[0][2], sc[0][3]);
      pf[2] = cvt_pk_bf16_f32(sc[1][0], sc[1][1]);
      pf[3] = cvt_pk_bf16_f32(sc[1][2], sc[1][3]);
      wave_lds_fence();
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        u32x4_t vt;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const int key = 16 * u + 4 * kq + (col >> 2), c = 2 * d + ((col & 3) >> 1);
          const uint2 v = tr_read(vbuf + key * (2 * D) + ((c ^ vswz<D>(key)) << 4) + 8 * (col & 1));
          vt[2 * u] = v.x;
          vt[2 * u + 1] = v.y;
        }
        o[d] = mfma16(vt, pf, o[d]);
      }
    }
  }
  l = xor32_sum(xor16_sum(l));
  wave_lds_fence();
  float* ob = reinterpret_cast<float*>(vbuf);            // [16][D]
#pragma unroll
  for (int d = 0; d < DT; ++d) *reinterpret_cast<f32x4_t*>(ob + col * D + 16 * d + 4 * kq) = o[d];
  if (lane < 16) {
    ml[w][lane][0] = m;
    ml[w][lane][1] = l;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < nr * (D / 4); e += 256) {
    const int r = e / (D / 4), c = 4 * (e % (D / 4));
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) M = fmaxf(M, ml[i][r][0]);
    const float ref = M == -INFINITY ? 0.f : M;
    f32x4_t y{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float f = exp2f(ml[i][r][0] - ref);
      L += f * ml[i][r][1];
      y += f * *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(smem + i * 64 * D) + r * D + c);
    }
    const size_t grow = qrow + r;
    if (a.P > 1) {
      *reinterpret_cast<f32x4_t*>(a.part_o + (grow * a.P + blockIdx.y) * D + c) = y;
      if (c == 0) {
        a.part_ml[(grow * a.P + blockIdx.y) * 2] = M;
        a.part_ml[(grow * a.P + blockIdx.y) * 2 + 1] = L;
      }
      continue;
    }
    const float inv = sink_inv(a, hk * R + r0 + r, M, L);
    const int oc = (hk * R + r0 + r) * a.DV + c;
    uint16_t* dst = out + s * a.og.ld + oc;
    if (a.og.vec) {
      if (c < a.DV) {
        const f32x4_t f = inv * out_gate4<uint16_t>(a.og, s, oc);
        *reinterpret_cast<uint2*>(dst) = make_uint2(cvt_pk_bf16_f32(y[0] * f[0], y[1] * f[1]), cvt_pk_bf16_f32(y[2] * f[2], y[3] * f[3]));
      }
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (c + i < a.DV) dst[i] = f2bf(y[i] * inv * out_gate<uint16_t>(a.og, s, oc + i));
    }
  }
}

// ------------------------------------------------------------------------------------------ prompt portions
// biases of one head in LDS, and whether a group's leave two workgroups a CU
constexpr int BIAS_PAD = 3;
__host__ __device__ __forceinline__ int bias_stride(int nb) { return (nb + 2 * BIAS_PAD) | 1; }
__host__ __device__ __forceinline__ bool bias_in_lds(int R, int nb) { return (int64_t)R * bias_stride(nb) <= 4096; }

// 1-D grid of n_tiles * G, tile major: in the tiles' order (those with the most keys first, so that long ones do not end
// the grid alone), and an XCD takes one key head of eight, whose keys its L2 then holds.
// A tile is 32 NW rows (row r of a portion and key head: token r / R, head r % R of the group).
template <int D, int NW, bool SHAPED>
__global__ void __launch_bounds__(64 * NW, D <= 128 ? 2 : 1) gqa_prompt_kernel(const uint16_t* __restrict__ q,
                                                                              const uint16_t* __restrict__ kc,
                                                                              const uint16_t* __restrict__ vc,
                                                                              const uint16_t* __restrict__ pk,
                                                                              const uint16_t* __restrict__ pv, GqaArgs a,
                                                                              uint16_t* __restrict__ out) {
  constexpr int NT = 64 * NW, CH = D / 8, NL = (64 * CH + NT - 1) / NT, KS = D / 16, DT = D / 32;
  constexpr bool EVEN = 64 * CH % NT == 0;
  constexpr int TILE = 64 * D * 2;
  extern __shared__ __attribute__((aligned(16))) char smem[];          // [2][K | V], then the group's biases (bias_stride)
  const int tile = blockIdx.x / a.G, hk = blockIdx.x - tile * a.G;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l32 = lane & 31, hi = lane >> 5;
  const int R = a.H / a.G, s = a.tile_seq[tile], m0 = a.tile_m0[tile];
  const int q0 = a.cu_q[s], n = a.cu_q[s + 1] - q0, rows = n * R, base = a.ctx_lens[s] - n;
  const int32_t* bt = a.block_tables + (size_t)s * a.max_blocks;
  const int pmax = base + (min(m0 + 32 * NW, rows) - 1) / R, nb = pmax / CFC_KV_BS + 1;
  const KeyTiles kt = key_tiles<64>(a, base + m0 / R, pmax);
  const int my = m0 + 32 * w + l32, mr = min(my, rows - 1), my_tok = mr / R, my_pos = base + my_tok;
  const int head = hk * R + (mr - my_tok * R);
  const int wp0 = base + min(m0 + 32 * w, rows - 1) / R, wp1 = base + min(m0 + 32 * w + 31, rows - 1) / R;

  u32x4_t qf[KS];
#pragma unroll
  for (int k = 0; k < KS; ++k)
    qf[k] = *reinterpret_cast<const u32x4_t*>(q + ((size_t)(q0 + my_tok) * a.H + head) * D + 16 * k + 8 * hi);

  u32x4_t ks[NL], vs[NL];
  int id[NL];
  auto key_of = [&](int t, int i) {          // index of piece i's key in its range
    const int e = min((tid + NT * i) / CH, 63);
    return t < kt.nat ? min(64 * t + e, kt.na - 1) : kt.lo + 64 * (t - kt.nat) + e;
  };
  auto ids = [&](int t) {
    t = min(t, kt.nt - 1);
    const bool pooled = t < kt.nat && a.pool;
#pragma unroll
    for (int i = 0; i < NL; ++i) id[i] = bt[min(key_page(a, pooled, key_of(t, i)), nb - 1)];
  };
  auto gload = [&](int t) {                  // unconditional: past the last tile it is read again, not used
    t = min(t, kt.nt - 1);
    const bool pooled = t < kt.nat && a.pool;
    const uint16_t *kb = pooled ? pk : kc, *vb = pooled ? pv : vc;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const size_t off = (size_t)key_row(a, pooled, id[i], hk, key_of(t, i)) * D + 8 * ((tid + NT * i) % CH);
      ks[i] = *reinterpret_cast<const u32x4_t*>(kb + off);
      vs[i] = *reinterpret_cast<const u32x4_t*>(vb + off);
    }
  };
  auto lwrite = [&](int buf) {
    char* kb = smem + buf * 2 * TILE;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = tid + NT * i, key = e / CH, c = e % CH;
      if (EVEN || e < 64 * CH) {
        *reinterpret_cast<u32x4_t*>(kb + key * (2 * D) + ((c ^ kswz<D>(key)) << 4)) = ks[i];
        *reinterpret_cast<u32x4_t*>(kb + TILE + key * (2 * D) + ((c ^ vswz<D>(key)) << 4)) = vs[i];
      }
    }
  };

  f32x16_t o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[d][r] = 0.f;
  float m = -INFINITY, lp[4] = {0.f, 0.f, 0.f, 0.f};

  ids(0);
  gload(0);
  ids(1);
  lwrite(0);
  // biases by falling distance, the ends repeated BIAS_PAD times: four neighbouring keys' are four neighbours here
  const int bs = SHAPED && a.bias ? bias_stride(a.nb) : 0;
  const float* lb = nullptr;
  float far_bias = 0.f;
  if constexpr (SHAPED) {
    if (a.bias) {
      far_bias = a.bias[(size_t)head * a.nb + a.nb - 1];
      float* tab = reinterpret_cast<float*>(smem + 4 * TILE);
      if (bias_in_lds(R, a.nb)) {
        for (int e = tid; e < R * bs; e += NT) {
          const int r = e / bs, i = e - r * bs;
          tab[e] = a.bias[(size_t)(hk * R + r) * a.nb + min(max(a.nb - 1 - (i - BIAS_PAD), 0), a.nb - 1)];
        }
        lb = tab + (head - hk * R) * bs + BIAS_PAD;
      }
    }
  }
  __syncthreads();
  for (int t = 0; t < kt.nt; ++t) {
    gload(t + 1);
    ids(t + 2);
    const bool far = t < kt.nat;
    const int k0 = far ? 64 * t : kt.lo + 64 * (t - kt.nat);
    // what this wave's rows see of the tile: nothing, some, all
    const int seen0 = a.pool ? pooled_seen(a, wp0) : kt.na, seen1 = a.pool ? pooled_seen(a, wp1) : kt.na;
    const bool none = far ? k0 >= seen1 : k0 > wp1 || (a.size > 0 && k0 + 63 < window_first(a, wp0) && k0 >= a.keep);
    const bool all = far ? k0 + 64 <= seen0 : k0 + 63 <= wp0 && (a.size == 0 || k0 >= window_first(a, wp1));
    if (!none) {
      const char* kb = smem + (t & 1) * 2 * TILE;
      const char* vb = kb + TILE;
      const float ref0 = m == -INFINITY ? 0.f : m;
      f32x16_t sc[2];
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const int key = 32 * h + l32;
#pragma unroll
        for (int r = 0; r < 16; ++r) sc[h][r] = SHAPED ? 0.f : -ref0;
        constexpr int KB = KS <= 8 ? KS : KS / 2;         // fragments in batches: one LDS round trip each
#pragma unroll
        for (int b0 = 0; b0 < KS; b0 += KB) {
          u32x4_t kf[KB];
#pragma unroll
          for (int k = 0; k < KB; ++k)
            kf[k] = *reinterpret_cast<const u32x4_t*>(kb + key * (2 * D) + (((2 * (b0 + k) + hi) ^ kswz<D>(key)) << 4));
#pragma unroll
          for (int k = 0; k < KB; ++k) sc[h] = mfma32(kf[k], qf[b0 + k], sc[h]);
          __builtin_amdgcn_sched_group_barrier(0x100, KB, 0);
          __builtin_amdgcn_sched_group_barrier(0x008, KB, 0);
        }
      }
      if constexpr (SHAPED) {
        const float far0 = far_bias - ref0;
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          float bv[16];                        // the biases, less the running maximum
#pragma unroll
          for (int r = 0; r < 16; ++r) bv[r] = far0;
          if (a.bias && wp0 - (k0 + 32 * h + 31) < a.nb - 1) {
#pragma unroll
            for (int g = 0; g < 4; ++g) {
              const int n = my_pos - (k0 + 32 * h + 8 * g + 4 * hi);          // the first key's distance
              if (lb) {
                const float* b = lb + min(max(a.nb - 1 - n, -BIAS_PAD), a.nb - 1);
#pragma unroll
                for (int i = 0; i < 4; ++i) bv[4 * g + i] = b[i] - ref0;
              } else {
#pragma unroll
                for (int i = 0; i < 4; ++i) bv[4 * g + i] = a.bias[(size_t)head * a.nb + min(max(n - i, 0), a.nb - 1)] - ref0;
              }
            }
          }
          if (a.capped == 3) {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
              const float t = sc[h][r] * sc[h][r];
              sc[h][r] = sc[h][r] * (a.k0 + t * (a.k1 + t * a.k2)) + bv[r];
            }
          } else if (a.capped) {
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[h][r] = cap_score<uint16_t>(a, sc[h][r], bv[r]);
          } else {
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[h][r] += bv[r];
          }
        }
      }
      if (!all) {
        const int mine = a.pool ? pooled_seen(a, my_pos) : kt.na;
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int j = k0 + 32 * h + 8 * (r >> 2) + 4 * hi + (r & 3);
            if (!(far ? j < mine : sees(a, my_pos, j))) sc[h][r] = -INFINITY;
          }
      }
      float ta = fmaxf(fmaxf(sc[0][0], sc[0][1]), sc[0][2]), tb = fmaxf(fmaxf(sc[1][0], sc[1][1]), sc[1][2]);
#pragma unroll
      for (int r = 3; r < 15; r += 2) {
        ta = fmaxf(fmaxf(ta, sc[0][r]), sc[0][r + 1]);
        tb = fmaxf(fmaxf(tb, sc[1][r]), sc[1][r + 1]);
      }
      const float tmax = xor32_max(fmaxf(fmaxf(ta, sc[0][15]), fmaxf(tb, sc[1][15])));
      if (!__all(m != -INFINITY && tmax <= RESCALE_AT)) {
        const float mn = fmaxf(m, ref0 + tmax), ref = mn == -INFINITY ? 0.f : mn;
        const float alpha = __builtin_amdgcn_exp2f(m - ref);
#pragma unroll
        for (int u = 0; u < 4; ++u) lp[u] *= alpha;
#pragma unroll
        for (int d = 0; d < DT; ++d) o[d] *= alpha;
        m = mn;
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int r = 0; r < 16; ++r) sc[h][r] -= ref - ref0;
      }
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          sc[h][r] = __builtin_amdgcn_exp2f(sc[h][r]);
          lp[r & 3] += sc[h][r];
        }
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int ss = 0; ss < 2; ++ss) {
          // operand slots 8 hi + j: keys 16 ss + 4 hi + j, then 8 further
          u32x4_t pf;
#pragma unroll
          for (int u = 0; u < 4; ++u) pf[u] = cvt_pk_bf16_f32(sc[h][8 * ss + 2 * u], sc[h][8 * ss + 2 * u + 1]);
          u32x4_t vt[DT];
#pragma unroll
          for (int d = 0; d < DT; ++d)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
              const int key = 32 * h + 16 * ss + 8 * u + 4 * hi + ((lane & 15) >> 2);
              const int c = 4 * d + 2 * ((lane >> 4) & 1) + ((lane & 3) >> 1);
              const uint2 v = tr_read(vb + key * (2 * D) + ((c ^ vswz<D>(key)) << 4) + 8 * (lane & 1));
              vt[d][2 * u] = v.x;
              vt[d][2 * u + 1] = v.y;
            }
#pragma unroll
          for (int d = 0; d < DT; ++d) o[d] = mfma32(vt[d], pf, o[d]);
        }
    }
    if (t + 1 < kt.nt) lwrite((t + 1) & 1);
    __syncthreads();
  }
  const float l = xor32_sum((lp[0] + lp[1]) + (lp[2] + lp[3]));
  if (my >= rows) return;
  const float inv = sink_inv(a, head, m, l);
  const int token = q0 + my_tok, oc = head * a.DV;
  uint16_t* dst = out + token * a.og.ld + oc;
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int c = 32 * d + 8 * g + 4 * hi;
      if (a.og.vec) {
        if (c < a.DV) {
          const f32x4_t f = inv * out_gate4<uint16_t>(a.og, token, oc + c);
          *reinterpret_cast<uint2*>(dst + c) = make_uint2(cvt_pk_bf16_f32(o[d][4 * g] * f[0], o[d][4 * g + 1] * f[1]),
                                                          cvt_pk_bf16_f32(o[d][4 * g + 2] * f[2], o[d][4 * g + 3] * f[3]));
        }
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (c + i < a.DV) dst[c + i] = f2bf(o[d][4 * g + i] * inv * out_gate<uint16_t>(a.og, token, oc + c + i));
      }
    }
}

// ------------------------------------------------------------------------------------------ any size, 32 bits
__device__ __forceinline__ float ldf(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// grid (tiles of 4 rows, P); rows are the flattened (token, head) rows of a sequence.  A lane scores one key of 64, then
// owns every 64th value column
template <typename ACT, int NC>
__global__ void __launch_bounds__(256) gqa_any_kernel(const ACT* __restrict__ q, const ACT* __restrict__ kc,
                                                     const ACT* __restrict__ vc, const ACT* __restrict__ pk,
                                                     const ACT* __restrict__ pv, GqaArgs a, ACT* __restrict__ out) {
  extern __shared__ float sq[];                 // [4][D] queries, [4][64] weights, [4][64] rows
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, D = a.D;
  const int per = (a.H + 3) / 4, s = a.tile_seq ? a.tile_seq[blockIdx.x] : blockIdx.x / per;
  const int m0 = a.tile_seq ? a.tile_m0[blockIdx.x] : blockIdx.x % per * 4;
  const int q0 = a.cu_q ? a.cu_q[s] : s, n = a.cu_q ? a.cu_q[s + 1] - q0 : 1, rows = n * a.H;
  const int mrow = min(m0 + w, rows - 1), head = mrow % a.H, hk = head / (a.H / a.G);
  const int pos = a.ctx_lens[s] - n + mrow / a.H;
  const size_t grow = (size_t)q0 * a.H + mrow;
  const int32_t* bt = a.block_tables + (size_t)s * a.max_blocks;
  float* myq = sq + w * D;
  float* pw = sq + 4 * D + 64 * w;
  int* rw = reinterpret_cast<int*>(sq + 4 * D + 256) + 64 * w;
  for (int c = lane; c < D; c += 64) myq[c] = ldf(q + grow * D + c);
  const KeyTiles kt = key_tiles<64>(a, pos, pos);
  const int t0 = (int)((int64_t)kt.nt * blockIdx.y / a.P), t1 = (int)((int64_t)kt.nt * (blockIdx.y + 1) / a.P);
  float o[NC], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int j = 0; j < NC; ++j) o[j] = 0.f;
  for (int t = t0; t < t1; ++t) {               // waves share nothing
    const bool far = t < kt.nat, pooled = far && a.pool;
    const int e = far ? 64 * t + lane : kt.lo + 64 * (t - kt.nat) + lane;
    const bool see = far ? e < kt.na : sees(a, pos, e);
    int row = 0;
    float sc = -INFINITY;
    if (see) {
      row = key_row(a, pooled, bt[key_page(a, pooled, e)], hk, e);
      const ACT* c = (pooled ? pk : kc) + (size_t)row * D;
      float s4[4] = {0.f, 0.f, 0.f, 0.f};
      for (int r = 0; r < D; r += 4)
#pragma unroll
        for (int u = 0; u < 4; ++u) s4[u] += myq[r + u] * ldf(c + r + u);
      sc = (s4[0] + s4[1]) + (s4[2] + s4[3]);
      if (a.capped) sc = cap_score<float>(a, sc, 0.f);
      if (a.bias) sc += a.bias[(size_t)head * a.nb + min(pos - e, a.nb - 1)];
    }
    const float mn = fmaxf(m, wave_max(sc)), ref = mn == -INFINITY ? 0.f : mn;
    const float alpha = exp2f(m - ref), p = exp2f(sc - ref);
    m = mn;
    l = l * alpha + wave_sum(p);
    wave_lds_fence();
    pw[lane] = p;
    rw[lane] = row;
    wave_lds_fence();
#pragma unroll
    for (int j = 0; j < NC; ++j) o[j] *= alpha;
    const ACT* vb = pooled ? pv : vc;
    for (int k = 0; k < 64; ++k) {
      const float pk_ = pw[k];
      if (pk_ == 0.f) continue;
      const ACT* c = vb + (size_t)rw[k] * D;
#pragma unroll
      for (int j = 0; j < NC; ++j)
        if (lane + 64 * j < D) o[j] += pk_ * ldf(c + lane + 64 * j);
    }
  }
  if (m0 + w >= rows) return;
  const float inv = sink_inv(a, head, m, l);
#pragma unroll
  for (int j = 0; j < NC; ++j) {
    const int c = lane + 64 * j;
    if (a.P > 1) {
      if (c < D) a.part_o[(grow * a.P + blockIdx.y) * D + c] = o[j];
    } else if (c < a.DV) {
      const int token = q0 + mrow / a.H, oc = head * a.DV + c;
      stf(out + token * a.og.ld + oc, o[j] * inv * out_gate<ACT>(a.og, token, oc));
    }
  }
  if (a.P > 1 && lane == 0) {
    a.part_ml[(grow * a.P + blockIdx.y) * 2] = m;
    a.part_ml[(grow * a.P + blockIdx.y) * 2 + 1] = l;
  }
}

template <int D, int NW, bool SHAPED>
int prompt_go(int grid, hipStream_t s, const void* q, const void* kc, const void* vc, const void* pk, const void* pv,
              const GqaArgs& a, void* out) {
  constexpr int tiles = 2 * 2 * 64 * D * 2, most = tiles + (SHAPED ? 16384 : 0);
  static bool raised = false;
  if (most > 65536 && !raised) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&gqa_prompt_kernel<D, NW, SHAPED>), hipFuncAttributeMaxDynamicSharedMemorySize, most);
    raised = true;
  }
  const int R = a.H / a.G, lds = tiles + (SHAPED && a.bias && bias_in_lds(R, a.nb) ? 4 * R * bias_stride(a.nb) : 0);
  gqa_prompt_kernel<D, NW, SHAPED><<<grid, 64 * NW, lds, s>>>((const uint16_t*)q, (const uint16_t*)kc, (const uint16_t*)vc,
                                                     (const uint16_t*)pk, (const uint16_t*)pv, a, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

constexpr int prompt_waves(int D) { return D == 64 || D == 128 ? 8 : 4; }

}  // namespace

// rows of one key head's prompt tile for cached heads of D columns (0: the general kernel's, 4 rows over all heads)
CFC_API int cfc_gqa_prompt_rows(int D) {
  return D == 32 || D == 64 || D == 96 || D == 128 || D == 160 || D == 192 || D == 256 ? 32 * prompt_waves(D) : 0;
}

// q [T][H][D] scaled by log2(e); caches [blocks][G][32][D], pooled [blocks][G][1 << le][D]; out [T][H][DV].
// kind 0: general (tiles of 4 rows over all heads; tile_seq null: one token per sequence), 1: decode, 2: prompt portions.
// chunk: the window is the row's own run of size positions.  capped 1, 2 or 3 (|score| <= 0.35, 0.25 cap): q scaled by 2 log2(e) / cap
// instead, cap2 = cap log2(e).  bias [H][nb] times log2(e), by distance.  gate: columns [T][H DV] of a product (gate_split 0:
// activations, else fp32 slabs; null: none) that, as oscale sigmoid(gate), multiply the output, whose rows have stride ldo
CFC_API int cfc_gqa_attention(int kind, int f32, const void* q, const void* kc, const void* vc, const void* pk, const void* pv,
                              const int32_t* block_tables, const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* tile_seq,
                              const int32_t* tile_m0, int n_tiles, int B, int H, int G, int D, int DV, int max_blocks, int size,
                              int keep, int pool, int le, int chunk, int capped, float cap2, const float* bias, int nb,
                              const float* sink, const void* gate, int gate_split, int64_t gate_ld, int64_t gate_plane, float oscale,
                              int P, int total_rows, float* part_o, float* part_ml, void* out, int64_t ldo, hipStream_t stream) {
  if (B <= 0 || (kind != 1 && n_tiles <= 0)) return 0;
  if (H < 1 || G < 1 || H % G || D < 32 || D % 32 || D > 1024 || DV < 1 || DV > D || max_blocks < 1 || P < 1 || P > MERGE_MAXP) return -1;
  if (size < 0 || keep < 0 || pool < 0 || (pool && (keep || !pk || !pv || le < 0 || le > 5 || (pool << le) < CFC_KV_BS || size < 1))) return -2;
  if (chunk && (size < 1 || pool)) return -2;
  if (capped < 0 || capped > 3 || (capped && !(cap2 > 0.f)) || (bias && nb < 1) || (bias && pool)) return -7;
  if (ldo < (int64_t)H * DV || (gate && (gate_split < 0 || gate_ld < (int64_t)H * DV))) return -8;
  if (P > 1 && (!part_o || !part_ml)) return -3;
  if (kind == 2 && (P != 1 || !cu_q || !tile_seq || !tile_m0)) return -4;
  if (kind != 0 && (f32 || cfc_gqa_prompt_rows(D) == 0)) return -5;
  OutGate og;
  og.p = gate; og.split = gate_split; og.pld = gate_ld; og.plane = gate_plane; og.scale = oscale; og.ld = ldo;
  const int esz = f32 ? 4 : 2, gsz = gate_split ? 4 : esz;
  og.vec = DV % 4 == 0 && ldo % 4 == 0 && ((uintptr_t)out & (4 * esz - 1)) == 0 &&
           (!gate || (gate_ld % 4 == 0 && gate_plane % 4 == 0 && ((uintptr_t)gate & (4 * gsz - 1)) == 0));
  const float h = 0.5f * LN2, h2 = h * h, h3 = h2 * h;
  const GqaArgs a{block_tables, cu_q, ctx_lens, tile_seq, tile_m0, n_tiles, H, G, D, DV, max_blocks, P, size, keep, pool, le,
                  chunk, capped, cap2, h * cap2, -h3 / 3.f * cap2, 2.f * h3 * h2 / 15.f * cap2, -17.f * h3 * h2 * h2 / 315.f * cap2,
                  bias, nb, og, sink, part_o, part_ml};
  const bool shaped = capped || bias;
  int rc = -6;
  if (kind == 2) {
#define GP(DD)                                                                                                       \
  case DD:                                                                                                           \
    rc = shaped ? prompt_go<DD, prompt_waves(DD), true>(n_tiles * G, stream, q, kc, vc, pk, pv, a, out)              \
                : prompt_go<DD, prompt_waves(DD), false>(n_tiles * G, stream, q, kc, vc, pk, pv, a, out);            \
    break
    switch (D) { GP(32); GP(64); GP(96); GP(128); GP(160); GP(192); GP(256); }
#undef GP
    return rc;
  }
  if (kind == 1) {
    const dim3 grid(B * G * ((H / G + 15) / 16), P);
#define GD(DD)                                                                                                            \
  case DD:                                                                                                                \
    if (shaped)                                                                                                           \
      gqa_decode_kernel<DD, true><<<grid, 256, 0, stream>>>((const uint16_t*)q, (const uint16_t*)kc, (const uint16_t*)vc, \
                                                            (const uint16_t*)pk, (const uint16_t*)pv, a, (uint16_t*)out); \
    else                                                                                                                  \
      gqa_decode_kernel<DD, false><<<grid, 256, 0, stream>>>((const uint16_t*)q, (const uint16_t*)kc, (const uint16_t*)vc, \
                                                             (const uint16_t*)pk, (const uint16_t*)pv, a, (uint16_t*)out); \
    rc = CFC_CHECK_LAUNCH();                                                                                              \
    break
    switch (D) { GD(32); GD(64); GD(96); GD(128); GD(160); GD(192); GD(256); }
#undef GD
  } else {
    const size_t lds = (size_t)(4 * D + 512) * 4;
#define GA(T, N)                                                                                                     \
  gqa_any_kernel<T, N><<<dim3(n_tiles, P), 256, lds, stream>>>((const T*)q, (const T*)kc, (const T*)vc, (const T*)pk, \
                                                               (const T*)pv, a, (T*)out)
    if (D <= 256) { if (f32) GA(float, 4); else GA(uint16_t, 4); }
    else if (f32) GA(float, 16);
    else GA(uint16_t, 16);
#undef GA
    rc = CFC_CHECK_LAUNCH();
  }
  if (rc || P == 1) return rc;
  if (f32) slice_merge_kernel<float><<<total_rows, 128, 0, stream>>>(part_o, part_ml, P, D, DV, sink, H, og, (float*)out);
  else slice_merge_kernel<uint16_t><<<total_rows, 128, 0, stream>>>(part_o, part_ml, P, D, DV, sink, H, og, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}
