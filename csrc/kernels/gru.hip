// Minimal gated recurrence: gate and candidate read the current token only, so the state is a linear recurrence
//   S_t = (1 - z_t) S_(t-1) + z_t c_t,   z = sigmoid(pre_z + bz),   c = u + 1/2 (u >= 0) or sigmoid(u),  u = pre_x + bx
// element by element, and the layer's output S_t silu(pre_g).  States are fp32, one row per sequence slot; a sequence's
// first token starts from zero whatever the slot holds.
//   * gru_step    one token per sequence, straight from a joint product's slabs
//   * gru_chunk   prompt portions, chunks of 64 tokens in parallel: each chunk's decay (the product of 1 - z) and what
//                 it adds to a state of zero
//   * carry       per sequence through its chunks: the state ahead of each, and the one the portion leaves (recur.h)
//   * gru_apply   the chunks again from their states: outputs
#include "recur.h"

namespace {

struct GruCols { const void* p; int split; int64_t ld, plane; };      // split 0: activations, else fp32 slabs

template <typename ACT, int V>
__device__ __forceinline__ Vec<V> gru_ld(const GruCols& a, int64_t t, int c) {
  const int64_t o = t * a.ld + c;
  if (a.split == 0) return ldv<V>(reinterpret_cast<const ACT*>(a.p) + o);
  Vec<V> y = zerov<V>();
  add_slabs<V>(y, reinterpret_cast<const float*>(a.p), a.split, a.plane, (size_t)o);
  return y;
}

// decay 1 - z and contribution z c of one token.  With t = exp(pre_z): 1 - z = 1 / (1 + t) and z = t / (1 + t), neither
// the other's difference from 1, so that small ones keep their digits; sigmoid(min(u, 0)) is 1/2 where u >= 0
template <typename ACT>
__device__ __forceinline__ void gru_gates(float pz, float u, float& a, float& b) {
  const float t = exp_of<ACT>(fminf(pz, 60.f)), v = exp_of<ACT>(fminf(u, 0.f));
  a = over1<ACT>(t);
  b = t * a * (fmaxf(u, 0.f) + v * over1<ACT>(v));
}

template <typename ACT>
__device__ __forceinline__ float silu(float g) { return g * over1<ACT>(exp_of<ACT>(fminf(-g, 60.f))); }

// V activations as loaded
template <typename ACT, int V> struct Raw;
template <> struct Raw<uint16_t, 4> {
  uint2 u;
  __device__ __forceinline__ void get(const uint16_t* p) { u = *reinterpret_cast<const uint2*>(p); }
  __device__ __forceinline__ float at(int e) const {
    const uint32_t w = e < 2 ? u.x : u.y;
    return __uint_as_float(e & 1 ? w & 0xffff0000u : w << 16);
  }
};
template <> struct Raw<float, 4> {
  float4 f;
  __device__ __forceinline__ void get(const float* p) { f = *reinterpret_cast<const float4*>(p); }
  __device__ __forceinline__ float at(int e) const { return e == 0 ? f.x : e == 1 ? f.y : e == 2 ? f.z : f.w; }
};
template <typename ACT> struct Raw<ACT, 1> {
  ACT u;
  __device__ __forceinline__ void get(const ACT* p) { u = *p; }
  __device__ __forceinline__ float at(int) const { return ld1(&u); }
};

template <typename ACT, int V>
__global__ void __launch_bounds__(64) gru_step_kernel(GruCols z, GruCols u, GruCols g, const float* __restrict__ bz,
                                                     const float* __restrict__ bx, const int32_t* __restrict__ slots,
                                                     const int32_t* __restrict__ ctx_lens, int W, float* __restrict__ state,
                                                     ACT* __restrict__ out, int64_t ldo, float oscale) {
  const int b = blockIdx.x, c = (blockIdx.y * 64 + threadIdx.x) * V;
  if (c >= W) return;
  float* sp = state + (size_t)slots[b] * W + c;
  Vec<V> S = ctx_lens[b] > 1 ? ldv<V>(sp) : zerov<V>();
  const Vec<V> zv = gru_ld<ACT, V>(z, b, c), uv = gru_ld<ACT, V>(u, b, c), gv = gru_ld<ACT, V>(g, b, c);
  const Vec<V> vz = ldv<V>(bz + c), vx = ldv<V>(bx + c);
  Vec<V> o;
#pragma unroll
  for (int e = 0; e < V; ++e) {
    float a, k;
    gru_gates<ACT>(zv.v[e] + vz.v[e], uv.v[e] + vx.v[e], a, k);
    S.v[e] = a * S.v[e] + k;
    o.v[e] = S.v[e] * silu<ACT>(gv.v[e]) * oscale;
  }
  stv<V>(sp, S);
  stv<V>(out + b * ldo + c, o);
}

constexpr int GRU_FLIGHT = 8;        // rows requested ahead of their use
struct GruRows { const void* p; int64_t ld; };      // activations

// chunks [n][2]: {first row, rows}; sums [n][2][W]: decay, contribution
template <typename ACT, int V>
__global__ void __launch_bounds__(64) gru_chunk_kernel(GruRows z, GruRows u, const float* __restrict__ bz,
                                                      const float* __restrict__ bx, const int32_t* __restrict__ chunks, int W,
                                                      float* __restrict__ sums) {
  const int c = (blockIdx.y * 64 + threadIdx.x) * V;
  if (c >= W) return;
  const int row0 = chunks[2 * blockIdx.x], n = chunks[2 * blockIdx.x + 1];
  const Vec<V> vz = ldv<V>(bz + c), vx = ldv<V>(bx + c);
  const ACT *zp = reinterpret_cast<const ACT*>(z.p) + row0 * z.ld + c, *up = reinterpret_cast<const ACT*>(u.p) + row0 * u.ld + c;
  Vec<V> A, B = zerov<V>();
#pragma unroll
  for (int e = 0; e < V; ++e) A.v[e] = 1.f;
  Raw<ACT, V> zv[GRU_FLIGHT], uv[GRU_FLIGHT];
#pragma unroll
  for (int i = 0; i < GRU_FLIGHT; ++i) {
    zv[i].get(zp + min(i, n - 1) * z.ld);
    uv[i].get(up + min(i, n - 1) * u.ld);
  }
  for (int r0 = 0; r0 < n; r0 += GRU_FLIGHT)
#pragma unroll
    for (int i = 0; i < GRU_FLIGHT; ++i) {
      const Raw<ACT, V> zr = zv[i], ur = uv[i];
      const int64_t next = min(r0 + GRU_FLIGHT + i, n - 1);      // past the last: read again, not used
      zv[i].get(zp + next * z.ld);
      uv[i].get(up + next * u.ld);
      if (r0 + i < n)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float a, k;
          gru_gates<ACT>(zr.at(e) + vz.v[e], ur.at(e) + vx.v[e], a, k);
          A.v[e] *= a;
          B.v[e] = a * B.v[e] + k;
        }
    }
  float* o = sums + (size_t)blockIdx.x * 2 * W + c;
  stv<V>(o, A);
  stv<V>(o + W, B);
}

template <typename ACT, int V>
__global__ void __launch_bounds__(64) gru_apply_kernel(GruRows z, GruRows u, GruRows g, const float* __restrict__ bz,
                                                      const float* __restrict__ bx, const int32_t* __restrict__ chunks, int W,
                                                      const float* __restrict__ sums, ACT* __restrict__ out, int64_t ldo,
                                                      float oscale) {
  const int c = (blockIdx.y * 64 + threadIdx.x) * V;
  if (c >= W) return;
  const int row0 = chunks[2 * blockIdx.x], n = chunks[2 * blockIdx.x + 1];
  const Vec<V> vz = ldv<V>(bz + c), vx = ldv<V>(bx + c);
  const ACT *zp = reinterpret_cast<const ACT*>(z.p) + row0 * z.ld + c, *up = reinterpret_cast<const ACT*>(u.p) + row0 * u.ld + c,
            *gp = reinterpret_cast<const ACT*>(g.p) + row0 * g.ld + c;
  Vec<V> S = ldv<V>(sums + (size_t)blockIdx.x * 2 * W + c);
  Raw<ACT, V> zv[GRU_FLIGHT], uv[GRU_FLIGHT], gv[GRU_FLIGHT];
#pragma unroll
  for (int i = 0; i < GRU_FLIGHT; ++i) {
    const int64_t r = min(i, n - 1);
    zv[i].get(zp + r * z.ld);
    uv[i].get(up + r * u.ld);
    gv[i].get(gp + r * g.ld);
  }
  for (int r0 = 0; r0 < n; r0 += GRU_FLIGHT)
#pragma unroll
    for (int i = 0; i < GRU_FLIGHT; ++i) {
      const Raw<ACT, V> zr = zv[i], ur = uv[i], gr = gv[i];
      const int64_t next = min(r0 + GRU_FLIGHT + i, n - 1);
      zv[i].get(zp + next * z.ld);
      uv[i].get(up + next * u.ld);
      gv[i].get(gp + next * g.ld);
      if (r0 + i < n) {
        Vec<V> o;
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float a, k;
          gru_gates<ACT>(zr.at(e) + vz.v[e], ur.at(e) + vx.v[e], a, k);
          S.v[e] = a * S.v[e] + k;
          o.v[e] = S.v[e] * silu<ACT>(gr.at(e)) * oscale;
        }
        stv<V>(out + (row0 + r0 + i) * ldo + c, o);
      }
    }
}

// vectors of four where every operand's rows allow them
bool gru_vec(const GruCols* a, int n, int W, int f32, const void* out, int64_t ldo) {
  bool v = W % 4 == 0 && ldo % 4 == 0 && ((uintptr_t)out & (f32 ? 15 : 7)) == 0;
  for (int i = 0; i < n; ++i)
    v = v && a[i].ld % 4 == 0 && a[i].plane % 4 == 0 && ((uintptr_t)a[i].p & (a[i].split == 0 && !f32 ? 7 : 15)) == 0;
  return v;
}

}  // namespace

// z, u, g: columns of products (pointer, split (0: activations, else fp32 slabs), row stride, slab stride); out rows of stride
// ldo, times oscale
CFC_API int cfc_gru_step(int f32, const void* z, int z_split, int64_t z_ld, int64_t z_plane, const void* u, int u_split,
                         int64_t u_ld, int64_t u_plane, const void* g, int g_split, int64_t g_ld, int64_t g_plane, const float* bz,
                         const float* bx, const int32_t* slots, const int32_t* ctx_lens, int B, int W, float* state, void* out,
                         int64_t ldo, float oscale, hipStream_t stream) {
  if (B <= 0) return 0;
  if (W < 1 || !slots || !ctx_lens || !state || ldo < W) return -1;
  const GruCols a[3] = {{z, z_split, z_ld, z_plane}, {u, u_split, u_ld, u_plane}, {g, g_split, g_ld, g_plane}};
#define GS(ACT, V) \
  gru_step_kernel<ACT, V><<<dim3(B, (W + 64 * V - 1) / (64 * V)), 64, 0, stream>>>(a[0], a[1], a[2], bz, bx, slots, ctx_lens, W, state, (ACT*)out, ldo, oscale)
  const bool v4 = gru_vec(a, 3, W, f32, out, ldo);
  if (f32) { if (v4) GS(float, 4); else GS(float, 1); }
  else if (v4) GS(uint16_t, 4);
  else GS(uint16_t, 1);
#undef GS
  return CFC_CHECK_LAUNCH();
}

// packed portions; z, u, g activations (pointer, row stride); chunks [n][2] {first row, rows}, chunk_cu [portions + 1]; sums
// scratch [n][2][W]
CFC_API int cfc_gru_prefill(int f32, const void* z, int64_t z_ld, const void* u, int64_t u_ld, const void* g, int64_t g_ld,
                            const float* bz, const float* bx, const int32_t* chunks, int n, const int32_t* chunk_cu,
                            const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* slots, int portions, int W, float* sums,
                            float* state, void* out, int64_t ldo, float oscale, hipStream_t stream) {
  if (n <= 0 || portions <= 0) return 0;
  if (W < 1 || !chunks || !chunk_cu || !cu_q || !ctx_lens || !slots || !sums || !state || ldo < W) return -1;
  const GruCols a[3] = {{z, 0, z_ld, 0}, {u, 0, u_ld, 0}, {g, 0, g_ld, 0}};
  const GruRows r[3] = {{z, z_ld}, {u, u_ld}, {g, g_ld}};
#define GP(ACT, V)                                                                                                    \
  do {                                                                                                                \
    const int gy = (W + 64 * V - 1) / (64 * V);                                                                       \
    gru_chunk_kernel<ACT, V><<<dim3(n, gy), 64, 0, stream>>>(r[0], r[1], bz, bx, chunks, W, sums);                    \
    carry_kernel<V><<<dim3(portions, gy), 64, 0, stream>>>(chunk_cu, cu_q, ctx_lens, slots, W, sums, state);      \
    gru_apply_kernel<ACT, V><<<dim3(n, gy), 64, 0, stream>>>(r[0], r[1], r[2], bz, bx, chunks, W, sums, (ACT*)out, ldo, oscale);   \
  } while (0)
  const bool v4 = gru_vec(a, 3, W, f32, out, ldo);
  if (f32) { if (v4) GP(float, 4); else GP(float, 1); }
  else if (v4) GP(uint16_t, 4);
  else GP(uint16_t, 1);
#undef GP
  return CFC_CHECK_LAUNCH();
}
