// Linear recurrence with a per-channel, data-dependent decay (the RWKV kind of time mixing), per head:
//   o_t = (S + diag(u) k_t v_t^T)^T r_t,   S <- diag(w_t) S + k_t v_t^T,   w_t = exp(-exp(z_t))
// with z_t = W2 tanh(low-rank projection) + w0; then o over its root mean square, times norm, times silu(gate).
// S [slots][H][D][D] fp32 (key channel, value channel); a sequence at position 0 starts from zeros.
//
// Prompt portions run in chunks of 16 tokens.  With L_t the running sum of log w inside a chunk, token i's
// output is  (r_i exp(L_(i-1)))^T S_chunk  +  sum_(j<i) [sum_c r_i k_j exp(L_(i-1) - L_j)] v_j  +  the bonus
// term, and the chunk's state step is  S <- exp(L_15) S + sum_j (k_j exp(L_15 - L_j)) v_j^T.  Every exponent
// is <= 0, whatever the decays, so nothing over- or underflows that the plain recurrence would keep.
//   * wkv_tanh   the low-rank activations as three bf16 parts (24 bits: W2's product on the bf16 matrix
//                cores is exact to fp32)
//   * wkv_prep   one wave per (chunk, head), all chunks in parallel: decays, the scaled r and k and the 16 x 16
//                coefficients, written in the fragment order of the scan's fp32 MFMAs
//   * wkv_scan   one workgroup per (sequence, head), a wave per 16 value channels: the state stays in the
//                accumulators over all chunks and is the B operand of the next one as it lies
//   * wkv_step   token by token: decoded tokens (one pass over the state: read, output, update), and prompt
//                portions of head sizes the chunked kernels are not built for
#include "common.h"

namespace {

__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ld1(const float* p) { return *p; }
__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

constexpr float LOG_DECAY_MIN = -104.f;      // exp(-104) is 0 in fp32
constexpr int CT = 16;                       // tokens per chunk
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float log_decay(float z) { return fmaxf(-expf(z), LOG_DECAY_MIN); }

// columns of a product: activations (split 0) or fp32 slabs
struct Cols {
  const void* p;
  int split;                // 0: activations
  int64_t ld, plane;
};

// in two steps, so that other loads can go out between the request and the wait: the first (up to) ASK slabs,
// then their sum and the rest
constexpr int ASK = 4;
template <typename ACT>
__device__ __forceinline__ void ldc_ask(const Cols& a, int64_t t, int c, float (&v)[ASK]) {
  const int64_t o = t * a.ld + c;
  if (a.split == 0) {
    v[0] = ld1(reinterpret_cast<const ACT*>(a.p) + o);
    return;
  }
  const float* p = reinterpret_cast<const float*>(a.p) + o;
#pragma unroll
  for (int u = 0; u < ASK; ++u) v[u] = p[(int64_t)min(u, a.split - 1) * a.plane];
}
template <typename ACT>
__device__ __forceinline__ float ldc_sum(const Cols& a, int64_t t, int c, const float (&v)[ASK]) {
  float s = v[0];
#pragma unroll
  for (int u = 1; u < ASK; ++u) s += u < a.split ? v[u] : 0.f;
  const float* p = reinterpret_cast<const float*>(a.p) + t * a.ld + c;
  for (int u = ASK; u < a.split; ++u) s += p[(int64_t)u * a.plane];
  return s;
}
template <typename ACT>
__device__ __forceinline__ float ldc(const Cols& a, int64_t t, int c) {
  float v[ASK];
  ldc_ask<ACT>(a, t, c, v);
  return ldc_sum<ACT>(a, t, c, v);
}

// out [T][3][RP]: high, middle and low bf16 parts of tanh(w1); columns past R zero
template <typename ACT>
__global__ void __launch_bounds__(256) wkv_tanh_kernel(Cols w1, int T, int R, int RP, uint16_t* __restrict__ out) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (int64_t)T * RP) return;
  const int64_t t = i / RP;
  const int c = (int)(i % RP);
  const float v = c < R ? tanhf(ldc<ACT>(w1, t, c)) : 0.f;
  const uint16_t hi = f2bf(v);
  const float r1 = v - bf2f(hi);
  const uint16_t mid = f2bf(r1);
  uint16_t* o = out + t * 3 * RP + c;
  o[0] = hi;
  o[RP] = mid;
  o[2 * RP] = f2bf(r1 - bf2f(mid));
}

// ---------------------------------------------------------------------------------- chunked prompt portions
// per (chunk, head): [ND][64][4] scaled r, [ND][64][4] scaled k, [64][4] coefficients, [16 ND] decays
template <int ND>
struct ChunkRec {
  static constexpr int R = 0, K = ND * 256, A = 2 * ND * 256, DEC = A + 256, SIZE = DEC + 16 * ND;
};

template <typename ACT, int ND, int WV>
__global__ void __launch_bounds__(64 * WV) wkv_prep_kernel(Cols r, Cols k, const uint16_t* __restrict__ th, int RP,
                                                          const uint16_t* __restrict__ w2, const float* __restrict__ w0,
                                                          const float* __restrict__ u, const int32_t* __restrict__ chunks,
                                                          int H, int D, float* __restrict__ rec) {
  constexpr int DP = 16 * ND, LD = DP + 4;
  using Rec = ChunkRec<ND>;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, col = lane & 15, q = lane >> 4;
  const int h = blockIdx.y * WV + wv;
  if (h >= H) return;                             // waves share nothing below
  float* L = smem + wv * (49 * LD);               // [17][LD]: L[t] = sum of log2 w before token t
  float* rs = L + 17 * LD;                        // [16][LD]
  float* ks = rs + 16 * LD;                       // [16][LD], then the coefficients [16][17] in its place
  const int row0 = chunks[2 * blockIdx.x], n = chunks[2 * blockIdx.x + 1];
  const int hc = h * D;
  // r and k, channel per lane
#pragma unroll
  for (int c0 = 0; c0 < DP; c0 += 64) {
    const int c = c0 + lane;
    if (c < DP) {
      const bool live = c < D;
      float a[CT], b[CT];
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        const int tt = row0 + min(t, n - 1), cc = hc + (live ? c : 0);
        a[t] = ld1(reinterpret_cast<const ACT*>(r.p) + tt * r.ld + cc);
        b[t] = ld1(reinterpret_cast<const ACT*>(k.p) + tt * k.ld + cc);
      }
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        rs[t * LD + c] = live && t < n ? a[t] : 0.f;
        ks[t * LD + c] = live && t < n ? b[t] : 0.f;
      }
    }
  }
  // z^T = W2 tanh^T + w0: lane holds channels 16 T + 4 q + i of token col.  Every load unconditional: one under a
  // branch would be waited for before the next goes out
  f32x4_t z[ND];
  float ur[ND][4];                                // u of the lane's channels of the diagonal, below
#pragma unroll
  for (int T = 0; T < ND; ++T)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      z[T][i] = w0[hc + min(16 * T + 4 * q + i, D - 1)];
      ur[T][i] = u[hc + min(16 * T + 4 * (lane & 3) + i, D - 1)];
    }
  const uint16_t* tr = th + (size_t)(row0 + min(col, n - 1)) * 3 * RP + 8 * q;
  for (int kk = 0; kk < RP; kk += 32) {
    bf16x8_t b[3];
#pragma unroll
    for (int p = 0; p < 3; ++p) b[p] = *reinterpret_cast<const bf16x8_t*>(tr + p * RP + kk);
#pragma unroll
    for (int T = 0; T < ND; ++T) {
      const int ch = min(16 * T + col, D - 1);
      const bf16x8_t a = *reinterpret_cast<const bf16x8_t*>(w2 + (size_t)(hc + ch) * RP + kk + 8 * q);
#pragma unroll
      for (int p = 0; p < 3; ++p) z[T] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b[p], z[T], 0, 0, 0);
    }
  }
#pragma unroll
  for (int T = 0; T < ND; ++T) {
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = 16 * T + 4 * q + i;
      const float l = log_decay(z[T][i]) * LOG2E;
      v[i] = c < D && col < n ? l : 0.f;
    }
    *reinterpret_cast<float4*>(L + (col + 1) * LD + 16 * T + 4 * q) = make_float4(v[0], v[1], v[2], v[3]);
  }
  auto sync = [] {                                // the wave's own LDS writes are visible to its lanes
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  };
  sync();
  float* out = rec + ((size_t)blockIdx.x * H + h) * Rec::SIZE;
#pragma unroll
  for (int c0 = 0; c0 < DP; c0 += 64) {
    const int c = c0 + lane;
    if (c < DP) {
      float s = 0.f;
      L[c] = 0.f;
#pragma unroll
      for (int t = 1; t <= CT; ++t) {
        s += L[t * LD + c];
        L[t * LD + c] = s;
      }
      out[Rec::DEC + c] = __builtin_amdgcn_exp2f(s);
    }
  }
  sync();
  // scaled r (row col, channels 16 T + 4 q ..) and scaled k (tokens 4 q + s, channel 16 T + col)
#pragma unroll
  for (int T = 0; T < ND; ++T) {
    const int c = 16 * T + 4 * q;
    const float4 rv = *reinterpret_cast<const float4*>(rs + col * LD + c), lv = *reinterpret_cast<const float4*>(L + col * LD + c);
    reinterpret_cast<float4*>(out + Rec::R)[T * 64 + lane] =
        make_float4(rv.x * __builtin_amdgcn_exp2f(lv.x), rv.y * __builtin_amdgcn_exp2f(lv.y), rv.z * __builtin_amdgcn_exp2f(lv.z), rv.w * __builtin_amdgcn_exp2f(lv.w));
    float kv[4];
    const float le = L[16 * LD + 16 * T + col];
#pragma unroll
    for (int s = 0; s < 4; ++s) kv[s] = ks[(4 * q + s) * LD + 16 * T + col] * __builtin_amdgcn_exp2f(le - L[(4 * q + s + 1) * LD + 16 * T + col]);
    reinterpret_cast<float4*>(out + Rec::K)[T * 64 + lane] = make_float4(kv[0], kv[1], kv[2], kv[3]);
  }
  // coefficients below the diagonal: two of the 120 pairs (i, j < i) per lane
  int pi[2], pj[2];
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int p = min(lane + 64 * e, 119);
    int i = (int)((1.f + sqrtf(1.f + 8.f * p)) * 0.5f);
    if (i * (i - 1) / 2 > p) --i;
    if ((i + 1) * i / 2 <= p) ++i;
    pi[e] = i;
    pj[e] = p - i * (i - 1) / 2;
  }
  float acc[2] = {0.f, 0.f};
#pragma unroll 2
  for (int c = 0; c < DP; c += 4)
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const float4 a = *reinterpret_cast<const float4*>(L + pi[e] * LD + c), b = *reinterpret_cast<const float4*>(L + (pj[e] + 1) * LD + c);
      const float4 x = *reinterpret_cast<const float4*>(rs + pi[e] * LD + c), y = *reinterpret_cast<const float4*>(ks + pj[e] * LD + c);
      acc[e] += x.x * y.x * __builtin_amdgcn_exp2f(a.x - b.x) + x.y * y.y * __builtin_amdgcn_exp2f(a.y - b.y) + x.z * y.z * __builtin_amdgcn_exp2f(a.z - b.z) +
                x.w * y.w * __builtin_amdgcn_exp2f(a.w - b.w);
    }
  // the diagonal: row lane / 4, a quarter of the channels
  float dg = 0.f;
  {
    const int i = lane >> 2;
#pragma unroll
    for (int T = 0; T < ND; ++T) {                // r and k past D are zero
      const int c = 16 * T + 4 * (lane & 3);
      const float4 a = *reinterpret_cast<const float4*>(rs + i * LD + c), b = *reinterpret_cast<const float4*>(ks + i * LD + c);
      dg += ur[T][0] * a.x * b.x + ur[T][1] * a.y * b.y + ur[T][2] * a.z * b.z + ur[T][3] * a.w * b.w;
    }
    dg += __shfl_xor(dg, 1, 64);
    dg += __shfl_xor(dg, 2, 64);
  }
  sync();
  float* am = ks;                                 // every read of k is done
#pragma unroll
  for (int e = 0; e < 4; ++e) am[(lane >> 2) * 17 + 4 * (lane & 3) + e] = 0.f;
  sync();
#pragma unroll
  for (int e = 0; e < 2; ++e)
    if (lane + 64 * e < 120) am[pi[e] * 17 + pj[e]] = acc[e];
  if ((lane & 3) == 0) am[(lane >> 2) * 17 + (lane >> 2)] = dg;
  sync();
  float av[4];
#pragma unroll
  for (int s = 0; s < 4; ++s) av[s] = am[col * 17 + 4 * q + s];
  reinterpret_cast<float4*>(out + Rec::A)[lane] = make_float4(av[0], av[1], av[2], av[3]);
}

struct ScanSeq {
  const int32_t* chunk_cu;    // [sequences + 1]
  const int32_t* chunks;      // [chunks][2]: first row, rows
  const int32_t* slots;       // [sequences]
  const int32_t* cu_q;
  const int32_t* ctx_lens;
};

__device__ __forceinline__ f32x4_t mfma4(float a, float b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// Records, v and g of the next SCAN_AHEAD chunks are on their way in registers while a chunk runs from LDS (two
// buffers, one barrier per chunk); a chunk's outputs wait for the head's mean square until the next barrier.
constexpr int SCAN_AHEAD = 4;

typedef unsigned short raw16_t;
template <typename ACT> struct RawOf { typedef uint32_t type; };
template <> struct RawOf<uint16_t> { typedef raw16_t type; };
template <typename ACT>
__device__ __forceinline__ typename RawOf<ACT>::type ld_raw(__amdgpu_buffer_rsrc_t b, int vo, int so) {
  if constexpr (sizeof(ACT) == 2) return __builtin_amdgcn_raw_buffer_load_b16(b, vo, so, 0);
  else return __builtin_amdgcn_raw_buffer_load_b32(b, vo, so, 0);
}
template <typename ACT>
__device__ __forceinline__ void st_raw(__amdgpu_buffer_rsrc_t b, int vo, int so, float y) {
  if constexpr (sizeof(ACT) == 2) __builtin_amdgcn_raw_buffer_store_b16((raw16_t)(cvt_pk_bf16_f32(y, y) & 0xffff), b, vo, so, 0);
  else __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(y), b, vo, so, 0);
}
template <typename ACT>
__device__ __forceinline__ float raw2f(typename RawOf<ACT>::type v) {
  return sizeof(ACT) == 2 ? __uint_as_float((uint32_t)v << 16) : __uint_as_float((uint32_t)v);
}
// buffer over `bytes` (< 2^31) from p, both uniform over the workgroup
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rows_of(const void* p, int64_t bytes) {
  // unsigned halves: readfirstlane returns int, whose sign would run into the upper half
  const uint32_t lo = __builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)p), hi = __builtin_amdgcn_readfirstlane((uint32_t)((uintptr_t)p >> 32));
  return __builtin_amdgcn_make_buffer_rsrc((void*)(((uintptr_t)hi << 32) | lo), (short)0, __builtin_amdgcn_readfirstlane((int)bytes), 0x00020000);
}
// sum over the 16 lanes of a row (four rotations within it)
__device__ __forceinline__ float row16_sum(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));   // row_ror:8
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x124, 0xf, 0xf, false));
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x122, 0xf, 0xf, false));
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x121, 0xf, 0xf, false));
  return x;
}

template <typename ACT, int ND>
__global__ void __launch_bounds__(64 * ND, 2) wkv_scan_kernel(const float* __restrict__ rec, Cols v, Cols g, ScanSeq sq, int H,
                                                             int D, const float* __restrict__ norm, float eps,
                                                             float* __restrict__ state, ACT* __restrict__ out, int64_t ldo) {
  using Rec = ChunkRec<ND>;
  using RAW = typename RawOf<ACT>::type;
  constexpr int NV4 = Rec::SIZE / 4, NT = 64 * ND, NLD = (NV4 + NT - 1) / NT;
  __shared__ __attribute__((aligned(16))) float buf[2][NLD * NT * 4];   // the last piece past the record: not read
  __shared__ __attribute__((aligned(16))) float red[2][ND][16];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, q = lane >> 4;
  const int h = blockIdx.x, s = blockIdx.y;
  const int c0 = sq.chunk_cu[s], nc = sq.chunk_cu[s + 1] - c0;
  if (nc <= 0) return;
  const int row0 = sq.cu_q[s], len = sq.cu_q[s + 1] - row0;
  const bool fresh = sq.ctx_lens[s] == len;
  const int vc = 16 * w + col;                    // value channel of this lane
  const bool live = vc < D;
  const int hv = h * D + min(vc, D - 1);
  float* st = state + (((size_t)sq.slots[s] * H + h) * D) * D + min(vc, D - 1);
  f32x4_t S[ND];
#pragma unroll
  for (int T = 0; T < ND; ++T)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int kc = 16 * T + 4 * q + i;
      S[T][i] = !fresh && live && kc < D ? st[(size_t)min(kc, D - 1) * D] : 0.f;
    }
  const float nw = norm[hv], rD = 1.f / (float)D;
  typedef float f4_t __attribute__((ext_vector_type(4)));      // arrays of these stay in registers
  f4_t rr[SCAN_AHEAD][NLD];
  RAW rv[SCAN_AHEAD][4], rg[SCAN_AHEAD][4];         // as loaded: a conversion would wait for them
  // buffers of the portion's rows: a chunk's place is a scalar offset, rows past the portion read as zero and are
  // not stored -- no bounds arithmetic, and no branch whose join would wait for every load in flight
  constexpr int EB = sizeof(ACT);
  const __amdgpu_buffer_rsrc_t vb = rows_of(reinterpret_cast<const ACT*>(v.p) + row0 * v.ld, len * v.ld * EB);
  const __amdgpu_buffer_rsrc_t gb = rows_of(reinterpret_cast<const ACT*>(g.p) + row0 * g.ld, len * g.ld * EB);
  const __amdgpu_buffer_rsrc_t ob = rows_of(out + row0 * ldo, len * ldo * EB);
  int vo[4], go[4], oo[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    vo[i] = ((4 * q + i) * (int)v.ld + hv) * EB;
    go[i] = ((4 * q + i) * (int)g.ld + hv) * EB;
    oo[i] = live ? ((4 * q + i) * (int)ldo + hv) * EB : 0x7ffffff0;
  }
  const float lm = live ? 1.f : 0.f;
  // chunk c (past the last: re-read, not used)
  auto load = [&](int c, int u) {
    c = __builtin_amdgcn_readfirstlane(min(c, nc - 1));
    const f4_t* p = reinterpret_cast<const f4_t*>(rec + ((size_t)(c0 + c) * H + h) * Rec::SIZE);
#pragma unroll
    for (int i = 0; i < NLD; ++i) rr[u][i] = p[min(tid + NT * i, NV4 - 1)];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      rv[u][i] = ld_raw<ACT>(vb, vo[i], c * CT * (int)v.ld * EB);
      rg[u][i] = ld_raw<ACT>(gb, go[i], c * CT * (int)g.ld * EB);
    }
  };
  auto store = [&](int b, int u) {
#pragma unroll
    for (int i = 0; i < NLD; ++i) reinterpret_cast<f4_t*>(buf[b])[tid + NT * i] = rr[u][i];
  };
  auto barrier = [] {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
  };
  f32x4_t o_prev{0.f, 0.f, 0.f, 0.f};
  float g_prev[4] = {0.f, 0.f, 0.f, 0.f};
  // outputs of chunk c from the mean squares in red[b]
  auto finish = [&](int c, int b) {
    float sv[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < ND; ++j) {
      const float4 a = *reinterpret_cast<const float4*>(&red[b][j][4 * q]);
      sv[0] += a.x; sv[1] += a.y; sv[2] += a.z; sv[3] += a.w;
    }
    const int so = __builtin_amdgcn_readfirstlane(max(c, 0) * CT * (int)ldo * EB);   // before the first: overwritten by it
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float r = __builtin_amdgcn_rsqf(sv[i] * rD + eps);
      const float y = o_prev[i] * r * nw * (g_prev[i] * __builtin_amdgcn_rcpf(1.f + __expf(-g_prev[i])));
      st_raw<ACT>(ob, oo[i], so, y);
    }
  };
#pragma unroll
  for (int u = 0; u < SCAN_AHEAD; ++u) load(u, u);
  store(0, 0);
  // chunk c from buf[u & 1] (its v and g in slot u); slot u then takes chunk c + SCAN_AHEAD
  auto chunk = [&](int c, int u) {
    barrier();
    const int b = u & 1;
    finish(c - 1, b ^ 1);
    float vv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      vv[i] = raw2f<ACT>(rv[u][i]);
      g_prev[i] = raw2f<ACT>(rg[u][i]);
    }
    load(c + SCAN_AHEAD, u);
    const float4* p = reinterpret_cast<const float4*>(buf[b]);
    f32x4_t o0{0.f, 0.f, 0.f, 0.f}, o1{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int T = 0; T < ND; ++T) {
      const float4 r = p[T * 64 + lane];
      o0 = mfma4(r.x, S[T][0], o0);
      o1 = mfma4(r.y, S[T][1], o1);
      o0 = mfma4(r.z, S[T][2], o0);
      o1 = mfma4(r.w, S[T][3], o1);
    }
    const float4 a = p[Rec::A / 4 + lane];
    o0 = mfma4(a.x, vv[0], o0);
    o1 = mfma4(a.y, vv[1], o1);
    o0 = mfma4(a.z, vv[2], o0);
    o1 = mfma4(a.w, vv[3], o1);
    float4 k[ND];
#pragma unroll
    for (int T = 0; T < ND; ++T) {
      const float4 d = p[Rec::DEC / 4 + 4 * T + q];
      k[T] = p[Rec::K / 4 + T * 64 + lane];
      S[T][0] *= d.x; S[T][1] *= d.y; S[T][2] *= d.z; S[T][3] *= d.w;
    }
#pragma unroll
    for (int T = 0; T < ND; ++T) S[T] = mfma4(k[T].x, vv[0], S[T]);
#pragma unroll
    for (int T = 0; T < ND; ++T) S[T] = mfma4(k[T].y, vv[1], S[T]);
#pragma unroll
    for (int T = 0; T < ND; ++T) S[T] = mfma4(k[T].z, vv[2], S[T]);
#pragma unroll
    for (int T = 0; T < ND; ++T) S[T] = mfma4(k[T].w, vv[3], S[T]);
    // sums of squares over the wave's 16 channels
    o_prev = o0 + o1;
    float ss[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      ss[i] = row16_sum(lm * o_prev[i] * o_prev[i]);
    }
    if (col == 0) *reinterpret_cast<float4*>(&red[b][w][4 * q]) = make_float4(ss[0], ss[1], ss[2], ss[3]);
    store(b ^ 1, (u + 1) % SCAN_AHEAD);
  };
  int c = 0;
  for (; c + SCAN_AHEAD <= nc; c += SCAN_AHEAD)
#pragma unroll
    for (int u = 0; u < SCAN_AHEAD; ++u) chunk(c + u, u);
#pragma unroll
  for (int u = 0; u < SCAN_AHEAD - 1; ++u)
    if (c + u < nc) chunk(c + u, u);
  barrier();
  finish(nc - 1, (nc - 1) & 1);
  if (live) {
#pragma unroll
    for (int T = 0; T < ND; ++T)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int kc = 16 * T + 4 * q + i;
        if (kc < D) st[(size_t)kc * D] = S[T][i];
      }
  }
}

// ---------------------------------------------------------------------------------- token by token
// one workgroup per (head, sequence); a thread owns V value channels of every NG-th key channel, so the
// state needs no synchronisation between tokens
constexpr int WS_T = 256, WS_NR = 4;
template <typename ACT, int V, bool ONE>      // ONE: a token per sequence
__global__ void __launch_bounds__(WS_T, ONE ? 6 : 4) wkv_step_kernel(Cols r, Cols k, Cols v, Cols g, Cols w1, int R, int RP,
                                                       const uint16_t* __restrict__ w2, const float* __restrict__ w0,
                                                       const float* __restrict__ u, const float* __restrict__ norm, float eps,
                                                       int H, int D, const int32_t* __restrict__ slots,
                                                       const int32_t* __restrict__ cu_q, const int32_t* __restrict__ ctx_lens,
                                                       float* __restrict__ state, ACT* __restrict__ out, int64_t ldo) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[16];
  const int nvec = (D + V - 1) / V, ng = WS_T / nvec;
  float* rs = sm;              // [D] each
  float* kk = rs + D;
  float* vs = kk + D;
  float* gs = vs + D;
  float* ws = gs + D;
  float* us = ws + D;          // u r k: the bonus
  float* th = us + D;          // [RP]
  float* part = th + RP;       // [ng][D]
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int q0 = ONE ? s : cu_q[s], n = ONE ? 1 : cu_q[s + 1] - q0;
  const bool fresh = ctx_lens[s] == n;
  float* st = state + ((size_t)slots[s] * H + h) * D * D;
  const int vx = tid % nvec, gy = tid / nvec, hc = h * D;
  const bool own = gy < ng;
  for (int t = 0; t < n; ++t) {
    const bool zero = fresh && t == 0;
    float S[WS_NR][V];
    auto ldS = [&](int i0) {
#pragma unroll
      for (int a = 0; a < WS_NR; ++a) {
        const int i = i0 + gy + a * ng;
#pragma unroll
        for (int e = 0; e < V; ++e) S[a][e] = 0.f;
        if (own && i < D && !zero) {
          if constexpr (V == 4) {
            const float4 f = *reinterpret_cast<const float4*>(st + (size_t)i * D + 4 * vx);
            S[a][0] = f.x; S[a][1] = f.y; S[a][2] = f.z; S[a][3] = f.w;
          } else {
            S[a][0] = st[(size_t)i * D + vx];
          }
        }
      }
    };
    const int64_t row = q0 + t;
    auto pick = [&](int e) {
      Cols s = r;
      const int w = e / D;
      s.p = w == 0 ? r.p : w == 1 ? k.p : w == 2 ? v.p : g.p;
      return s;
    };
    // the small operands are asked for ahead of the state: loads return in order
    float ask[ASK], ask1[ASK];
    const int e0 = min(tid, 4 * D - 1), z0 = min(tid, R - 1), wc = min(tid >> 2, D - 1);
    uint4 wq[2];
    ldc_ask<ACT>(pick(e0), row, hc + e0 % D, ask);
    ldc_ask<ACT>(w1, row, z0, ask1);
#pragma unroll
    for (int y = 0; y < 2; ++y)
      wq[y] = *reinterpret_cast<const uint4*>(w2 + (size_t)(hc + wc) * RP + min(8 * (tid & 3) + 32 * y, RP - 8));
    const float w0v = w0[hc + wc];
    ldS(0);
    if (tid < 4 * D) rs[tid] = ldc_sum<ACT>(pick(e0), row, hc + e0 % D, ask);
    if (tid < RP) th[tid] = tid < R ? tanhf(ldc_sum<ACT>(w1, row, z0, ask1)) : 0.f;
    for (int e = tid + WS_T; e < 4 * D; e += WS_T) rs[e] = ldc<ACT>(pick(e), row, hc + e % D);
    for (int c = tid + WS_T; c < RP; c += WS_T) th[c] = c < R ? tanhf(ldc<ACT>(w1, row, c)) : 0.f;
    __syncthreads();
    // four threads per channel over the low rank
    for (int c0 = 0; c0 < D; c0 += WS_T / 4) {
      const int c = c0 + (tid >> 2), p = tid & 3;
      float z = 0.f;
      auto dot = [&](const uint4& w, int x) {
        float wv[8];
        unpack8(w, wv);
#pragma unroll
        for (int e = 0; e < 8; ++e) z += wv[e] * th[x + e];
      };
      if (c < D) {
        if (c0 == 0) {
          dot(wq[0], 8 * p);
          if (RP > 32) dot(wq[1], 8 * p + 32);
        }
        for (int x = 8 * p + (c0 == 0 ? 64 : 0); x < RP; x += 32)
          dot(*reinterpret_cast<const uint4*>(w2 + (size_t)(hc + c) * RP + x), x);
      }
      z += __shfl_xor(z, 1, 64);
      z += __shfl_xor(z, 2, 64);
      if (c < D && p == 0) ws[c] = expf(log_decay(z + (c0 == 0 ? w0v : w0[hc + c])));
    }
    for (int c = tid; c < D; c += WS_T) us[c] = u[hc + c] * rs[c] * kk[c];
    __syncthreads();
    float o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = 0.f;
    float vv[V];
#pragma unroll
    for (int e = 0; e < V; ++e) vv[e] = own ? vs[min(V * vx + e, D - 1)] : 0.f;
    for (int i0 = 0; i0 < D; i0 += WS_NR * ng) {
      if (i0) ldS(i0);
#pragma unroll
      for (int a = 0; a < WS_NR; ++a) {
        const int i = i0 + gy + a * ng;
        if (!own || i >= D) continue;
        const float ri = rs[i], ki = kk[i], wi = ws[i], bi = us[i];
#pragma unroll
        for (int e = 0; e < V; ++e) {
          o[e] += ri * S[a][e] + bi * vv[e];
          S[a][e] = wi * S[a][e] + ki * vv[e];
        }
        if constexpr (V == 4) *reinterpret_cast<float4*>(st + (size_t)i * D + 4 * vx) = make_float4(S[a][0], S[a][1], S[a][2], S[a][3]);
        else st[(size_t)i * D + vx] = S[a][0];
      }
    }
    if (own)
#pragma unroll
      for (int e = 0; e < V; ++e)
        if (V * vx + e < D) part[gy * D + V * vx + e] = o[e];
    __syncthreads();
    float y[2], ss = 0.f;                        // D <= 2 WS_T
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int c = tid + m * WS_T;
      y[m] = 0.f;
      if (c < D) {
        for (int a = 0; a < ng; ++a) y[m] += part[a * D + c];
        ss += y[m] * y[m];
      }
    }
    if (ONE && D <= 64 && tid >= 64) return;     // one wave holds the head
    const float rr = 1.f / sqrtf((D <= 64 ? wave_sum(ss) : block_sum(ss, red)) / (float)D + eps);
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int c = tid + m * WS_T;
      if (c < D) {
        const float gg = gs[c];
        st1(out + row * ldo + hc + c, y[m] * rr * norm[hc + c] * (gg / (1.f + expf(-gg))));
      }
    }
    if constexpr (!ONE) __syncthreads();         // the next token overwrites what this one read
  }
}

template <typename ACT, int ND>
int chunked_go(hipStream_t s, const Cols& r, const Cols& k, const Cols& v, const Cols& g, const uint16_t* th, int RP,
               const uint16_t* w2, const float* w0, const float* u, const float* norm, float eps, int H, int D, int n_chunks,
               int n_seq, const ScanSeq& sq, float* rec, float* state, void* out, int64_t ldo) {
  constexpr int WV = ND <= 4 ? 4 : 2;
  constexpr int lds = WV * 49 * (16 * ND + 4) * 4;
  wkv_prep_kernel<ACT, ND, WV><<<dim3(n_chunks, (H + WV - 1) / WV), 64 * WV, lds, s>>>(r, k, th, RP, w2, w0, u, sq.chunks, H, D, rec);
  if (const int e = (int)hipGetLastError()) return e;
  wkv_scan_kernel<ACT, ND><<<dim3(H, n_seq), 64 * ND, 0, s>>>(rec, v, g, sq, H, D, norm, eps, state, (ACT*)out, ldo);
  return CFC_CHECK_LAUNCH();
}

}  // namespace

constexpr int WKV_MAX_CHUNKED = 128;

// floats of scratch per (chunk, head); 0: no chunked kernel for this head size
CFC_API int cfc_wkv_chunk_floats(int D) {
  if (D < 1 || D > WKV_MAX_CHUNKED) return 0;
  const int nd = D <= 64 ? (D + 15) / 16 : D <= 96 ? 6 : 8;
  return 2 * nd * 256 + 256 + 16 * nd;
}

// out [T][3][RP] bf16 parts of tanh(w1) (split 0: w1 are activations)
CFC_API int cfc_wkv_tanh(int f32, const void* w1, int split, int64_t ld, int64_t plane, int T, int R, int RP, void* out,
                         hipStream_t stream) {
  if (T <= 0) return 0;
  if (R < 1 || RP < R || RP % 32 || split < 0) return -1;
  const Cols c{w1, split, ld, plane};
  const int64_t n = ((int64_t)T * RP + 255) / 256;
  if (f32) wkv_tanh_kernel<float><<<(unsigned)n, 256, 0, stream>>>(c, T, R, RP, (uint16_t*)out);
  else wkv_tanh_kernel<uint16_t><<<(unsigned)n, 256, 0, stream>>>(c, T, R, RP, (uint16_t*)out);
  return CFC_CHECK_LAUNCH();
}

// r, k, v, g: activations with row strides; th from cfc_wkv_tanh; chunks [n][2] = {first row, rows <= 16} in
// sequence order, chunk_cu [sequences + 1]; rec: cfc_wkv_chunk_floats(D) floats per (chunk, head)
CFC_API int cfc_wkv_chunked(int f32, const void* r, int64_t ldr, const void* k, int64_t ldk, const void* v, int64_t ldv,
                            const void* g, int64_t ldg, const void* th, int RP, const void* w2, const float* w0,
                            const float* u, const float* norm, float eps, int H, int D, int n_chunks, int n_seq,
                            const int32_t* chunk_cu, const int32_t* chunks, const int32_t* slots, const int32_t* cu_q,
                            const int32_t* ctx_lens, float* rec, float* state, void* out, int64_t ldo, hipStream_t stream) {
  if (n_seq <= 0 || n_chunks <= 0) return 0;
  if (H < 1 || D < 1 || D > WKV_MAX_CHUNKED || RP < 32 || RP % 32 || n_seq > 65535) return -1;
  // 32-bit offsets within a portion
  const int64_t ldm = ldo > ldv ? (ldo > ldg ? ldo : ldg) : (ldv > ldg ? ldv : ldg);
  if (((int64_t)n_chunks + 4) * CT * ldm * (f32 ? 4 : 2) >= 0x7fffff00ll) return -4;
  const Cols cr{r, 0, ldr, 0}, ck{k, 0, ldk, 0}, cv{v, 0, ldv, 0}, cg{g, 0, ldg, 0};
  const ScanSeq sq{chunk_cu, chunks, slots, cu_q, ctx_lens};
#define WC(ACT, ND)                                                                                                      \
  return chunked_go<ACT, ND>(stream, cr, ck, cv, cg, (const uint16_t*)th, RP, (const uint16_t*)w2, w0, u, norm, eps, H, \
                             D, n_chunks, n_seq, sq, rec, state, out, ldo)
#define WN(ACT)                                      \
  switch (D <= 64 ? (D + 15) / 16 : D <= 96 ? 6 : 8) { \
    case 1: WC(ACT, 1);                              \
    case 2: WC(ACT, 2);                              \
    case 3: WC(ACT, 3);                              \
    case 4: WC(ACT, 4);                              \
    case 6: WC(ACT, 6);                              \
    default: WC(ACT, 8);                             \
  }
  if (f32) WN(float)
  WN(uint16_t)
#undef WN
#undef WC
}

// one token per sequence (cu_q null) or portions, token by token.  Each operand: pointer, split (0:
// activations, else fp32 slabs), row stride, slab stride
CFC_API int cfc_wkv_step(int f32, const void* r, const void* k, const void* v, const void* g, int split, int64_t ld,
                         int64_t plane, const void* w1, int split1, int64_t ld1, int64_t plane1, int R, int RP,
                         const void* w2, const float* w0, const float* u, const float* norm, float eps, int H, int D, int n_seq,
                         const int32_t* slots, const int32_t* cu_q, const int32_t* ctx_lens, float* state, void* out,
                         int64_t ldo, hipStream_t stream) {
  if (n_seq <= 0) return 0;
  if (H < 1 || D < 1 || D > 2 * WS_T || R < 1 || RP < R || RP % 32 || RP > 2048 || split < 0 || split1 < 0 || n_seq > 65535) return -1;
  const int V = D % 4 == 0 ? 4 : 1;
  if ((D + V - 1) / V > WS_T) return -1;
  const int ng = WS_T / ((D + V - 1) / V);
  const size_t lds = (size_t)(6 * D + RP + ng * D) * 4;
  const Cols cr{r, split, ld, plane}, ck{k, split, ld, plane}, cv{v, split, ld, plane}, cg{g, split, ld, plane},
      c1{w1, split1, ld1, plane1};
#define ST1(ACT, VV, ONE)                                                                                                     \
  wkv_step_kernel<ACT, VV, ONE><<<dim3(H, n_seq), WS_T, lds, stream>>>(cr, ck, cv, cg, c1, R, RP, (const uint16_t*)w2, w0, u, \
                                                                      norm, eps, H, D, slots, cu_q, ctx_lens, state, (ACT*)out, ldo)
#define ST(ACT, VV)                  \
  do {                               \
    if (cu_q) ST1(ACT, VV, false);   \
    else ST1(ACT, VV, true);         \
  } while (0)
  if (f32) { if (V == 4) ST(float, 4); else ST(float, 1); }
  else if (V == 4) ST(uint16_t, 4);
  else ST(uint16_t, 1);
#undef ST
#undef ST1
  return CFC_CHECK_LAUNCH();
}
