// Latent attention: every head's keys and values are products of one normalised latent row
// per token, and a few rotated key dimensions are shared by all heads.  Only those two are
// cached (one row per position).
//
// A prompt portion expands keys and values from the cache rows (a library product) and runs
// the causal attention of chunk_attend.hip.  A decode step, or a portion of a few tokens, moves
// the key product to the query's side instead (w_uk[h]^T q_h), so that the cache rows themselves
// are keys and, their first part, values of all heads at once; the value product follows on
// the weighted sum.  Kernels here:
//
//  * latent_rows_kernel: the two norms and the shared rotated part of a projected row.
//  * latent_absorb_kernel: query side of a step, with the cache row of the new token.
//  * latent_attend_kernel: keys dealt to workgroups, partial results per workgroup.
//  * latent_values_kernel: merge, value product and output gate.
#include "elem.h"

namespace {

constexpr int kLatThreads = 256;
constexpr float kLatLog2e = 1.4426950408889634f;

int round8(int n) { return (n + 7) & ~7; }
__device__ __forceinline__ int round8d(int n) { return (n + 7) & ~7; }

__device__ __forceinline__ float load_in(const socket_latent& a, int64_t i) {
  return a.in_f32 ? ((const float*)a.in)[i] : bf16_bits_to_f32(((const uint16_t*)a.in)[i]);
}

// The cache row of token (b, t), by the whole workgroup.
template <class DT>
__device__ __forceinline__ void cache_row(const socket_latent& a, int b, int t, float* red) {
  const int64_t p = a.pos ? *a.pos : a.pos0 + t;
  if (p < 0 || p >= a.n_pos) return;                    // (uniform)
  const int64_t row = b * a.in_stride_b + t * a.in_stride_t;
  const int64_t dst = b * a.cache_stride_b + p * a.cache_stride_t;
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.rank; i += kLatThreads) {
    const float x = load_in(a, row + a.c_off + i);
    ss = fmaf(x, x, ss);
  }
  const float rs = rsqrt_f32(block_sum(ss, red) / (float)a.rank + a.eps);
  const int rank_p = round8d(a.rank), rot_p = round8d(a.rot), half = a.rot / 2;
  for (int i = threadIdx.x; i < rank_p; i += kLatThreads)
    store_elem<DT>(a.cache, dst + i, i < a.rank ? load_in(a, row + a.c_off + i) * rs * a.c_norm[i] : 0.f);
  for (int i = threadIdx.x; i < rot_p; i += kLatThreads) {
    float y = 0.f;
    if (i < a.rot) {
      const int pair = i < half ? i : i - half;
      const float u = load_in(a, row + a.rot_off + pair), v = load_in(a, row + a.rot_off + pair + half);
      const float2 f = *reinterpret_cast<const float2*>(a.cos_sin + (p * half + pair) * 2);
      y = i < half ? fmaf(u, f.x, -(v * f.y)) : fmaf(v, f.x, u * f.y);
    }
    store_elem<DT>(a.cache, dst + rank_p + i, y);
  }
}

template <class DT>
__global__ __launch_bounds__(kLatThreads) void latent_rows_kernel(socket_latent a) {
  __shared__ float red[2][4];
  const int t = blockIdx.x, b = blockIdx.y;
  if (a.cq_out) {
    const int64_t src = b * a.in_stride_b + t * a.in_stride_t + a.cq_off, dst = ((int64_t)b * a.T + t) * a.q_rank;
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.q_rank; i += kLatThreads) {
      const float x = load_in(a, src + i);
      ss = fmaf(x, x, ss);
    }
    const float rs = rsqrt_f32(block_sum(ss, red[0]) / (float)a.q_rank + a.eps);
    for (int i = threadIdx.x; i < a.q_rank; i += kLatThreads) store_elem<DT>(a.cq_out, dst + i, load_in(a, src + i) * rs * a.q_norm[i]);
  }
  cache_row<DT>(a, b, t, red[1]);
}

template <class DT>
__global__ __launch_bounds__(256) void rotate_tail_kernel(void* q, int T, int H, int dim, int rot, const float* cos_sin,
                                                          int64_t pos0, int64_t items) {
  const int64_t w = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (w >= items) return;
  const int half = rot / 2, pair = (int)(w % half);
  const int64_t head = w / half, t = head / H % T;
  const int64_t at = head * (dim + rot) + dim + pair;
  const float u = load_elem<DT>(q, at), v = load_elem<DT>(q, at + half);
  const float2 f = *reinterpret_cast<const float2*>(cos_sin + ((pos0 + t) * half + pair) * 2);
  store_elem<DT>(q, at, fmaf(u, f.x, -(v * f.y)));
  store_elem<DT>(q, at + half, fmaf(v, f.x, u * f.y));
}

// ---- query side of a step ---------------------------------------------------------------------
//
// Grid (rank in slices of 64 columns, then one workgroup for what is not a product; heads; tokens).
// 8 lanes of 8 columns side by side, 32 groups of lanes down the head's rows of w_uk.
constexpr int kAbsCols = 64, kAbsGroups = kLatThreads / 8, kAbsRows = 4;

template <class DT, bool VEC>
__global__ __launch_bounds__(kLatThreads) void latent_absorb_kernel(socket_latent a) {
  __shared__ __attribute__((aligned(16))) float part[kAbsGroups][kAbsCols + 4];
  __shared__ float red[4];
  const int tid = threadIdx.x, h = blockIdx.y, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank), rot_p = round8d(a.rot), width = rank_p + rot_p;
  const float* q = a.q + ((int64_t)blockIdx.z * a.H + h) * (a.dim + a.rot);
  const int64_t dst = ((int64_t)blockIdx.z * a.H + h) * width;
  if (blockIdx.x == gridDim.x - 1) {
    const int64_t p0 = a.pos ? *a.pos : a.pos0 + t;
    const int64_t p = p0 < 0 ? 0 : (p0 >= a.n_pos ? a.n_pos - 1 : p0);
    const int half = a.rot / 2;
    for (int i = tid; i < rot_p; i += kLatThreads) {
      float y = 0.f;
      if (i < a.rot) {
        const int pair = i < half ? i : i - half;
        const float u = q[a.dim + pair], v = q[a.dim + pair + half];
        const float2 f = *reinterpret_cast<const float2*>(a.cos_sin + (p * half + pair) * 2);
        y = i < half ? fmaf(u, f.x, -(v * f.y)) : fmaf(v, f.x, u * f.y);
      }
      store_elem<DT>(a.q_lat, dst + rank_p + i, y);
    }
    if (a.append && h == 0) cache_row<DT>(a, b, t, red);
    return;
  }
  const int c0 = blockIdx.x * kAbsCols, lane8 = tid & 7, grp = tid >> 3, c = c0 + lane8 * 8;
  float acc[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) acc[e] = 0.f;
  const int64_t w0 = (int64_t)h * a.dim * a.rank;
  for (int d0 = 0; d0 < a.dim; d0 += kAbsGroups * kAbsRows) {
    float w[kAbsRows][8], x[kAbsRows];
#pragma unroll
    for (int i = 0; i < kAbsRows; ++i) {
      const int d = d0 + i * kAbsGroups + grp;
#pragma unroll
      for (int e = 0; e < 8; ++e) w[i][e] = 0.f;
      x[i] = 0.f;
      if (d < a.dim) {
        x[i] = q[d];
        if constexpr (VEC) {
          if (c < a.rank) load_vec<DT, 8>(a.w_uk, w0 + (int64_t)d * a.rank + c, w[i]);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (c + e < a.rank) w[i][e] = load_elem<DT>(a.w_uk, w0 + (int64_t)d * a.rank + c + e);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < kAbsRows; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = fmaf(x[i], w[i][e], acc[e]);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) part[grp][lane8 * 8 + e] = acc[e];
  __syncthreads();
  if (tid < kAbsCols && c0 + tid < rank_p) {
    float s = 0.f;
#pragma unroll
    for (int g = 0; g < kAbsGroups; ++g) s += part[g][tid];
    store_elem<DT>(a.q_lat, dst + c0 + tid, s);          // (columns past the rank: zero)
  }
}

// ---- attention over the cache rows ------------------------------------------------------------
//
// A wave takes 16 keys at a time (tiles dealt round the launch's waves) and 16 heads, and keeps its
// own running maximum; nothing is shared until the end.  Keys go from memory straight into
// the registers that are the first product's operand, S^T[key, head] = K Q^T (16x16x32), and from
// there into the wave's own LDS rows, of which the second, O^T[dim, head] = V^T P^T (16x16x16),
// needs columns: a lane reads 8 neighbouring dims of four keys and so feeds eight accumulators,
// accumulator i holding dims 8 m + i of a block of 128.  The weights a lane computes are the
// operand it has to supply; they enter as a sum of two bf16 numbers.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 la_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(short)))) short la_s16x4;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float la_f32x4;

__device__ __forceinline__ la_f32x4 mfma_k32(const uint4& x, const uint4& y, la_f32x4 c) {
  union {
    uint4 u;
    la_bf16x8 v;
  } a, b;
  a.u = x;
  b.u = y;
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ la_f32x4 mfma_k16(const uint2& x, const uint2& y, la_f32x4 c) {
  union {
    uint2 u;
    la_s16x4 v;
  } a, b;
  a.u = x;
  b.u = y;
  return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pack2(float lo, float hi) {
  return (uint32_t)f32_to_bf16_bits(lo) | ((uint32_t)f32_to_bf16_bits(hi) << 16);
}
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

constexpr int kAttWaves = 4;

template <int KS>
constexpr int att_pitch() { return KS * 32 + 8; }      // elements of an LDS row

template <int KS, int NV>
__global__ __launch_bounds__(kAttWaves * 64, 1) void latent_attend_kernel(socket_latent_attention a) {
  constexpr int PITCH = att_pitch<KS>();
  static_assert(KS * 32 >= NV * 128, "values are a prefix of the keys");
  extern __shared__ __attribute__((aligned(16))) uint16_t la_lds[];
  __shared__ float sm[kAttWaves][16], sl[kAttWaves][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int x16 = lane & 15, quarter = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank), width = rank_p + round8d(a.rot);
  const int64_t p = (a.pos ? *a.pos : a.pos0) + t;
  const int len = (int)(p < 0 ? 0 : (p >= a.n_pos ? a.n_pos : p + 1));
  const int n_tiles = (len + 15) / 16, stride = a.splits * kAttWaves;
  uint16_t* mine = la_lds + wave * 16 * PITCH;

  uint4 qf[KS], kr[KS];
  const bool head_ok = h0 + x16 < a.H;
  const uint16_t* q = (const uint16_t*)a.q_lat + ((int64_t)blockIdx.z * a.H + (head_ok ? h0 + x16 : 0)) * width;
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int d = (4 * ks + quarter) * 8;
    qf[ks] = head_ok && d < width ? *reinterpret_cast<const uint4*>(q + d) : make_uint4(0, 0, 0, 0);
  }
  auto fetch = [&](int tile) __attribute__((always_inline)) {
    const int j = min(tile * 16 + x16, len - 1);
    const uint16_t* row = (const uint16_t*)a.cache + b * a.cache_stride_b + j * a.cache_stride_t;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = (4 * ks + quarter) * 8;
      kr[ks] = d < width ? *reinterpret_cast<const uint4*>(row + d) : make_uint4(0, 0, 0, 0);
    }
  };
  la_f32x4 o[NV * 8];
#pragma unroll
  for (int i = 0; i < NV * 8; ++i) o[i] = la_f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const float c1 = a.scale * kLatLog2e;
  int tile = split * kAttWaves + wave;
  if (tile < n_tiles) fetch(tile);
  for (; tile < n_tiles; tile += stride) {
    la_f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      s = mfma_k32(kr[ks], qf[ks], s);
      *reinterpret_cast<uint4*>(mine + x16 * PITCH + (4 * ks + quarter) * 8) = kr[ks];
    }
    if (tile + stride < n_tiles) fetch(tile + stride);
    float mb = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = tile * 16 + 4 * quarter + r;
      s[r] = j < len ? s[r] * c1 : -INFINITY;
      mb = fmaxf(mb, s[r]);
    }
    mb = fmaxf(mb, lane_xor16(mb));
    mb = fmaxf(mb, lane_xor32(mb));                     // (finite: a tile has a visible key)
    const float mn = fmaxf(m, mb), alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    l *= alpha;
    if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
      for (int i = 0; i < NV * 8; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[i][r] *= alpha;
    }
    float w[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      w[r] = __builtin_amdgcn_exp2f(s[r] - mn);
      l += w[r];
    }
    const uint2 ph = make_uint2(pack2(w[0], w[1]), pack2(w[2], w[3]));
    const uint2 pl = make_uint2(pack2(w[0] - __uint_as_float(ph.x << 16), w[1] - __uint_as_float(ph.x & 0xffff0000u)),
                                pack2(w[2] - __uint_as_float(ph.y << 16), w[3] - __uint_as_float(ph.y & 0xffff0000u)));
    wave_lds_fence();
#pragma unroll
    for (int nv = 0; nv < NV; ++nv) {
      uint4 v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = *reinterpret_cast<const uint4*>(mine + (4 * quarter + j) * PITCH + nv * 128 + x16 * 8);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const uint32_t sel = (i & 1) ? 0x07060302u : 0x05040100u;
        const uint2 f = make_uint2(__builtin_amdgcn_perm((&v[1].x)[i >> 1], (&v[0].x)[i >> 1], sel),
                                   __builtin_amdgcn_perm((&v[3].x)[i >> 1], (&v[2].x)[i >> 1], sel));
        o[nv * 8 + i] = mfma_k16(f, ph, o[nv * 8 + i]);
        o[nv * 8 + i] = mfma_k16(f, pl, o[nv * 8 + i]);
      }
    }
    wave_lds_fence();                                   // (the rows are rewritten by the next tile)
  }

  // ---- the workgroup's waves together
  l += lane_xor16(l);
  l += lane_xor32(l);
  if (quarter == 0) {
    sm[wave][x16] = m;
    sl[wave][x16] = l;
  }
  __syncthreads();
  float top = -INFINITY, sum = 0.f;
#pragma unroll
  for (int w = 0; w < kAttWaves; ++w) top = fmaxf(top, sm[w][x16]);
  const bool none = top == -INFINITY;
  if (!none)
#pragma unroll
    for (int w = 0; w < kAttWaves; ++w) sum += sl[w][x16] * __builtin_amdgcn_exp2f(sm[w][x16] - top);
  const float f = none ? 0.f : __builtin_amdgcn_exp2f(m - top);
  float* acc = reinterpret_cast<float*>(la_lds);        // [16][rank_p]
  for (int w = 0; w < kAttWaves; ++w) {
    if (wave == w) {
#pragma unroll
      for (int nv = 0; nv < NV; ++nv)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = nv * 128 + 8 * (4 * quarter + r);
          if (d < rank_p) {
            float* at = acc + x16 * rank_p + d;
            float4 lo = make_float4(o[nv * 8][r] * f, o[nv * 8 + 1][r] * f, o[nv * 8 + 2][r] * f, o[nv * 8 + 3][r] * f);
            float4 hi = make_float4(o[nv * 8 + 4][r] * f, o[nv * 8 + 5][r] * f, o[nv * 8 + 6][r] * f, o[nv * 8 + 7][r] * f);
            if (w > 0) {
              const float4 pl = *reinterpret_cast<const float4*>(at), ph = *reinterpret_cast<const float4*>(at + 4);
              lo = make_float4(lo.x + pl.x, lo.y + pl.y, lo.z + pl.z, lo.w + pl.w);
              hi = make_float4(hi.x + ph.x, hi.y + ph.y, hi.z + ph.z, hi.w + ph.w);
            }
            *reinterpret_cast<float4*>(at) = lo;
            *reinterpret_cast<float4*>(at + 4) = hi;
          }
        }
    }
    __syncthreads();
  }
  const int64_t part = ((int64_t)blockIdx.z * a.splits + split) * a.H + h0;
  const int heads = min(16, a.H - h0);
  for (int i = threadIdx.x * 4; i < heads * rank_p; i += kAttWaves * 256)
    *reinterpret_cast<float4*>(a.o + part * rank_p + i) = *reinterpret_cast<const float4*>(acc + i);
  if (wave == 0 && quarter == 0 && head_ok) {
    a.ml[(part + x16) * 2] = top;
    a.ml[(part + x16) * 2 + 1] = sum;
  }
}

// ---- value side of a step -----------------------------------------------------------------------
//
// Grid (rows of w_uv in slices of 16, heads, tokens).  The first weights are requested before the
// partial results are merged.
constexpr int kValRows = 4;               // per wave
constexpr int kMaxSplits = 256;

template <class DT, bool VEC>
__global__ __launch_bounds__(kLatThreads) void latent_values_kernel(socket_latent_attention a) {
  extern __shared__ __attribute__((aligned(16))) float lv_lds[];   // rank_p
  __shared__ float share[kMaxSplits];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.y, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank);
  const int d0 = (blockIdx.x * (kLatThreads / 64) + wave) * kValRows;
  const int64_t w0 = ((int64_t)h * a.vdim + d0) * a.rank;
  float w[kValRows][8];
  auto request = [&](int c) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kValRows; ++i) {
#pragma unroll
      for (int e = 0; e < 8; ++e) w[i][e] = 0.f;
      if (d0 + i < a.vdim) {
        if constexpr (VEC) {
          if (c < a.rank) load_vec<DT, 8>(a.w_uv, w0 + (int64_t)i * a.rank + c, w[i]);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (c + e < a.rank) w[i][e] = load_elem<DT>(a.w_uv, w0 + (int64_t)i * a.rank + c + e);
        }
      }
    }
  };
  request(lane * 8);
  float gate = 0.f;
  const int64_t g0 = b * a.gate_stride_b + t * a.gate_stride_t + (int64_t)h * a.vdim;
  if (a.gate && lane < kValRows && d0 + lane < a.vdim)
    gate = a.gate_f32 ? ((const float*)a.gate)[g0 + d0 + lane] : load_elem<DT>(a.gate, g0 + d0 + lane);
  const int64_t part = (int64_t)blockIdx.z * a.splits * a.H + h;
  if (a.ml) {
    // (a.splits <= 256: a lane per split)
    __shared__ float red[4], red2[4];
    const float m = tid < a.splits ? a.ml[(part + (int64_t)tid * a.H) * 2] : -INFINITY;
    const float l = tid < a.splits ? a.ml[(part + (int64_t)tid * a.H) * 2 + 1] : 0.f;
    const float mw = wave_reduce_to_last<true>(m);
    if (lane == 63) red[wave] = mw;
    __syncthreads();
    const float top = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float f = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - top);
    const float total = block_sum(l * f, red2);
    if (tid < a.splits) share[tid] = total > 0.f ? f / total : 0.f;
    __syncthreads();
  } else {
    if (tid == 0) share[0] = 1.f;
    __syncthreads();
  }
  for (int c = tid * 2; c < rank_p; c += kLatThreads * 2) {
    float2 s = make_float2(0.f, 0.f);
#pragma unroll 8
    for (int k = 0; k < a.splits; ++k) {
      const float2 v = *reinterpret_cast<const float2*>(a.o + (part + (int64_t)k * a.H) * rank_p + c);
      const float f = share[k];
      s.x = f > 0.f ? fmaf(f, v.x, s.x) : s.x;          // (an empty split's values are not read into the sum)
      s.y = f > 0.f ? fmaf(f, v.y, s.y) : s.y;
    }
    *reinterpret_cast<float2*>(lv_lds + c) = s;
  }
  __syncthreads();
  float acc[kValRows];
#pragma unroll
  for (int i = 0; i < kValRows; ++i) acc[i] = 0.f;
  for (int c0 = 0; c0 < a.rank; c0 += 512) {
    const int c = c0 + lane * 8;
    if (c0 > 0) request(c);
    float x[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = 0.f;
    if (c < rank_p) load_vec<DType_f32, 8>(lv_lds, c, x);
#pragma unroll
    for (int i = 0; i < kValRows; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[i] = fmaf(w[i][e], x[e], acc[i]);
  }
#pragma unroll
  for (int i = 0; i < kValRows; ++i) acc[i] = group_sum<64>(acc[i]);
  if (lane < kValRows && d0 + lane < a.vdim) {
    float y = acc[0];
#pragma unroll
    for (int i = 1; i < kValRows; ++i) y = lane == i ? acc[i] : y;
    if (a.gate) y *= sigmoid_f32(gate);
    store_elem<DT>(a.out, ((int64_t)blockIdx.z * a.H + h) * a.vdim + d0 + lane, y);
  }
}

int check_latent(const socket_latent* p) {
  SOCKET_REQUIRE(p && p->cos_sin, SOCKET_ERR_NULL);
  const socket_latent& a = *p;
  SOCKET_REQUIRE(a.dtype == SOCKET_F32 || a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.dtype == SOCKET_BF16 || a.in_f32, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.B <= 65535 && a.T > 0 && a.H > 0 && a.dim > 0 && a.rank > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.rot > 0 && a.rot % 2 == 0 && a.n_pos > 0 && (!a.pos || a.T == 1), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.pos || (a.pos0 >= 0 && a.pos0 + a.T <= a.n_pos), SOCKET_ERR_SHAPE);
  return SOCKET_OK;
}

template <int KS, int NV>
int launch_attend(const socket_latent_attention& a, hipStream_t s) {
  auto kern = latent_attend_kernel<KS, NV>;
  size_t lds = (size_t)kAttWaves * 16 * att_pitch<KS>() * 2;
  const size_t merge = (size_t)16 * round8(a.rank) * 4;
  if (merge > lds) lds = merge;
  if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return SOCKET_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3((unsigned)a.splits, (unsigned)((a.H + 15) / 16), (unsigned)(a.B * a.T)),
                     dim3(kAttWaves * 64), lds, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

}  // namespace

extern "C" int socket_latent_rows(const socket_latent* args, void* stream) {
  const int rc = check_latent(args);
  if (rc != SOCKET_OK) return rc;
  const socket_latent& a = *args;
  SOCKET_REQUIRE(a.in && a.cache && a.c_norm && (!a.cq_out || a.q_norm), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(!a.cq_out || a.q_rank > 0, SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)a.T, (unsigned)a.B), block(kLatThreads);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == SOCKET_F32) hipLaunchKernelGGL((latent_rows_kernel<DType_f32>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((latent_rows_kernel<DType_bf16>), grid, block, 0, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_rotate_tail(void* q, int dtype, int B, int T, int H, int dim, int rot, const float* cos_sin,
                                  int64_t n_pos, int64_t pos0, void* stream) {
  SOCKET_REQUIRE(q && cos_sin, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(dtype == SOCKET_F32 || dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(B > 0 && T > 0 && H > 0 && dim >= 0 && rot > 0 && rot % 2 == 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(pos0 >= 0 && pos0 + T <= n_pos, SOCKET_ERR_SHAPE);
  const int64_t items = (int64_t)B * T * H * (rot / 2);
  SOCKET_REQUIRE((items + 255) / 256 < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((items + 255) / 256)), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == SOCKET_F32) hipLaunchKernelGGL((rotate_tail_kernel<DType_f32>), grid, block, 0, s, q, T, H, dim, rot, cos_sin, pos0, items);
  else hipLaunchKernelGGL((rotate_tail_kernel<DType_bf16>), grid, block, 0, s, q, T, H, dim, rot, cos_sin, pos0, items);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_latent_absorb(const socket_latent* args, void* stream) {
  const int rc = check_latent(args);
  if (rc != SOCKET_OK) return rc;
  const socket_latent& a = *args;
  SOCKET_REQUIRE(a.q && a.w_uk && a.q_lat && (!a.append || (a.in && a.cache && a.c_norm)), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.H <= 65535 && (int64_t)a.B * a.T <= 65535, SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((a.rank + kAbsCols - 1) / kAbsCols + 1), (unsigned)a.H, (unsigned)(a.B * a.T)), block(kLatThreads);
  hipStream_t s = (hipStream_t)stream;
  const bool vec = a.rank % 8 == 0 && socket_aligned16(a.w_uk);
  if (a.dtype == SOCKET_F32) {
    if (vec) hipLaunchKernelGGL((latent_absorb_kernel<DType_f32, true>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((latent_absorb_kernel<DType_f32, false>), grid, block, 0, s, a);
  } else {
    if (vec) hipLaunchKernelGGL((latent_absorb_kernel<DType_bf16, true>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((latent_absorb_kernel<DType_bf16, false>), grid, block, 0, s, a);
  }
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_latent_attend(const socket_latent_attention* args, void* stream) {
  SOCKET_REQUIRE(args && args->q_lat && args->cache && args->o && args->ml, SOCKET_ERR_NULL);
  const socket_latent_attention& a = *args;
  SOCKET_REQUIRE(a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.T > 0 && a.H > 0 && a.rank > 0 && a.rot >= 0 && (!a.pos || a.T == 1), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE((int64_t)a.B * a.T <= 65535 && a.H <= 65535 * 16 && a.splits >= 1 && a.splits <= kMaxSplits, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.n_pos > 0 && a.n_pos < (1LL << 30) && (a.pos || (a.pos0 >= 0 && a.pos0 + a.T <= a.n_pos)), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.cache_stride_b % 8 == 0 && a.cache_stride_t % 8 == 0 && socket_aligned16(a.cache) &&
                 socket_aligned16(a.q_lat) && socket_aligned16(a.o), SOCKET_ERR_ALIGN);
  const int rank_p = round8(a.rank), width = rank_p + round8(a.rot);
  hipStream_t s = (hipStream_t)stream;
  if (rank_p <= 128 && width <= 128) return launch_attend<4, 1>(a, s);
  if (rank_p <= 128 && width <= 192) return launch_attend<6, 1>(a, s);
  if (rank_p <= 256 && width <= 320) return launch_attend<10, 2>(a, s);
  if (rank_p <= 512 && width <= 576) return launch_attend<18, 4>(a, s);
  if (rank_p <= 512 && width <= 640) return launch_attend<20, 4>(a, s);
  return SOCKET_ERR_UNSUPPORTED;
}

extern "C" int socket_latent_values(const socket_latent_attention* args, void* stream) {
  SOCKET_REQUIRE(args && args->o && args->w_uv && args->out, SOCKET_ERR_NULL);
  const socket_latent_attention& a = *args;
  SOCKET_REQUIRE(a.dtype == SOCKET_F32 || a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.T > 0 && a.H > 0 && a.H <= 65535 && a.rank > 0 && a.vdim > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE((int64_t)a.B * a.T <= 65535 && a.splits >= 1 && a.splits <= kMaxSplits && (a.ml || a.splits == 1), SOCKET_ERR_SHAPE);
  const int rank_p = round8(a.rank);
  SOCKET_REQUIRE((size_t)rank_p * 4 <= 40 * 1024, SOCKET_ERR_UNSUPPORTED);
  const int per_wg = kLatThreads / 64 * kValRows;
  const dim3 grid((unsigned)((a.vdim + per_wg - 1) / per_wg), (unsigned)a.H, (unsigned)(a.B * a.T)), block(kLatThreads);
  const size_t lds = (size_t)rank_p * 4;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = a.rank % 8 == 0 && socket_aligned16(a.w_uv);
  if (a.dtype == SOCKET_F32) {
    if (vec) hipLaunchKernelGGL((latent_values_kernel<DType_f32, true>), grid, block, lds, s, a);
    else hipLaunchKernelGGL((latent_values_kernel<DType_f32, false>), grid, block, lds, s, a);
  } else {
    if (vec) hipLaunchKernelGGL((latent_values_kernel<DType_bf16, true>), grid, block, lds, s, a);
    else hipLaunchKernelGGL((latent_values_kernel<DType_bf16, false>), grid, block, lds, s, a);
  }
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}
