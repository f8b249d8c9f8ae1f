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

// V neighbouring elements of a projected row.
template <int V>
__device__ __forceinline__ void load_in(const socket_latent& a, int64_t i, float* out) {
  if (a.in_f32) load_vec<DType_f32, V>(a.in, i, out);
  else load_vec<DType_bf16, V>(a.in, i, out);
}

// Element i of a rotate-half of `rot` elements at position p: x(k) gives the element before.
template <class X>
__device__ __forceinline__ float rotated(const float* cos_sin, int64_t p, int rot, int i, X x) {
  const int half = rot / 2, pair = i < half ? i : i - half;
  const float2 f = *reinterpret_cast<const float2*>(cos_sin + (p * half + pair) * 2);
  const float u = x(pair), v = x(pair + half);
  return i < half ? fmaf(u, f.x, -(v * f.y)) : fmaf(v, f.x, u * f.y);
}

// The cache row of token (b, t) and, with QUERY, its normed query latent, by a workgroup of N lanes.
template <class DT, int V, bool QUERY, int N>
__device__ __forceinline__ void project_row(const socket_latent& a, int b, int t, float (*red)[4]) {
  const int64_t p = a.pos ? *a.pos : a.pos0 + t;
  const bool ok = p >= 0 && p < a.n_pos;                // (uniform)
  const int64_t row = b * a.in_stride_b + t * a.in_stride_t;
  const int64_t dst = b * a.cache_stride_b + p * a.cache_stride_t, cq = ((int64_t)b * a.T + t) * a.q_rank;
  float sc = 0.f, sq = 0.f;
  for (int i = threadIdx.x * V; i < a.rank; i += N * V) {
    float x[V];
    load_in<V>(a, row + a.c_off + i, x);
#pragma unroll
    for (int e = 0; e < V; ++e) sc = fmaf(x[e], x[e], sc);
  }
  if constexpr (QUERY) {
    for (int i = threadIdx.x * V; i < a.q_rank; i += N * V) {
      float x[V];
      load_in<V>(a, row + a.cq_off + i, x);
#pragma unroll
      for (int e = 0; e < V; ++e) sq = fmaf(x[e], x[e], sq);
    }
  }
  const float rc = rsqrt_f32(block_sum(sc, red[0]) / (float)a.rank + a.eps);
  if constexpr (QUERY) {
    const float rq = rsqrt_f32(block_sum(sq, red[1]) / (float)a.q_rank + a.eps);
    for (int i = threadIdx.x * V; i < a.q_rank; i += N * V) {
      float x[V], w[V];
      load_in<V>(a, row + a.cq_off + i, x);
      load_vec<DType_f32, V>(a.q_norm, i, w);
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] = x[e] * rq * w[e];
      store_vec<DT, V>(a.cq_out, cq + i, x);
    }
  }
  if (!ok) return;
  const int rank_p = round8d(a.rank), rot_p = round8d(a.rot);
  for (int i = threadIdx.x * V; i < rank_p; i += N * V) {
    float x[V], w[V];
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = w[e] = 0.f;
    if (i < a.rank) {
      load_in<V>(a, row + a.c_off + i, x);
      load_vec<DType_f32, V>(a.c_norm, i, w);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = x[e] * rc * w[e];
    store_vec<DT, V>(a.cache, dst + i, x);
  }
  for (int i = N - 1 - threadIdx.x; i < rot_p; i += N) {          // (the lanes with the least to do so far)
    const float y = i < a.rot ? rotated(a.cos_sin, p, a.rot, i, [&](int k) {
      float x;
      load_in<1>(a, row + a.rot_off + k, &x);
      return x;
    }) : 0.f;
    store_elem<DT>(a.cache, dst + rank_p + i, y);
  }
}

template <class DT, int V>
__global__ __launch_bounds__(kLatThreads) void latent_rows_kernel(socket_latent a) {
  __shared__ float red[2][4];
  if (a.cq_out) project_row<DT, V, true, kLatThreads>(a, blockIdx.y, blockIdx.x, red);
  else project_row<DT, V, false, kLatThreads>(a, blockIdx.y, blockIdx.x, red);
}

// V pairs per lane.
template <class DT, int V>
__global__ __launch_bounds__(256) void rotate_tail_kernel(void* q, int T, int H, int dim, int rot, const float* cos_sin,
                                                          int64_t pos0, int64_t items) {
  const int64_t w = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (w >= items) return;
  const int half = rot / 2, units = half / V;
  const int64_t head = w / units, t = head / H % T;
  const int pair = (int)(w % units) * V;
  const int64_t at = head * (dim + rot) + dim + pair;
  float u[V], v[V], f[2 * V];
  load_vec<DT, V>(q, at, u);
  load_vec<DT, V>(q, at + half, v);
  const float* cs = cos_sin + ((pos0 + t) * half + pair) * 2;
  if constexpr (V == 8) {
    load_vec<DType_f32, 8>(cs, 0, f);
    load_vec<DType_f32, 8>(cs, 8, f + 8);
  } else {
    f[0] = cs[0];
    f[1] = cs[1];
  }
#pragma unroll
  for (int e = 0; e < V; ++e) {
    const float x = fmaf(u[e], f[2 * e], -(v[e] * f[2 * e + 1])), y = fmaf(v[e], f[2 * e], u[e] * f[2 * e + 1]);
    u[e] = x;
    v[e] = y;
  }
  store_vec<DT, V>(q, at, u);
  store_vec<DT, V>(q, at + half, v);
}

// ---- query side of a step ---------------------------------------------------------------------
//
// Grid (rank in slices of 64 columns, then one workgroup for what is not a product; heads; tokens).
// 8 lanes of 8 columns side by side, 32 groups of lanes down the head's rows of w_uk.
constexpr int kAbsCols = 64, kAbsGroups = kLatThreads / 8, kAbsRows = 4;

template <class DT, bool VEC>
__global__ __launch_bounds__(kLatThreads) void latent_absorb_kernel(socket_latent a) {
  __shared__ __attribute__((aligned(16))) float part[kAbsGroups][kAbsCols + 4];
  __shared__ float red[2][4];
  const int tid = threadIdx.x, h = blockIdx.y, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank), rot_p = round8d(a.rot), width = rank_p + rot_p;
  const float* q = a.q + ((int64_t)blockIdx.z * a.H + h) * (a.dim + a.rot);
  const int64_t dst = ((int64_t)blockIdx.z * a.H + h) * width;
  if (blockIdx.x == gridDim.x - 1) {
    const int64_t p0 = a.pos ? *a.pos : a.pos0 + t;
    const int64_t p = p0 < 0 ? 0 : (p0 >= a.n_pos ? a.n_pos - 1 : p0);
    for (int i = tid; i < rot_p; i += kLatThreads)
      store_elem<DT>(a.q_lat, dst + rank_p + i,
                     i < a.rot ? rotated(a.cos_sin, p, a.rot, i, [&](int k) { return q[a.dim + k]; }) : 0.f);
    if (a.append && h == 0) project_row<DT, 1, false, kLatThreads>(a, b, t, red);
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
// A workgroup takes tiles of 64 keys (dealt round the launch's workgroups) for 16 RT heads; the
// next tile's rows are in registers while a tile in LDS is worked on.  A wave has one 16-key
// subtile and 16 heads of the first product, S^T[key, head] = K Q^T; the waves agree on the
// tile's maxima and hand the weights on through LDS, each as a sum of two bf16 numbers; in the
// second, O^T[dim, head] = V^T P^T, a wave has 64 dims and every head and key.  That product's key
// rows are the columns of the LDS tile: a lane reads 4 neighbouring dims of eight keys and so feeds
// four accumulators, accumulator i holding dims 4 m + i of the wave's block.  The keys of a 32-key
// step are in the order the weights come in: slots 0 .. 3 are keys 4 quarter + r of the first
// subtile, slots 4 .. 7 those of the second.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 la_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float la_f32x4;

__device__ __forceinline__ la_f32x4 mfma_bf16(const uint4& x, const uint4& y, la_f32x4 c) {
  union {
    uint4 u;
    la_bf16x8 v;
  } a, b;
  a.u = x;
  b.u = y;
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pack2(float lo, float hi) {
  typedef __bf16 bf2 __attribute__((ext_vector_type(2)));
  typedef float f2 __attribute__((ext_vector_type(2)));
  union {
    bf2 v;
    uint32_t u;
  } r;
  r.v = __builtin_convertvector(f2{lo, hi}, bf2);
  return r.u;
}

constexpr int kAttThreads = 512, kAttWaves = kAttThreads / 64;
constexpr int kAttKeys = 64, kAttSub = kAttKeys / 16;
constexpr int kAttBlock = 64;             // dims of a wave in the second product

// KS: key dims in steps of 32; RT: heads in tiles of 16.
template <int KS, int RT>
__global__ __launch_bounds__(kAttThreads, 1) void latent_attend_kernel(socket_latent_attention a) {
  constexpr int PITCH = KS * 32 + 16;     // elements of an LDS row (four rows are half the banks apart)
  constexpr int PIECES = KS * 4, PER = kAttKeys * PIECES / kAttThreads;
  static_assert(KS % 2 == 0 && kAttKeys * PIECES % kAttThreads == 0 && RT * kAttSub <= kAttWaves, "work does not deal out");
  extern __shared__ __attribute__((aligned(16))) uint16_t la_lds[];        // kAttKeys x PITCH
  __shared__ uint2 ph[RT][kAttSub][64], pl[RT][kAttSub][64];
  __shared__ float top[RT][kAttSub][16], shrink[RT][16], sums[RT][kAttSub][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int x16 = lane & 15, quarter = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * 16 * RT, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank), width = rank_p + round8d(a.rot);
  const uint16_t* rows = (const uint16_t*)a.cache + b * a.cache_stride_b;

  // (the first rows are requested before the position is known: rows that are not visible become zero
  // on their way into LDS)
  uint4 kr[PER];
  auto fetch = [&](int tile) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = tid + i * kAttThreads, piece = at % PIECES;
      const int64_t j = min((int64_t)tile * kAttKeys + at / PIECES, a.n_pos - 1);
      kr[i] = piece * 8 < width ? *reinterpret_cast<const uint4*>(rows + j * a.cache_stride_t + piece * 8) : make_uint4(0, 0, 0, 0);
    }
  };
  fetch(split);
  const int rt = wave / kAttSub, sub = wave % kAttSub;
  const bool scores = rt < RT;
  uint4 qf[KS];
  {
    const int h = h0 + rt * 16 + x16;
    const bool live = scores && h < a.H;
    const uint16_t* q = (const uint16_t*)a.q_lat + ((int64_t)blockIdx.z * a.H + (live ? h : 0)) * width;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = (4 * ks + quarter) * 8;
      qf[ks] = live && d < width ? *reinterpret_cast<const uint4*>(q + d) : make_uint4(0, 0, 0, 0);
    }
  }
  const int64_t p = (a.pos ? *a.pos : a.pos0) + t;
  const int len = (int)(p < 0 ? 0 : (p >= a.n_pos ? a.n_pos : p + 1));
  const int n_tiles = (len + kAttKeys - 1) / kAttKeys;

  la_f32x4 o[RT][4];
#pragma unroll
  for (int r = 0; r < RT; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) o[r][i] = la_f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const float c1 = a.scale * kLatLog2e;
  const int d0 = wave * kAttBlock;
  const bool values = d0 < rank_p;
  for (int tile = split; tile < n_tiles; tile += a.splits) {
    __syncthreads();                                    // the previous tile has been consumed
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = tid + i * kAttThreads, key = at / PIECES;
      const bool seen = tile * kAttKeys + key < len;
      *reinterpret_cast<uint4*>(la_lds + key * PITCH + at % PIECES * 8) = seen ? kr[i] : make_uint4(0, 0, 0, 0);
    }
    __syncthreads();
    if (tile + a.splits < n_tiles) fetch(tile + a.splits);
    la_f32x4 s = {0.f, 0.f, 0.f, 0.f};
    if (scores) {
      const uint16_t* k = la_lds + (16 * sub + x16) * PITCH + quarter * 8;
      la_f32x4 s1 = {0.f, 0.f, 0.f, 0.f};                // (two sums: neighbouring products do not wait for each other)
#pragma unroll
      for (int ks = 0; ks < KS; ks += 2) {
        s = mfma_bf16(*reinterpret_cast<const uint4*>(k + ks * 32), qf[ks], s);
        s1 = mfma_bf16(*reinterpret_cast<const uint4*>(k + ks * 32 + 32), qf[ks + 1], s1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) s[r] += s1[r];
      float mb = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[r] = tile * kAttKeys + 16 * sub + 4 * quarter + r < len ? s[r] * c1 : -INFINITY;
        mb = fmaxf(mb, s[r]);
      }
      mb = fmaxf(mb, lane_xor16(mb));
      mb = fmaxf(mb, lane_xor32(mb));
      if (quarter == 0) top[rt][sub][x16] = mb;
    }
    __syncthreads();
    if (scores) {
      float mn = m;
#pragma unroll
      for (int i = 0; i < kAttSub; ++i) mn = fmaxf(mn, top[rt][i][x16]);   // (finite: a tile has a visible key)
      const float alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      l *= alpha;
      float w[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        w[r] = __builtin_amdgcn_exp2f(s[r] - mn);
        l += w[r];
      }
      const uint2 hi = make_uint2(pack2(w[0], w[1]), pack2(w[2], w[3]));
      ph[rt][sub][lane] = hi;
      pl[rt][sub][lane] = make_uint2(pack2(w[0] - __uint_as_float(hi.x << 16), w[1] - __uint_as_float(hi.x & 0xffff0000u)),
                                     pack2(w[2] - __uint_as_float(hi.y << 16), w[3] - __uint_as_float(hi.y & 0xffff0000u)));
      if (sub == 0 && quarter == 0) shrink[rt][x16] = alpha;
    }
    __syncthreads();
    if (values) {                                       // (wave-uniform)
#pragma unroll
      for (int r = 0; r < RT; ++r) {
        const float alpha = shrink[r][x16];
        if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[r][i][e] *= alpha;
        }
      }
#pragma unroll
      for (int c = 0; c < kAttSub / 2; ++c) {
        uint2 v[8];
#pragma unroll
        for (int k = 0; k < 8; ++k)
          v[k] = *reinterpret_cast<const uint2*>(la_lds + (32 * c + 16 * (k >> 2) + 4 * quarter + (k & 3)) * PITCH + d0 + x16 * 4);
        uint4 hi[RT], lo[RT];
#pragma unroll
        for (int r = 0; r < RT; ++r) {
          const uint2 h0_ = ph[r][2 * c][lane], h1 = ph[r][2 * c + 1][lane], l0 = pl[r][2 * c][lane], l1 = pl[r][2 * c + 1][lane];
          hi[r] = make_uint4(h0_.x, h0_.y, h1.x, h1.y);
          lo[r] = make_uint4(l0.x, l0.y, l1.x, l1.y);
        }
        uint4 f[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const uint32_t sel = (i & 1) ? 0x07060302u : 0x05040100u;
          uint32_t w[4];
#pragma unroll
          for (int k = 0; k < 4; ++k)
            w[k] = __builtin_amdgcn_perm(i < 2 ? v[2 * k + 1].x : v[2 * k + 1].y, i < 2 ? v[2 * k].x : v[2 * k].y, sel);
          f[i] = make_uint4(w[0], w[1], w[2], w[3]);
#pragma unroll
          for (int r = 0; r < RT; ++r) o[r][i] = mfma_bf16(f[i], hi[r], o[r][i]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int r = 0; r < RT; ++r) o[r][i] = mfma_bf16(f[i], lo[r], o[r][i]);
      }
    }
  }

  const int64_t part = ((int64_t)blockIdx.z * a.splits + split) * a.H + h0;
  if (values && split < n_tiles) {
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int d = d0 + 4 * (4 * quarter + e), h = r * 16 + x16;
        if (h0 + h < a.H && d < rank_p)
          *reinterpret_cast<float4*>(a.o + (part + h) * rank_p + d) = make_float4(o[r][0][e], o[r][1][e], o[r][2][e], o[r][3][e]);
      }
  }
  if (scores) {
    l += lane_xor16(l);
    l += lane_xor32(l);
    if (quarter == 0) sums[rt][sub][x16] = l;
  }
  __syncthreads();
  if (scores && sub == 0 && quarter == 0 && h0 + rt * 16 + x16 < a.H) {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < kAttSub; ++i) sum += sums[rt][i][x16];
    *reinterpret_cast<float2*>(a.ml + (part + rt * 16 + x16) * 2) = make_float2(m, sum);
  }
}

// ---- value side of a step -----------------------------------------------------------------------
//
// Grid (rows of w_uv in slices of 64, heads, tokens).  The first weights are requested before the
// partial results are merged, which eight groups of lanes share.
constexpr int kValThreads = 1024, kValWaves = kValThreads / 64;
constexpr int kValRows = 4;               // per wave
constexpr int kValGroups = 8, kValLanes = kValThreads / kValGroups;
constexpr int kMaxSplits = 256;
constexpr int kMaxMerge = 4 * kValLanes;  // widest row whose merge the groups share

template <class DT, bool VEC>
__global__ __launch_bounds__(kValThreads) void latent_values_kernel(socket_latent_attention a) {
  extern __shared__ __attribute__((aligned(16))) float lv_lds[];   // rank_p, then kValGroups x rank_p
  __shared__ float share[kMaxSplits], red[kValWaves], red2[kValWaves];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.y, b = blockIdx.z / a.T, t = blockIdx.z % a.T;
  const int rank_p = round8d(a.rank);
  const int d0 = (blockIdx.x * kValWaves + wave) * kValRows;
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
    float2 ml = make_float2(-INFINITY, 0.f);           // (a lane per split: at most 256)
    if (tid < a.splits) ml = *reinterpret_cast<const float2*>(a.ml + (part + (int64_t)tid * a.H) * 2);
    const float mw = wave_reduce_to_last<true>(ml.x);
    if (lane == 63) red[wave] = mw;
    __syncthreads();
    const float top = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float f = ml.x == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(ml.x - top);
    const float total = block_sum(ml.y * f, red2);
    if (tid < a.splits) share[tid] = total > 0.f ? f / total : 0.f;
    __syncthreads();
  } else {
    if (tid == 0) share[0] = 1.f;
    __syncthreads();
  }
  if (a.splits > 1 && rank_p <= kMaxMerge) {
    const int grp = tid / kValLanes, c = tid % kValLanes * 4;
    float* mine = lv_lds + (1 + grp) * rank_p;
    if (c < rank_p) {
      float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
      for (int k = grp; k < a.splits; k += kValGroups) {
        const float f = share[k];                       // (0: the split saw nothing and wrote nothing)
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (f > 0.f) v = *reinterpret_cast<const float4*>(a.o + (part + (int64_t)k * a.H) * rank_p + c);
        s = make_float4(fmaf(f, v.x, s.x), fmaf(f, v.y, s.y), fmaf(f, v.z, s.z), fmaf(f, v.w, s.w));
      }
      *reinterpret_cast<float4*>(mine + c) = s;
    }
    __syncthreads();
    if (tid < rank_p) {
      float s = 0.f;
#pragma unroll
      for (int g = 0; g < kValGroups; ++g) s += lv_lds[(1 + g) * rank_p + tid];
      lv_lds[tid] = s;
    }
  } else {
    for (int c = tid; c < rank_p; c += kValThreads) {
      float s = 0.f;
      for (int k = 0; k < a.splits; ++k)
        if (share[k] > 0.f) s = fmaf(share[k], a.o[(part + (int64_t)k * a.H) * rank_p + c], s);
      lv_lds[c] = s;
    }
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

template <int KS, int RT>
int launch_attend(const socket_latent_attention& a, hipStream_t s) {
  auto kern = latent_attend_kernel<KS, RT>;
  const size_t lds = (size_t)kAttKeys * (KS * 32 + 16) * 2;
  if (lds > 32 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return SOCKET_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3((unsigned)a.splits, (unsigned)((a.H + 16 * RT - 1) / (16 * RT)), (unsigned)(a.B * a.T)),
                     dim3(kAttThreads), lds, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

template <int KS>
int launch_attend_heads(const socket_latent_attention& a, hipStream_t s) {
  // (two tiles of heads per workgroup once there are more workgroups than CUs; neighbours share the L2 before)
  const int64_t wgs = (int64_t)a.splits * ((a.H + 15) / 16) * a.B * a.T;
  return a.H <= 16 || wgs <= socket_device_limits().cu_count ? launch_attend<KS, 1>(a, s) : launch_attend<KS, 2>(a, s);
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
  const bool vec = a.rank % 8 == 0 && a.c_off % 8 == 0 && a.in_stride_b % 8 == 0 && a.in_stride_t % 8 == 0 &&
                   a.cache_stride_b % 8 == 0 && a.cache_stride_t % 8 == 0 && socket_aligned16(a.in) && socket_aligned16(a.cache) &&
                   socket_aligned16(a.c_norm) &&
                   (!a.cq_out || (a.q_rank % 8 == 0 && a.cq_off % 8 == 0 && socket_aligned16(a.cq_out) && socket_aligned16(a.q_norm)));
  if (a.dtype == SOCKET_F32) {
    if (vec) hipLaunchKernelGGL((latent_rows_kernel<DType_f32, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((latent_rows_kernel<DType_f32, 1>), grid, block, 0, s, a);
  } else {
    if (vec) hipLaunchKernelGGL((latent_rows_kernel<DType_bf16, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((latent_rows_kernel<DType_bf16, 1>), grid, block, 0, s, a);
  }
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_rotate_tail(void* q, int dtype, int B, int T, int H, int dim, int rot, const float* cos_sin,
                                  int64_t n_pos, int64_t pos0, void* stream) {
  SOCKET_REQUIRE(q && cos_sin, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(dtype == SOCKET_F32 || dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(B > 0 && T > 0 && H > 0 && dim >= 0 && rot > 0 && rot % 2 == 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(pos0 >= 0 && pos0 + T <= n_pos, SOCKET_ERR_SHAPE);
  const bool v8 = dim % 8 == 0 && rot % 16 == 0 && socket_aligned16(q) && socket_aligned16(cos_sin);
  const int64_t items = (int64_t)B * T * H * (rot / 2) / (v8 ? 8 : 1);
  SOCKET_REQUIRE((items + 255) / 256 < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((items + 255) / 256)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define SOCKET_ROT(DT, V) hipLaunchKernelGGL((rotate_tail_kernel<DT, V>), grid, block, 0, s, q, T, H, dim, rot, cos_sin, pos0, items)
  if (dtype == SOCKET_F32) {
    if (v8) SOCKET_ROT(DType_f32, 8);
    else SOCKET_ROT(DType_f32, 1);
  } else {
    if (v8) SOCKET_ROT(DType_bf16, 8);
    else SOCKET_ROT(DType_bf16, 1);
  }
#undef SOCKET_ROT
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
  SOCKET_REQUIRE(rank_p <= kAttWaves * kAttBlock, SOCKET_ERR_UNSUPPORTED);
  if (width <= 128) return launch_attend_heads<4>(a, s);
  if (width <= 192) return launch_attend_heads<6>(a, s);
  if (width <= 320) return launch_attend_heads<10>(a, s);
  if (width <= 576) return launch_attend_heads<18>(a, s);
  if (width <= 640) return launch_attend_heads<20>(a, s);
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
  const int per_wg = kValWaves * kValRows;
  const dim3 grid((unsigned)((a.vdim + per_wg - 1) / per_wg), (unsigned)a.H, (unsigned)(a.B * a.T)), block(kValThreads);
  const size_t lds = (size_t)rank_p * 4 * (rank_p <= kMaxMerge ? 1 + kValGroups : 1);
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
