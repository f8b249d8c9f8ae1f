// Row kernels of decoders whose residual stream is kept in fp32 and whose sublayer
// outputs are normalised before they are added to it:
//
//  * residual_norm_kernel: pending sublayer output -> its norm -> residual add -> average
//    with the results of earlier layers -> the next sublayer's norm, one launch per step
//    between two sublayers (the embedding lookup rides in the first).
//  * rows_linear_kernel: the matrix-vector products of a decode step, with that step
//    as an optional prologue, and a gated unit, a second scaled term, or the residual sum
//    and the average over depth as epilogue.
//  * gated_unit_kernel: the gated unit alone, for prompts.
#include "elem.h"

namespace {

constexpr int kRowThreads = 256;

// One row of the step described at socket_residual_norm by a workgroup of kRowThreads
// lanes.  `buf`: LDS, `dim` floats; a lane reads back only what it wrote itself.  V = 4
// (dim a multiple of 4) or 1.  emit(i, v): V normalised elements at column i.
template <class DT, int V, bool DEPTH, class Emit>
__device__ __forceinline__ void residual_row(const socket_residual& a, int64_t row, float* buf, float (*red)[4],
                                             bool store_x, Emit emit) {
  const int dim = a.dim;
  const int64_t base = row * dim;
  float rs_y = 1.f;
  if (a.a) {
    float ss = 0.f;
    for (int i = threadIdx.x * V; i < dim; i += kRowThreads * V) {
      float y[V];
      if (a.pending_f32) load_vec<DType_f32, V>(a.a, base + i, y);
      else load_vec<DT, V>(a.a, base + i, y);
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] *= a.scale_a;
      if (a.b) {
        float z[V];
        if (a.pending_f32) load_vec<DType_f32, V>(a.b, base + i, z);
        else load_vec<DT, V>(a.b, base + i, z);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] = fmaf(a.scale_b, z[e], y[e]);
      }
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf(y[e], y[e], ss);
      store_vec<DType_f32, V>(buf, i, y);
    }
    if (a.post_w) rs_y = rsqrt_f32(block_sum(ss, red[0]) / (float)dim + a.eps);
  }
  int64_t src = a.x_stride ? row * a.x_stride : base;
  if (!a.x) {
    int64_t id = a.ids64 ? ((const int64_t*)a.ids)[row] : (int64_t)((const int32_t*)a.ids)[row];
    id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
    src = id * dim;
  }
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < dim; i += kRowThreads * V) {
    float x[V];
    if (a.x) load_vec<DType_f32, V>(a.x, src + i, x);
    else {
      load_vec<DT, V>(a.embed, src + i, x);
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] *= a.embed_scale;
    }
    if (a.a) {
      float y[V];
      load_vec<DType_f32, V>(buf, i, y);
      if (a.post_w) {
        float w[V];
        load_vec<DType_f32, V>(a.post_w, i, w);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] = y[e] * rs_y * w[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] += y[e];
    }
    if constexpr (DEPTH) {
      const socket_depth_mix& d = a.depth;
      store_vec<DType_f32, V>(d.result, base + i, x);
      const float own = d.w[d.n];
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] *= own;
#pragma unroll 4
      for (int j = 0; j < d.n; ++j) {
        float p[V];
        load_vec<DType_f32, V>(d.past, j * d.past_stride + base + i, p);
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] = fmaf(d.w[j], p[e], x[e]);
      }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(x[e], x[e], ss);
    store_vec<DType_f32, V>(buf, i, x);
    if (store_x && a.x_out) store_vec<DType_f32, V>(a.x_out, base + i, x);
  }
  const float rs = rsqrt_f32(block_sum(ss, red[1]) / (float)dim + a.eps);
  for (int i = threadIdx.x * V; i < dim; i += kRowThreads * V) {
    float x[V], w[V];
    load_vec<DType_f32, V>(buf, i, x);
    load_vec<DType_f32, V>(a.pre_w, i, w);
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = x[e] * rs * w[e];
    emit(i, x);
  }
}

template <class DT, int V, bool DEPTH>
__global__ __launch_bounds__(kRowThreads) void residual_norm_kernel(socket_residual a) {
  extern __shared__ __attribute__((aligned(16))) float row_buf[];
  __shared__ float red[2][4];
  const int64_t row = blockIdx.x;
  residual_row<DT, V, DEPTH>(a, row, row_buf, red, true, [&](int i, const float* v) {
    if (a.h_out) store_vec<DT, V>(a.h_out, row * a.dim + i, v);
  });
}

__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f32(1.702f * g) * (u + 1.f);
}

__device__ __forceinline__ float gated_unit(int kind, float g, float u, float limit) {
  return kind == 1 ? clamped_glu(g, u, limit) : g * sigmoid_f32(g) * u;
}

template <class DT, int V>
__global__ __launch_bounds__(256) void gated_unit_kernel(const void* __restrict__ gu, void* __restrict__ out,
                                                         int64_t rows, int ff, int kind, float limit) {
  const int64_t per_row = ff / V;
  const int64_t t = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (t >= rows * per_row) return;
  const int64_t r = t / per_row, j = (t % per_row) * V;
  float g[V], u[V];
  load_vec<DT, V>(gu, r * 2 * ff + j, g);
  load_vec<DT, V>(gu, r * 2 * ff + ff + j, u);
#pragma unroll
  for (int e = 0; e < V; ++e) g[e] = gated_unit(kind, g[e], u[e], limit);
  store_vec<DT, V>(out, r * ff + j, g);
}

constexpr int kVec = 8;                    // weights per lane and load
constexpr int kDepth = 4;                  // loads in flight per matrix
constexpr int kChunkElems = 64 * kVec * kDepth;
constexpr int kWgPerCu = 4;                // workgroups per CU of the persistent (NORM) launch

typedef uint32_t rl_u32x4 __attribute__((ext_vector_type(4)));

// kDepth weight vectors of row n, elements [kc * kChunkElems, ...), zero past K (FULL: K is a
// multiple of kChunkElems, no element is past it).
template <bool FULL>
__device__ __forceinline__ void fetch_row(rl_u32x4 (&v)[kDepth], const uint16_t* w, int64_t n, int K, int kc, int lane) {
#pragma unroll
  for (int u = 0; u < kDepth; ++u) {
    const int k = kc * kChunkElems + (u * 64 + lane) * kVec;
    v[u] = (FULL || k < K) ? __builtin_nontemporal_load(reinterpret_cast<const rl_u32x4*>(w + n * K + k)) : rl_u32x4{0, 0, 0, 0};
  }
}

template <int M, bool FULL>
__device__ __forceinline__ void mul_chunk(float (&acc)[M], const rl_u32x4 (&v)[kDepth], const uint16_t* x, int64_t xs, int K,
                                          int kc, int lane) {
#pragma unroll
  for (int u = 0; u < kDepth; ++u) {
    const int k = kc * kChunkElems + (u * 64 + lane) * kVec;
    if (!FULL && k >= K) continue;
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const uint4 xv = *reinterpret_cast<const uint4*>(x + m * xs + k);
      const uint32_t xw[4] = {xv.x, xv.y, xv.z, xv.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        acc[m] = fmaf(__uint_as_float(v[u][i] << 16), __uint_as_float(xw[i] << 16), acc[m]);
        acc[m] = fmaf(__uint_as_float(v[u][i] & 0xffff0000u), __uint_as_float(xw[i] & 0xffff0000u), acc[m]);
      }
    }
  }
}

// One wave per output feature; wave g of the launch takes features g, g + waves, ...
// TWO: 0 one product, 1 the gated unit (w1 and w2 share the input row), 2 a second scaled
// product (x2 . w2).  NORM: the input row is residual_row's, in LDS (M rows of K1), and the
// launch is persistent so that few workgroups pay for it; the first weights are requested
// before it starts, and a wave's weight vectors run through two register buffers, so that
// it streams without a gap from its first row to its last.  RES: the residual sum and the
// average over depth in the epilogue; a wave takes one feature, whose earlier results its lanes
// gather (one each) before the weights arrive.
template <int M, bool NORM, int TWO, bool FULL, bool RES>
__global__ __launch_bounds__(kRowThreads) void rows_linear_kernel(socket_rows_linear a, socket_residual nrm) {
  extern __shared__ __attribute__((aligned(16))) float rl_lds[];
  __shared__ float red[2][4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int waves = gridDim.x * (kRowThreads / 64);
  int n = blockIdx.x * (kRowThreads / 64) + wave;   // (wave-uniform)
  const uint16_t* w1 = (const uint16_t*)a.w1;
  const uint16_t* w2 = (const uint16_t*)a.w2;
  const uint16_t* x1 = (const uint16_t*)a.x1;
  const uint16_t* x2 = TWO == 2 ? (const uint16_t*)a.x2 : x1;
  const int K1 = a.K1, K2 = TWO == 2 ? a.K2 : K1;
  const int nk1 = (K1 + kChunkElems - 1) / kChunkElems;
  const int nk = TWO == 2 ? nk1 + (K2 + kChunkElems - 1) / kChunkElems : nk1;
  rl_u32x4 wa[kDepth], ga[TWO == 1 ? kDepth : 1], wb[kDepth], gb[TWO == 1 ? kDepth : 1];
  float bias1 = 0.f, bias2 = 0.f;          // of the row whose first chunk was requested last
  auto fetch = [&](rl_u32x4 (&v)[kDepth], auto& g, int row, int kc) __attribute__((always_inline)) {
    if (kc == 0) {
      if (a.b1) bias1 = load_elem<DType_bf16>(a.b1, row);
      if (TWO == 1 && a.b2) bias2 = load_elem<DType_bf16>(a.b2, row);
    }
    if (TWO == 2 && kc >= nk1) fetch_row<FULL>(v, w2, row, K2, kc - nk1, lane);
    else fetch_row<FULL>(v, w1, row, K1, kc, lane);
    if constexpr (TWO == 1) fetch_row<FULL>(g, w2, row, K1, kc, lane);
  };
  if (n < a.N) fetch(wa, ga, n, 0);
  float before[M], mixed[M], own = 1.f;    // RES: the stream, this lane's share of the average
  if constexpr (RES) {
    const socket_depth_mix& d = a.depth;
    if (d.w) own = d.w[d.n];
#pragma unroll
    for (int m = 0; m < M; ++m) {
      before[m] = mixed[m] = 0.f;
      if (n >= a.N) continue;
      const int64_t at = (int64_t)m * a.N + n;
      before[m] = a.res[at];
      if (d.w)
        for (int j = lane; j < d.n; j += 64) mixed[m] = fmaf(d.w[j], d.past[j * d.past_stride + at], mixed[m]);
    }
  }
  if constexpr (NORM) {
    uint16_t* xs = reinterpret_cast<uint16_t*>(rl_lds + K1);
    for (int m = 0; m < M; ++m) {
      residual_row<DType_bf16, 4, false>(nrm, m, rl_lds, red, blockIdx.x == 0,
                                  [&](int i, const float* v) { store_vec<DType_bf16, 4>(xs, (int64_t)m * K1 + i, v); });
      __syncthreads();
    }
    x1 = x2 = xs;
  }
  float acc[M], acc2[M];
#pragma unroll
  for (int m = 0; m < M; ++m) acc[m] = acc2[m] = 0.f;
  int kc = 0;
  auto step = [&](rl_u32x4 (&cv)[kDepth], auto& cg, rl_u32x4 (&nv)[kDepth], auto& ng) __attribute__((always_inline)) {
    const bool row_ends = kc + 1 == nk;
    const int n2 = row_ends ? n + waves : n, kc2 = row_ends ? 0 : kc + 1;
    const float c1 = bias1, c2 = bias2;
    if (n2 < a.N) fetch(nv, ng, n2, kc2);
    if (TWO == 2 && kc >= nk1) mul_chunk<M, FULL>(acc2, cv, x2, K2, K2, kc - nk1, lane);
    else mul_chunk<M, FULL>(acc, cv, x1, K1, K1, kc, lane);
    if constexpr (TWO == 1) mul_chunk<M, FULL>(acc2, cg, x1, K1, K1, kc, lane);
    if (row_ends) {
#pragma unroll
      for (int m = 0; m < M; ++m) {
        float o = wave_reduce_to_last<false>(acc[m]);
        if (TWO) {
          const float o2 = wave_reduce_to_last<false>(acc2[m]);
          o = TWO == 1 ? gated_unit(a.kind, o + c1, o2 + c2, a.limit) : fmaf(a.s2, o2, a.s1 * o) + c1;
        } else {
          o = a.s1 * o + c1;
        }
        if constexpr (RES) {
          o += before[m];
          const float past = wave_reduce_to_last<false>(mixed[m]);
          if (lane == 63 && a.depth.w) a.depth.result[(int64_t)m * a.N + n] = o;
          o = fmaf(own, o, past);
        }
        if (lane == 63) {
          if (a.y_f32) ((float*)a.y)[(int64_t)m * a.N + n] = o;
          else ((uint16_t*)a.y)[(int64_t)m * a.N + n] = f32_to_bf16_bits(o);
        }
        acc[m] = acc2[m] = 0.f;
      }
    }
    n = n2;
    kc = kc2;
  };
  while (n < a.N) {
    step(wa, ga, wb, gb);
    if (n >= a.N) break;
    step(wb, gb, wa, ga);
  }
}

template <int M, bool NORM, int TWO, bool FULL, bool RES = false>
int launch_rows_linear(const socket_rows_linear& a, hipStream_t s) {
  const SocketDeviceLimits& lim = socket_device_limits();
  size_t lds = 0;
  int n_wg = (a.N + kRowThreads / 64 - 1) / (kRowThreads / 64);
  auto kern = rows_linear_kernel<M, NORM, TWO, FULL, RES>;
  socket_residual nrm{};
  if (NORM) {
    nrm = *a.norm;
    lds = (size_t)a.K1 * 4 + (size_t)M * a.K1 * 2;
    if (lds + 256 > (size_t)lim.max_lds_per_block) return SOCKET_ERR_UNSUPPORTED;
    if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return SOCKET_ERR_LAUNCH;
    n_wg = n_wg < lim.cu_count * kWgPerCu ? n_wg : lim.cu_count * kWgPerCu;
  }
  hipLaunchKernelGGL(kern, dim3((unsigned)n_wg), dim3(kRowThreads), lds, s, a, nrm);
  return SOCKET_OK;
}

template <int M, bool FULL>
int dispatch_form(const socket_rows_linear& a, hipStream_t s) {
  const int two = a.kind != 0 ? 1 : (a.x2 ? 2 : 0);
  if (a.res) return launch_rows_linear<M, false, 0, FULL, true>(a, s);
  if (a.norm) return two == 1 ? launch_rows_linear<M, true, 1, FULL>(a, s) : launch_rows_linear<M, true, 0, FULL>(a, s);
  if (two == 1) return launch_rows_linear<M, false, 1, FULL>(a, s);
  return two == 2 ? launch_rows_linear<M, false, 2, FULL>(a, s) : launch_rows_linear<M, false, 0, FULL>(a, s);
}

template <int M>
int dispatch_rows_linear(const socket_rows_linear& a, hipStream_t s) {
  const bool full = a.K1 % kChunkElems == 0 && (!a.x2 || a.K2 % kChunkElems == 0);
  return full ? dispatch_form<M, true>(a, s) : dispatch_form<M, false>(a, s);
}

int check_residual(const socket_residual* a) {
  SOCKET_REQUIRE(a && a->pre_w, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a->x || (a->embed && a->ids), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a->x || a->vocab > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a->a || !a->b, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(!a->depth.w || (a->depth.result && a->depth.n >= 0 && (a->depth.past || a->depth.n == 0)), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a->x_stride >= 0 && (a->x_stride == 0 || a->x_out != a->x), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a->dim > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a->dtype == SOCKET_F32 || a->dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  if (a->dim % 4 == 0) {
    const void* ptrs[] = {a->x, a->embed, a->a, a->b, a->post_w, a->pre_w, a->x_out, a->h_out};
    for (const void* p : ptrs) SOCKET_REQUIRE(p == nullptr || socket_aligned16(p), SOCKET_ERR_ALIGN);
    SOCKET_REQUIRE(a->x_stride % 4 == 0 && (!a->depth.w || (a->depth.past_stride % 4 == 0 && socket_aligned16(a->depth.past) &&
                                                            socket_aligned16(a->depth.result))), SOCKET_ERR_ALIGN);
  }
  return SOCKET_OK;
}

}  // namespace

extern "C" int socket_residual_norm(const socket_residual* args, int64_t rows, void* stream) {
  const int rc = check_residual(args);
  if (rc != SOCKET_OK) return rc;
  SOCKET_REQUIRE(rows > 0 && rows < (1LL << 31), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(args->dim <= 32768, SOCKET_ERR_UNSUPPORTED);
  const size_t lds = (size_t)args->dim * 4;
  hipStream_t s = (hipStream_t)stream;
#define SOCKET_RN(DT, V)                                                                                            \
  do {                                                                                                              \
    auto kern = args->depth.w ? residual_norm_kernel<DT, V, true> : residual_norm_kernel<DT, V, false>;                                                                        \
    if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),                                 \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
      return SOCKET_ERR_LAUNCH;                                                                                     \
    hipLaunchKernelGGL(kern, dim3((unsigned)rows), dim3(kRowThreads), lds, s, *args);                               \
  } while (0)
  const bool v4 = args->dim % 4 == 0;
  if (args->dtype == SOCKET_F32) {
    if (v4) SOCKET_RN(DType_f32, 4);
    else SOCKET_RN(DType_f32, 1);
  } else {
    if (v4) SOCKET_RN(DType_bf16, 4);
    else SOCKET_RN(DType_bf16, 1);
  }
#undef SOCKET_RN
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_rows_linear_bf16(const socket_rows_linear* args, void* stream) {
  SOCKET_REQUIRE(args && args->w1 && args->y, SOCKET_ERR_NULL);
  const socket_rows_linear& a = *args;
  SOCKET_REQUIRE(a.kind >= 0 && a.kind <= 2, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.M >= 1 && a.N >= 1 && a.K1 >= 1, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.M <= 4 && a.K1 % 8 == 0, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(socket_aligned16(a.w1) && (!a.w2 || socket_aligned16(a.w2)), SOCKET_ERR_ALIGN);
  SOCKET_REQUIRE(a.kind == 0 || a.w2, SOCKET_ERR_NULL);
  if (a.norm) {
    const int rc = check_residual(a.norm);
    if (rc != SOCKET_OK) return rc;
    SOCKET_REQUIRE(!a.x2 && !a.res && !a.norm->depth.w && a.norm->dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
    SOCKET_REQUIRE(a.norm->dim == a.K1 && (a.norm->x_out == nullptr || a.norm->x_out != a.norm->x), SOCKET_ERR_SHAPE);
  } else {
    SOCKET_REQUIRE(a.x1 != nullptr, SOCKET_ERR_NULL);
    SOCKET_REQUIRE(socket_aligned16(a.x1), SOCKET_ERR_ALIGN);
  }
  if (a.res) {
    SOCKET_REQUIRE(a.kind == 0 && !a.x2 && a.y_f32 && (const void*)a.res != a.y, SOCKET_ERR_UNSUPPORTED);
    SOCKET_REQUIRE(!a.depth.w || (a.depth.result && a.depth.n >= 0 && (a.depth.past || a.depth.n == 0)), SOCKET_ERR_NULL);
  }
  if (a.x2) {
    SOCKET_REQUIRE(a.w2 && a.kind == 0, SOCKET_ERR_NULL);
    SOCKET_REQUIRE(a.K2 >= 8 && a.K2 % 8 == 0, SOCKET_ERR_UNSUPPORTED);
    SOCKET_REQUIRE(socket_aligned16(a.x2), SOCKET_ERR_ALIGN);
  }
  hipStream_t s = (hipStream_t)stream;
  int rc;
  switch (a.M) {
    case 1: rc = dispatch_rows_linear<1>(a, s); break;
    case 2: rc = dispatch_rows_linear<2>(a, s); break;
    case 3: rc = dispatch_rows_linear<3>(a, s); break;
    default: rc = dispatch_rows_linear<4>(a, s); break;
  }
  if (rc != SOCKET_OK) return rc;
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_gated_unit(const void* gu, void* out, int dtype, int64_t rows, int ff, int kind, float limit,
                                 void* stream) {
  SOCKET_REQUIRE(gu && out, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(kind == 1 || kind == 2, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(dtype == SOCKET_F32 || dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(rows > 0 && ff > 0, SOCKET_ERR_SHAPE);
  const bool v8 = ff % 8 == 0 && socket_aligned16(gu) && socket_aligned16(out);
  const int64_t items = rows * (v8 ? ff / 8 : ff);
  SOCKET_REQUIRE((items + 255) / 256 < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((items + 255) / 256)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define SOCKET_CG(DT, V) hipLaunchKernelGGL((gated_unit_kernel<DT, V>), grid, block, 0, s, gu, out, rows, ff, kind, limit)
  if (dtype == SOCKET_F32) {
    if (v8) SOCKET_CG(DType_f32, 8);
    else SOCKET_CG(DType_f32, 1);
  } else {
    if (v8) SOCKET_CG(DType_bf16, 8);
    else SOCKET_CG(DType_bf16, 1);
  }
#undef SOCKET_CG
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}
