// Rotary embedding and attention inside chunks of the position axis, with an optional
// soft cap on the scores and keys that serve as values before their rotation.
//
// A query sees the keys of its own chunk only (chunks of `chunk` positions counted from
// position 0), so what a sequence has to keep is one ring of `chunk` rows per kv head:
// position p lives in slot p % chunk, and the visible keys of a decode step are the
// slots 0 .. p % chunk, a plain prefix.  A prompt portion reads the keys it brings from
// its own projections and older keys of its first chunk from the ring; the rows of its
// last chunk are stored into the ring after the attention has read it.  Full causal attention is
// the case of one endless chunk; values may be narrower or wider than keys, a second key segment
// may be shared by all heads, and the output may be gated.
#include "elem.h"

namespace {

// Work items of a token: V elements of the first rotated half of a head with the V that
// are paired with them, V elements of a head's unrotated rest, or V zeros of the padding.
template <class DT, int V>
__global__ __launch_bounds__(256) void rope_half_kernel(socket_rope_half a) {
  const int t = blockIdx.x, b = blockIdx.y;
  const int64_t p = a.pos ? *a.pos : a.pos0 + t;
  const bool ok = p >= 0 && p < a.n_pos;
  const int half = a.rot_dims / 2;
  const int pair_units = half / V, rest_units = (a.D - a.rot_dims) / V, units = pair_units + rest_units;
  const int heads = a.H + a.G;
  const int slot = (int)(ok ? p % a.chunk : 0);
  if (a.pos && a.ring_len && ok && threadIdx.x == 0 && blockIdx.z == 0) a.ring_len[b] = slot + 1;
  const int64_t row = b * a.proj_stride_b + t * a.proj_stride_t;
  const float* cs = a.cos_sin + (ok ? p : 0) * half * 2;
  for (int w = blockIdx.z * 256 + threadIdx.x; w < heads * units; w += gridDim.z * 256) {
    const int head = w / units, u = w % units;
    const bool is_q = head < a.H;
    const int g = head - a.H;
    const int64_t src = row + (is_q ? a.q_off + (int64_t)head * a.D : a.k_off + (int64_t)g * a.D);
    const bool pair = u < pair_units;
    const int d0 = pair ? u * V : a.rot_dims + (u - pair_units) * V;
    float x[V], y[V], rx[V], ry[V];
    load_vec<DT, V>(a.proj, src + d0, x);
#pragma unroll
    for (int e = 0; e < V; ++e) rx[e] = x[e];
    if (pair) {
      load_vec<DT, V>(a.proj, src + d0 + half, y);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float2 f = *reinterpret_cast<const float2*>(cs + (d0 + e) * 2);
        rx[e] = fmaf(x[e], f.x, -(y[e] * f.y));
        ry[e] = fmaf(y[e], f.x, x[e] * f.y);
      }
    }
    if (is_q) {
      const int64_t o = (((int64_t)b * a.T + t) * a.H + head) * a.q_pitch;
      store_vec<DT, V>(a.q_out, o + d0, rx);
      if (pair) store_vec<DT, V>(a.q_out, o + d0 + half, ry);
    } else if (!a.pos) {
      const int64_t o = (((int64_t)b * a.T + t) * a.G + g) * a.D;
      store_vec<DT, V>(a.k_out, o + d0, rx);
      if (pair) store_vec<DT, V>(a.k_out, o + d0 + half, ry);
    } else if (ok) {
      const int64_t o = b * a.ring_stride_b + g * a.ring_stride_g + slot * a.ring_stride_s;
      store_vec<DT, V>(a.k_ring, o + d0, rx);
      store_vec<DT, V>(a.v_ring, o + d0, x);
      if (pair) {
        store_vec<DT, V>(a.k_ring, o + d0 + half, ry);
        store_vec<DT, V>(a.v_ring, o + d0 + half, y);
      }
    }
  }
  if (a.q_pitch > a.D) {
    const int pad = a.q_pitch - a.D;
    for (int w = blockIdx.z * 256 + threadIdx.x; w < a.H * pad; w += gridDim.z * 256)
      store_elem<DT>(a.q_out, (((int64_t)b * a.T + t) * a.H + w / pad) * a.q_pitch + a.D + w % pad, 0.f);
  }
}

template <class DT, int V>
__global__ __launch_bounds__(256) void ring_store_kernel(const void* k, int64_t k_sb, int64_t k_st, int64_t k_sg,
                                                         const void* v, int64_t v_sb, int64_t v_st, int64_t v_sg,
                                                         void* k_ring, void* v_ring, int64_t r_sb, int64_t r_sg,
                                                         int64_t r_ss, int t_first, int G, int D, int chunk,
                                                         int64_t pos0) {
  const int t = t_first + blockIdx.x, b = blockIdx.y;
  const int slot = (int)((pos0 + t) % chunk);
  for (int w = threadIdx.x; w < G * (D / V); w += 256) {
    const int g = w / (D / V), d = w % (D / V) * V;
    float x[V];
    const int64_t o = b * r_sb + g * r_sg + slot * r_ss + d;
    load_vec<DT, V>(k, b * k_sb + t * k_st + g * k_sg + d, x);
    store_vec<DT, V>(k_ring, o, x);
    load_vec<DT, V>(v, b * v_sb + t * v_st + g * v_sg + d, x);
    store_vec<DT, V>(v_ring, o, x);
  }
}

// Where key j (position) of sequence b, kv head g lies: the portion's own rows from
// `fresh_from` on, the ring before that.
struct KeySource {
  const char *k_new, *v_new, *k_ring, *v_ring;   // of (b, g)
  int64_t k_st, v_st, r_ss;                      // bytes per token / slot
  int64_t fresh_from;
  int chunk;
  __device__ __forceinline__ const char* key(int64_t j) const {
    return j >= fresh_from ? k_new + (j - fresh_from) * k_st : k_ring + (j % chunk) * r_ss;
  }
  __device__ __forceinline__ const char* value(int64_t j) const {
    return j >= fresh_from ? v_new + (j - fresh_from) * v_st : v_ring + (j % chunk) * r_ss;
  }
};

template <class DT>
__device__ __forceinline__ KeySource key_source(const socket_chunk_attention& a, int b, int g, int64_t pos) {
  constexpr int es = sizeof(typename DT::storage);
  KeySource s;
  s.k_new = (const char*)a.k_new + (b * a.k_stride_b + g * a.k_stride_g) * es;
  s.v_new = (const char*)a.v_new + (b * a.v_stride_b + g * a.v_stride_g) * es;
  s.k_ring = (const char*)a.k_ring + (b * a.ring_stride_b + g * a.ring_stride_g) * es;
  s.v_ring = (const char*)a.v_ring + (b * a.ring_stride_b + g * a.ring_stride_g) * es;
  s.k_st = a.k_stride_t * es;
  s.v_st = a.v_stride_t * es;
  s.r_ss = a.ring_stride_s * es;
  s.fresh_from = a.pos ? pos + 1 : a.k_from;     // (a decode step's own key is in the ring already)
  s.chunk = a.chunk;
  return s;
}

// Any value width up to 1024, any type, all arithmetic fp32: one wave per query row.  A block of
// 64 keys, one key per lane for the scores; for the values a lane owns dims lane, lane + 64, ...
constexpr int kSimpleWaves = 4;
constexpr int kSimpleDims = 16;   // dims per lane

template <class DT>
__global__ __launch_bounds__(kSimpleWaves * 64) void chunk_attend_simple_kernel(socket_chunk_attention a) {
  extern __shared__ __attribute__((aligned(16))) float ca_lds[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t r = (int64_t)blockIdx.x * kSimpleWaves + wave;
  const int b = blockIdx.y;
  const bool live = r < (int64_t)a.T * a.H;        // (wave-uniform; no barrier below)
  if (!live) return;
  const int t = (int)(r / a.H), h = (int)(r % a.H), g = h / (a.H / a.G);
  const int Dq = a.D + a.D2, Dv = a.Dv;
  float* qs = ca_lds + wave * (Dq + 64);
  float* ps = qs + Dq;
  const int64_t i = a.pos ? *a.pos : a.pos0 + t;
  const KeySource src = key_source<DT>(a, b, g, i);
  const int64_t q0 = b * a.q_stride_b + t * a.q_stride_t + h * a.q_stride_h;
  for (int d = lane; d < Dq; d += 64) qs[d] = load_elem<DT>(a.q, q0 + d);
  float acc[kSimpleDims];
#pragma unroll
  for (int e = 0; e < kSimpleDims; ++e) acc[e] = 0.f;
  float m = -INFINITY, l = 0.f;
  __builtin_amdgcn_wave_barrier();
  if (i >= 0) {
    for (int64_t j0 = i / a.chunk * a.chunk; j0 <= i; j0 += 64) {
      const int64_t j = j0 + lane;
      float s = -INFINITY;
      if (j <= i) {
        const char* kp = src.key(j);
        s = 0.f;
        for (int d = 0; d < a.D; ++d) s = fmaf(qs[d], load_elem<DT>(kp, d), s);
        for (int d = 0; d < a.D2; ++d)
          s = fmaf(qs[a.D + d], load_elem<DT>(a.k2, b * a.k2_stride_b + j * a.k2_stride_t + d), s);
        s *= a.scale;
        if (a.softcap > 0.f) s = a.softcap * tanhf(s / a.softcap);
      }
      float mb = wave_reduce_to_last<true>(s);
      mb = __shfl(mb, 63, 64);
      const float mn = fmaxf(m, mb);
      const float alpha = expf(m - mn);            // (m = -inf on the first block: 0)
      const float p = j <= i ? expf(s - mn) : 0.f;
      l = l * alpha + p;                            // (per lane; summed at the end)
      m = mn;
      ps[lane] = p;
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int e = 0; e < kSimpleDims; ++e) acc[e] *= alpha;
      const int nj = (int)min((int64_t)64, i - j0 + 1);
      for (int jj = 0; jj < nj; ++jj) {
        const float pj = ps[jj];
        const char* vp = src.value(j0 + jj);
#pragma unroll
        for (int e = 0; e < kSimpleDims; ++e)
          if (lane + 64 * e < Dv) acc[e] = fmaf(pj, load_elem<DT>(vp, lane + 64 * e), acc[e]);
      }
      __builtin_amdgcn_wave_barrier();
    }
  }
  l = __shfl(wave_reduce_to_last<false>(l), 63, 64);
  const float inv = l > 0.f ? 1.f / l : 0.f;
  const int64_t o0 = (((int64_t)b * a.T + t) * a.H + h) * Dv;
  const int64_t g0 = b * a.gate_stride_b + t * a.gate_stride_t + (int64_t)h * Dv;
#pragma unroll
  for (int e = 0; e < kSimpleDims; ++e) {
    const int d = lane + 64 * e;
    if (d < Dv) store_elem<DT>(a.out, o0 + d, acc[e] * inv * (a.gate ? sigmoid_f32(load_elem<DT>(a.gate, g0 + d)) : 1.f));
  }
}

// ---- bf16 portions on the matrix cores --------------------------------------------------------
//
// A workgroup takes a tile of query rows of one kv head, the heads of its group packed next to
// each other (row r = token r / Gq, head r % Gq), so that a K / V tile in LDS serves them all.
// Both products are v_mfma_f32_16x16x32_bf16 in the transposed orientation (the query row is the
// N index: lane x holds row x % 16 in every accumulator):
//   S^T[key, row] = K . Q^T,   O^T[dim, row] = V^T . P^T
// so the weights a lane computes are the operand it has to supply.  V is transposed on its way
// into LDS: rows of NK + 8 elements, the 4-key groups of a row at group ^ (dim / 8 % (NK / 4)).
// Weights are computed in fp32 and enter the second product as a sum of two bf16 numbers.
//
// With a soft cap the scores are bounded by it, and exp(score) needs no running maximum
// while exp(+-cap) is far from the fp32 range (ONLINE = false): p = exp(cap tanh(s / cap)) with
// tanh(y) = 1 - 2 / (exp(2 y) + 1).
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 ca_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float ca_f32x4;

__device__ __forceinline__ ca_f32x4 mfma_bf16(const uint4& a, const uint4& b, ca_f32x4 c) {
  union {
    uint4 u;
    ca_bf16x8 v;
  } x, y;
  x.u = a;
  y.u = b;
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.v, y.v, c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pack_bf16x2(float lo, float hi) {
  typedef __bf16 bf2 __attribute__((ext_vector_type(2)));
  typedef float f2 __attribute__((ext_vector_type(2)));
  union {
    bf2 v;
    uint32_t u;
  } r;
  r.v = __builtin_convertvector(f2{lo, hi}, bf2);
  return r.u;
}

constexpr float kMaxOfflineCap = 60.f;   // exp(60) * 2^31 keys < 3.4e38, exp(-60) > 1.2e-38
constexpr float kLog2e = 1.4426950408889634f;

// DP: key dims (both segments), DVP: value dims, rounded up; SHARED: there is a second segment.
// NK: keys of a tile (32 where 64 would leave one wave per SIMD).
template <int DP, int DVP, int RW, int NK, bool ONLINE, bool SHARED>
__global__ __launch_bounds__(256, NK == 32 ? 2 : 1) void chunk_attend_mma_kernel(socket_chunk_attention a) {
  constexpr int CH = DP / 8;                 // 16-byte pieces per key
  constexpr int KS = DP / 32;
  constexpr int DB = DVP / 16;
  constexpr int KP = CH + 1;                 // pitch of a K row in pieces (odd: 16 rows hit 16 bank groups)
  constexpr int kVtPitch = NK + 8, GROUPS = NK / 4, NB = NK / 16;
  constexpr int TASKS = GROUPS * CH;             // (piece, four keys) per tile
  constexpr int PER = (TASKS + 255) / 256;
  constexpr int TASKS_V = GROUPS * (DVP / 8), PER_V = (TASKS_V + 255) / 256;
  constexpr int ROWS = 64 * RW;              // rows per workgroup
  __shared__ __attribute__((aligned(16))) uint4 k_lds[NK * KP];
  __shared__ __attribute__((aligned(16))) uint16_t vt_lds[DVP * kVtPitch];
  const int Dq = SHARED ? a.D + a.D2 : a.D, Dv = a.Dv;

  const int Gq = a.H / a.G;
  // kv heads are neighbours in the launch order: with eight of them each XCD's L2 serves one head's
  // keys.  Later tiles see more keys and come first.
  const int heads = a.G * a.B, tiles = gridDim.x / heads;
  const int hb = blockIdx.x % heads, tile = tiles - 1 - blockIdx.x / heads;
  const int g = hb % a.G, b = hb / a.G;
  const int64_t R = (int64_t)a.T * Gq, r0 = (int64_t)tile * ROWS;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int prow = lane & 15, quarter = lane >> 4;

  // (positions as 32-bit offsets from the first key of the tile's first chunk)
  const int64_t i_first = a.pos0 + r0 / Gq;
  const int64_t base = i_first / a.chunk * a.chunk;
  const int end = (int)(a.pos0 + min(r0 + ROWS - 1, R - 1) / Gq - base) + 1;   // keys [0, end)
  const KeySource src = key_source<DType_bf16>(a, b, g, 0);
  const int64_t wr0 = min(r0 + wave * 16 * RW, R - 1), wr1 = min(r0 + wave * 16 * RW + 16 * RW - 1, R - 1);
  const int iw0 = (int)(a.pos0 + wr0 / Gq - base), iw1 = (int)(a.pos0 + wr1 / Gq - base);
  const int cw0 = iw0 / a.chunk * a.chunk, cw1 = iw1 / a.chunk * a.chunk;      // (base is a chunk's start)
  const bool wave_live = r0 + wave * 16 * RW < R;

  uint4 qf[RW][KS];
  int row_i[RW], row_c[RW];                  // position and chunk start of the lane's rows; nothing visible: i < c
#pragma unroll
  for (int w = 0; w < RW; ++w) {
    const int64_t r = r0 + (wave * RW + w) * 16 + prow;
    const bool live = r < R;
    const int64_t t = (live ? r : 0) / Gq;
    row_i[w] = live ? (int)(a.pos0 + t - base) : -1;
    row_c[w] = live ? row_i[w] / a.chunk * a.chunk : 0;
    const uint16_t* q = (const uint16_t*)a.q + b * a.q_stride_b + t * a.q_stride_t +
                        (g * Gq + (live ? r : 0) % Gq) * a.q_stride_h;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = (4 * ks + quarter) * 8;
      qf[w][ks] = (live && d < Dq) ? *reinterpret_cast<const uint4*>(q + d) : make_uint4(0, 0, 0, 0);
    }
  }
  ca_f32x4 o[RW][DB];
  float l[RW], m[RW];
#pragma unroll
  for (int w = 0; w < RW; ++w) {
    l[w] = 0.f;
    m[w] = -INFINITY;
#pragma unroll
    for (int db = 0; db < DB; ++db) o[w][db] = ca_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float c1 = a.softcap > 0.f ? 2.f * kLog2e * a.scale / a.softcap : a.scale * kLog2e;
  const float c2 = a.softcap * kLog2e;

  uint4 kr[PER][4], vr[PER_V][4];
  const char* k2 = SHARED ? (const char*)a.k2 + b * a.k2_stride_b * 2 : nullptr;
  auto fetch = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int task = tid + p * 256, piece = task % CH, key0 = 4 * (task / CH);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        kr[p][i] = make_uint4(0, 0, 0, 0);
        if (p < PER_V) vr[p][i] = make_uint4(0, 0, 0, 0);
        const int64_t j = base + min(j0 + key0 + i, end - 1);   // (a live row past the end; masked below)
        if (task < TASKS && piece * 8 < Dq) {
          if (SHARED && piece * 8 >= a.D)
            kr[p][i] = *reinterpret_cast<const uint4*>(k2 + j * a.k2_stride_t * 2 + (piece * 8 - a.D) * 2);
          else
            kr[p][i] = *reinterpret_cast<const uint4*>(src.key(j) + piece * 16);
        }
        if (DVP == DP && task < TASKS && piece * 8 < Dv) vr[p][i] = *reinterpret_cast<const uint4*>(src.value(j) + piece * 16);
        if constexpr (DVP != DP) {
          const int vpiece = task % (DVP / 8), vkey0 = 4 * (task / (DVP / 8));
          const int64_t jv = base + min(j0 + vkey0 + i, end - 1);
          if (p < PER_V && task < TASKS_V && vpiece * 8 < Dv)
            vr[p][i] = *reinterpret_cast<const uint4*>(src.value(jv) + vpiece * 16);
        }
      }
    }
  };
  auto store = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int task = tid + p * 256;
      if (task < TASKS) {
        const int piece = task % CH, key0 = 4 * (task / CH);
#pragma unroll
        for (int i = 0; i < 4; ++i) k_lds[(key0 + i) * KP + piece] = kr[p][i];
      }
    }
#pragma unroll
    for (int p = 0; p < PER_V; ++p) {
      const int task = tid + p * 256, piece = task % (DVP / 8), key0 = 4 * (task / (DVP / 8));
      if (task >= TASKS_V) continue;
      const uint32_t w[4][4] = {{vr[p][0].x, vr[p][0].y, vr[p][0].z, vr[p][0].w},
                                {vr[p][1].x, vr[p][1].y, vr[p][1].z, vr[p][1].w},
                                {vr[p][2].x, vr[p][2].y, vr[p][2].z, vr[p][2].w},
                                {vr[p][3].x, vr[p][3].y, vr[p][3].z, vr[p][3].w}};
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const uint32_t sel = (e & 1) ? 0x07060302u : 0x05040100u;
        uint2 t;
        t.x = __builtin_amdgcn_perm(w[1][e >> 1], w[0][e >> 1], sel);
        t.y = __builtin_amdgcn_perm(w[3][e >> 1], w[2][e >> 1], sel);
        *reinterpret_cast<uint2*>(vt_lds + (piece * 8 + e) * kVtPitch + (((key0 >> 2) ^ (piece & (GROUPS - 1))) << 2)) = t;
      }
    }
  };

  fetch(0);
  for (int j0 = 0; j0 < end; j0 += NK) {
    __syncthreads();   // the previous tile has been consumed
    store();
    __syncthreads();
    if (j0 + NK < end) fetch(j0 + NK);
    if (!wave_live || j0 > iw1 || j0 + NK - 1 < cw0) continue;   // (wave-uniform)
    const bool open = j0 + NK - 1 <= iw0 && j0 >= cw1;

    ca_f32x4 s[RW][NB];
#pragma unroll
    for (int w = 0; w < RW; ++w)
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) s[w][nb] = ca_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) {
        const uint4 kf = k_lds[(nb * 16 + prow) * KP + 4 * ks + quarter];
#pragma unroll
        for (int w = 0; w < RW; ++w) s[w][nb] = mfma_bf16(kf, qf[w][ks], s[w][nb]);
      }
#pragma unroll
    for (int w = 0; w < RW; ++w) {
      // (ONLINE) scores in base-2 units, masked, and the rescale by the new maximum
      float shift = 0.f;
      if constexpr (ONLINE) {
        float mb = -INFINITY;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = j0 + nb * 16 + 4 * quarter + r;
            float x = s[w][nb][r] * c1;
            if (a.softcap > 0.f) x = c2 - 2.f * c2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(x) + 1.f);
            if (!open && !(j <= row_i[w] && j >= row_c[w])) x = -INFINITY;
            s[w][nb][r] = x;
            mb = fmaxf(mb, x);
          }
        mb = fmaxf(mb, lane_xor16(mb));
        mb = fmaxf(mb, lane_xor32(mb));
        const float mn = fmaxf(m[w], mb);
        const bool blind = mn == -INFINITY;
        const float alpha = blind ? 1.f : __builtin_amdgcn_exp2f(m[w] - mn);
        shift = blind ? 0.f : mn;
        m[w] = mn;
        l[w] *= alpha;
        if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
          for (int db = 0; db < DB; ++db)
#pragma unroll
            for (int r = 0; r < 4; ++r) o[w][db][r] *= alpha;
        }
      }
#pragma unroll
      for (int nb = 0; nb < NB; ++nb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float p;
          if constexpr (ONLINE) {
            p = __builtin_amdgcn_exp2f(s[w][nb][r] - shift);
          } else {
            const int j = j0 + nb * 16 + 4 * quarter + r;
            const float t = __builtin_amdgcn_exp2f(s[w][nb][r] * c1);
            p = __builtin_amdgcn_exp2f(fmaf(-2.f * c2, __builtin_amdgcn_rcpf(t + 1.f), c2));
            if (!open && !(j <= row_i[w] && j >= row_c[w])) p = 0.f;
          }
          s[w][nb][r] = p;
          l[w] += p;
        }
    }
#pragma unroll
    for (int c = 0; c < NB / 2; ++c) {
      uint4 ph[RW], pl[RW];   // slots 0..3: keys 32c + 4q + r, slots 4..7: keys 32c + 16 + 4q + r
#pragma unroll
      for (int w = 0; w < RW; ++w) {
        uint32_t* h = &ph[w].x;
        uint32_t* lo = &pl[w].x;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float x = s[w][2 * c + (i >> 1)][2 * (i & 1)], y = s[w][2 * c + (i >> 1)][2 * (i & 1) + 1];
          h[i] = pack_bf16x2(x, y);
          lo[i] = pack_bf16x2(x - __uint_as_float(h[i] << 16), y - __uint_as_float(h[i] & 0xffff0000u));
        }
      }
#pragma unroll
      for (int db = 0; db < DB; ++db) {
        const uint16_t* vrow = vt_lds + (db * 16 + prow) * kVtPitch;
        const int swz = (2 * db + (prow >> 3)) & (GROUPS - 1);
        const uint2 lo = *reinterpret_cast<const uint2*>(vrow + (((8 * c + quarter) ^ swz) << 2));
        const uint2 hi = *reinterpret_cast<const uint2*>(vrow + (((8 * c + 4 + quarter) ^ swz) << 2));
        const uint4 vf = make_uint4(lo.x, lo.y, hi.x, hi.y);
#pragma unroll
        for (int w = 0; w < RW; ++w) {
          o[w][db] = mfma_bf16(vf, ph[w], o[w][db]);
          o[w][db] = mfma_bf16(vf, pl[w], o[w][db]);
        }
      }
    }
  }
#pragma unroll
  for (int w = 0; w < RW; ++w) {
    float sum = l[w];
    sum += lane_xor16(sum);
    sum += lane_xor32(sum);
    const int64_t r = r0 + (wave * RW + w) * 16 + prow;
    if (r >= R) continue;
    const float inv = 1.f / sum;
    const int64_t t = r / Gq, h = g * Gq + r % Gq;
    uint16_t* out = (uint16_t*)a.out + (((int64_t)b * a.T + t) * a.H + h) * Dv;
    const int64_t g0 = b * a.gate_stride_b + t * a.gate_stride_t + h * Dv;
#pragma unroll
    for (int db = 0; db < DB; ++db) {
      const int d = db * 16 + 4 * quarter;
      if (SHARED && a.gate && d < Dv) {
        float gate[4];
        load_vec<DType_bf16, 4>(a.gate, g0 + d, gate);
#pragma unroll
        for (int r = 0; r < 4; ++r) o[w][db][r] *= sigmoid_f32(gate[r]);
      }
      if (d < Dv)
        *reinterpret_cast<uint2*>(out + d) = make_uint2(pack_bf16x2(o[w][db][0] * inv, o[w][db][1] * inv),
                                                        pack_bf16x2(o[w][db][2] * inv, o[w][db][3] * inv));
    }
  }
}

bool mma_fits(const socket_chunk_attention& a) {
  if (a.force_simple || a.pos || a.dtype != SOCKET_BF16 || a.D % 8 != 0 || a.D + a.D2 > 256) return false;
  if (a.k2 ? a.Dv > 256 || a.softcap > 0.f : a.Dv != a.D || a.gate) return false;
  if (a.Dv % 8 != 0 || a.D2 % 8 != 0) return false;
  const int64_t strides[] = {a.q_stride_b, a.q_stride_t, a.q_stride_h, a.k_stride_b, a.k_stride_t, a.k_stride_g,
                             a.v_stride_b, a.v_stride_t, a.v_stride_g, a.ring_stride_b, a.ring_stride_g, a.ring_stride_s,
                             a.k2_stride_b, a.k2_stride_t, a.gate_stride_b, a.gate_stride_t};
  for (int64_t st : strides)
    if (st % 8 != 0) return false;
  const void* ptrs[] = {a.q, a.k_new, a.v_new, a.k_ring, a.v_ring, a.out, a.k2, a.gate};
  for (const void* p : ptrs)
    if (!socket_aligned16(p)) return false;
  return a.chunk == INT32_MAX ? a.pos0 + a.T < (1LL << 30) : (int64_t)a.T + a.chunk < (1LL << 30);
}

template <int DP, int DVP, int RW, bool SHARED, int NK = 64>
int launch_mma(const socket_chunk_attention& a, hipStream_t s) {
  const int64_t rows = (int64_t)a.T * (a.H / a.G);
  const int64_t n = (rows + 64 * RW - 1) / (64 * RW) * a.G * a.B;
  SOCKET_REQUIRE(n < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)n), block(256);
  if constexpr (!SHARED) {
    if (a.softcap > 0.f && a.softcap <= kMaxOfflineCap) {
      hipLaunchKernelGGL((chunk_attend_mma_kernel<DP, DVP, RW, NK, false, false>), grid, block, 0, s, a);
      SOCKET_LAUNCH_CHECK();
      return SOCKET_OK;
    }
  }
  hipLaunchKernelGGL((chunk_attend_mma_kernel<DP, DVP, RW, NK, true, SHARED>), grid, block, 0, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

}  // namespace

extern "C" int socket_rope_half_rows(const socket_rope_half* args, void* stream) {
  SOCKET_REQUIRE(args && args->proj && args->q_out && (args->cos_sin || args->rot_dims == 0), SOCKET_ERR_NULL);
  const socket_rope_half& a = *args;
  SOCKET_REQUIRE(a.pos ? (a.k_ring && a.v_ring) : a.k_out != nullptr, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.dtype == SOCKET_F32 || a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.B <= 65535 && a.T > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.D > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.rot_dims >= 0 && a.rot_dims % 2 == 0 && a.rot_dims <= a.D && a.q_pitch >= a.D, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.chunk > 0 && a.n_pos > 0 && (!a.pos || a.T == 1), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.pos || (a.pos0 >= 0 && a.pos0 + a.T <= a.n_pos), SOCKET_ERR_SHAPE);
  const int per = a.dtype == SOCKET_F32 ? 4 : 8;
  const bool v8 = a.D % 8 == 0 && a.rot_dims % 16 == 0 && a.q_off % per == 0 && a.k_off % per == 0 &&
                  a.proj_stride_b % per == 0 && a.proj_stride_t % per == 0 && a.q_pitch % per == 0 &&
                  a.ring_stride_b % per == 0 && a.ring_stride_g % per == 0 && a.ring_stride_s % per == 0 &&
                  socket_aligned16(a.proj) && socket_aligned16(a.q_out) &&
                  (!a.k_out || socket_aligned16(a.k_out)) && (!a.k_ring || socket_aligned16(a.k_ring)) &&
                  (!a.v_ring || socket_aligned16(a.v_ring));
  const int items = (a.H + a.G) * (v8 ? (a.D - a.rot_dims / 2) / 8 : a.D - a.rot_dims / 2);
  int gz = a.T >= 64 ? 1 : (items + 255) / 256;
  if (gz > 64) gz = 64;
  const dim3 grid((unsigned)a.T, (unsigned)a.B, (unsigned)(gz < 1 ? 1 : gz)), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == SOCKET_F32) {
    if (v8) hipLaunchKernelGGL((rope_half_kernel<DType_f32, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((rope_half_kernel<DType_f32, 1>), grid, block, 0, s, a);
  } else {
    if (v8) hipLaunchKernelGGL((rope_half_kernel<DType_bf16, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((rope_half_kernel<DType_bf16, 1>), grid, block, 0, s, a);
  }
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_chunk_ring_store(const void* k, int64_t k_sb, int64_t k_st, int64_t k_sg, const void* v,
                                       int64_t v_sb, int64_t v_st, int64_t v_sg, void* k_ring, void* v_ring,
                                       int64_t ring_sb, int64_t ring_sg, int64_t ring_ss, int dtype, int B, int T,
                                       int G, int D, int chunk, int64_t pos0, void* stream) {
  SOCKET_REQUIRE(k && v && k_ring && v_ring, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(dtype == SOCKET_F32 || dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(B > 0 && B <= 65535 && T > 0 && G > 0 && D > 0 && chunk > 0 && pos0 >= 0, SOCKET_ERR_SHAPE);
  const int64_t last = pos0 + T - 1, first = last / chunk * chunk;
  const int t_first = first > pos0 ? (int)(first - pos0) : 0;
  const int per = dtype == SOCKET_F32 ? 4 : 8;
  const bool v8 = D % 8 == 0 && k_sb % per == 0 && k_st % per == 0 && k_sg % per == 0 && v_sb % per == 0 &&
                  v_st % per == 0 && v_sg % per == 0 && ring_sb % per == 0 && ring_sg % per == 0 && ring_ss % per == 0 &&
                  socket_aligned16(k) && socket_aligned16(v) && socket_aligned16(k_ring) && socket_aligned16(v_ring);
  const dim3 grid((unsigned)(T - t_first), (unsigned)B), block(256);
  hipStream_t s = (hipStream_t)stream;
#define SOCKET_RS(DT, V)                                                                                          \
  hipLaunchKernelGGL((ring_store_kernel<DT, V>), grid, block, 0, s, k, k_sb, k_st, k_sg, v, v_sb, v_st, v_sg, k_ring, \
                     v_ring, ring_sb, ring_sg, ring_ss, t_first, G, D, chunk, pos0)
  if (dtype == SOCKET_F32) {
    if (v8) SOCKET_RS(DType_f32, 8);
    else SOCKET_RS(DType_f32, 1);
  } else {
    if (v8) SOCKET_RS(DType_bf16, 8);
    else SOCKET_RS(DType_bf16, 1);
  }
#undef SOCKET_RS
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_chunk_attend(const socket_chunk_attention* args, void* stream) {
  SOCKET_REQUIRE(args && args->q && args->out, SOCKET_ERR_NULL);
  socket_chunk_attention a = *args;
  if (a.Dv == 0) a.Dv = a.D;
  SOCKET_REQUIRE((a.k_ring && a.v_ring) || (!a.pos && a.k_from == 0), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.pos || (a.k_from >= 0 && a.k_from <= a.pos0), SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.k2 ? (a.D2 > 0 && !a.pos && a.k_from == 0) : a.D2 == 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.Dv > 0 && (a.D + a.D2 + 64) * 4 * kSimpleWaves <= 48 * 1024, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.pos || (a.k_new && a.v_new), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.dtype == SOCKET_F32 || a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.B <= 65535 && a.T > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.chunk > 0 && (!a.pos || a.T == 1) && a.pos0 >= 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.D > 0 && a.Dv <= 64 * kSimpleDims, SOCKET_ERR_UNSUPPORTED);
  hipStream_t s = (hipStream_t)stream;
  if (mma_fits(a)) {
    if (a.k2) {
      const int dq = a.D + a.D2;
      if (dq <= 64 && a.Dv <= 64) return launch_mma<64, 64, 2, true>(a, s);
      if (dq <= 96 && a.Dv <= 96) return launch_mma<96, 96, 2, true>(a, s);
      if (dq <= 128 && a.Dv <= 128) return launch_mma<128, 128, 2, true, 32>(a, s);
      if (dq <= 192 && a.Dv <= 128) return launch_mma<192, 128, 2, true, 32>(a, s);
      return launch_mma<256, 256, 1, true, 32>(a, s);
    }
    if (a.D <= 32) return launch_mma<32, 32, 2, false>(a, s);
    if (a.D <= 64) return launch_mma<64, 64, 2, false>(a, s);
    if (a.D <= 96) return launch_mma<96, 96, 2, false>(a, s);
    if (a.D <= 128) return launch_mma<128, 128, 2, false>(a, s);
    if (a.D <= 192) return launch_mma<192, 192, 1, false>(a, s);
    return launch_mma<256, 256, 1, false>(a, s);
  }
  const int64_t rows = (int64_t)a.T * a.H;
  SOCKET_REQUIRE((rows + kSimpleWaves - 1) / kSimpleWaves < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((rows + kSimpleWaves - 1) / kSimpleWaves), (unsigned)a.B), block(kSimpleWaves * 64);
  const size_t lds = (size_t)kSimpleWaves * (a.D + a.D2 + 64) * 4;
  if (a.dtype == SOCKET_F32) hipLaunchKernelGGL((chunk_attend_simple_kernel<DType_f32>), grid, block, lds, s, a);
  else hipLaunchKernelGGL((chunk_attend_simple_kernel<DType_bf16>), grid, block, lds, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}
