// Gated linear recurrences with a decay per head and key channel, with or without the
// delta rule, or with the generalized delta rule (the definition stands at socket_recurrence in socket_hip.h): one token per
// call for decoding, chunks of tokens on the matrix cores for prompts.  fp32 throughout;
// only the projected rows that come in and the gated rows that go out have the model's type.
//
// Chunk form.  Inside a chunk let b_t be the running sum of log g (per channel, <= 0) and
// S0 the state before the chunk.  Unrolling the recurrence,
//   o_t = (q_t e^{b_t})^T S0 + sum_{s <= t} Aqk[t,s] u_s,   Aqk[t,s] = sum_c q_tc k_sc e^{b_tc - b_sc}
//   u_t = beta_t (v_t - (k_t e^{b_t})^T S0 - sum_{s < t} Akk[t,s] u_s)     (delta rule)
//   S   = diag(e^{b_C}) S0 + sum_s (k_s e^{b_C - b_s}) u_s^T
// so with L = diag(beta) Akk (strictly lower), U = (I + L)^{-1} diag(beta) (V - K^ S0) = Ubar - W S0.
// Everything without S0 is worked out for all chunks at once (recurrence_prep_kernel); only
// U = Ubar - W S0, O = Q^ S0 + Aqk U and the update of S run in sequence over the chunks
// (recurrence_scan_kernel), independently per (sequence, head, 16 value columns).
//
// e^{b_t - b_s} must not be split as e^{b_t} e^{-b_s}: the second factor overflows under
// strong decay.  Tokens are grouped in blocks of 16 with sums pl local to the block and
// block totals tot; for s in an earlier block the exponent splits at the start of t's
// block into two parts that are both <= 0.  Inside a block the split at the block's
// start is used while its total stays above kMildDecay, else the exponent is taken per
// pair on the vector ALU.
//
// All products are v_mfma_f32_16x16x4_f32 (fp32 operands).  Its operands hold one k index
// per lane quarter; a step r of four takes k = 4 * quarter + r of a 16-wide tile, so that
// a lane's four values are one 16-byte vector ("fragment order": lane (quarter, x) holds row x,
// columns 4 quarter .. + 3 of a tile), and an accumulator (rows 4 quarter + r, column x) is
// directly the second operand of the next product.
#include "elem.h"

namespace {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float rc_f32x4;

__device__ __forceinline__ rc_f32x4 mfma4(const float4& a, const rc_f32x4& b, rc_f32x4 c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], c, 0, 0, 0);
  return c;
}

// ---- what both forms share: inputs of one (sequence, head) -------------------------------

constexpr float kRcLog2e = 1.4426950408889634f;

__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }   // v_exp_f32

// log2 of a channel's decay factor for z = low-rank product + bias; a_exp = exp(a_log[h]).
__device__ __forceinline__ float log2_decay(const socket_recurrence& a, float a_exp, float z) {
  if (a.decay_kind == 2) return -a.decay_rate * kRcLog2e * sigmoid_f32(z);
  const float f = a.decay_kind == 0 ? a_exp : a.inv_tau;
  return -f * kRcLog2e * softplus_f32(a.decay_kind == 0 ? z : -z);
}

__device__ __forceinline__ float gate_act(int kind, float x) {
  const float s = sigmoid_f32(x);
  return kind == 0 ? s : x * s;
}

__device__ __forceinline__ int conv_channels(const socket_recurrence& a) { return 2 * a.Hk * a.dk + a.H * a.dv; }

constexpr int kTapsAtOnce = 4;   // rows requested together

// q | k | v channel `ch` of token t (column `col` of the projected row), after the short
// convolution and its activation.  Rows before the portion come from half `parity` of the
// convolution state.  N channels at once, N = 1 or 8 (aligned).
template <class DT, int N>
__device__ __forceinline__ void conv_input(const socket_recurrence& a, int b, int t, int col, int ch, int parity,
                                           float* out) {
  const int64_t row = b * a.proj_stride_b + col;
  if (a.taps < 1) {
    load_vec<DT, N>(a.proj, row + t * a.proj_stride_t, out);
    return;
  }
  const int n1 = a.taps - 1, C = conv_channels(a);
#pragma unroll
  for (int e = 0; e < N; ++e) out[e] = 0.f;
  for (int m0 = 0; m0 < a.taps; m0 += kTapsAtOnce) {
    float x[kTapsAtOnce][N], w[kTapsAtOnce][N];
#pragma unroll
    for (int i = 0; i < kTapsAtOnce; ++i) {
      const int m = m0 + i, tt = t - n1 + m;
#pragma unroll
      for (int e = 0; e < N; ++e) x[i][e] = w[i][e] = 0.f;
      if (m < a.taps) {
        load_vec<DType_f32, N>(a.conv_w, (int64_t)m * C + ch, w[i]);
        if (tt >= 0) load_vec<DT, N>(a.proj, row + tt * a.proj_stride_t, x[i]);
        else if (!a.fresh) load_vec<DT, N>(a.conv_state, (((int64_t)parity * a.B + b) * n1 + (tt + n1)) * C + ch, x[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < kTapsAtOnce; ++i)
#pragma unroll
      for (int e = 0; e < N; ++e) out[e] = fmaf(x[i][e], w[i][e], out[e]);
  }
#pragma unroll
  for (int e = 0; e < N; ++e) out[e] *= sigmoid_f32(out[e]);
}

// ---- one token ------------------------------------------------------------------------------

// Rows of the low-rank products of one head: the decay's dk rows, then the gate's dv rows (none
// without gate_w), y[r] = w[r, :] . x.  16 lanes per row; kRowsAtOnce rows of a lane group are
// requested before the first is summed, so that a head's matrices (which no cache holds from one
// token to the next) cost one trip to memory.
constexpr int kRowsAtOnce = 8;

// One lane's 8 elements as loaded, so that eight rows in flight take few registers.
template <class DT>
struct Raw8 {
  uint4 v[8 / DT::kPer16B];
  __device__ __forceinline__ void load(const void* p, int64_t i) {
#pragma unroll
    for (int k = 0; k < 8 / DT::kPer16B; ++k)
      v[k] = *reinterpret_cast<const uint4*>((const typename DT::storage*)p + i + k * DT::kPer16B);
  }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int k = 0; k < 8 / DT::kPer16B; ++k) v[k] = make_uint4(0, 0, 0, 0);
  }
  __device__ __forceinline__ void get(float* out) const {
#pragma unroll
    for (int k = 0; k < 8 / DT::kPer16B; ++k) unpack16<DT>(v[k], out + k * DT::kPer16B);
  }
};

// By lanes tid = 0 .. nt - 1 (a multiple of 64).  TANH: of the decay's columns.
template <class DT, bool TANH>
__device__ __forceinline__ void low_rank_rows(const socket_recurrence& a, int h, int64_t row0, int tid, int nt, float* gs,
                                              float* gate) {
  constexpr int ROWS = DT::kPer16B == 8 ? kRowsAtOnce : kRowsAtOnce / 2;
  const int sub = tid & 15, grp = tid >> 4, ngrp = nt >> 4;
  const int n = a.dk + (a.gate_w ? a.dv : 0);
  const bool vec = a.decay_rank % 8 == 0 && a.decay_rank <= 128 && (row0 + a.decay_off) % 8 == 0 &&
                   (!a.gate_w || (a.gate_rank % 8 == 0 && a.gate_rank <= 128 && (row0 + a.gate_off) % 8 == 0));
  if (vec) {
    Raw8<DT> xd, xg;
    xd.zero();
    xg.zero();
    if (sub * 8 < a.decay_rank) xd.load(a.proj, row0 + a.decay_off + sub * 8);
    if (a.gate_w && sub * 8 < a.gate_rank) xg.load(a.proj, row0 + a.gate_off + sub * 8);
    float xt[8];
    if constexpr (TANH) {
      xd.get(xt);
#pragma unroll
      for (int e = 0; e < 8; ++e) xt[e] = tanh_f32(xt[e]);
    }
    for (int c0 = 0; c0 < n; c0 += ngrp * ROWS) {   // (all lanes take part in the sums)
      Raw8<DT> w[ROWS];
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        const int c = c0 + i * ngrp + grp;
        w[i].zero();
        if (c < a.dk) {
          if (sub * 8 < a.decay_rank) w[i].load(a.decay_w, ((int64_t)h * a.dk + c) * a.decay_rank + sub * 8);
        } else if (c < n) {
          if (sub * 8 < a.gate_rank) w[i].load(a.gate_w, ((int64_t)h * a.dv + c - a.dk) * a.gate_rank + sub * 8);
        }
      }
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        const int c = c0 + i * ngrp + grp;
        float x[8], y[8], t = 0.f;
        (c < a.dk ? xd : xg).get(x);
        if constexpr (TANH) {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = xt[e];      // (no gate here)
        }
        w[i].get(y);
#pragma unroll
        for (int e = 0; e < 8; ++e) t = fmaf(y[e], x[e], t);
        t = group_sum<16>(t);
        if (c < n && sub == 0) (c < a.dk ? gs : gate - a.dk)[c] = t;
      }
    }
    return;
  }
  for (int c0 = 0; c0 < n; c0 += ngrp) {
    const int c = c0 + grp;
    float t = 0.f;
    if (c < n) {
      const bool decay = c < a.dk;
      const void* w = decay ? a.decay_w : a.gate_w;
      const int rank = decay ? a.decay_rank : a.gate_rank;
      const int64_t wr = (decay ? (int64_t)h * a.dk + c : (int64_t)h * a.dv + c - a.dk) * rank;
      const int64_t xr = row0 + (decay ? a.decay_off : a.gate_off);
      for (int r = sub; r < rank; r += 16) {
        const float x = load_elem<DT>(a.proj, xr + r);
        t = fmaf(load_elem<DT>(w, wr + r), TANH && decay ? tanh_f32(x) : x, t);
      }
    }
    t = group_sum<16>(t);
    if (c < n && sub == 0) (c < a.dk ? gs : gate - a.dk)[c] = t;
  }
}

// How a workgroup's lanes cover a state: `nc` lanes of VEC columns across (nc_shift: its base-2
// logarithm, -1 if it is no power of two) and RG rows side by side.
struct StepShape {
  int nc, nc_shift, RG;
};

// One workgroup per (head, sequence); grid (heads per q / k head, q / k heads, sequences).  The
// state lives in registers: a lane owns VEC neighbouring columns of every RG-th row; sums
// over the rows go through LDS.  GENERAL: rule 1.
template <class DT, int VEC, int ROWS, bool GENERAL>
__global__ __launch_bounds__(1024) void recurrence_step_kernel(socket_recurrence a, StepShape sh) {
  extern __shared__ __attribute__((aligned(16))) float rs_lds[];
  const int hk = blockIdx.y, h = hk * gridDim.x + blockIdx.x, b = blockIdx.z;
  const int tid = threadIdx.x, nt = blockDim.x, lane = tid & 63;
  const int dk = a.dk, dv = a.dv;
  const bool delta = GENERAL || a.beta_off >= 0;
  float* qs = rs_lds;             // dk
  float* ks = qs + dk;            // dk
  float* gs = ks + dk;            // dk: low-rank product, then decay
  float* vs = gs + dk;            // dv
  float* gate = vs + dv;          // dv
  float* os = gate + dv;          // dv: sums over the rows
  float* red = os + dv;           // 16
  float* rates = red + 16;        // GENERAL: dk, removal rate per key channel
  float* part = rates + (GENERAL ? dk : 0);   // RG * dv
  const int RG = sh.RG;
  const int rg = sh.nc_shift >= 0 ? tid >> sh.nc_shift : tid / sh.nc;
  const int col = (tid - rg * sh.nc) * VEC;
  const bool active = rg < RG;

  // the state, requested before anything else, then the small operands of later phases
  float* Sp = a.state + ((int64_t)b * a.H + h) * dk * dv + rg * dv + col;
  float S[ROWS][VEC];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) S[i][e] = 0.f;
    if (active && rg + i * RG < dk) load_vec<DType_f32, VEC>(Sp, i * RG * dv, S[i]);
  }
  const int64_t row0 = b * a.proj_stride_b;
  const float bias = (a.decay_bias && tid < dk) ? a.decay_bias[h * dk + tid] : 0.f;
  const float nw = tid < dv ? a.norm_w[(GENERAL && a.norm_per_head ? h * dv : 0) + tid] : 0.f;
  const float beta_z = !GENERAL && delta ? load_elem<DT>(a.proj, row0 + a.beta_off + h) : 0.f;
  const int half = nt >> 1;
  if (tid < half) {
    // half of the waves: the low-rank products
    low_rank_rows<DT, GENERAL>(a, h, row0, tid, half, gs, gate);
  } else {
    // the other half meanwhile: q, k and v through the convolution, whose inputs move up by one
    // in the other half of its state (heads that share q / k write the same values).  Both halves
    // are read, so that the loads do not wait for the position.
    const int n1 = a.taps - 1, C = conv_channels(a);
    const int64_t pos = *a.pos;
    if constexpr (GENERAL)
      for (int c = tid - half; c < dk; c += half) {
        const float z = load_elem<DT>(a.proj, row0 + a.rate_off + h * dk + c);
        rates[c] = sigmoid_f32(z + (a.rate_bias ? a.rate_bias[h * dk + c] : 0.f));
      }
    for (int i = tid - half; i < 2 * dk + dv; i += half) {
      const int which = (i >= dk) + (i >= 2 * dk);
      const int at = which == 2 ? h * dv + i - 2 * dk : hk * dk + i - which * dk;
      const int ch = which * a.Hk * dk + at;
      const float now = load_elem<DT>(a.proj, row0 + (which == 0 ? a.q_off : which == 1 ? a.k_off : a.v_off) + at);
      float y = now;
      if (!GENERAL && a.taps >= 1) {
        y = 0.f;
        const int64_t s0 = (int64_t)b * n1 * C + ch, other = (int64_t)a.B * n1 * C;
        for (int m0 = 0; m0 < a.taps; m0 += kTapsAtOnce) {
          float w[kTapsAtOnce], x0[kTapsAtOnce], x1[kTapsAtOnce];
#pragma unroll
          for (int u = 0; u < kTapsAtOnce; ++u) {
            const int m = m0 + u;
            w[u] = x0[u] = x1[u] = 0.f;
            if (m < a.taps) w[u] = a.conv_w[m * C + ch];
            if (m < n1) {
              x0[u] = load_elem<DT>(a.conv_state, s0 + m * C);
              x1[u] = load_elem<DT>(a.conv_state, s0 + other + m * C);
            }
          }
          const bool odd = pos & 1;
#pragma unroll
          for (int u = 0; u < kTapsAtOnce; ++u) {
            const int m = m0 + u;
            const float x = m < n1 ? (odd ? x1[u] : x0[u]) : now;
            y = fmaf(x, w[u], y);
            if (m >= 1 && m <= n1) store_elem<DT>(a.conv_state, s0 + (odd ? 0 : other) + (m - 1) * C, x);
          }
        }
        y *= sigmoid_f32(y);
      }
      qs[i < 2 * dk ? i : i + dk] = y;     // q | k | (decays) | v
    }
    if (!a.gate_w)
      for (int c = tid - half; c < dv; c += half) gate[c] = load_elem<DT>(a.proj, row0 + a.gate_off + h * dv + c);
  }
  const float a_exp = a.decay_kind == 0 ? exp_f32(a.a_log[h]) : 0.f;
  __syncthreads();
  if (tid < dk) gs[tid] = exp2_fast(log2_decay(a, a_exp, gs[tid] + bias));   // (dk <= 256 <= nt)
  float q_mul = a.q_scale, k_mul = 1.f;
  if (GENERAL || a.unit_qk) {
    // (every wave takes both sums for itself: no further barrier)
    float sq = 0.f, sk = 0.f;
    for (int c = lane; c < dk; c += 64) {
      sq = fmaf(qs[c], qs[c], sq);
      sk = fmaf(ks[c], ks[c], sk);
    }
    if (!GENERAL) q_mul *= rsqrt_f32(group_sum<64>(sq) + 1e-6f);
    k_mul = rsqrt_f32(group_sum<64>(sk) + 1e-6f);
  }
  __syncthreads();

  auto column_sum = [&](int c) __attribute__((always_inline)) {
    float s = 0.f;
#pragma unroll 8
    for (int r = 0; r < RG; ++r) s += part[r * dv + c];
    return s;
  };
  // decay (GENERAL: later), and what the state holds for this key
  float u[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) u[e] = 0.f;
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = rg + i * RG;
    if (active && row < dk) {
      const float g = gs[row], k = ks[row] * k_mul;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        if (!GENERAL) S[i][e] *= g;
        u[e] = fmaf(S[i][e], k, u[e]);
      }
    }
  }
  if (delta) {
    if (active) store_vec<DType_f32, VEC>(part, rg * dv + col, u);
    __syncthreads();
    if (tid < dv) os[tid] = GENERAL ? column_sum(tid) : sigmoid_f32(beta_z) * (vs[tid] - column_sum(tid));   // (dv <= 256 <= nt)
    __syncthreads();
  }
  float o[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) o[e] = 0.f;
  float v[VEC];
  if (active) load_vec<DType_f32, VEC>(delta ? os : vs, col, u);
  if (GENERAL && active) load_vec<DType_f32, VEC>(vs, col, v);
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = rg + i * RG;
    if (active && row < dk) {
      const float k = ks[row] * k_mul, q = qs[row] * q_mul;
      const float gone = GENERAL ? -rates[row] * k : 0.f;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        if constexpr (GENERAL) S[i][e] = fmaf(ks[row], v[e], fmaf(gone, u[e], S[i][e] * gs[row]));
        else S[i][e] = fmaf(k, u[e], S[i][e]);
        o[e] = fmaf(S[i][e], q, o[e]);
      }
    }
  }
  if (active) store_vec<DType_f32, VEC>(part, rg * dv + col, o);   // (its last readers passed a barrier since)
#pragma unroll
  for (int i = 0; i < ROWS; ++i)
    if (active && rg + i * RG < dk) store_vec<DType_f32, VEC>(Sp, i * RG * dv, S[i]);
  __syncthreads();
  const float s = tid < dv ? column_sum(tid) : 0.f;
  const float rs = rsqrt_f32(block_sum(s * s, red) / (float)dv + a.eps);
  if (tid < dv) store_elem<DT>(a.out, ((int64_t)b * a.H + h) * dv + tid, s * rs * nw * gate_act(a.gate_kind, gate[tid]));
}

// ---- chunks of tokens -----------------------------------------------------------------------

constexpr int kPrepThreads = 1024;
constexpr int kPrepWaves = kPrepThreads / 64;
constexpr float kMildDecay = -60.f;   // a block's total log2 decay above which 2^{-pl} is safe in fp32

// Workspace of one (chunk, head, sequence), in floats.  kt / vt: 16-wide tiles of dk / dv.
// extra: what rule 1 adds to the read-out and to the state whatever the state was.
struct ChunkSpace {
  int kt, vt, nb;
  bool extra = false;
  __host__ __device__ int64_t w() const { return 0; }
  __host__ __device__ int64_t q() const { return (int64_t)nb * kt * 256; }
  __host__ __device__ int64_t kT() const { return 2 * (int64_t)nb * kt * 256; }
  __host__ __device__ int64_t u() const { return 3 * (int64_t)nb * kt * 256; }
  __host__ __device__ int64_t aqk() const { return u() + (int64_t)nb * vt * 256; }
  __host__ __device__ int64_t gamma() const { return aqk() + (int64_t)nb * nb * 256; }
  __host__ __device__ int64_t o() const { return gamma() + (int64_t)kt * 16; }
  __host__ __device__ int64_t s() const { return o() + (int64_t)nb * vt * 256; }
  __host__ __device__ int64_t size() const { return extra ? s() + (int64_t)kt * vt * 256 : o(); }
};

// Channels [0, 16 tiles) of token rows [0, 16 NB) of q, k or v into LDS rows of `pitch`
// floats; rows past the portion and channels past `width` are zero.
template <class DT>
__device__ __forceinline__ void stage_rows(const socket_recurrence& a, int b, int t_first, int n_rows, int rows, int col0,
                                           int ch0, int width, int padded, float* dst, int pitch, bool vec) {
  if (vec) {
    const int per = padded / 8;
    for (int w = threadIdx.x; w < rows * per; w += kPrepThreads) {
      const int r = w / per, c = w % per * 8;
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = 0.f;
      if (r < n_rows && c < width) conv_input<DT, 8>(a, b, t_first + r, col0 + c, ch0 + c, (int)(a.pos0 & 1), x);
      *reinterpret_cast<float4*>(dst + r * pitch + c) = make_float4(x[0], x[1], x[2], x[3]);
      *reinterpret_cast<float4*>(dst + r * pitch + c + 4) = make_float4(x[4], x[5], x[6], x[7]);
    }
  } else {
    for (int w = threadIdx.x; w < rows * padded; w += kPrepThreads) {
      const int r = w / padded, c = w % padded;
      float x = 0.f;
      if (r < n_rows && c < width) conv_input<DT, 1>(a, b, t_first + r, col0 + c, ch0 + c, (int)(a.pos0 & 1), &x);
      dst[r * pitch + c] = x;
    }
  }
}

// By one wave: the tile d = -L (strictly lower, fragment order) becomes (I + L)^{-1}, a column per lane.
__device__ __forceinline__ void invert_diagonal(float* d, int x16, int quarter) {
  float x[16];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    x[r] = r == x16 ? 1.f : 0.f;
#pragma unroll
    for (int s0 = 0; s0 < r; s0 += 4) {
      const float4 m = *reinterpret_cast<const float4*>(d + ((s0 >> 2) * 16 + r) * 4);
      x[r] = fmaf(m.x, x[s0], x[r]);
      if (s0 + 1 < r) x[r] = fmaf(m.y, x[s0 + 1], x[r]);
      if (s0 + 2 < r) x[r] = fmaf(m.z, x[s0 + 2], x[r]);
      if (s0 + 3 < r) x[r] = fmaf(m.w, x[s0 + 3], x[r]);
    }
  }
  if (quarter == 0)
#pragma unroll
    for (int r = 0; r < 16; ++r) d[((x16 >> 2) * 16 + r) * 4 + (x16 & 3)] = x[r];
}

template <class DT, int NB>
__global__ __launch_bounds__(kPrepThreads) void recurrence_prep_kernel(socket_recurrence a, int vec) {
  constexpr int C = 16 * NB;
  extern __shared__ __attribute__((aligned(16))) float rp_lds[];
  const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int x16 = lane & 15, quarter = lane >> 4;
  const int dk = a.dk, dv = a.dv, hk = h / (a.H / a.Hk);
  const bool delta = a.beta_off >= 0;
  const ChunkSpace sp{(dk + 15) / 16, (dv + 15) / 16, NB};
  const int dkp = sp.kt * 16, dvp = sp.vt * 16;
  const int kp = dkp + 4, vp = dvp + 4;          // LDS pitches
  const int t_first = a.t0 + chunk * C;          // token of the portion
  const int n_rows = min(C, a.t0 + a.n - t_first);

  float* qs = rp_lds;                            // C x kp; later V, C x vp
  float* ks = qs + C * (kp > vp ? kp : vp);      // C x kp
  float* pl = ks + C * kp;                       // C x kp: log2 decay, then its running sum inside the block
  float* tot = pl + C * kp;                      // NB x dkp
  float* lk = tot + NB * dkp;                    // NB x NB tiles in fragment order: -L, inverses on the diagonal
  float* beta = lk + NB * NB * 256;              // C

  float* ws = (float*)a.workspace + (((int64_t)b * a.H + h) * gridDim.x + chunk) * sp.size();

  // ---- inputs
  stage_rows<DT>(a, b, t_first, n_rows, C, a.q_off + hk * dk, hk * dk, dk, dkp, qs, kp, vec);
  stage_rows<DT>(a, b, t_first, n_rows, C, a.k_off + hk * dk, a.Hk * dk + hk * dk, dk, dkp, ks, kp, vec);
  const float a_exp = a.decay_kind == 0 ? exp_f32(a.a_log[h]) : 0.f;
#pragma unroll 4
  for (int w = tid; w < C * dkp; w += kPrepThreads) {
    const int r = w / dkp, c = w % dkp;
    float g = 0.f;
    if (r < n_rows && c < dk) {
      const int64_t zi = ((int64_t)b * a.T + t_first + r) * a.H * dk + h * dk + c;
      g = log2_decay(a, a_exp, (a.decay_z_f32 ? ((const float*)a.decay_z)[zi] : load_elem<DT>(a.decay_z, zi)) +
                                   (a.decay_bias ? a.decay_bias[h * dk + c] : 0.f));
    }
    pl[r * kp + c] = g;
  }
  if (tid < C)
    beta[tid] = (delta && tid < n_rows)
                    ? sigmoid_f32(load_elem<DT>(a.proj, b * a.proj_stride_b + (t_first + tid) * a.proj_stride_t + a.beta_off + h))
                    : 0.f;
  __syncthreads();

  // ---- unit vectors and the scale of q; running sums of the log2 decay inside each block
  for (int r = wave; r < C; r += kPrepWaves) {
    float qm = a.q_scale, km = 1.f;
    if (a.unit_qk) {
      float sq = 0.f, sk = 0.f;
      for (int c = lane; c < dkp; c += 64) {
        sq = fmaf(qs[r * kp + c], qs[r * kp + c], sq);
        sk = fmaf(ks[r * kp + c], ks[r * kp + c], sk);
      }
      qm *= rsqrt_f32(group_sum<64>(sq) + 1e-6f);
      km = rsqrt_f32(group_sum<64>(sk) + 1e-6f);
    }
    for (int c = lane; c < dkp; c += 64) {
      qs[r * kp + c] *= qm;
      ks[r * kp + c] *= km;
    }
  }
  for (int w = tid; w < NB * dkp; w += kPrepThreads) {
    const int blk = w / dkp, c = w % dkp;
    float s = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      s += pl[(blk * 16 + r) * kp + c];
      pl[(blk * 16 + r) * kp + c] = s;
    }
    tot[blk * dkp + c] = s;
  }
  __syncthreads();

  // ---- Aqk and -L, tile (I, J): lane (quarter, x) holds row x of block I against keys
  // 4 quarter + r of block J (the transposed product, which leaves fragment order)
  for (int unit = wave; unit < NB * (NB + 1) / 2; unit += kPrepWaves) {
    int I = 0, J = unit;
    while (J > I) J -= ++I;
    const int t = 16 * I + x16, s = 16 * J + x16;
    rc_f32x4 aq = {0.f, 0.f, 0.f, 0.f}, ak = {0.f, 0.f, 0.f, 0.f};
    bool mild = true;
    if (I == J) {
      bool low = false;
      for (int c = lane; c < dkp; c += 64) low |= tot[I * dkp + c] < kMildDecay;
      mild = __builtin_amdgcn_ballot_w64(low) == 0;
    }
    if (mild) {
      for (int j = 0; j < sp.kt; ++j) {
        const int c = 16 * j + 4 * quarter;
        float4 kk = *reinterpret_cast<const float4*>(ks + s * kp + c);
        const float4 ps = *reinterpret_cast<const float4*>(pl + s * kp + c);
        float4 e = make_float4(-ps.x, -ps.y, -ps.z, -ps.w);
        if (I != J) {
          for (int m = J; m < I; ++m) {
            const float4 tm = *reinterpret_cast<const float4*>(tot + m * dkp + c);
            e.x += tm.x;
            e.y += tm.y;
            e.z += tm.z;
            e.w += tm.w;
          }
        }
        kk.x *= exp2_fast(e.x);
        kk.y *= exp2_fast(e.y);
        kk.z *= exp2_fast(e.z);
        kk.w *= exp2_fast(e.w);
        const float4 pt = *reinterpret_cast<const float4*>(pl + t * kp + c);
        const float4 f = make_float4(exp2_fast(pt.x), exp2_fast(pt.y), exp2_fast(pt.z), exp2_fast(pt.w));
        const float4 qt = *reinterpret_cast<const float4*>(qs + t * kp + c);
        aq = mfma4(kk, rc_f32x4{qt.x * f.x, qt.y * f.y, qt.z * f.z, qt.w * f.w}, aq);
        if (delta) {
          const float4 kt = *reinterpret_cast<const float4*>(ks + t * kp + c);
          ak = mfma4(kk, rc_f32x4{kt.x * f.x, kt.y * f.y, kt.z * f.z, kt.w * f.w}, ak);
        }
      }
    } else {
      for (int c = 0; c < dkp; ++c) {
        const float pt = pl[t * kp + c], qt = qs[t * kp + c], kt = ks[t * kp + c];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int sr = 16 * J + 4 * quarter + r;
          const float w = ks[sr * kp + c] * exp2_fast(fminf(pt - pl[sr * kp + c], 0.f));
          aq[r] = fmaf(qt, w, aq[r]);
          ak[r] = fmaf(kt, w, ak[r]);
        }
      }
    }
    const float bt = beta[t];
    float4 q4, k4;
    float* q4p = &q4.x;
    float* k4p = &k4.x;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int sr = 16 * J + 4 * quarter + r;
      q4p[r] = sr <= t ? aq[r] : 0.f;
      k4p[r] = sr < t ? -bt * ak[r] : 0.f;
    }
    *reinterpret_cast<float4*>(ws + sp.aqk() + (I * NB + J) * 256 + lane * 4) = q4;
    if (delta) *reinterpret_cast<float4*>(lk + (I * NB + J) * 256 + lane * 4) = k4;
  }

  // ---- Q^ and K^T (for the update) fragments, the chunk's total decay
  for (int item = wave; item < 2 * NB * sp.kt; item += kPrepWaves) {
    const bool is_q = item < NB * sp.kt;
    const int w = is_q ? item : item - NB * sp.kt;
    if (is_q) {
      const int rt = w / sp.kt, ct = w % sp.kt;
      const int t = 16 * rt + x16, c = 16 * ct + 4 * quarter;
      float4 e = *reinterpret_cast<const float4*>(pl + t * kp + c);
      for (int m = 0; m < rt; ++m) {
        const float4 tm = *reinterpret_cast<const float4*>(tot + m * dkp + c);
        e.x += tm.x;
        e.y += tm.y;
        e.z += tm.z;
        e.w += tm.w;
      }
      const float4 q = *reinterpret_cast<const float4*>(qs + t * kp + c);
      *reinterpret_cast<float4*>(ws + sp.q() + (rt * sp.kt + ct) * 256 + lane * 4) =
          make_float4(q.x * exp2_fast(e.x), q.y * exp2_fast(e.y), q.z * exp2_fast(e.z), q.w * exp2_fast(e.w));
    } else {
      const int ct = w / NB, rt = w % NB;
      const int c = 16 * ct + x16;
      float after = 0.f;
      for (int m = rt; m < NB; ++m) after += tot[m * dkp + c];
      float4 o;
      float* op = &o.x;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * rt + 4 * quarter + r;
        op[r] = ks[t * kp + c] * exp2_fast(after - pl[t * kp + c]);
      }
      *reinterpret_cast<float4*>(ws + sp.kT() + (ct * NB + rt) * 256 + lane * 4) = o;
    }
  }
  for (int c = tid; c < dkp; c += kPrepThreads) {
    float s = 0.f;
    for (int m = 0; m < NB; ++m) s += tot[m * dkp + c];
    ws[sp.gamma() + c] = exp2_fast(s);
  }
  __syncthreads();

  // ---- (I + L_II)^{-1} of the diagonal tiles, a column per lane; V over q's rows meanwhile
  if (delta && wave < NB) invert_diagonal(lk + (wave * NB + wave) * 256, x16, quarter);
  stage_rows<DT>(a, b, t_first, n_rows, C, a.v_off + h * dv, 2 * a.Hk * dk + h * dv, dv, dvp, qs, vp, vec);
  __syncthreads();

  // ---- Ubar = T beta V and W = T beta K^, a 16-column tile per wave: forward substitution over
  // the blocks; a finished block's accumulator is the next product's operand
  const int n_tiles = delta ? sp.vt + sp.kt : sp.vt;
  for (int tile = wave; tile < n_tiles; tile += kPrepWaves) {
    const bool is_v = tile < sp.vt;
    const int ct = is_v ? tile : tile - sp.vt;
    const int c = 16 * ct + x16;
    rc_f32x4 X[NB];
    float before = 0.f;
#pragma unroll
    for (int I = 0; I < NB; ++I) {
      rc_f32x4 acc;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * I + 4 * quarter + r;
        const float v = is_v ? qs[t * vp + c] : ks[t * kp + c] * exp2_fast(before + pl[t * kp + c]);
        acc[r] = delta ? beta[t] * v : v;
      }
      if (!is_v) before += tot[I * dkp + c];
      if (delta) {
#pragma unroll
        for (int J = 0; J < I; ++J)
          acc = mfma4(*reinterpret_cast<const float4*>(lk + (I * NB + J) * 256 + lane * 4), X[J], acc);
        X[I] = mfma4(*reinterpret_cast<const float4*>(lk + (I * NB + I) * 256 + lane * 4), acc, rc_f32x4{0.f, 0.f, 0.f, 0.f});
      } else {
        X[I] = acc;
      }
      if (is_v) {
        *reinterpret_cast<rc_f32x4*>(ws + sp.u() + (I * sp.vt + ct) * 256 + lane * 4) = X[I];
      } else {
        float* w = ws + sp.w() + (I * sp.kt + ct) * 256;
#pragma unroll
        for (int r = 0; r < 4; ++r) w[((x16 >> 2) * 16 + 4 * quarter + r) * 4 + (x16 & 3)] = X[I][r];
      }
    }
  }
}

// ---- chunks of the generalized delta rule ---------------------------------------------------
//
// With y_t = S_{t-1}^T n_t, c_t = a_t * n_t and b_t the running sum of log g,
//   y_t = (n_t e^{b_{t-1}})^T S0 + sum_{s < t} M[t,s] v_s - L[t,s] y_s
//   o_t = (q_t e^{b_t})^T S0 + sum_{s <= t} Aqk[t,s] v_s - Aqc[t,s] y_s
//   S   = diag(e^{b_C}) S0 + sum_s (k_s e^{b_C - b_s}) v_s^T - (c_s e^{b_C - b_s}) y_s^T
// where M, L pair n_t e^{b_{t-1}} with k_s e^{-b_s}, c_s e^{-b_s}, and Aqk, Aqc pair q_t e^{b_t} with
// them.  With U = -Y the sequential part is the delta rule's, U = Ubar - W S0, O = Q^ S0 + Aqc U,
// S = diag(e^{b_C}) S0 + C^T U, plus two terms that do not depend on S0: Obar = Aqk V and Sbar = K^T V.
// W = (I + L)^{-1} (n e^{b-}), Ubar = -(I + L)^{-1} M V.
//
// A token's log2 decay is bounded (decay kind 2), so a chunk's sum stays far inside fp32's exponent
// range and e^{b_t - b_s} is taken as e^{b_t} e^{-b_s} (the host checks the bound).
constexpr int kGeneralItems = 2;         // (row, 4 channels) pieces per lane
constexpr float kMaxChunkDecay = 100.f;  // log2; exponents of that size and their products are normal numbers

template <class DT, int NB>
__global__ __launch_bounds__(kPrepThreads) void general_prep_kernel(socket_recurrence a, int vec, int late_v) {
  constexpr int C = 16 * NB;
  extern __shared__ __attribute__((aligned(16))) float rp_lds[];
  const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int x16 = lane & 15, quarter = lane >> 4;
  const int dk = a.dk, dv = a.dv;
  const ChunkSpace sp{(dk + 15) / 16, (dv + 15) / 16, NB, true};
  const int dkp = sp.kt * 16, dvp = sp.vt * 16;
  const int kp = dkp + 4, vp = dvp + 4;          // LDS pitches
  const int t_first = a.t0 + chunk * C;
  const int n_rows = min(C, a.t0 + a.n - t_first);

  float* qs = rp_lds;                            // C x kp: q, then q e^b
  float* us = qs + C * kp;                       // C x kp: log2 decay, its running sum in the block, then n e^{b-}
  float* ks = us + C * kp;                       // C x kp: k, then k e^{-b}
  float* cs = ks + C * kp;                       // C x kp: rates, then a n e^{-b}
  float* vs = late_v ? qs : cs + C * kp;         // C x vp; late_v (wide heads): over q once that has been used
  float* tot = cs + C * kp + (late_v ? 0 : C * vp);   // NB x dkp
  float* lk = tot + NB * dkp;                    // tiles (I, J) in fragment order: -L, inverses on the diagonal
  float* mk = lk + NB * NB * 256;                // M
  float* ak = mk + NB * NB * 256;                // Aqk
  float* kn = ak + NB * NB * 256;                // C: 1 / |k|

  float* ws = (float*)a.workspace + (((int64_t)b * a.H + h) * gridDim.x + chunk) * sp.size();

  // ---- inputs
  stage_rows<DT>(a, b, t_first, n_rows, C, a.q_off + h * dk, h * dk, dk, dkp, qs, kp, vec);
  stage_rows<DT>(a, b, t_first, n_rows, C, a.k_off + h * dk, a.Hk * dk + h * dk, dk, dkp, ks, kp, vec);
  stage_rows<DT>(a, b, t_first, n_rows, C, a.rate_off + h * dk, 0, dk, dkp, cs, kp, vec && a.rate_off % 8 == 0);
  if (!late_v) stage_rows<DT>(a, b, t_first, n_rows, C, a.v_off + h * dv, 2 * a.Hk * dk + h * dv, dv, dvp, vs, vp, vec);
#pragma unroll 4
  for (int w = tid; w < C * dkp; w += kPrepThreads) {
    const int r = w / dkp, c = w % dkp;
    float g = 0.f;
    if (r < n_rows && c < dk) {
      const int64_t zi = ((int64_t)b * a.T + t_first + r) * a.H * dk + h * dk + c;
      g = log2_decay(a, 0.f, (a.decay_z_f32 ? ((const float*)a.decay_z)[zi] : load_elem<DT>(a.decay_z, zi)) +
                                 (a.decay_bias ? a.decay_bias[h * dk + c] : 0.f));
    }
    us[r * kp + c] = g;
  }
  __syncthreads();

  // ---- norms of the keys; running sums of the log2 decay inside each block
  for (int r = wave; r < C; r += kPrepWaves) {
    float sk = 0.f;
    for (int c = lane; c < dkp; c += 64) sk = fmaf(ks[r * kp + c], ks[r * kp + c], sk);
    sk = group_sum<64>(sk);
    if (lane == 0) kn[r] = rsqrt_f32(sk + 1e-6f);
  }
  for (int w = tid; w < NB * dkp; w += kPrepThreads) {
    const int blk = w / dkp, c = w % dkp;
    float s = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      s += us[(blk * 16 + r) * kp + c];
      us[(blk * 16 + r) * kp + c] = s;
    }
    tot[blk * dkp + c] = s;
  }
  __syncthreads();

  // ---- the four scaled operands, in place (a row's sums are read by the row after it: registers between)
  const int quads = dkp / 4;
  float4 nq[kGeneralItems], nu[kGeneralItems], nk[kGeneralItems], nc[kGeneralItems];
#pragma unroll
  for (int it = 0; it < kGeneralItems; ++it) {
    const int w = tid + it * kPrepThreads, r = w / quads, c = w % quads * 4;
    if (r >= C) continue;
    float4 off = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int m = 0; m < (r >> 4); ++m) {
      const float4 tm = *reinterpret_cast<const float4*>(tot + m * dkp + c);
      off.x += tm.x;
      off.y += tm.y;
      off.z += tm.z;
      off.w += tm.w;
    }
    const float4 in = *reinterpret_cast<const float4*>(us + r * kp + c);
    const float4 ex = (r & 15) ? *reinterpret_cast<const float4*>(us + (r - 1) * kp + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    const float4 q = *reinterpret_cast<const float4*>(qs + r * kp + c), k = *reinterpret_cast<const float4*>(ks + r * kp + c);
    const float4 z = *reinterpret_cast<const float4*>(cs + r * kp + c);
    const float n = kn[r];
    const float* offp = &off.x;
    const float* inp = &in.x;
    const float* exp_ = &ex.x;
    const float* qp = &q.x;
    const float* kq = &k.x;
    const float* zp = &z.x;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float bt = offp[e] + inp[e], grow = exp2_fast(-bt), u = kq[e] * n;
      const float rate = sigmoid_f32(zp[e] + (a.rate_bias && c + e < dk ? a.rate_bias[h * dk + c + e] : 0.f));
      (&nq[it].x)[e] = qp[e] * a.q_scale * exp2_fast(bt);
      (&nu[it].x)[e] = u * exp2_fast(offp[e] + exp_[e]);
      (&nk[it].x)[e] = kq[e] * grow;
      (&nc[it].x)[e] = rate * u * grow;
    }
  }
  __syncthreads();
#pragma unroll
  for (int it = 0; it < kGeneralItems; ++it) {
    const int w = tid + it * kPrepThreads, r = w / quads, c = w % quads * 4;
    if (r >= C) continue;
    *reinterpret_cast<float4*>(qs + r * kp + c) = nq[it];
    *reinterpret_cast<float4*>(us + r * kp + c) = nu[it];
    *reinterpret_cast<float4*>(ks + r * kp + c) = nk[it];
    *reinterpret_cast<float4*>(cs + r * kp + c) = nc[it];
  }
  __syncthreads();

  // ---- tile (I, J) of the four products, against k in one wave and against c in another: lane
  // (quarter, x) holds row x of block I against tokens 4 quarter + r of block J
  for (int item = wave; item < NB * (NB + 1); item += kPrepWaves) {
    const bool with_k = item & 1;
    int I = 0, J = item >> 1;
    while (J > I) J -= ++I;
    const int t = 16 * I + x16, s = 16 * J + x16;
    const float* right = with_k ? ks : cs;
    rc_f32x4 aq = {0.f, 0.f, 0.f, 0.f}, au = {0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < sp.kt; ++j) {
      const int c = 16 * j + 4 * quarter;
      const float4 kk = *reinterpret_cast<const float4*>(right + s * kp + c);
      const float4 qt = *reinterpret_cast<const float4*>(qs + t * kp + c);
      const float4 ut = *reinterpret_cast<const float4*>(us + t * kp + c);
      aq = mfma4(kk, rc_f32x4{qt.x, qt.y, qt.z, qt.w}, aq);
      au = mfma4(kk, rc_f32x4{ut.x, ut.y, ut.z, ut.w}, au);
    }
    float4 q4, u4;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int sr = 16 * J + 4 * quarter + r;
      (&q4.x)[r] = sr <= t ? aq[r] : 0.f;
      (&u4.x)[r] = sr < t ? (with_k ? au[r] : -au[r]) : 0.f;
    }
    const int at = (I * NB + J) * 256 + lane * 4;
    if (with_k) {
      *reinterpret_cast<float4*>(ak + at) = q4;
      *reinterpret_cast<float4*>(mk + at) = u4;
    } else {
      *reinterpret_cast<float4*>(ws + sp.aqk() + at) = q4;
      *reinterpret_cast<float4*>(lk + at) = u4;
    }
  }

  // ---- Q^ and C^T fragments, the chunk's total decay
  auto total = [&](int c) __attribute__((always_inline)) {
    float s = 0.f;
#pragma unroll
    for (int m = 0; m < NB; ++m) s += tot[m * dkp + c];
    return exp2_fast(s);
  };
  for (int item = wave; item < 2 * NB * sp.kt; item += kPrepWaves) {
    const bool is_q = item < NB * sp.kt;
    const int w = is_q ? item : item - NB * sp.kt;
    if (is_q) {
      const int rt = w / sp.kt, ct = w % sp.kt;
      *reinterpret_cast<float4*>(ws + sp.q() + (rt * sp.kt + ct) * 256 + lane * 4) =
          *reinterpret_cast<const float4*>(qs + (16 * rt + x16) * kp + 16 * ct + 4 * quarter);
    } else {
      const int ct = w / NB, rt = w % NB;
      const int c = 16 * ct + x16;
      const float after = total(c);
      float4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) (&o.x)[r] = cs[(16 * rt + 4 * quarter + r) * kp + c] * after;
      *reinterpret_cast<float4*>(ws + sp.kT() + (ct * NB + rt) * 256 + lane * 4) = o;
    }
  }
  for (int c = tid; c < dkp; c += kPrepThreads) ws[sp.gamma() + c] = total(c);
  __syncthreads();

  if (wave < NB) invert_diagonal(lk + (wave * NB + wave) * 256, x16, quarter);
  if (late_v) stage_rows<DT>(a, b, t_first, n_rows, C, a.v_off + h * dv, 2 * a.Hk * dk + h * dv, dv, dvp, vs, vp, vec);
  __syncthreads();

  // ---- a 16-column tile per wave: Ubar with Obar, W, then the tiles of Sbar
  const int solves = sp.vt + sp.kt;
  for (int item = wave; item < solves + sp.kt * sp.vt; item += kPrepWaves) {
    if (item >= solves) {
      const int j = (item - solves) / sp.vt, ct = (item - solves) % sp.vt;
      const int c = 16 * j + x16;
      const float after = total(c);
      rc_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int I = 0; I < NB; ++I) {
        float4 k;
        rc_f32x4 v;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * I + 4 * quarter + r;
          (&k.x)[r] = ks[t * kp + c] * after;
          v[r] = vs[t * vp + 16 * ct + x16];
        }
        acc = mfma4(k, v, acc);
      }
      *reinterpret_cast<rc_f32x4*>(ws + sp.s() + (j * sp.vt + ct) * 256 + lane * 4) = acc;
      continue;
    }
    const bool is_v = item < sp.vt;
    const int ct = is_v ? item : item - sp.vt;
    const int c = 16 * ct + x16;
    rc_f32x4 X[NB], B[NB];
#pragma unroll
    for (int I = 0; I < NB; ++I)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * I + 4 * quarter + r;
        B[I][r] = is_v ? vs[t * vp + c] : us[t * kp + c];
      }
#pragma unroll
    for (int I = 0; I < NB; ++I) {
      rc_f32x4 acc = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f};
      if (is_v) {
#pragma unroll
        for (int J = 0; J <= I; ++J) {
          acc = mfma4(*reinterpret_cast<const float4*>(mk + (I * NB + J) * 256 + lane * 4), B[J], acc);
          o = mfma4(*reinterpret_cast<const float4*>(ak + (I * NB + J) * 256 + lane * 4), B[J], o);
        }
        *reinterpret_cast<rc_f32x4*>(ws + sp.o() + (I * sp.vt + ct) * 256 + lane * 4) = o;
      } else {
        acc = B[I];
      }
#pragma unroll
      for (int J = 0; J < I; ++J)
        acc = mfma4(*reinterpret_cast<const float4*>(lk + (I * NB + J) * 256 + lane * 4), X[J], acc);
      X[I] = mfma4(*reinterpret_cast<const float4*>(lk + (I * NB + I) * 256 + lane * 4), acc, rc_f32x4{0.f, 0.f, 0.f, 0.f});
      if (is_v) {
        *reinterpret_cast<rc_f32x4*>(ws + sp.u() + (I * sp.vt + ct) * 256 + lane * 4) = -X[I];
      } else {
        float* w = ws + sp.w() + (I * sp.kt + ct) * 256;
#pragma unroll
        for (int r = 0; r < 4; ++r) w[((x16 >> 2) * 16 + 4 * quarter + r) * 4 + (x16 & 3)] = X[I][r];
      }
    }
  }
}

constexpr int kScanThreads = 256;
constexpr int kScanWaves = 4;

// The chunks of one (16 value columns, head, sequence) in order.  Wave w takes row block w of
// U and O and state tiles w, w + 4, ...; U and S pass through LDS.  KT: 16-row state tiles.
// EXTRA: rule 1's additions to the read-outs and the state.
template <int KT, int NB, bool DELTA, bool EXTRA>
__global__ __launch_bounds__(kScanThreads, 1) void recurrence_scan_kernel(socket_recurrence a, int n_chunks, int slices) {
  constexpr int C = 16 * NB;
  constexpr int OWN = (KT + kScanWaves - 1) / kScanWaves;
  __shared__ __attribute__((aligned(16))) float s_lds[KT * 256];
  __shared__ __attribute__((aligned(16))) float u_lds[NB * 256];
  // workgroups go to the XCDs round-robin by id: the slices of one (sequence, head) share an
  // XCD (whose L2 then serves their common W, Q^ and K^T) when the heads are a multiple of 8
  const int bh_n = a.B * a.H;
  const int slice = blockIdx.x / bh_n, bh = blockIdx.x % bh_n;
  const int h = bh % a.H, b = bh / a.H;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int x16 = lane & 15, quarter = lane >> 4;
  const ChunkSpace sp{(a.dk + 15) / 16, (a.dv + 15) / 16, NB, EXTRA};
  const int kt = sp.kt;
  const int col = 16 * slice + x16;
  const bool col_ok = col < a.dv;
  float* Sg = a.state + (int64_t)bh * a.dk * a.dv;
  const float* ws = (const float*)a.workspace + (int64_t)bh * n_chunks * sp.size();
  (void)slices;

  rc_f32x4 S[OWN];
#pragma unroll
  for (int i = 0; i < OWN; ++i) {
    const int j = wave + i * kScanWaves;
    S[i] = rc_f32x4{0.f, 0.f, 0.f, 0.f};
    if (!a.fresh && j < kt && col_ok) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * j + 4 * quarter + r;
        if (row < a.dk) S[i][r] = Sg[(int64_t)row * a.dv + col];
      }
    }
    if (j < KT) *reinterpret_cast<rc_f32x4*>(s_lds + j * 256 + lane * 4) = S[i];
  }
  const bool rows_mine = wave < NB;
  const int wb = rows_mine ? wave : 0;
  float4 fw[DELTA ? KT : 1], fq[KT], fk[OWN][NB], fa[NB], fg[OWN];
  rc_f32x4 fu, fo = {0.f, 0.f, 0.f, 0.f}, fs[EXTRA ? OWN : 1];
  auto fetch = [&](int n) __attribute__((always_inline)) {
    const float* c = ws + (int64_t)n * sp.size() + lane * 4;
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      const int jj = j < kt ? j : kt - 1;   // (tiles past dk meet zero state)
      if (DELTA) fw[j] = *reinterpret_cast<const float4*>(c + sp.w() + (wb * kt + jj) * 256);
      fq[j] = *reinterpret_cast<const float4*>(c + sp.q() + (wb * kt + jj) * 256);
    }
    fu = *reinterpret_cast<const rc_f32x4*>(c + sp.u() + (wb * sp.vt + slice) * 256);
    if (EXTRA) fo = *reinterpret_cast<const rc_f32x4*>(c + sp.o() + (wb * sp.vt + slice) * 256);
#pragma unroll
    for (int J = 0; J < NB; ++J) fa[J] = *reinterpret_cast<const float4*>(c + sp.aqk() + (wb * NB + (J <= wb ? J : wb)) * 256);
#pragma unroll
    for (int i = 0; i < OWN; ++i) {
      const int j = wave + i * kScanWaves, jj = j < kt ? j : kt - 1;
#pragma unroll
      for (int I = 0; I < NB; ++I) fk[i][I] = *reinterpret_cast<const float4*>(c + sp.kT() + (jj * NB + I) * 256);
      fg[i] = *reinterpret_cast<const float4*>(ws + (int64_t)n * sp.size() + sp.gamma() + 16 * jj + 4 * quarter);
      if (EXTRA) fs[i] = *reinterpret_cast<const rc_f32x4*>(c + sp.s() + (jj * sp.vt + slice) * 256);
    }
  };
  fetch(0);
  __syncthreads();
  for (int n = 0; n < n_chunks; ++n) {
    // a fragment's registers take the next chunk's as soon as it has been used: every load has
    // about one chunk's time to arrive
    const float* nx = ws + (int64_t)min(n + 1, n_chunks - 1) * sp.size() + lane * 4;
    rc_f32x4 u = fu, o = fo, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      const int jj = j < kt ? j : kt - 1;
      const rc_f32x4 s = *reinterpret_cast<const rc_f32x4*>(s_lds + j * 256 + lane * 4);
      if (DELTA) {
        y = mfma4(fw[j], s, y);
        fw[j] = *reinterpret_cast<const float4*>(nx + sp.w() + (wb * kt + jj) * 256);
      }
      o = mfma4(fq[j], s, o);
      fq[j] = *reinterpret_cast<const float4*>(nx + sp.q() + (wb * kt + jj) * 256);
    }
    if (DELTA) {
#pragma unroll
      for (int r = 0; r < 4; ++r) u[r] -= y[r];
    }
    fu = *reinterpret_cast<const rc_f32x4*>(nx + sp.u() + (wb * sp.vt + slice) * 256);
    if (EXTRA) fo = *reinterpret_cast<const rc_f32x4*>(nx + sp.o() + (wb * sp.vt + slice) * 256);
    if (rows_mine) *reinterpret_cast<rc_f32x4*>(u_lds + wave * 256 + lane * 4) = u;
    __syncthreads();   // U complete, S read by everyone
    rc_f32x4 ub[NB];
#pragma unroll
    for (int I = 0; I < NB; ++I) ub[I] = *reinterpret_cast<const rc_f32x4*>(u_lds + I * 256 + lane * 4);
#pragma unroll
    for (int i = 0; i < OWN; ++i) {
      const int j = wave + i * kScanWaves, jj = j < kt ? j : kt - 1;
      S[i][0] *= fg[i].x;
      S[i][1] *= fg[i].y;
      S[i][2] *= fg[i].z;
      S[i][3] *= fg[i].w;
      fg[i] = *reinterpret_cast<const float4*>(nx - lane * 4 + sp.gamma() + 16 * jj + 4 * quarter);
      if (EXTRA) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][r] += fs[i][r];
        fs[i] = *reinterpret_cast<const rc_f32x4*>(nx + sp.s() + (jj * sp.vt + slice) * 256);
      }
#pragma unroll
      for (int I = 0; I < NB; ++I) {
        S[i] = mfma4(fk[i][I], ub[I], S[i]);
        fk[i][I] = *reinterpret_cast<const float4*>(nx + sp.kT() + (jj * NB + I) * 256);
      }
      if (j < kt) *reinterpret_cast<rc_f32x4*>(s_lds + j * 256 + lane * 4) = S[i];
    }
    if (rows_mine) {
#pragma unroll
      for (int J = 0; J < NB; ++J) {
        if (J <= wave) o = mfma4(fa[J], ub[J], o);
        fa[J] = *reinterpret_cast<const float4*>(nx + sp.aqk() + (wb * NB + (J <= wb ? J : wb)) * 256);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = n * C + 16 * wave + 4 * quarter + r;
        if (t < a.n && col_ok) a.o_buf[(((int64_t)b * a.n + t) * a.H + h) * a.dv + col] = o[r];
      }
    }
    __syncthreads();   // S complete, U read by everyone
  }
#pragma unroll
  for (int i = 0; i < OWN; ++i) {
    const int j = wave + i * kScanWaves;
    if (j < kt && col_ok) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * j + 4 * quarter + r;
        if (row < a.dk) Sg[(int64_t)row * a.dv + col] = S[i][r];
      }
    }
  }
}

// The read-outs' norm and gate: LPH lanes per (token, head), V neighbouring values each and
// LPH * V apart.
template <class DT, int LPH, int V>
__global__ __launch_bounds__(256) void recurrence_out_kernel(socket_recurrence a) {
  const int sub = threadIdx.x % LPH;
  const int64_t w = (int64_t)blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const bool live = w < (int64_t)a.B * a.n * a.H;    // (every lane takes part in the sum)
  const int64_t wl = live ? w : 0;
  const int h = (int)(wl % a.H), dv = a.dv;
  const int64_t bt = wl / a.H;
  const int t = (int)(bt % a.n), b = (int)(bt / a.n);
  const float* o = a.o_buf + wl * dv;
  float ss = 0.f;
  for (int c = sub * V; c < dv; c += LPH * V) {
    float x[V];
    load_vec<DType_f32, V>(o, c, x);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(x[e], x[e], ss);
  }
  const float rs = rsqrt_f32(group_sum<LPH>(ss) / (float)dv + a.eps);
  if (!live) return;
  const int64_t dst = ((int64_t)b * a.T + a.t0 + t) * a.H * dv + (int64_t)h * dv;
  const int64_t gsrc = a.gate_w ? dst : b * a.proj_stride_b + (a.t0 + t) * a.proj_stride_t + a.gate_off + h * dv;
  for (int c = sub * V; c < dv; c += LPH * V) {
    float x[V], g[V], nw[V];
    load_vec<DType_f32, V>(o, c, x);
    load_vec<DT, V>(a.gate_w ? a.gate_z : a.proj, gsrc + c, g);
    load_vec<DType_f32, V>(a.norm_w, (a.norm_per_head ? h * dv : 0) + c, nw);
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = x[e] * rs * nw[e] * gate_act(a.gate_kind, g[e]);
    store_vec<DT, V>(a.out, dst + c, x);
  }
}

// The last taps - 1 inputs of a portion (older ones from the state where the portion is shorter).
// One lane per channel, rows in ascending order: row m reads row m + T of the same half at most.
template <class DT>
__global__ __launch_bounds__(256) void conv_tail_kernel(socket_recurrence a) {
  const int C = conv_channels(a), ch = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (ch >= C) return;
  const int qk = a.Hk * a.dk, n1 = a.taps - 1;
  const int col = ch < qk ? a.q_off + ch : (ch < 2 * qk ? a.k_off + ch - qk : a.v_off + ch - 2 * qk);
  const int64_t from = ((int64_t)(a.pos0 & 1) * a.B + b) * n1 * C + ch;
  const int64_t to = ((int64_t)((a.pos0 + a.T) & 1) * a.B + b) * n1 * C + ch;
  for (int m = 0; m < n1; ++m) {
    const int t = a.T - n1 + m;
    float x = 0.f;
    if (t >= 0) x = load_elem<DT>(a.proj, b * a.proj_stride_b + t * a.proj_stride_t + col);
    else if (!a.fresh) x = load_elem<DT>(a.conv_state, from + (int64_t)(t + n1) * C);
    store_elem<DT>(a.conv_state, to + (int64_t)m * C, x);
  }
}

template <class DT>
__global__ __launch_bounds__(256) void tanh_rows_kernel(const void* x, int64_t x_stride, void* y, int64_t items, int cols) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i < items) store_elem<DT>(y, i, tanh_f32(load_elem<DT>(x, i / cols * x_stride + i % cols)));
}

int chunk_blocks(int dk, int rule) { return dk <= (rule == 1 ? 64 : 128) ? 4 : 2; }

int check_recurrence(const socket_recurrence* p) {
  SOCKET_REQUIRE(p && p->proj && p->state && p->out && p->norm_w, SOCKET_ERR_NULL);
  const socket_recurrence& a = *p;
  SOCKET_REQUIRE(a.dtype == SOCKET_F32 || a.dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.B > 0 && a.B <= 65535 && a.T > 0 && a.H > 0 && a.H <= 65535 && a.Hk > 0 && a.H % a.Hk == 0 && a.dk > 0 && a.dv > 0,
                 SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.dk <= 256 && a.dv <= 256, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE((a.taps < 1 || a.conv_w) && (a.taps <= 1 || a.conv_state), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.taps >= 0 && a.taps <= 32, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.rule == 0 || a.rule == 1, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.rule == 1 ? a.decay_kind == 2 : (a.decay_kind == 0 || a.decay_kind == 1) && !a.decay_tanh, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.rule == 0 || (a.H == a.Hk && a.taps == 0 && !a.gate_w && a.decay_tanh && a.rate_off >= 0), SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.rule == 0 || (a.decay_rate >= 0.f && a.decay_rate * kRcLog2e * 16 * chunk_blocks(a.dk, 1) <= kMaxChunkDecay),
                 SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.gate_kind == 0 || a.gate_kind == 1, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(a.decay_kind != 0 || a.a_log, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(socket_aligned16(a.state) && socket_aligned16(a.proj), SOCKET_ERR_ALIGN);
  return SOCKET_OK;
}

template <class DT>
int launch_step(const socket_recurrence& a, hipStream_t s) {
  const int vec = a.dv % 4 == 0 ? 4 : 1;
  const int nc = a.dv / vec;
  // lanes enough to hold the state in at most 16 registers each where 1024 allow it
  int nt = 256;
  auto rows_of = [&](int n) { const int rg = n / nc; return (a.dk + rg - 1) / rg; };
  const int want = 16 / vec;
  while (nt < 1024 && rows_of(nt) > want) nt *= 2;
  const int rows = rows_of(nt);
  StepShape sh{nc, -1, nt / nc};
  if ((nc & (nc - 1)) == 0)
    for (sh.nc_shift = 0; (1 << sh.nc_shift) < nc; ++sh.nc_shift) {}
  const bool general = a.rule == 1;
  const size_t lds = (size_t)((general ? 4 : 3) * a.dk + 3 * a.dv + 16 + sh.RG * a.dv) * 4;
  SOCKET_REQUIRE(lds <= 48 * 1024, SOCKET_ERR_UNSUPPORTED);
  const dim3 grid((unsigned)(a.H / a.Hk), (unsigned)a.Hk, (unsigned)a.B), block((unsigned)nt);
#define SOCKET_STEP(V, R)                                                                                        \
  do {                                                                                                           \
    if (general) hipLaunchKernelGGL((recurrence_step_kernel<DT, V, R, true>), grid, block, lds, s, a, sh);       \
    else hipLaunchKernelGGL((recurrence_step_kernel<DT, V, R, false>), grid, block, lds, s, a, sh);              \
  } while (0)
  if (vec == 4) {
    if (rows <= 4) SOCKET_STEP(4, 4);
    else if (rows <= 8) SOCKET_STEP(4, 8);
    else if (rows <= 16) SOCKET_STEP(4, 16);
    else return SOCKET_ERR_UNSUPPORTED;
  } else {
    if (rows <= 16) SOCKET_STEP(1, 16);
    else if (rows <= 32) SOCKET_STEP(1, 32);
    else if (rows <= 64) SOCKET_STEP(1, 64);
    else return SOCKET_ERR_UNSUPPORTED;
  }
#undef SOCKET_STEP
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

template <class DT, int NB>
int launch_prep(const socket_recurrence& a, int n_chunks, bool vec, hipStream_t s) {
  constexpr int C = 16 * NB;
  const ChunkSpace sp{(a.dk + 15) / 16, (a.dv + 15) / 16, NB};
  const int dkp = sp.kt * 16, kp = dkp + 4, vp = sp.vt * 16 + 4;
  const size_t lds = (size_t)(C * (kp > vp ? kp : vp) + 2 * C * kp + NB * dkp + NB * NB * 256 + C) * 4;
  SOCKET_REQUIRE(lds <= (size_t)socket_device_limits().max_lds_per_block, SOCKET_ERR_UNSUPPORTED);
  auto kern = recurrence_prep_kernel<DT, NB>;
  if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return SOCKET_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3((unsigned)n_chunks, (unsigned)a.H, (unsigned)a.B), dim3(kPrepThreads), lds, s, a, vec ? 1 : 0);
  return SOCKET_OK;
}

template <class DT, int NB>
int launch_general_prep(const socket_recurrence& a, int n_chunks, bool vec, hipStream_t s) {
  constexpr int C = 16 * NB;
  const int dkp = (a.dk + 15) / 16 * 16, dvp = (a.dv + 15) / 16 * 16;
  const size_t limit = (size_t)socket_device_limits().max_lds_per_block, own_v = (size_t)C * (dvp + 4) * 4;
  size_t lds = (size_t)(4 * C * (dkp + 4) + NB * dkp + 3 * NB * NB * 256 + C) * 4;
  const int late_v = lds + own_v > limit && dvp <= dkp ? 1 : 0;
  if (!late_v) lds += own_v;
  SOCKET_REQUIRE(lds <= limit, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(C * dkp / 4 <= kGeneralItems * kPrepThreads, SOCKET_ERR_UNSUPPORTED);
  auto kern = general_prep_kernel<DT, NB>;
  if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return SOCKET_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3((unsigned)n_chunks, (unsigned)a.H, (unsigned)a.B), dim3(kPrepThreads), lds, s, a, vec ? 1 : 0,
                     late_v);
  return SOCKET_OK;
}

template <int NB, bool DELTA, bool EXTRA = false>
int launch_scan(const socket_recurrence& a, int n_chunks, hipStream_t s) {
  const int kt = (a.dk + 15) / 16, slices = (a.dv + 15) / 16;
  const dim3 grid((unsigned)((int64_t)slices * a.B * a.H)), block(kScanThreads);
#define SOCKET_SCAN(KT) hipLaunchKernelGGL((recurrence_scan_kernel<KT, NB, DELTA, EXTRA>), grid, block, 0, s, a, n_chunks, slices)
  if constexpr (NB == 4) {
    if (kt <= 2) SOCKET_SCAN(2);
    else if (kt <= 4) SOCKET_SCAN(4);
    else if (kt <= 6) SOCKET_SCAN(6);
    else SOCKET_SCAN(8);
  } else {
    if (EXTRA && kt <= 8) SOCKET_SCAN(8);
    else if (kt <= 12) SOCKET_SCAN(12);
    else SOCKET_SCAN(16);
  }
#undef SOCKET_SCAN
  return SOCKET_OK;
}

}  // namespace

extern "C" int socket_recurrence_step(const socket_recurrence* args, void* stream) {
  const int rc = check_recurrence(args);
  if (rc != SOCKET_OK) return rc;
  const socket_recurrence& a = *args;
  SOCKET_REQUIRE(a.pos && a.decay_w && a.decay_rank > 0, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.T == 1 && !a.fresh, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(!a.gate_w || a.gate_rank > 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(socket_aligned16(a.decay_w) && (!a.gate_w || socket_aligned16(a.gate_w)), SOCKET_ERR_ALIGN);
  hipStream_t s = (hipStream_t)stream;
  return a.dtype == SOCKET_F32 ? launch_step<DType_f32>(a, s) : launch_step<DType_bf16>(a, s);
}

extern "C" int socket_recurrence_chunk(int dk, int rule) { return 16 * chunk_blocks(dk, rule); }

extern "C" size_t socket_recurrence_workspace_bytes(int B, int n, int H, int dk, int dv, int rule) {
  if (B <= 0 || n <= 0 || H <= 0 || dk <= 0 || dv <= 0) return 0;
  const int nb = chunk_blocks(dk, rule), C = 16 * nb;
  const ChunkSpace sp{(dk + 15) / 16, (dv + 15) / 16, nb, rule == 1};
  return (size_t)B * H * ((n + C - 1) / C) * sp.size() * sizeof(float);
}

extern "C" int socket_recurrence_scan(const socket_recurrence* args, void* stream) {
  const int rc = check_recurrence(args);
  if (rc != SOCKET_OK) return rc;
  const socket_recurrence& a = *args;
  SOCKET_REQUIRE(a.decay_z && a.o_buf && a.workspace && (!a.gate_w || a.gate_z), SOCKET_ERR_NULL);
  SOCKET_REQUIRE(a.t0 >= 0 && a.n > 0 && a.t0 + a.n <= a.T && a.pos0 >= 0, SOCKET_ERR_SHAPE);
  SOCKET_REQUIRE(a.workspace_bytes >= socket_recurrence_workspace_bytes(a.B, a.n, a.H, a.dk, a.dv, a.rule), SOCKET_ERR_WORKSPACE);
  SOCKET_REQUIRE(socket_aligned16(a.workspace), SOCKET_ERR_ALIGN);
  hipStream_t s = (hipStream_t)stream;
  const int nb = chunk_blocks(a.dk, a.rule), C = 16 * nb, n_chunks = (a.n + C - 1) / C;
  const int per = 8;
  const bool vec = a.dk % 8 == 0 && a.dv % 8 == 0 && a.q_off % per == 0 && a.k_off % per == 0 && a.v_off % per == 0 &&
                   a.proj_stride_b % per == 0 && a.proj_stride_t % per == 0 &&
                   (a.taps < 1 || socket_aligned16(a.conv_w)) && (a.taps <= 1 || socket_aligned16(a.conv_state));
  const bool delta = a.beta_off >= 0;
  int st;
  if (a.rule == 1) {
    if (nb == 4)
      st = a.dtype == SOCKET_F32 ? launch_general_prep<DType_f32, 4>(a, n_chunks, vec, s)
                                 : launch_general_prep<DType_bf16, 4>(a, n_chunks, vec, s);
    else
      st = a.dtype == SOCKET_F32 ? launch_general_prep<DType_f32, 2>(a, n_chunks, vec, s)
                                 : launch_general_prep<DType_bf16, 2>(a, n_chunks, vec, s);
  } else if (nb == 4)
    st = a.dtype == SOCKET_F32 ? launch_prep<DType_f32, 4>(a, n_chunks, vec, s) : launch_prep<DType_bf16, 4>(a, n_chunks, vec, s);
  else
    st = a.dtype == SOCKET_F32 ? launch_prep<DType_f32, 2>(a, n_chunks, vec, s) : launch_prep<DType_bf16, 2>(a, n_chunks, vec, s);
  if (st != SOCKET_OK) return st;
  SOCKET_LAUNCH_CHECK();
  if (a.rule == 1) st = nb == 4 ? launch_scan<4, true, true>(a, n_chunks, s) : launch_scan<2, true, true>(a, n_chunks, s);
  else if (nb == 4) st = delta ? launch_scan<4, true>(a, n_chunks, s) : launch_scan<4, false>(a, n_chunks, s);
  else st = delta ? launch_scan<2, true>(a, n_chunks, s) : launch_scan<2, false>(a, n_chunks, s);
  if (st != SOCKET_OK) return st;
  SOCKET_LAUNCH_CHECK();
  const int64_t items = (int64_t)a.B * a.n * a.H;
  SOCKET_REQUIRE((items + 3) / 4 < (1LL << 31), SOCKET_ERR_SHAPE);
  const bool v8 = vec && a.gate_off % 8 == 0 && socket_aligned16(a.out) && socket_aligned16(a.o_buf) &&
                  socket_aligned16(a.norm_w) && (!a.gate_w || socket_aligned16(a.gate_z));
#define SOCKET_OUT(DT, LPH, V)                                                                                    \
  hipLaunchKernelGGL((recurrence_out_kernel<DT, LPH, V>), dim3((unsigned)((items + 256 / LPH - 1) / (256 / LPH))), \
                     dim3(256), 0, s, a)
  if (a.dtype == SOCKET_F32) {
    if (v8) SOCKET_OUT(DType_f32, 16, 8);
    else SOCKET_OUT(DType_f32, 64, 1);
  } else {
    if (v8) SOCKET_OUT(DType_bf16, 16, 8);
    else SOCKET_OUT(DType_bf16, 64, 1);
  }
#undef SOCKET_OUT
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_tanh_rows(const void* x, int64_t x_stride, void* y, int dtype, int64_t rows, int cols, void* stream) {
  SOCKET_REQUIRE(x && y, SOCKET_ERR_NULL);
  SOCKET_REQUIRE(dtype == SOCKET_F32 || dtype == SOCKET_BF16, SOCKET_ERR_UNSUPPORTED);
  SOCKET_REQUIRE(rows > 0 && cols > 0 && x_stride >= cols, SOCKET_ERR_SHAPE);
  const int64_t items = rows * cols;
  SOCKET_REQUIRE((items + 255) / 256 < (1LL << 31), SOCKET_ERR_SHAPE);
  const dim3 grid((unsigned)((items + 255) / 256)), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == SOCKET_F32) hipLaunchKernelGGL((tanh_rows_kernel<DType_f32>), grid, block, 0, s, x, x_stride, y, items, cols);
  else hipLaunchKernelGGL((tanh_rows_kernel<DType_bf16>), grid, block, 0, s, x, x_stride, y, items, cols);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}

extern "C" int socket_recurrence_conv_tail(const socket_recurrence* args, void* stream) {
  const int rc = check_recurrence(args);
  if (rc != SOCKET_OK) return rc;
  const socket_recurrence& a = *args;
  if (a.taps <= 1) return SOCKET_OK;
  const int C = 2 * a.Hk * a.dk + a.H * a.dv;
  const dim3 grid((unsigned)((C + 255) / 256), (unsigned)a.B), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == SOCKET_F32) hipLaunchKernelGGL((conv_tail_kernel<DType_f32>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((conv_tail_kernel<DType_bf16>), grid, block, 0, s, a);
  SOCKET_LAUNCH_CHECK();
  return SOCKET_OK;
}
