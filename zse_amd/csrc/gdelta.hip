// The generalized delta rule: a recurrent mixer with a matrix state S [D, D] per head whose rows
// decay each at its own rate and lose, per row, what they held along the key.
//
//   u_t = k_t / sqrt(sum k_t^2 + 1e-6)
//   S <- diag(w_t) S - (a_t * u_t) (u_t^T S) + k_t v_t^T       (both terms read the old S)
//   o_t = S^T r_t
//
// with w_t = exp(-exp(-1/2) sigmoid(z_t)) and a_t = sigmoid(y_t) per key channel; the read-out is
// divided by its root mean square over the head, times a gain per channel of all heads and
// sigmoid(g_t).
//
// The recurrence never mixes value channels: column e of S and o depends on column e alone, and
// k_t = |k_t| u_t, so with d = sum_i u_i S_i (old) a row becomes w_i S_i + u_i (|k| v_e - a_i d).
//
// Three ways through it, one arithmetic:
//  - the walk (gdelta_kernel): DS neighbouring lanes own one column of S, each a share of its rows in
//    registers (row chunks of four, dealt out in turn), and walk the tokens of their request; the
//    two sums over the rows are joined across the lanes by lane permutations inside the wave, no
//    local memory and no barrier.  u, r, w and a of a group of tokens wait in local memory.  The
//    order of every sum follows from the channel numbers alone: in the 32-bit library, which has
//    only this one, a request's values are the same bits however its tokens are cut into steps.
//  - single tokens (gdelta_token_kernel): a block a head, a thread a column's share of the rows, the
//    state read and written in whole lines.
//  - long portions (gdelta_chunk_kernel, gdelta_scan_kernel): chunks of 32 tokens as matrix products on the
//    32-bit matrix cores.  With b_t the product of a chunk's decays up to token t (b_0 = 1; a decay is at least
//    exp(-exp(-1/2)), so 1 / b stays below 3e8) and the rows
//        B_t = u_t b_(t-1),   A_t = -(a_t u_t) / b_t,   K_t = k_t / b_t,   R_t = r_t b_t
//    what the tokens of a chunk find along their keys is Y = B S_0 + L Y + M V with L = B A^T and
//    M = B K^T below the diagonal, so with T = (I - L)^-1
//        Y = (T B) S_0 + P V,                        P = T M
//        O = (R + Q T B) S_0 + (N + Q P) V           Q = R A^T, N = R K^T up to the diagonal
//        S = b_32 (S_0 + A^T (T B) S_0 + (K + P^T A)^T V)
//    The first kernel makes, for all chunks side by side, everything that does not know S_0 or V and lays it
//    out as the operands of the second, which goes through a request's chunks in order: a block a head and
//    16 value channels, its waves sharing out the rows of S, which stays in the accumulators (the order
//    in which they lie there is a valid order of contraction, so they are operands as they are).
#include "common.h"
#include "packed_call.h"

extern "C" int zk_steplist_register(const char* name, int nargs, void* fn);
#define ZK_ENTER(fn) \
  static const int fn##_entered = zk_steplist_register(#fn, zk_packed::Call<fn>::nargs, (void*)zk_packed::Call<fn>::call);

#define GD_COLS_LONG 16           // value channels a block takes when portions are long

__device__ __forceinline__ float gd_sum8(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x141, 0xf, 0xf, false));   // row_half_mirror
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0xB1, 0xf, 0xf, false));    // quad_perm [1,0,3,2]
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x4E, 0xf, 0xf, false));    // quad_perm [2,3,0,1]
  return x;
}
__device__ __forceinline__ float gd_sum16(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x140, 0xf, 0xf, false));   // row_mirror
  return gd_sum8(x);
}
__device__ __forceinline__ float gd_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---- the decays and removal rates of a step's tokens
//
//   w = exp(-exp(-1/2) sigmoid(W2 tanh(low) + w0)),   a = sigmoid(y + a0)
//
// rows: float [T, ld] with y at column 0 (n of them) and low (rank of them) at low_off.  A block
// takes GD_TOKENS tokens and 256 channels; tanh(low) of its tokens waits in local memory.
#define GD_TOKENS 8
template <bool VEC>
__global__ __launch_bounds__(256) void gdelta_gates_kernel(const float* __restrict__ rows, int ld, int low_off, int rank,
                                                           const act_t* __restrict__ w2, const float* __restrict__ w0,
                                                           const float* __restrict__ a0, float* __restrict__ decay,
                                                           float* __restrict__ rate, int T, int n) {
  extern __shared__ __attribute__((aligned(16))) float low[];          // [rank][GD_TOKENS]
  const int t0 = blockIdx.y * GD_TOKENS, nt = min(GD_TOKENS, T - t0);
  for (int i = threadIdx.x; i < rank * GD_TOKENS; i += 256) {
    const int k = i / GD_TOKENS, tt = i % GD_TOKENS;
    low[i] = tt < nt ? tanhf(rows[(size_t)(t0 + tt) * ld + low_off + k]) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= n) return;
  float acc[GD_TOKENS];
#pragma unroll
  for (int tt = 0; tt < GD_TOKENS; tt++) acc[tt] = 0.f;
  const act_t* wr = w2 + (size_t)c * rank;
  auto add = [&](int k, float x) {
    const float4 p = *(const float4*)(low + k * GD_TOKENS), q = *(const float4*)(low + k * GD_TOKENS + 4);
    acc[0] = fmaf(x, p.x, acc[0]);
    acc[1] = fmaf(x, p.y, acc[1]);
    acc[2] = fmaf(x, p.z, acc[2]);
    acc[3] = fmaf(x, p.w, acc[3]);
    acc[4] = fmaf(x, q.x, acc[4]);
    acc[5] = fmaf(x, q.y, acc[5]);
    acc[6] = fmaf(x, q.z, acc[6]);
    acc[7] = fmaf(x, q.w, acc[7]);
  };
  if (VEC) {
    for (int k = 0; k < rank; k += 8) {
      act_t v[8];
#if ZSE_ACT_BF16
      *(uint4*)v = *(const uint4*)(wr + k);
#else
      *(float4*)v = *(const float4*)(wr + k);
      *(float4*)(v + 4) = *(const float4*)(wr + k + 4);
#endif
#pragma unroll
      for (int e = 0; e < 8; e++) add(k + e, to_f32(v[e]));
    }
  } else {
    for (int k = 0; k < rank; k++) add(k, to_f32(wr[k]));
  }
  const float shift = w0[c], bias = a0 ? a0[c] : 0.f;
  for (int tt = 0; tt < nt; tt++) {
    const size_t at = (size_t)(t0 + tt) * n + c;
    float x = acc[0];
#pragma unroll
    for (int i = 1; i < GD_TOKENS; i++) x = i == tt ? acc[i] : x;
    decay[at] = expf(-0.6065306597126334f * gd_sigmoid(x + shift));
    rate[at] = gd_sigmoid(rows[(size_t)(t0 + tt) * ld + c] + bias);
  }
}

// ---- the walk.  DS lanes share a column (8 or 16), each holds CH chunks of four rows of S (4 CH DS rows in
// all, D padded with zeros).  raw (may be null): float [T, H * D], the read-outs before their norm, for a
// head that spans several blocks.
template <int CH, int DS>
__global__ __launch_bounds__(1024) void gdelta_kernel(const act_t* __restrict__ rkv, int ld, int k_off, int v_off,
                                                      const act_t* __restrict__ g, int ldg, const float* __restrict__ decay,
                                                      const float* __restrict__ rate, const float* __restrict__ gain,
                                                      float* __restrict__ state, int slot_words, int offset_words,
                                                      const int* __restrict__ q_start, const int* __restrict__ slot_of_req,
                                                      act_t* __restrict__ out, float* __restrict__ raw, int H, int D,
                                                      float eps, int COLS, int GRP) {
  constexpr int DMAX = 4 * CH * DS, RD = 4 * CH;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* rs = lds;                                 // [GRP][DMAX] each
  float* us = rs + GRP * DMAX;
  float* ws = us + GRP * DMAX;
  float* as = ws + GRP * DMAX;
  float* ov = as + GRP * DMAX;                     // [GRP][COLS]: |k| v going in, the read-out coming back
  float* kn = ov + GRP * COLS;                     // [GRP]: |k|
  const int r = blockIdx.x, h = blockIdx.y, e0 = blockIdx.z * COLS, tid = threadIdx.x, nt = blockDim.x;
  const int lane = tid & 63, wave = tid >> 6, nw = nt >> 6;
  const int col = tid / DS, j = tid % DS, e = e0 + col;
  const int t0 = q_start[r], t1 = q_start[r + 1];
  if (t1 <= t0) return;
  const bool live = e < D;
  const int cols = min(COLS, D - e0);
  float* S = state + (size_t)slot_of_req[r] * slot_words + offset_words + (size_t)h * D * D;
  float s[RD];
#pragma unroll
  for (int i = 0; i < CH; i++)
#pragma unroll
    for (int c = 0; c < 4; c++) {
      const int d = 4 * (j + DS * i) + c;
      s[4 * i + c] = (live && d < D) ? S[(size_t)d * D + e] : 0.f;
    }
  for (int c0 = t0; c0 < t1; c0 += GRP) {
    const int n = min(GRP, t1 - c0);
    __syncthreads();
    for (int i = tid; i < n * DMAX; i += nt) {
      const int tt = i / DMAX, d = i % DMAX;
      const bool in = d < D;
      const act_t* row = rkv + (size_t)(c0 + tt) * ld + (size_t)h * D + d;
      const size_t at = ((size_t)(c0 + tt) * H + h) * D + d;
      rs[i] = in ? to_f32(row[0]) : 0.f;
      us[i] = in ? to_f32(row[k_off]) : 0.f;
      ws[i] = in ? decay[at] : 0.f;                // padding rows of S stay zero
      as[i] = in ? rate[at] : 0.f;
    }
    for (int i = tid; i < n * COLS; i += nt) {
      const int tt = i / COLS, c = i % COLS;
      ov[i] = c < cols ? to_f32(rkv[(size_t)(c0 + tt) * ld + v_off + (size_t)h * D + e0 + c]) : 0.f;
    }
    __syncthreads();
    // unit keys: 16 lanes a row, their sum of squares joined inside the lanes' row
    for (int tt = tid >> 4; tt < n; tt += nt >> 4) {
      float* row = us + tt * DMAX;
      const int l16 = tid & 15;
      float ss = 0.f;
      for (int d = l16; d < DMAX; d += 16) ss = fmaf(row[d], row[d], ss);
      const float norm = sqrtf(gd_sum16(ss) + 1e-6f), inv = 1.0f / norm;
      for (int d = l16; d < DMAX; d += 16) row[d] *= inv;
      if (l16 == 0) kn[tt] = norm;
    }
    __syncthreads();
    for (int tt = 0; tt < n; tt++) {
      const float4* r4 = (const float4*)(rs + tt * DMAX) + j;
      const float4* u4 = (const float4*)(us + tt * DMAX) + j;
      const float4* w4 = (const float4*)(ws + tt * DMAX) + j;
      const float4* a4 = (const float4*)(as + tt * DMAX) + j;
      const float kv = kn[tt] * ov[tt * COLS + col];
      float4 uu[CH];
      float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
#pragma unroll
      for (int i = 0; i < CH; i++) {
        uu[i] = u4[DS * i];
        d0 = fmaf(s[4 * i], uu[i].x, d0);
        d1 = fmaf(s[4 * i + 1], uu[i].y, d1);
        d2 = fmaf(s[4 * i + 2], uu[i].z, d2);
        d3 = fmaf(s[4 * i + 3], uu[i].w, d3);
      }
      const float dot = DS == 16 ? gd_sum16((d0 + d1) + (d2 + d3)) : gd_sum8((d0 + d1) + (d2 + d3));
      d0 = d1 = d2 = d3 = 0.f;
#pragma unroll
      for (int i = 0; i < CH; i++) {
        const float4 ww = w4[DS * i], aa = a4[DS * i], rr = r4[DS * i];
        s[4 * i] = fmaf(ww.x, s[4 * i], uu[i].x * fmaf(-aa.x, dot, kv));
        s[4 * i + 1] = fmaf(ww.y, s[4 * i + 1], uu[i].y * fmaf(-aa.y, dot, kv));
        s[4 * i + 2] = fmaf(ww.z, s[4 * i + 2], uu[i].z * fmaf(-aa.z, dot, kv));
        s[4 * i + 3] = fmaf(ww.w, s[4 * i + 3], uu[i].w * fmaf(-aa.w, dot, kv));
        d0 = fmaf(s[4 * i], rr.x, d0);
        d1 = fmaf(s[4 * i + 1], rr.y, d1);
        d2 = fmaf(s[4 * i + 2], rr.z, d2);
        d3 = fmaf(s[4 * i + 3], rr.w, d3);
      }
      const float o = DS == 16 ? gd_sum16((d0 + d1) + (d2 + d3)) : gd_sum8((d0 + d1) + (d2 + d3));
      // a column's v of this token was read (by its lanes, all in one wave) before the read-out
      // takes its place
      if (j == 0) ov[tt * COLS + col] = o;
    }
    __syncthreads();
    if (raw != nullptr) {                          // the head spans several blocks: its norm comes later
      for (int i = tid; i < n * COLS; i += nt) {
        const int tt = i / COLS, c = i % COLS;
        if (c < cols) raw[((size_t)(c0 + tt) * H + h) * D + e0 + c] = ov[i];
      }
      continue;
    }
    for (int tt = wave; tt < n; tt += nw) {        // unit RMS over the head's read-out, gain, gate
      float ss = 0.f;
      for (int c = lane; c < D; c += 64) ss = fmaf(ov[tt * COLS + c], ov[tt * COLS + c], ss);
      ss = wave_sum(ss);
      const float inv = 1.0f / sqrtf(ss / (float)D + eps);
      const act_t* gr = g + (size_t)(c0 + tt) * ldg + (size_t)h * D;
      act_t* orow = out + ((size_t)(c0 + tt) * H + h) * D;
      for (int c = lane; c < D; c += 64)
        orow[c] = from_f32<act_t>(ov[tt * COLS + c] * inv * gain[(size_t)h * D + c] * gd_sigmoid(to_f32(gr[c])));
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < CH; i++)
#pragma unroll
      for (int c = 0; c < 4; c++) {
        const int d = 4 * (j + DS * i) + c;
        if (d < D) S[(size_t)d * D + e] = s[4 * i + c];
      }
  }
}

// One wave per (token, head): out = raw / sqrt(mean(raw^2) + eps) * gain * sigmoid(g).
__global__ __launch_bounds__(64) void gdelta_finish_kernel(const float* __restrict__ raw, const act_t* __restrict__ g, int ldg,
                                                           const float* __restrict__ gain, const int* __restrict__ positions,
                                                           act_t* __restrict__ out, int H, int D, float eps) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const float* rr = raw + ((size_t)t * H + h) * D;
  act_t* orow = out + ((size_t)t * H + h) * D;
  if (positions[t] < 0) {                          // a padding row of a captured step
    for (int c = lane; c < D; c += 64) orow[c] = from_f32<act_t>(0.f);
    return;
  }
  float ss = 0.f;
  for (int c = lane; c < D; c += 64) ss = fmaf(rr[c], rr[c], ss);
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)D + eps);
  const act_t* gr = g + (size_t)t * ldg + (size_t)h * D;
  for (int c = lane; c < D; c += 64)
    orow[c] = from_f32<act_t>(rr[c] * inv * gain[(size_t)h * D + c] * gd_sigmoid(to_f32(gr[c])));
}

#if ZSE_ACT_BF16
// ---- single tokens: a block per (head, token), P = threads / D threads a column, each RP = D / P of its
// rows.  Every row with a negative position (padding) comes out as 0.
template <int RP>
__global__ __launch_bounds__(1024) void gdelta_token_kernel(const act_t* __restrict__ rkv, int ld, int k_off, int v_off,
                                                            const act_t* __restrict__ g, int ldg,
                                                            const float* __restrict__ decay, const float* __restrict__ rate,
                                                            const float* __restrict__ gain, float* __restrict__ state,
                                                            int slot_words, int offset_words,
                                                            const int* __restrict__ positions,
                                                            const int* __restrict__ req_of_token,
                                                            const int* __restrict__ slot_of_req, act_t* __restrict__ out,
                                                            int H, int D, float eps) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* us = lds;                   // [D] each
  float* rs = us + D;
  float* ws = rs + D;
  float* as = ws + D;
  float* part = as + D;              // [P][D]
  __shared__ float red[17];
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, P = blockDim.x / D;
  const int e = tid % D, p = tid / D;
  act_t* orow = out + ((size_t)t * H + h) * D;
  if (positions[t] < 0) {
    if (p == 0) orow[e] = from_f32<act_t>(0.f);
    return;
  }
  float* S = state + (size_t)slot_of_req[req_of_token[t]] * slot_words + offset_words + (size_t)h * D * D;
  float s[RP];
#pragma unroll
  for (int i = 0; i < RP; i++) s[i] = S[(size_t)(p * RP + i) * D + e];
  const act_t* row = rkv + (size_t)t * ld + (size_t)h * D;
  const float v = to_f32(row[v_off + e]);
  float kk = 0.f;
  if (p == 0) {
    const size_t at = ((size_t)t * H + h) * D + e;
    kk = to_f32(row[k_off + e]);
    us[e] = kk;
    rs[e] = to_f32(row[e]);
    ws[e] = decay[at];
    as[e] = rate[at];
  }
  const float norm = sqrtf(block_sum(kk * kk, red) + 1e-6f);      // its barriers also make us, rs, ws, as visible
  const float inv = 1.0f / norm;
  float dot = 0.f;
#pragma unroll
  for (int i = 0; i < RP; i++) dot = fmaf(us[p * RP + i] * inv, s[i], dot);
  part[p * D + e] = dot;
  __syncthreads();
  dot = 0.f;
  for (int q = 0; q < P; q++) dot += part[q * D + e];
  __syncthreads();
  float o = 0.f;
  const float kv = norm * v;
#pragma unroll
  for (int i = 0; i < RP; i++) {
    const int d = p * RP + i;
    s[i] = fmaf(ws[d], s[i], us[d] * inv * fmaf(-as[d], dot, kv));
    o = fmaf(s[i], rs[d], o);
  }
#pragma unroll
  for (int i = 0; i < RP; i++) S[(size_t)(p * RP + i) * D + e] = s[i];
  part[p * D + e] = o;
  __syncthreads();
  o = 0.f;
  if (p == 0)
    for (int q = 0; q < P; q++) o += part[q * D + e];
  const float ms = block_sum(p == 0 ? o * o : 0.f, red) / (float)D;
  if (p == 0)
    orow[e] = from_f32<act_t>(o * (1.0f / sqrtf(ms + eps)) * gain[(size_t)h * D + e] *
                              gd_sigmoid(to_f32(g[(size_t)t * ldg + (size_t)h * D + e])));
}
#endif

#if ZSE_ACT_BF16
// ---- long portions, chunk by chunk
typedef float gd_f4 __attribute__((ext_vector_type(4)));
#define GD_CHUNK 32
#define GD_SMALL 36                // the distance between rows of a 32 x 32 matrix in local memory

__device__ __forceinline__ gd_f4 gd_mfma(float a, float b, gd_f4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// What gdelta_chunk_kernel leaves for a (chunk, head), in floats: per 16 channels the operands T B, R + Q T B, A^T,
// K + P^T A (two tiles of 64 lanes x 4 each), the three lower tiles of N + Q P, and b_32.
template <int D>
struct GdWork {
  static constexpr int TILES = D / 16, PER_TILE = 4 * 2 * 64 * 4, N_AT = TILES * PER_TILE, B_AT = N_AT + 3 * 64 * 4;
  static constexpr int FLOATS = B_AT + D;
};

// A block per (chunk, head, request), 8 waves.  Lane l of a wave has lr = l % 16 and g = l / 16: an operand's
// row and its four places in a step of the contraction, or an accumulator's column and its rows 4 g + i.
template <int D>
__global__ __launch_bounds__(512) void gdelta_chunk_kernel(const act_t* __restrict__ rkv, int ld, int k_off,
                                                           const float* __restrict__ decay, const float* __restrict__ rate,
                                                           const int* __restrict__ q_start, int H, int first_chunk,
                                                           float* __restrict__ work) {
  constexpr int LD = D + 4, PARTS = 512 / D, PER = GD_CHUNK / PARTS, NT = D / 16;
  using Wk = GdWork<D>;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* Bm = lds;                               // [32][LD] each
  float* Rm = Bm + GD_CHUNK * LD;
  float* Am = Rm + GD_CHUNK * LD;
  float* Km = Am + GD_CHUNK * LD;
  float* Lm = Km + GD_CHUNK * LD;                // [32][GD_SMALL] each: L, then T
  float* Mm = Lm + GD_CHUNK * GD_SMALL;
  float* Qm = Mm + GD_CHUNK * GD_SMALL;
  float* Nm = Qm + GD_CHUNK * GD_SMALL;
  float* Pm = Nm + GD_CHUNK * GD_SMALL;
  float* kn = Pm + GD_CHUNK * GD_SMALL;          // [32]
  float* pp = kn + GD_CHUNK;                     // [PARTS][D]
  const int h = blockIdx.y, r = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int base = (first_chunk + blockIdx.x) * GD_CHUNK;
  const int n = q_start[r + 1] - q_start[r];
  if (base >= n) return;
  const int m = min(GD_CHUNK, n - base), t0 = q_start[r] + base;
  float* out = work + (((size_t)r * gridDim.x + blockIdx.x) * H + h) * Wk::FLOATS;

  // key lengths, a wave four tokens
  for (int t = wave; t < GD_CHUNK; t += 8) {
    float ss = 0.f;
    if (t < m)
      for (int d = lane; d < D; d += 64) {
        const float x = to_f32(rkv[(size_t)(t0 + t) * ld + k_off + (size_t)h * D + d]);
        ss = fmaf(x, x, ss);
      }
    ss = wave_sum(ss);
    if (lane == 0) kn[t] = sqrtf(ss + 1e-6f);
  }
  // the four scaled rows: a thread PER tokens of a channel; tokens past the portion's end change nothing (decay 1, rows 0)
  {
    const int d = tid % D, part = tid / D;
    float w[PER], prod = 1.f;
#pragma unroll
    for (int i = 0; i < PER; i++) {
      const int t = part * PER + i;
      w[i] = t < m ? decay[((size_t)(t0 + t) * H + h) * D + d] : 1.f;
      prod *= w[i];
    }
    pp[part * D + d] = prod;
    __syncthreads();
    float b = 1.f;
    for (int q = 0; q < part; q++) b *= pp[q * D + d];
#pragma unroll
    for (int i = 0; i < PER; i++) {
      const int t = part * PER + i;
      float kk = 0.f, rr = 0.f, aa = 0.f;
      if (t < m) {
        const act_t* row = rkv + (size_t)(t0 + t) * ld + (size_t)h * D + d;
        rr = to_f32(row[0]);
        kk = to_f32(row[k_off]);
        aa = rate[((size_t)(t0 + t) * H + h) * D + d];
      }
      const float u = kk / kn[t];
      Bm[t * LD + d] = u * b;
      b *= w[i];
      const float ib = 1.0f / b;
      Rm[t * LD + d] = rr * b;
      Am[t * LD + d] = -(aa * u) * ib;
      Km[t * LD + d] = kk * ib;
    }
    if (part == PARTS - 1) out[Wk::B_AT + d] = b;
  }
  __syncthreads();
  // L, M, Q, N: a wave one of them and 16 of its rows
  {
    const int mt = wave >> 2;
    const float* X = (wave & 1) ? Rm : Bm;
    const float* Z = (wave & 2) ? Km : Am;
    float* dst = (wave & 1) ? ((wave & 2) ? Nm : Qm) : ((wave & 2) ? Mm : Lm);
    const int strict = (wave & 1) ? 0 : 1;
    gd_f4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    for (int j = 0; j < NT; j++) {
      const gd_f4 x = *(const gd_f4*)(X + (mt * 16 + lr) * LD + 16 * j + 4 * g);
      const gd_f4 z0 = *(const gd_f4*)(Z + lr * LD + 16 * j + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; i++) acc[0] = gd_mfma(x[i], z0[i], acc[0]);
      if (mt == 1) {
        const gd_f4 z1 = *(const gd_f4*)(Z + (16 + lr) * LD + 16 * j + 4 * g);
#pragma unroll
        for (int i = 0; i < 4; i++) acc[1] = gd_mfma(x[i], z1[i], acc[1]);
      }
    }
#pragma unroll
    for (int nt = 0; nt < 2; nt++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = mt * 16 + 4 * g + i, c = nt * 16 + lr;
        dst[t * GD_SMALL + c] = c + strict <= t ? acc[nt][i] : 0.f;
      }
  }
  __syncthreads();
  // T = (I - L)^-1: the two diagonal blocks by substitution, a lane a column, then T21 = T22 (L21 T11)
  if (wave == 0) {
    float x[16];
    const int o = (lane >> 4 & 1) * 16, c = lane & 15;
#pragma unroll
    for (int t = 0; t < 16; t++) x[t] = t == c ? 1.f : 0.f;
#pragma unroll
    for (int s = 0; s < 15; s++)
#pragma unroll
      for (int t = s + 1; t < 16; t++) x[t] = fmaf(Lm[(o + t) * GD_SMALL + o + s], x[s], x[t]);
    __builtin_amdgcn_wave_barrier();
    if (lane < 32) {
#pragma unroll
      for (int t = 0; t < 16; t++) Lm[(o + t) * GD_SMALL + o + c] = x[t];
    }
    __threadfence_block();
    __builtin_amdgcn_wave_barrier();
    gd_f4 z = {0.f, 0.f, 0.f, 0.f}, t21 = {0.f, 0.f, 0.f, 0.f};
    const gd_f4 l21 = *(const gd_f4*)(Lm + (16 + lr) * GD_SMALL + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; i++) z = gd_mfma(l21[i], Lm[(4 * g + i) * GD_SMALL + lr], z);
    const gd_f4 t22 = *(const gd_f4*)(Lm + (16 + lr) * GD_SMALL + 16 + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; i++) t21 = gd_mfma(t22[i], z[i], t21);
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < 4; i++) Lm[(16 + 4 * g + i) * GD_SMALL + lr] = t21[i];
  }
  __syncthreads();
  // a tile of a lower triangular 32 x 32 product X Z, (mt, nt) with nt <= mt
  auto lower = [&](const float* X, const float* Z, int mt, int nt, gd_f4 acc) {
    for (int kt = nt; kt <= mt; kt++) {
      const gd_f4 x = *(const gd_f4*)(X + (mt * 16 + lr) * GD_SMALL + 16 * kt + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; i++) acc = gd_mfma(x[i], Z[(16 * kt + 4 * g + i) * GD_SMALL + 16 * nt + lr], acc);
    }
    return acc;
  };
  const int lower_m = wave % 3 > 0, lower_n = wave % 3 > 1;            // waves 0, 1, 2 (and 3, 4, 5): tiles (0, 0), (1, 0), (1, 1)
  if (wave < 3) {
    const gd_f4 acc = lower(Lm, Mm, lower_m, lower_n, gd_f4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
    for (int i = 0; i < 4; i++) Pm[(16 * lower_m + 4 * g + i) * GD_SMALL + 16 * lower_n + lr] = acc[i];
  }
  if (wave == 3) {                                                      // above the diagonal: nothing
#pragma unroll
    for (int i = 0; i < 4; i++) Pm[(4 * g + i) * GD_SMALL + 16 + lr] = 0.f;
  }
  // T B, 16 channels at a time
  constexpr int MINE = (NT + 7) / 8;
  gd_f4 tb[MINE][2];
#pragma unroll
  for (int q = 0; q < MINE; q++) {
    const int nt = wave + 8 * q;
    tb[q][0] = tb[q][1] = gd_f4{0.f, 0.f, 0.f, 0.f};
    if (nt < NT) {
      const gd_f4 t00 = *(const gd_f4*)(Lm + lr * GD_SMALL + 4 * g), t10 = *(const gd_f4*)(Lm + (16 + lr) * GD_SMALL + 4 * g),
                  t11 = *(const gd_f4*)(Lm + (16 + lr) * GD_SMALL + 16 + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float b0 = Bm[(4 * g + i) * LD + 16 * nt + lr], b1 = Bm[(16 + 4 * g + i) * LD + 16 * nt + lr];
        tb[q][0] = gd_mfma(t00[i], b0, tb[q][0]);
        tb[q][1] = gd_mfma(t10[i], b0, tb[q][1]);
        tb[q][1] = gd_mfma(t11[i], b1, tb[q][1]);
      }
    }
  }
  __syncthreads();
  if (wave >= 3 && wave < 6) {                                          // N + Q P
    gd_f4 acc;
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] = Nm[(16 * lower_m + 4 * g + i) * GD_SMALL + 16 * lower_n + lr];
    acc = lower(Qm, Pm, lower_m, lower_n, acc);
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < 4; i++) Nm[(16 * lower_m + 4 * g + i) * GD_SMALL + 16 * lower_n + lr] = acc[i];
    __threadfence_block();
    __builtin_amdgcn_wave_barrier();
    *(gd_f4*)(out + Wk::N_AT + ((wave - 3) * 64 + lane) * 4) =
        *(const gd_f4*)(Nm + (16 * lower_m + lr) * GD_SMALL + 16 * lower_n + 4 * g);
  }
#pragma unroll
  for (int q = 0; q < MINE; q++) {
    const int nt = wave + 8 * q;
    if (nt >= NT) continue;
    const int col = 16 * nt + lr;
    gd_f4 rq[2], kp[2], at[2];
#pragma unroll
    for (int tt = 0; tt < 2; tt++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int row = (16 * tt + 4 * g + i) * LD + col;
        rq[tt][i] = Rm[row];
        kp[tt][i] = Km[row];
        at[tt][i] = Am[row];
      }
    const gd_f4 q00 = *(const gd_f4*)(Qm + lr * GD_SMALL + 4 * g), q10 = *(const gd_f4*)(Qm + (16 + lr) * GD_SMALL + 4 * g),
                q11 = *(const gd_f4*)(Qm + (16 + lr) * GD_SMALL + 16 + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      rq[0] = gd_mfma(q00[i], tb[q][0][i], rq[0]);
      rq[1] = gd_mfma(q10[i], tb[q][0][i], rq[1]);
      rq[1] = gd_mfma(q11[i], tb[q][1][i], rq[1]);
      const float* p0 = Pm + (4 * g + i) * GD_SMALL;                    // row 4 g + i of P, as a column of P^T
      const float* p1 = p0 + 16 * GD_SMALL;
      kp[0] = gd_mfma(p0[lr], at[0][i], kp[0]);
      kp[0] = gd_mfma(p1[lr], at[1][i], kp[0]);
      kp[1] = gd_mfma(p1[16 + lr], at[1][i], kp[1]);
    }
    // back into local memory (these columns are this wave's own), to be read along the rows
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int tt = 0; tt < 2; tt++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int row = (16 * tt + 4 * g + i) * LD + col;
        Bm[row] = tb[q][tt][i];
        Rm[row] = rq[tt][i];
      }
    __threadfence_block();
    __builtin_amdgcn_wave_barrier();
    gd_f4* o4 = (gd_f4*)(out + nt * Wk::PER_TILE) + lane;
#pragma unroll
    for (int tt = 0; tt < 2; tt++) {
      o4[(0 + tt) * 64] = *(const gd_f4*)(Bm + (16 * tt + lr) * LD + 16 * nt + 4 * g);
      o4[(2 + tt) * 64] = *(const gd_f4*)(Rm + (16 * tt + lr) * LD + 16 * nt + 4 * g);
      o4[(4 + tt) * 64] = at[tt];
      o4[(6 + tt) * 64] = kp[tt];
    }
  }
}

// A block per (head, 16 value channels, request): through the chunks [first_chunk, first_chunk + per_pass) in
// order.  NW waves, each ST tiles of 16 rows of S in its accumulators.
template <int D, int NW>
__global__ __launch_bounds__(NW * 64) void gdelta_scan_kernel(const act_t* __restrict__ rkv, int ld, int v_off,
                                                              const float* __restrict__ work, float* __restrict__ state,
                                                              int slot_words, int offset_words,
                                                              const int* __restrict__ q_start,
                                                              const int* __restrict__ slot_of_req, float* __restrict__ raw,
                                                              int H, int first_chunk, int per_pass) {
  constexpr int ST = D / 16 / NW, NN = (3 + NW - 1) / NW;
  using Wk = GdWork<D>;
  __shared__ gd_f4 part[2][NW][4][64];               // partial Y (two tiles), partial O (two tiles)
  // the value channels of one head read the same operands: neighbours in the launch differ by the head, so
  // that (with heads in whole eights) a head's blocks meet in one L2
  const int h = blockIdx.x % H, e0 = blockIdx.x / H * 16, r = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, lr = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int q0 = q_start[r], n = q_start[r + 1] - q0;
  if (first_chunk * GD_CHUNK >= n) return;
  const int chunks = min(per_pass, (n - first_chunk * GD_CHUNK + GD_CHUNK - 1) / GD_CHUNK);
  float* S0 = state + (size_t)slot_of_req[r] * slot_words + offset_words + (size_t)h * D * D + e0 + lr;
  gd_f4 S[ST];
#pragma unroll
  for (int j = 0; j < ST; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) S[j][i] = S0[(size_t)(16 * (wave * ST + j) + 4 * g + i) * D];
  struct Operands {
    gd_f4 tb[ST][2], rq[ST][2], at[ST][2], kp[ST][2], bc[ST], nq[NN];
    act_t v[2][4];          // as they lie in memory: turned into floats where they are used, so that nothing waits for them here
  };
  auto fetch = [&](int c, Operands& x) {
    const float* w = work + (((size_t)r * per_pass + c) * H + h) * Wk::FLOATS;
#pragma unroll
    for (int j = 0; j < ST; j++) {
      const gd_f4* f = (const gd_f4*)(w + (wave * ST + j) * Wk::PER_TILE) + lane;
#pragma unroll
      for (int tt = 0; tt < 2; tt++) {
        x.tb[j][tt] = f[tt * 64];
        x.rq[j][tt] = f[(2 + tt) * 64];
        x.at[j][tt] = f[(4 + tt) * 64];
        x.kp[j][tt] = f[(6 + tt) * 64];
      }
      x.bc[j] = *(const gd_f4*)(w + Wk::B_AT + 16 * (wave * ST + j) + 4 * g);
    }
#pragma unroll
    for (int q = 0; q < NN; q++)
      x.nq[q] = *((const gd_f4*)(w + Wk::N_AT) + min(wave + q * NW, 2) * 64 + lane);
    const int t = (first_chunk + c) * GD_CHUNK;
#pragma unroll
    for (int tt = 0; tt < 2; tt++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int at = min(t + 16 * tt + 4 * g + i, n - 1);      // (rows past the portion's end meet zeros in K, A and N)
        x.v[tt][i] = rkv[(size_t)(q0 + at) * ld + v_off + (size_t)h * D + e0 + lr];
      }
  };
  // the read-outs of a chunk: two waves add up the partial sums of 16 tokens each
  auto read_out = [&](int c) {
    if (wave >= 2) return;
    gd_f4 sum = part[c & 1][0][2 + wave][lane];
#pragma unroll
    for (int w = 1; w < NW; w++) sum += part[c & 1][w][2 + wave][lane];
    const int t = (first_chunk + c) * GD_CHUNK + 16 * wave + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; i++)
      if (t + i < n) raw[((size_t)(q0 + t + i) * H + h) * D + e0 + lr] = sum[i];
  };
  Operands x, next;
  fetch(0, x);
  for (int c = 0; c < chunks; c++) {
    // The stores of the chunk before, then the next chunk's loads, then this one's arithmetic: whoever waits for
    // the loads at the end of the turn waits for nothing younger.  (Always a fetch, the last chunk's twice: a
    // branch around it would make the waits behind it wait for everything.)
    if (c > 0) read_out(c - 1);
    fetch(min(c + 1, chunks - 1), next);
    const int buf = c & 1;
    float v[2][4];
    gd_f4 y[2], o[2];
#pragma unroll
    for (int tt = 0; tt < 2; tt++) {
      y[tt] = o[tt] = gd_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 4; i++) v[tt][i] = to_f32(x.v[tt][i]);
    }
#pragma unroll
    for (int j = 0; j < ST; j++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int tt = 0; tt < 2; tt++) y[tt] = gd_mfma(x.tb[j][tt][i], S[j][i], y[tt]);
    part[buf][wave][0][lane] = y[0];
    part[buf][wave][1][lane] = y[1];
#pragma unroll
    for (int j = 0; j < ST; j++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int tt = 0; tt < 2; tt++) o[tt] = gd_mfma(x.rq[j][tt][i], S[j][i], o[tt]);
#pragma unroll
    for (int q = 0; q < NN; q++) {
      // the three lower tiles of N + Q P, a wave one (or two) of them; a wave without one adds zeros
      const int idx = wave + q * NW;
      const float on0 = idx == 0 ? 1.f : 0.f, on1 = idx == 1 || idx == 2 ? 1.f : 0.f;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float nv = x.nq[q][i];
        o[0] = gd_mfma(nv * on0, v[0][i], o[0]);
        o[1] = gd_mfma(nv * on1, idx == 2 ? v[1][i] : v[0][i], o[1]);
      }
    }
    part[buf][wave][2][lane] = o[0];
    part[buf][wave][3][lane] = o[1];
#pragma unroll
    for (int tt = 0; tt < 2; tt++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < ST; j++) S[j] = gd_mfma(x.kp[j][tt][i], v[tt][i], S[j]);
    __syncthreads();          // two buffers: one barrier a chunk suffices
#pragma unroll
    for (int tt = 0; tt < 2; tt++) {
      gd_f4 sum = part[buf][0][tt][lane];
#pragma unroll
      for (int w = 1; w < NW; w++) sum += part[buf][w][tt][lane];
      y[tt] = sum;
    }
#pragma unroll
    for (int tt = 0; tt < 2; tt++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < ST; j++) S[j] = gd_mfma(x.at[j][tt][i], y[tt][i], S[j]);
#pragma unroll
    for (int j = 0; j < ST; j++) S[j] *= x.bc[j];
    x = next;
  }
  read_out(chunks - 1);
#pragma unroll
  for (int j = 0; j < ST; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) S0[(size_t)(16 * (wave * ST + j) + 4 * g + i) * D] = S[j][i];
}

template <int D, int NW>
static int gdelta_chunked_sizes(const act_t* rkv, int ld, int k_off, int v_off, const float* decay, const float* rate, float* state,
                                int slot_words, int offset_words, const int* q_start, const int* slot_of_req, float* raw,
                                float* work, size_t work_floats, int R, int max_q_len, int H, hipStream_t s) {
  constexpr size_t lds = ((size_t)4 * GD_CHUNK * (D + 4) + 5 * GD_CHUNK * GD_SMALL + GD_CHUNK + 512) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    if (hipFuncSetAttribute((const void*)gdelta_chunk_kernel<D>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return zk_fail("zk_gdelta_chunked: the chunk kernel's local memory was refused");
    raised = true;
  }
  const int total = (max_q_len + GD_CHUNK - 1) / GD_CHUNK;
  const long long room = (long long)(work_floats / ((size_t)GdWork<D>::FLOATS * H * R));
  ZK_REQUIRE(room >= 1, "zk_gdelta_chunked: the workspace does not hold a chunk of every request");
  const int per_pass = (int)(room < total ? room : total);
  for (int first = 0; first < total; first += per_pass) {
    gdelta_chunk_kernel<D><<<dim3(per_pass, H, R), 512, lds, s>>>(rkv, ld, k_off, decay, rate, q_start, H, first, work);
    gdelta_scan_kernel<D, NW><<<dim3(H * (D / 16), R), NW * 64, 0, s>>>(rkv, ld, v_off, work, state, slot_words, offset_words, q_start,
                                                                      slot_of_req, raw, H, first, per_pass);
  }
  return 0;
}
#endif

extern "C" {

// rows: float [T, ld]: n removal-rate numbers (before bias and sigmoid), and at column low_off ``rank`` numbers
// before their tanh.  w2: [n, rank] in the storage type; w0: float [n]; a0 (may be null): float [n].
// decay, rate: float [T, n].
int zk_gdelta_gates(const float* rows, int ld, int low_off, int rank, const void* w2, const float* w0, const float* a0,
                    float* decay, float* rate, int T, int n, void* stream) {
  ZK_REQUIRE(T >= 0 && n > 0 && rank > 0 && ld >= n && low_off >= 0 && ld >= low_off + rank, "zk_gdelta_gates: bad sizes");
  ZK_REQUIRE(rank <= 1024, "zk_gdelta_gates: a rank of more than 1024 is not supported");
  if (T == 0) return 0;
  dim3 grid((n + 255) / 256, (T + GD_TOKENS - 1) / GD_TOKENS);
  ZK_REQUIRE(grid.y <= 65535, "zk_gdelta_gates: too many tokens");
  const size_t lds = (size_t)rank * GD_TOKENS * sizeof(float);
  if (rank % 8 == 0 && (uintptr_t)w2 % 16 == 0)
    gdelta_gates_kernel<true><<<grid, 256, lds, (hipStream_t)stream>>>(rows, ld, low_off, rank, (const act_t*)w2, w0, a0, decay,
                                                                      rate, T, n);
  else
    gdelta_gates_kernel<false><<<grid, 256, lds, (hipStream_t)stream>>>(rows, ld, low_off, rank, (const act_t*)w2, w0, a0, decay,
                                                                       rate, T, n);
  return zk_launch_status("zk_gdelta_gates");
}

// rkv: [T, ld] activations: H heads of D at column 0 (r), at k_off and at v_off.  g: [T, ldg], H heads of
// D (the output gate before its sigmoid).  decay, rate: float [T, H * D]; gain: float [H * D].
// state: request r's S [H, D, D] lies at state[slot_of_req[r] * slot_words + offset_words].
// out: [T, H * D].  Requests are rows [q_start[r], q_start[r + 1]).  raw: float scratch [T, H * D], used by
// heads that span several blocks.  max_q_len: the longest portion of the step.
int zk_gdelta(const void* rkv, int ld, int k_off, int v_off, const void* g, int ldg, const float* decay, const float* rate,
              const float* gain, float* state, int slot_words, int offset_words, const int* q_start, const int* slot_of_req,
              const int* positions, void* out, float* raw, int T, int R, int max_q_len, int H, int D, float eps,
              void* stream) {
  ZK_REQUIRE(T >= 0 && R >= 0 && H > 0 && D > 0, "zk_gdelta: bad sizes");
  ZK_REQUIRE(D <= 256, "zk_gdelta: up to 256 channels a head");
  ZK_REQUIRE(H <= 65535 && T <= 0x7fffffff / H, "zk_gdelta: too many heads");
  ZK_REQUIRE(state != nullptr && (long long)slot_words >= (long long)offset_words + (long long)H * D * D,
             "zk_gdelta: the state does not fit its slot");
  ZK_REQUIRE(ld >= k_off + H * D && ld >= v_off + H * D && ldg >= H * D && k_off >= 0 && v_off >= 0, "zk_gdelta: rows too short");
  ZK_REQUIRE(raw != nullptr && positions != nullptr, "zk_gdelta: needs scratch");
  if (R == 0 || T == 0) return 0;
  const int DMAX = D <= 32 ? 32 : D <= 64 ? 64 : D <= 128 ? 128 : 256;
  // long portions: few columns a block, so that a head spreads over more compute units; the heads' norm
  // then follows in a kernel of its own
  const int DS = DMAX >= 128 ? 16 : 8;
  const int most = 512 / DS;
  const int per_block = (max_q_len > 16 && D > GD_COLS_LONG) ? GD_COLS_LONG : most;
  const int blocks_e = (D + per_block - 1) / per_block;
  const int unit = 64 / DS;                                             // columns of a wave
  const int cols = D < per_block ? (D + unit - 1) / unit * unit : per_block;
  const int threads = cols * DS;
  const int GRP = DMAX == 256 ? 8 : 16;
  const size_t lds = ((size_t)GRP * (4 * DMAX + cols) + GRP) * sizeof(float);
  dim3 grid(R, H, blocks_e);
  float* raw_arg = blocks_e > 1 ? raw : nullptr;
#define LAUNCH(C, L)                                                                                                     \
  gdelta_kernel<C, L><<<grid, threads, lds, (hipStream_t)stream>>>((const act_t*)rkv, ld, k_off, v_off, (const act_t*)g, \
                                                                   ldg, decay, rate, gain, state, slot_words,            \
                                                                   offset_words, q_start, slot_of_req, (act_t*)out,      \
                                                                   raw_arg, H, D, eps, cols, GRP)
  if (DMAX == 32) LAUNCH(1, 8);
  else if (DMAX == 64) LAUNCH(2, 8);
  else if (DMAX == 128) LAUNCH(2, 16);
  else LAUNCH(4, 16);
#undef LAUNCH
  if (blocks_e > 1) {
    dim3 fg(T, H);
    gdelta_finish_kernel<<<fg, 64, 0, (hipStream_t)stream>>>(raw, (const act_t*)g, ldg, gain, positions, (act_t*)out, H, D, eps);
  }
  return zk_launch_status("zk_gdelta");
}

#if ZSE_ACT_BF16
// 1 if zk_gdelta_token takes heads of this size.
int zk_gdelta_token_supports(int D) { return D == 32 || D == 64 || D == 128 || D == 256; }

// As zk_gdelta for steps in which every request brings one token (T rows; row t belongs to request
// req_of_token[t], rows with a negative position are padding and come out as 0).
int zk_gdelta_token(const void* rkv, int ld, int k_off, int v_off, const void* g, int ldg, const float* decay,
                    const float* rate, const float* gain, float* state, int slot_words, int offset_words,
                    const int* positions, const int* req_of_token, const int* slot_of_req, void* out, int T, int H, int D,
                    float eps, void* stream) {
  ZK_REQUIRE(T >= 0 && T <= 65535 && H > 0 && zk_gdelta_token_supports(D), "zk_gdelta_token: bad sizes");
  ZK_REQUIRE(state != nullptr && (long long)slot_words >= (long long)offset_words + (long long)H * D * D,
             "zk_gdelta_token: the state does not fit its slot");
  ZK_REQUIRE(ld >= k_off + H * D && ld >= v_off + H * D && ldg >= H * D && k_off >= 0 && v_off >= 0,
             "zk_gdelta_token: rows too short");
  if (T == 0) return 0;
  const int threads = 1024, P = threads / D;
  const size_t lds = (size_t)(4 + P) * D * sizeof(float);
  dim3 grid(H, T);
#define LAUNCH(RP)                                                                                                         \
  gdelta_token_kernel<RP><<<grid, threads, lds, (hipStream_t)stream>>>((const act_t*)rkv, ld, k_off, v_off, (const act_t*)g, \
                                                                       ldg, decay, rate, gain, state, slot_words,          \
                                                                       offset_words, positions, req_of_token, slot_of_req, \
                                                                       (act_t*)out, H, D, eps)
  if (D == 32) LAUNCH(1);
  else if (D == 64) LAUNCH(4);
  else if (D == 128) LAUNCH(16);
  else LAUNCH(64);
#undef LAUNCH
  return zk_launch_status("zk_gdelta_token");
}
// Floats that zk_gdelta_chunked's workspace takes for one chunk of 32 tokens of one head (0: heads of this size
// are not taken).
int zk_gdelta_chunk_floats(int D) {
  switch (D) {
    case 32: return GdWork<32>::FLOATS;
    case 64: return GdWork<64>::FLOATS;
    case 128: return GdWork<128>::FLOATS;
    case 256: return GdWork<256>::FLOATS;
    default: return 0;
  }
}

// As zk_gdelta (raw is always used), in chunks of 32 tokens.  work: scratch of work_floats floats, at least
// R * H * zk_gdelta_chunk_floats(D); with room for fewer chunks than the longest portion has, the portions
// are taken in several passes.
int zk_gdelta_chunked(const void* rkv, int ld, int k_off, int v_off, const void* g, int ldg, const float* decay,
                      const float* rate, const float* gain, float* state, int slot_words, int offset_words,
                      const int* q_start, const int* slot_of_req, const int* positions, void* out, float* raw, float* work,
                      size_t work_floats, int T, int R, int max_q_len, int H, int D, float eps, void* stream) {
  ZK_REQUIRE(T >= 0 && R >= 0 && H > 0 && zk_gdelta_chunk_floats(D) > 0, "zk_gdelta_chunked: bad sizes");
  ZK_REQUIRE(H <= 65535 && R <= 65535 && max_q_len > 0, "zk_gdelta_chunked: too many heads or requests, or no tokens");
  ZK_REQUIRE(state != nullptr && (long long)slot_words >= (long long)offset_words + (long long)H * D * D,
             "zk_gdelta_chunked: the state does not fit its slot");
  ZK_REQUIRE(ld >= k_off + H * D && ld >= v_off + H * D && ldg >= H * D && k_off >= 0 && v_off >= 0,
             "zk_gdelta_chunked: rows too short");
  ZK_REQUIRE(raw != nullptr && positions != nullptr && work != nullptr && (uintptr_t)work % 16 == 0,
             "zk_gdelta_chunked: needs scratch");
  if (R == 0 || T == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const act_t* x = (const act_t*)rkv;
  int rc;
#define RUN(N, NW)                                                                                                            \
  rc = gdelta_chunked_sizes<N, NW>(x, ld, k_off, v_off, decay, rate, state, slot_words, offset_words, q_start, slot_of_req, raw, \
                                   work, work_floats, R, max_q_len, H, s)
  if (D == 32) RUN(32, 2);
  else if (D == 64) RUN(64, 4);
  else if (D == 128) RUN(128, 4);
  else RUN(256, 8);
#undef RUN
  if (rc) return rc;
  gdelta_finish_kernel<<<dim3(T, H), 64, 0, s>>>(raw, (const act_t*)g, ldg, gain, positions, (act_t*)out, H, D, eps);
  return zk_launch_status("zk_gdelta_chunked");
}
#endif

}  // extern "C"

ZK_ENTER(zk_gdelta_gates)
ZK_ENTER(zk_gdelta)
#if ZSE_ACT_BF16
ZK_ENTER(zk_gdelta_token)
ZK_ENTER(zk_gdelta_chunked)
#endif
