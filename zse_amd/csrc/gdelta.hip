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
#endif

}  // extern "C"

ZK_ENTER(zk_gdelta_gates)
ZK_ENTER(zk_gdelta)
#if ZSE_ACT_BF16
ZK_ENTER(zk_gdelta_token)
#endif
