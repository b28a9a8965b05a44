// The short causal convolution over time, channel by channel:
//
//   u = x + in_bias;   y_t = bias + sum_j w[:, j] u_(t - taps + 1 + j);   (+ u_t);   (silu)
//
// rows before a sequence's start being zero (not in_bias).  The taps - 1 rows of u before a
// request's next token are float rows in its state slot, the youngest first; a step reads them for its
// first tokens and renews them.
//
// A thread owns V neighbouring channels (16 bytes of bfloat16) of a run of ``span`` tokens of one
// request and carries the taps - 1 rows before the current token in registers, so a row is read
// once a run.  Runs are counted from the request's first token of the step: only the first of
// them reads the state (span >= taps - 1), and its threads renew it, each its own columns, after
// they have read them.  One launch serves every kind of step.
#include "common.h"
#include "packed_call.h"

extern "C" int zk_steplist_register(const char* name, int nargs, void* fn);
#define ZK_ENTER(fn) \
  static const int fn##_entered = zk_steplist_register(#fn, zk_packed::Call<fn>::nargs, (void*)zk_packed::Call<fn>::call);

#define CONV_SPAN 8
#define CONV_MOST_TAPS (CONV_SPAN + 1)

template <int V>
__device__ __forceinline__ void conv_get(const act_t* p, float (&v)[V]) {
  if constexpr (V == 8) {
#if ZSE_ACT_BF16
    typedef __bf16 b8 __attribute__((ext_vector_type(8)));
    const b8 q = *(const b8*)p;
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] = (float)q[e];
#else
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
#endif
  } else {
    v[0] = to_f32(p[0]);
  }
}
template <int V>
__device__ __forceinline__ void conv_put(act_t* p, const float (&v)[V]) {
  if constexpr (V == 8) {
#if ZSE_ACT_BF16
    typedef __bf16 b8 __attribute__((ext_vector_type(8)));
    b8 q;
#pragma unroll
    for (int e = 0; e < 8; e++) q[e] = (__bf16)v[e];
    *(b8*)p = q;
#else
    *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
    *(float4*)(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
#endif
  } else {
    p[0] = from_f32<act_t>(v[0]);
  }
}
template <int V>
__device__ __forceinline__ void conv_get_state(const float* p, float (&v)[V]) {
  if constexpr (V == 8) {
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
  } else {
    v[0] = p[0];
  }
}
template <int V>
__device__ __forceinline__ void conv_put_state(float* p, const float (&v)[V]) {
  if constexpr (V == 8) {
    *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
    *(float4*)(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
  } else {
    p[0] = v[0];
  }
}

// TAPS: the number of taps where the launch knows it at compile time, 0: ``taps`` (up to 9)
template <int V, int TAPS>
__global__ __launch_bounds__(256) void conv_rows_kernel(const act_t* __restrict__ x, int ld_in,
                                                        const float* __restrict__ in_bias, const float* __restrict__ w,
                                                        const float* __restrict__ bias, float* __restrict__ state,
                                                        int slot_words, int offset_words, const int* __restrict__ q_start,
                                                        const int* __restrict__ slot_of_req, act_t* __restrict__ out,
                                                        int ld_out, int T, int R, int C, int taps_given, int residual,
                                                        int act) {
  constexpr int MOST = TAPS ? TAPS : CONV_MOST_TAPS, BACK = MOST > 1 ? MOST - 1 : 1;
  const int taps = TAPS ? TAPS : taps_given;
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (c >= C) return;
  const int r = blockIdx.z, first = blockIdx.y * CONV_SPAN;
  const int t0 = q_start[r];
  if (r == R) {                          // rows behind the last request: padding of a captured step
    if (first == 0) {
      float zero[V];
#pragma unroll
      for (int e = 0; e < V; e++) zero[e] = 0.f;
      for (int t = t0; t < T; t++) conv_put<V>(out + (size_t)t * ld_out + c, zero);
    }
    return;
  }
  const int n = q_start[r + 1] - t0;
  if (first >= n) return;
  const int last = min(n, first + CONV_SPAN);
  float ib[V], b0[V], wt[MOST][V];
#pragma unroll
  for (int e = 0; e < V; e++) {
    ib[e] = in_bias ? in_bias[c + e] : 0.f;
    b0[e] = bias ? bias[c + e] : 0.f;
#pragma unroll
    for (int j = 0; j < MOST; j++) wt[j][e] = j < taps ? w[(size_t)(c + e) * taps + j] : 0.f;
  }
  auto input = [&](int i, float (&v)[V]) {
    conv_get<V>(x + (size_t)(t0 + i) * ld_in + c, v);
#pragma unroll
    for (int e = 0; e < V; e++) v[e] += ib[e];
  };
  float* st = taps > 1 ? state + (size_t)slot_of_req[r] * slot_words + offset_words + c : nullptr;
  // back[b]: the row b + 1 places before the current token
  float back[BACK][V];
#pragma unroll
  for (int b = 0; b < BACK; b++)
    if (b < taps - 1) {
      if (first - 1 - b >= 0) input(first - 1 - b, back[b]);
      else conv_get_state<V>(st + (size_t)(b - first) * C, back[b]);      // only in the first run
    }
  if (first == 0 && taps > 1) {
    // the state the next step finds: row a is the row a + 1 places before it, one of this step's
    // rows or one of those just read
#pragma unroll
    for (int a = 0; a < BACK; a++)
      if (a < taps - 1) {
        float v[V];
        if (n - 1 - a >= 0) {
          input(n - 1 - a, v);
        } else {
#pragma unroll
          for (int e = 0; e < V; e++) v[e] = 0.f;
#pragma unroll
          for (int b = 0; b < BACK; b++)
            if (b == a - n) {
#pragma unroll
              for (int e = 0; e < V; e++) v[e] = back[b][e];
            }
        }
        conv_put_state<V>(st + (size_t)a * C, v);
      }
  }
  for (int i = first; i < last; i++) {
    float cur[V], acc[V];
    input(i, cur);
#pragma unroll
    for (int e = 0; e < V; e++) acc[e] = b0[e];
#pragma unroll
    for (int b = BACK - 1; b >= 0; b--)
      if (b < taps - 1) {
#pragma unroll
        for (int e = 0; e < V; e++) {
          float wj = 0.f;
          if (TAPS) {
            wj = wt[MOST - 2 - b < 0 ? 0 : MOST - 2 - b][e];
          } else {
#pragma unroll
            for (int j = 0; j < MOST; j++) wj = j == taps - 2 - b ? wt[j][e] : wj;
          }
          acc[e] = fmaf(wj, back[b][e], acc[e]);
        }
      }
#pragma unroll
    for (int e = 0; e < V; e++) {
      float wj = wt[0][e];
#pragma unroll
      for (int j = 0; j < MOST; j++) wj = j == taps - 1 ? wt[j][e] : wj;
      acc[e] = fmaf(wj, cur[e], acc[e]);
      if (residual) acc[e] = cur[e] + acc[e];
      if (act == 1) acc[e] = acc[e] / (1.0f + expf(-acc[e]));      // silu
    }
    conv_put<V>(out + (size_t)(t0 + i) * ld_out + c, acc);
#pragma unroll
    for (int b = BACK - 1; b > 0; b--)
#pragma unroll
      for (int e = 0; e < V; e++) back[b][e] = back[b - 1][e];
#pragma unroll
    for (int e = 0; e < V; e++) back[0][e] = cur[e];
  }
}

extern "C" {

// The most taps zk_conv_rows takes.
int zk_conv_rows_most_taps() { return CONV_MOST_TAPS; }

// x: [T, ld_in] activations, out: [T, ld_out] (another buffer), of which the first C channels take
// part; w: float [C, taps]; in_bias, bias (either may be null): float [C]; the state of request r is
// taps - 1 float rows of C at state[slot_of_req[r] * slot_words + offset_words], renewed by this
// launch.  Requests are rows [q_start[r], q_start[r + 1]) of the step, q_start has R + 1 entries;
// rows behind q_start[R] are padding and come out as 0.  max_q_len: no request brings more tokens
// than this.  residual: the input (with in_bias) is added to the sum; act: 0 none, 1 silu.
int zk_conv_rows(const void* x, int ld_in, const float* in_bias, const float* w, const float* bias, float* state, int slot_words,
                 int offset_words, const int* q_start, const int* slot_of_req, void* out, int ld_out, int T, int R,
                 int max_q_len, int C, int taps, int residual, int act, void* stream) {
  ZK_REQUIRE(T >= 0 && R >= 0 && R < 65535 && C > 0 && taps >= 1 && max_q_len >= 0, "zk_conv_rows: bad sizes");
  ZK_REQUIRE(taps <= CONV_MOST_TAPS, "zk_conv_rows: too many taps");
  ZK_REQUIRE(ld_in >= C && ld_out >= C && (act == 0 || act == 1), "zk_conv_rows: bad strides or activation");
  ZK_REQUIRE(x != out, "zk_conv_rows: not in place");
  ZK_REQUIRE(taps == 1 || (state != nullptr && (long long)slot_words >= (long long)offset_words + (long long)(taps - 1) * C),
             "zk_conv_rows: the state does not fit its slot");
  if (T == 0) return 0;
  auto aligned = [](const void* p, size_t n) { return (uintptr_t)p % n == 0; };
  const bool vec = C % 8 == 0 && ld_in % 8 == 0 && ld_out % 8 == 0 && aligned(x, 16) && aligned(out, 16) &&
                   (taps == 1 || (aligned(state, 16) && slot_words % 4 == 0 && offset_words % 4 == 0));
  const int runs = max_q_len > 0 ? (max_q_len + CONV_SPAN - 1) / CONV_SPAN : 1;
  ZK_REQUIRE(runs <= 65535, "zk_conv_rows: too many tokens");
  const int per = vec ? 8 : 1, columns = (C + per - 1) / per;
  // few runs: narrow blocks, so that they spread over the compute units
  const int threads = (long long)((columns + 255) / 256) * runs * R >= 512 ? 256 : 64;
  dim3 grid((columns + threads - 1) / threads, runs, R + 1);
#define LAUNCH(V, N)                                                                                                  \
  conv_rows_kernel<V, N><<<grid, threads, 0, (hipStream_t)stream>>>((const act_t*)x, ld_in, in_bias, w, bias, state,  \
                                                                    slot_words, offset_words, q_start, slot_of_req,   \
                                                                    (act_t*)out, ld_out, T, R, C, taps, residual, act)
  if (vec) {
    if (taps == 2) LAUNCH(8, 2);
    else if (taps == 3) LAUNCH(8, 3);
    else if (taps == 4) LAUNCH(8, 4);
    else LAUNCH(8, 0);
  } else {
    LAUNCH(1, 0);
  }
#undef LAUNCH
  return zk_launch_status("zk_conv_rows");
}

}  // extern "C"

ZK_ENTER(zk_conv_rows)
