// Between two sublayers of a pre-norm layer: a sublayer's result joins the float residual stream,
// and the next sublayer's input is made from the new stream, one launch, one block a token.
//
//   write:  h <- h + g * y                       (g: a gain per channel; the layer scale)
//       or  h <- h + y / sqrt(mean(y^2) + e) * g (y brought to unit root mean square first)
//   read :  n = (h - mean(h)) / sqrt(var(h) + eps) * w + b     (var: the mean squared deviation)
//           out = n,  or n + conv(n) where every request brings one token (see below)
//           raw = h rounded to the activation type, for a product that reads the stream itself
//
// conv(n)_t = sum_j c[:, j] n_(t - taps + 1 + j), channel by channel, rows before a sequence's start
// being zero.  The taps - 1 rows before a request's next token are float rows in its state slot.
// In a step of single tokens the thread of (token, channel) is the only one that touches its
// column of the state and moves it on itself; longer portions take n to the kernel of
// shortconv.hip.  n is rounded to the activation type before the convolution reads it either way,
// so both give the same bits.
//
// ``zk_norm_stream``: the stream itself replaced by its norm (an embedding's norm).
// ``zk_token_gate``: gelu_tanh(z) * e with e a slice of the token's row of a table.
// Everything is float; y, raw and out have the activation type (y may be float planes).
#include "common.h"
#include "packed_call.h"

extern "C" int zk_steplist_register(const char* name, int nargs, void* fn);
#define ZK_ENTER(fn) \
  static const int fn##_entered = zk_steplist_register(#fn, zk_packed::Call<fn>::nargs, (void*)zk_packed::Call<fn>::call);

struct SublayerConv {
  const float* w;              // [W, taps]; null: no convolution here
  float* state;
  const int* positions;
  const int* req_of_token;
  const int* slot_of_req;
  int taps, slot_words, offset_words;
};

// V consecutive numbers of a row as floats
template <int V>
__device__ __forceinline__ void get_floats(const float* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const float4 q = *(const float4*)p;
    v[0] = q.x, v[1] = q.y, v[2] = q.z, v[3] = q.w;
  } else {
    v[0] = p[0];
  }
}
template <int V>
__device__ __forceinline__ void put_floats(float* p, const float (&v)[V]) {
  if constexpr (V == 4) *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
  else p[0] = v[0];
}
template <int V>
__device__ __forceinline__ void get_acts(const act_t* p, float (&v)[V]) {
#if ZSE_ACT_BF16
  if constexpr (V == 4) {
    typedef __bf16 b4 __attribute__((ext_vector_type(4)));
    const b4 q = *(const b4*)p;
#pragma unroll
    for (int e = 0; e < 4; e++) v[e] = (float)q[e];
  } else {
    v[0] = (float)p[0];
  }
#else
  get_floats<V>(p, v);
#endif
}
template <int V>
__device__ __forceinline__ void put_acts(act_t* p, const float (&v)[V]) {
#if ZSE_ACT_BF16
  if constexpr (V == 4) {
    typedef __bf16 b4 __attribute__((ext_vector_type(4)));
    b4 q;
#pragma unroll
    for (int e = 0; e < 4; e++) q[e] = (__bf16)v[e];
    *(b4*)p = q;
  } else {
    p[0] = (__bf16)v[0];
  }
#else
  put_floats<V>(p, v);
#endif
}

template <int V>
__global__ __launch_bounds__(1024) void sublayer_step_kernel(float* __restrict__ h, const void* __restrict__ y, int y_parts,
                                                             size_t y_plane, const float* __restrict__ y_gain, int y_unit,
                                                             float y_eps, act_t* __restrict__ raw,
                                                             const float* __restrict__ norm_w,
                                                             const float* __restrict__ norm_b, float eps,
                                                             act_t* __restrict__ out, SublayerConv cv, int W) {
  extern __shared__ __attribute__((aligned(16))) float row[];          // [W]
  __shared__ float red[17];
  const int t = blockIdx.x, tid = threadIdx.x, nt = blockDim.x;
  const size_t base = (size_t)t * W;
  float* hr = h + base;
  auto result = [&](int c, float (&v)[V]) {
    if (y_parts > 0) {
      const float* p = (const float*)y + base + c;
      get_floats<V>(p, v);
      for (int k = 1; k < y_parts; k++) {
        float u[V];
        get_floats<V>(p + (size_t)k * y_plane, u);
#pragma unroll
        for (int e = 0; e < V; e++) v[e] += u[e];
      }
    } else {
      get_acts<V>((const act_t*)y + base + c, v);
    }
  };
  float inv_y = 1.f;
  if (y != nullptr && y_unit) {
    float ss = 0.f;
    for (int c = tid * V; c < W; c += nt * V) {
      float v[V];
      result(c, v);
#pragma unroll
      for (int e = 0; e < V; e++) ss = fmaf(v[e], v[e], ss);
      put_floats<V>(row + c, v);
    }
    inv_y = 1.0f / sqrtf(block_sum(ss, red) / (float)W + y_eps);
  }
  float sum = 0.f;
  for (int c = tid * V; c < W; c += nt * V) {
    float x[V];
    get_floats<V>(hr + c, x);
    if (y != nullptr) {
      float v[V], g[V];
      if (y_unit) get_floats<V>(row + c, v);       // what this thread put there
      else result(c, v);
      if (y_gain) {
        get_floats<V>(y_gain + c, g);
      } else {
#pragma unroll
        for (int e = 0; e < V; e++) g[e] = 1.f;
      }
#pragma unroll
      for (int e = 0; e < V; e++) x[e] = fmaf(v[e] * inv_y, g[e], x[e]);
      put_floats<V>(hr + c, x);
    }
    if (raw != nullptr) put_acts<V>(raw + base + c, x);
    if (out != nullptr) {
      put_floats<V>(row + c, x);
#pragma unroll
      for (int e = 0; e < V; e++) sum += x[e];
    }
  }
  if (out == nullptr) return;
  const float mean = block_sum(sum, red) / (float)W;
  float dev = 0.f;
  for (int c = tid * V; c < W; c += nt * V) {
    float x[V];
    get_floats<V>(row + c, x);
#pragma unroll
    for (int e = 0; e < V; e++) {
      const float d = x[e] - mean;
      dev = fmaf(d, d, dev);
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(dev, red) / (float)W + eps);
  const bool conv = cv.w != nullptr;
  const bool padding = conv && cv.positions[t] < 0;          // a padding row of a captured step
  float* st = (conv && !padding && cv.taps > 1)
                  ? cv.state + (size_t)cv.slot_of_req[cv.req_of_token[t]] * cv.slot_words + cv.offset_words : nullptr;
  for (int c = tid * V; c < W; c += nt * V) {
    float x[V], g[V], b[V];
    get_floats<V>(row + c, x);
    get_floats<V>(norm_w + c, g);
    if (norm_b) {
      get_floats<V>(norm_b + c, b);
    } else {
#pragma unroll
      for (int e = 0; e < V; e++) b[e] = 0.f;
    }
#pragma unroll
    for (int e = 0; e < V; e++) x[e] = fmaf((x[e] - mean) * inv, g[e], b[e]);
    if (conv) {
      float acc[V];
#pragma unroll
      for (int e = 0; e < V; e++) {
        x[e] = padding ? 0.f : to_f32(from_f32<act_t>(x[e]));
        acc[e] = 0.f;
      }
      if (!padding) {
        // oldest row first; a row moves to the place of the one before it once that one is in hand
        for (int a = cv.taps - 2; a >= 0; a--) {
          float v[V];
          get_floats<V>(st + (size_t)a * W + c, v);
          if (a < cv.taps - 2) put_floats<V>(st + (size_t)(a + 1) * W + c, v);
#pragma unroll
          for (int e = 0; e < V; e++) acc[e] = fmaf(cv.w[(size_t)(c + e) * cv.taps + cv.taps - 2 - a], v[e], acc[e]);
        }
#pragma unroll
        for (int e = 0; e < V; e++) acc[e] = fmaf(cv.w[(size_t)(c + e) * cv.taps + cv.taps - 1], x[e], acc[e]);
        if (cv.taps > 1) put_floats<V>(st + c, x);
      }
#pragma unroll
      for (int e = 0; e < V; e++) x[e] += acc[e];
    }
    put_acts<V>(out + base + c, x);
  }
}

// A sum over the block with one barrier: every wave leaves its own, every thread adds them up in order.  Each
// use in a kernel has its own ``red`` (16 floats), so nothing is read after it was overwritten.
__device__ __forceinline__ float rows_sum(float x, float* red) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x140, 0xf, 0xf, false));   // row_mirror
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x141, 0xf, 0xf, false));   // row_half_mirror
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0xB1, 0xf, 0xf, false));    // quad_perm [1,0,3,2]
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x4E, 0xf, 0xf, false));    // quad_perm [2,3,0,1]
  x += __shfl_xor(x, 16, 64);
  x += __shfl_xor(x, 32, 64);
  const int nw = blockDim.x >> 6;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
  __syncthreads();
  float t = red[0];
  for (int w = 1; w < nw; w++) t += red[w];
  return t;
}

// The same for rows of whole groups of four channels, a thread a group: everything the row needs is asked for
// at once, before the first sum.  TAPS: 0 without the convolution, 2 to 4 taps known to the
// compiler (their weights and state rows are asked for at once too), -1 any other number.
template <int TAPS>
__global__ __launch_bounds__(1024) void sublayer_row_kernel(float* __restrict__ h, const void* __restrict__ y, int y_parts,
                                                            size_t y_plane, const float* __restrict__ y_gain, int y_unit,
                                                            float y_eps, act_t* __restrict__ raw,
                                                            const float* __restrict__ norm_w, const float* __restrict__ norm_b,
                                                            float eps, act_t* __restrict__ out, SublayerConv cv, int W) {
  __shared__ float red[3][16];
  constexpr int N = TAPS > 0 ? TAPS : 1;
  const int t = blockIdx.x, c = threadIdx.x * 4;
  const bool in = c < W;
  const size_t at = (size_t)t * W + (in ? c : 0);
  const int taps = TAPS > 0 ? TAPS : cv.taps;
  float x[4] = {}, v[4] = {}, g[4] = {1.f, 1.f, 1.f, 1.f}, nw[4], nb[4] = {}, cw[4 * N], older[N][4];
  const bool padding = TAPS != 0 && cv.positions[t] < 0;          // a padding row of a captured step
  float* st = (TAPS != 0 && !padding && taps > 1)
                  ? cv.state + (size_t)cv.slot_of_req[cv.req_of_token[t]] * cv.slot_words + cv.offset_words + c : nullptr;
  if (in) {
    get_floats<4>(h + at, x);
    if (y != nullptr) {
      if (y_parts > 0) {
        const float* p = (const float*)y + at;
        get_floats<4>(p, v);
        for (int k = 1; k < y_parts; k++) {
          float u[4];
          get_floats<4>(p + (size_t)k * y_plane, u);
#pragma unroll
          for (int e = 0; e < 4; e++) v[e] += u[e];
        }
      } else {
        get_acts<4>((const act_t*)y + at, v);
      }
      if (y_gain) get_floats<4>(y_gain + c, g);
    }
    if (out != nullptr) {
      get_floats<4>(norm_w + c, nw);
      if (norm_b) get_floats<4>(norm_b + c, nb);
    }
    if (TAPS > 0) {
#pragma unroll
      for (int q = 0; q < N; q++) {
        float u[4];
        get_floats<4>(cv.w + (size_t)c * N + 4 * q, u);
#pragma unroll
        for (int e = 0; e < 4; e++) cw[4 * q + e] = u[e];
      }
      if (!padding) {
#pragma unroll
        for (int a = 0; a < N - 1; a++) get_floats<4>(st + (size_t)a * W, older[a]);
      }
    }
  }
  if (y != nullptr) {
    float inv_y = 1.f;
    if (y_unit) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
      inv_y = 1.0f / sqrtf(rows_sum(ss, red[0]) / (float)W + y_eps);
    }
#pragma unroll
    for (int e = 0; e < 4; e++) x[e] = fmaf(v[e] * inv_y, g[e], x[e]);
    if (in) put_floats<4>(h + at, x);
  }
  if (in && raw != nullptr) put_acts<4>(raw + at, x);
  if (out == nullptr) return;
  const float mean = rows_sum(in ? (x[0] + x[1]) + (x[2] + x[3]) : 0.f, red[1]) / (float)W;
  float dev = 0.f;
  if (in) {
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float d = x[e] - mean;
      dev = fmaf(d, d, dev);
    }
  }
  const float inv = 1.0f / sqrtf(rows_sum(dev, red[2]) / (float)W + eps);
  if (!in) return;
#pragma unroll
  for (int e = 0; e < 4; e++) x[e] = fmaf((x[e] - mean) * inv, nw[e], nb[e]);
  if (TAPS != 0) {
    float acc[4] = {};
#pragma unroll
    for (int e = 0; e < 4; e++) x[e] = padding ? 0.f : to_f32(from_f32<act_t>(x[e]));
    if (!padding) {
      if (TAPS > 0) {
#pragma unroll
        for (int a = N - 2; a >= 0; a--)
#pragma unroll
          for (int e = 0; e < 4; e++) acc[e] = fmaf(cw[e * N + N - 2 - a], older[a][e], acc[e]);
#pragma unroll
        for (int a = 1; a < N - 1; a++) put_floats<4>(st + (size_t)a * W, older[a - 1]);
#pragma unroll
        for (int e = 0; e < 4; e++) acc[e] = fmaf(cw[e * N + N - 1], x[e], acc[e]);
      } else {
        for (int a = taps - 2; a >= 0; a--) {
          float u[4];
          get_floats<4>(st + (size_t)a * W, u);
          if (a < taps - 2) put_floats<4>(st + (size_t)(a + 1) * W, u);
#pragma unroll
          for (int e = 0; e < 4; e++) acc[e] = fmaf(cv.w[(size_t)(c + e) * taps + taps - 2 - a], u[e], acc[e]);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) acc[e] = fmaf(cv.w[(size_t)(c + e) * taps + taps - 1], x[e], acc[e]);
      }
      if (taps > 1) put_floats<4>(st, x);
    }
#pragma unroll
    for (int e = 0; e < 4; e++) x[e] += acc[e];
  }
  put_acts<4>(out + at, x);
}

// h <- (h - mean) / sqrt(var + eps) * w + b, in place and in float
__global__ __launch_bounds__(1024) void norm_stream_kernel(float* __restrict__ h, const float* __restrict__ w,
                                                           const float* __restrict__ b, float eps, int W) {
  __shared__ float red[17];
  float* hr = h + (size_t)blockIdx.x * W;
  float sum = 0.f;
  for (int c = threadIdx.x; c < W; c += blockDim.x) sum += hr[c];
  const float mean = block_sum(sum, red) / (float)W;
  float dev = 0.f;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    const float d = hr[c] - mean;
    dev = fmaf(d, d, dev);
  }
  const float inv = 1.0f / sqrtf(block_sum(dev, red) / (float)W + eps);
  for (int c = threadIdx.x; c < W; c += blockDim.x) hr[c] = fmaf((hr[c] - mean) * inv, w[c], b ? b[c] : 0.f);
}

__global__ void token_gate_kernel(const float* __restrict__ z, const act_t* __restrict__ table, const int* __restrict__ tokens,
                                  int ld_table, int column, act_t* __restrict__ out, int T, int n) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (size_t)T * n) return;
  const int t = (int)(i / n), c = (int)(i - (size_t)t * n);
  const float x = z[i];
  const float g = 0.5f * x * (1.0f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
  out[i] = from_f32<act_t>(g * to_f32(table[(size_t)tokens[t] * ld_table + column + c]));
}

extern "C" {

// h: float [T, W], updated in place when y is given (y: [T, W] activations, or y_parts float planes
// [y_parts, T, W] added up in order).  y_gain: float [W] or null (1).  y_unit: y is divided by its
// root mean square (y_eps inside the root) first.  raw (may be null): [T, W], the new stream in
// the activation type.  out (may be null): [T, W], the layer norm of the new stream (norm_b may be
// null), through the convolution when conv_w (float [W, taps]) is given: the step then brings one
// token for each request (rows with a negative position are padding and come out as 0), and
// the state of request r is taps - 1 float rows of W at
// state[slot_of_req[r] * slot_words + offset_words], moved on by this launch.
int zk_sublayer_step(float* h, const void* y, int y_parts, const float* y_gain, int y_unit, float y_eps, void* raw,
                     const float* norm_w, const float* norm_b, float eps, void* out, const float* conv_w, int taps,
                     float* state, int slot_words, int offset_words, const int* positions, const int* req_of_token,
                     const int* slot_of_req, int T, int W, void* stream) {
  ZK_REQUIRE(T >= 0 && W > 0 && y_parts >= 0 && h != nullptr, "zk_sublayer_step: bad sizes");
  ZK_REQUIRE(out == nullptr || norm_w != nullptr, "zk_sublayer_step: the norm needs its gain");
  ZK_REQUIRE((size_t)W * 4 <= 96 * 1024, "zk_sublayer_step: rows of more than 24576 channels are not supported");
  ZK_REQUIRE(conv_w == nullptr || (out != nullptr && taps >= 1 && positions != nullptr && req_of_token != nullptr &&
                                   slot_of_req != nullptr),
             "zk_sublayer_step: a convolution needs an output, its taps and the step's arrays");
  ZK_REQUIRE(conv_w == nullptr || taps == 1 ||
                 (state != nullptr && (long long)slot_words >= (long long)offset_words + (long long)(taps - 1) * W),
             "zk_sublayer_step: the convolution's state does not fit its slot");
  if (T == 0) return 0;
  SublayerConv cv{conv_w, state, positions, req_of_token, slot_of_req, taps, slot_words, offset_words};
  auto aligned = [](const void* p, size_t n) { return (uintptr_t)p % n == 0; };
  const size_t act4 = 4 * sizeof(act_t);
  const bool vec = W % 4 == 0 && aligned(h, 16) && aligned(y_gain, 16) && aligned(norm_w, 16) && aligned(norm_b, 16) &&
                   aligned(conv_w, 16) && aligned(raw, act4) && aligned(out, act4) && aligned(y, y_parts > 0 ? 16 : act4) &&
                   (conv_w == nullptr || (aligned(state, 16) && slot_words % 4 == 0 && offset_words % 4 == 0));
  if (vec && W <= 4096) {
    // (which kernel follows from the width and the operands' places alone, and the block from the width: the order
    // of a row's sums does not follow from how many rows a step brings)
    const int width = (W / 4 + 63) / 64 * 64;
#define ROW(N)                                                                                                            \
  sublayer_row_kernel<N><<<T, width, 0, (hipStream_t)stream>>>(h, y, y_parts, (size_t)T * W, y_gain, y_unit, y_eps, (act_t*)raw, \
                                                               norm_w, norm_b, eps, (act_t*)out, cv, W)
    if (conv_w == nullptr) ROW(0);
    else if (taps == 2) ROW(2);
    else if (taps == 3) ROW(3);
    else if (taps == 4) ROW(4);
    else ROW(-1);
#undef ROW
    return zk_launch_status("zk_sublayer_step");
  }
  const size_t lds = (size_t)W * 4;
  if (lds > 48 * 1024) {
    static bool raised = false;
    if (!raised) {
      hipFuncSetAttribute((const void*)sublayer_step_kernel<4>, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
      hipFuncSetAttribute((const void*)sublayer_step_kernel<1>, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
      raised = true;
    }
  }
  // in the 32-bit library the block is always 256 wide: the order of a row's sums must not follow
  // from how many rows a step brings
  const int threads = (ZSE_ACT_BF16 && T <= 64 && W >= 2048) ? 512 : 256;
  if (vec)
    sublayer_step_kernel<4><<<T, threads, lds, (hipStream_t)stream>>>(h, y, y_parts, (size_t)T * W, y_gain, y_unit, y_eps,
                                                                     (act_t*)raw, norm_w, norm_b, eps, (act_t*)out, cv, W);
  else
    sublayer_step_kernel<1><<<T, threads, lds, (hipStream_t)stream>>>(h, y, y_parts, (size_t)T * W, y_gain, y_unit, y_eps,
                                                                     (act_t*)raw, norm_w, norm_b, eps, (act_t*)out, cv, W);
  return zk_launch_status("zk_sublayer_step");
}

// h: float [T, W], replaced by its layer norm (b may be null).
int zk_norm_stream(float* h, const float* w, const float* b, float eps, int T, int W, void* stream) {
  ZK_REQUIRE(T >= 0 && W > 0 && h != nullptr && w != nullptr, "zk_norm_stream: bad arguments");
  if (T == 0) return 0;
  norm_stream_kernel<<<T, 256, 0, (hipStream_t)stream>>>(h, w, b, eps, W);
  return zk_launch_status("zk_norm_stream");
}

// z: float [T, n]; table: rows ld_table apart in the storage type, of which columns
// [column, column + n) are read at the rows tokens[t]; out: [T, n] activations, gelu_tanh(z) * table.
int zk_token_gate(const float* z, const void* table, const int* tokens, int ld_table, int column, void* out, int T, int n,
                  void* stream) {
  ZK_REQUIRE(T >= 0 && n > 0 && column >= 0 && ld_table >= column + n, "zk_token_gate: bad sizes");
  if (T == 0) return 0;
  const size_t total = (size_t)T * n;
  token_gate_kernel<<<(unsigned)((total + 255) / 256), 256, 0, (hipStream_t)stream>>>(z, (const act_t*)table, tokens, ld_table,
                                                                                     column, (act_t*)out, T, n);
  return zk_launch_status("zk_token_gate");
}

}  // extern "C"

ZK_ENTER(zk_sublayer_step)
ZK_ENTER(zk_norm_stream)
ZK_ENTER(zk_token_gate)
