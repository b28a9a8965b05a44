// A routed feed-forward: every token goes through ``top`` of E small gated layers.
//
//   s = sigmoid(router logits),  the ``top`` largest are chosen (the lower index among equals)
//   expert e of token t sees  x' = s_e x_t  (the weight multiplies the input, not the output)
//   g = min(Wg x', limit),  u = clamp(Wu x', -limit, limit),  y = g sigmoid(1.702 g) (u + 1)
//   out_t = sum over the chosen experts, in the order they were chosen, of Wd y
//
// Variants, as parameters of the ``_ext`` entry points: scores softmax(router logits) over all experts
// instead of sigmoids; the weight on the expert's output instead of its input (out_t = sum s_e Wd y);
// y = silu(g) u instead of the clamped form; experts without a gate, y = max(Wu x', 0)^2, whose
// weights are [E][F][W].  A shared layer's rows may be added to the experts' sum, times the sigmoid of
// a number a row.  ``zk_moe_route_groups`` chooses by s + a correction per
// expert, among the experts of the best groups only, and may bring the weights to a sum.
// Identity experts are numbers from E on that the router may choose: such an expert has no weights and gives
// its input back, so it adds s x_t.
//
// Two ways through the experts.  Few tokens (decoding): one block per (token, choice) multiplies
// the expert's rows by the token's row, and the weights stream once per choice.  Many tokens
// (bfloat16 only): the (token, choice) pairs are sorted by expert on the device, and a grouped
// matrix-core product runs over tiles of one expert's rows each, which it reads from where they are (or,
// where the weights multiply the inputs, from scaled rows gathered in that order); nothing comes back to the host, so a step can be written down and repeated.  Either
// way a row's sums run in an order fixed by the channel numbers, and a token's result does not
// depend on what else is in the step.
#include "common.h"
#include "packed_call.h"

extern "C" int zk_steplist_register(const char* name, int nargs, void* fn);
#define ZK_ENTER(fn) \
  static const int fn##_entered = zk_steplist_register(#fn, zk_packed::Call<fn>::nargs, (void*)zk_packed::Call<fn>::call);

#define MOE_MAX_EXPERTS 1024
#define MOE_MAX_TOP 16

__device__ __forceinline__ float clamped_swiglu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
}

__device__ __forceinline__ float expert_act(float g, float u, float limit, int act) {
  return act == 1 ? g / (1.0f + expf(-g)) * u : clamped_swiglu(g, u, limit);
}
#define MOE_NO_GATE 2             // act: experts without gate rows, the square of relu
__device__ __forceinline__ float square_of_relu(float x) {
  x = fmaxf(x, 0.f);
  return x * x;
}

// ---- the router: one wave per token
__global__ __launch_bounds__(64) void moe_route_kernel(const float* __restrict__ logits, int ld, int E, int top,
                                                       int* __restrict__ ids, float* __restrict__ wts, int softmax) {
  const int t = blockIdx.x, lane = threadIdx.x;
  float s[MOE_MAX_EXPERTS / 64];
  if (softmax) {
    // scores exp(z - max) / sum over all experts, in float
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++) {
      const int e = lane + 64 * i;
      s[i] = e < E ? logits[(size_t)t * ld + e] : -INFINITY;
      mx = fmaxf(mx, s[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++) {
      const int e = lane + 64 * i;
      s[i] = e < E ? expf(s[i] - mx) : 0.f;
      sum += s[i];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++) s[i] = (lane + 64 * i) < E ? s[i] / sum : -1.f;
  } else {
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++) {
      const int e = lane + 64 * i;
      s[i] = e < E ? 1.0f / (1.0f + expf(-logits[(size_t)t * ld + e])) : -1.f;
    }
  }
  for (int k = 0; k < top; k++) {
    float best = -2.f;
    int at = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++)
      if (s[i] > best) {
        best = s[i];
        at = lane + 64 * i;
      }
    // the largest score of the wave, the lowest index among equals
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oa = __shfl_xor(at, o, 64);
      if (ob > best || (ob == best && oa < at)) {
        best = ob;
        at = oa;
      }
    }
    if (lane == 0) {
      ids[(size_t)t * top + k] = at;
      wts[(size_t)t * top + k] = best;
    }
#pragma unroll
    for (int i = 0; i < MOE_MAX_EXPERTS / 64; i++)
      if (lane + 64 * i == at) s[i] = -1.f;
  }
}

// ---- the router with a correction per expert and groups of neighbouring experts: one wave per token.
// Choice scores c = s + correction (s = sigmoid of the logits, or their softmax).  With groups, the E
// experts form ``groups`` runs of E / groups; a group's value is the sum of its ``group_best`` (1 or 2) largest c
// (of one, where it has one), and only experts of the ``keep`` best groups can be chosen.  The ``top`` largest c are
// chosen, the lower number among equals, of groups as of experts.  Weights: s, divided by the
// chosen ones' sum (+ 1e-20) when ``normalise``, times ``scale``.
__global__ __launch_bounds__(64) void moe_route_groups_kernel(const float* __restrict__ logits, int ld,
                                                              const float* __restrict__ correction, int E, int top,
                                                              int groups, int keep, int softmax, int normalise, float scale,
                                                              int group_best, int* __restrict__ ids,
                                                              float* __restrict__ wts) {
  __shared__ float sc[MOE_MAX_EXPERTS], ch[MOE_MAX_EXPERTS], gv[MOE_MAX_EXPERTS];
  const int t = blockIdx.x, lane = threadIdx.x;
  const float* z = logits + (size_t)t * ld;
  float mx = 0.f, sum = 1.f;
  if (softmax) {
    mx = -INFINITY;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, z[e]);
    mx = wave_max(mx);
    sum = 0.f;
    for (int e = lane; e < E; e += 64) sum += expf(z[e] - mx);
    sum = wave_sum(sum);
  }
  for (int e = lane; e < E; e += 64) {
    const float s = softmax ? expf(z[e] - mx) / sum : 1.0f / (1.0f + expf(-z[e]));
    sc[e] = s;
    ch[e] = correction ? s + correction[e] : s;
  }
  __syncthreads();
  // the largest of v[0..n) still in the race, the lowest number among equals; one that was taken is
  // left at -inf by its taker.  Always a number below n, whatever the values are.
  auto best_of = [&](const float* v, int n) {
    float best = -INFINITY;
    int at = 0x7fffffff;
    for (int e = lane; e < n; e += 64)
      if (v[e] > best) {
        best = v[e];
        at = e;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oa = __shfl_xor(at, o, 64);
      if (ob > best || (ob == best && oa < at)) {
        best = ob;
        at = oa;
      }
    }
    return at < n ? at : 0;
  };
  if (groups > 1 && keep < groups) {
    const int size = E / groups;
    for (int g = lane; g < groups; g += 64) {
      float a = -INFINITY, b = -INFINITY;
      for (int i = 0; i < size; i++) {
        const float c = ch[g * size + i];
        if (c > a) {
          b = a;
          a = c;
        } else if (c > b) {
          b = c;
        }
      }
      gv[g] = (size > 1 && group_best > 1) ? a + b : a;
    }
    __syncthreads();
    for (int k = 0; k < keep; k++) {
      const int g = best_of(gv, groups);
      __syncthreads();
      if (lane == 0) gv[g] = NAN;                  // kept: out of the race, told apart from the rest
      __syncthreads();
    }
    for (int e = lane; e < E; e += 64)
      if (!isnan(gv[e / size])) ch[e] = -INFINITY;
    __syncthreads();
  }
  float total = 0.f;
  for (int k = 0; k < top; k++) {
    const int e = best_of(ch, E);
    __syncthreads();
    const float s = sc[e];
    total += s;
    if (lane == 0) {
      ids[(size_t)t * top + k] = e;
      wts[(size_t)t * top + k] = s * scale;
      ch[e] = -INFINITY;
    }
    __syncthreads();
  }
  if (normalise && lane == 0) {
    for (int k = 0; k < top; k++) {
      const float s = sc[ids[(size_t)t * top + k]];
      wts[(size_t)t * top + k] = s / (total + 1e-20f) * scale;
    }
  }
}

// Eight consecutive weights as floats (rows in whole groups of eight are read 16 bytes a lane).
__device__ __forceinline__ void load8(const float* p, float v[8]) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void load8(const __bf16* p, float v[8]) {
  typedef __bf16 b8 __attribute__((ext_vector_type(8)));
  const b8 t = *(const b8*)p;
#pragma unroll
  for (int i = 0; i < 8; i++) v[i] = (float)t[i];
}

// A wave's sum with the steps inside a row of 16 lanes done by lane permutations of the vector unit
// (lane i with 15 - i, with 7 - i, inside the quads), the two steps across rows through local memory.
__device__ __forceinline__ float wave_sum_rows(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x140, 0xf, 0xf, false));   // row_mirror
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x141, 0xf, 0xf, false));   // row_half_mirror
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0xB1, 0xf, 0xf, false));    // quad_perm [1,0,3,2]
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x4E, 0xf, 0xf, false));    // quad_perm [2,3,0,1]
  x += __shfl_xor(x, 16, 64);
  x += __shfl_xor(x, 32, 64);
  return x;
}

// The dot product of a weight row and a row in local memory, over a wave; the same order of sums
// whatever the step (eight channels a lane in turn where rows are whole groups of eight).
__device__ __forceinline__ float row_dot(const act_t* __restrict__ w, const float* __restrict__ x, int n, int lane) {
  float a = 0.f;
  if ((n & 7) == 0) {
    for (int i = lane * 8; i < n; i += 512) {
      float v[8];
      load8(w + i, v);
#pragma unroll
      for (int c = 0; c < 8; c++) a = fmaf(v[c], x[i + c], a);
    }
  } else {
    for (int i = lane; i < n; i += 64) a = fmaf(to_f32(w[i]), x[i], a);
  }
  return wave_sum_rows(a);
}

// ---- few tokens: y[(t, k), n] = act(Wg[e] x', Wu[e] x'), a wave per row pair
__global__ __launch_bounds__(256) void moe_gate_up_kernel(const act_t* __restrict__ x, const int* __restrict__ ids,
                                                          const float* __restrict__ wts, const act_t* __restrict__ w_gu,
                                                          act_t* __restrict__ y, int top, int W, int F, float limit,
                                                          int rows_per_block, int act, int on_out, int experts) {
  extern __shared__ float xs[];                   // [W]
  const int pair = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int e = ids[pair];
  if (e >= experts) return;                       // an identity expert: nothing to multiply, the whole block alike
  const float s = wts[pair];
  const int t = pair / top;
  const act_t* xr = x + (size_t)t * W;
  for (int i = tid; i < W; i += 256) xs[i] = on_out ? to_f32(xr[i]) : to_f32(from_f32<act_t>(s * to_f32(xr[i])));
  __syncthreads();
  const act_t* wg = w_gu + (size_t)e * (act == MOE_NO_GATE ? 1 : 2) * F * W;
  const int n0 = blockIdx.y * rows_per_block;
  for (int n = n0 + wave; n < min(F, n0 + rows_per_block); n += 4) {
    if (act == MOE_NO_GATE) {
      const float u = row_dot(wg + (size_t)n * W, xs, W, lane);
      if (lane == 0) y[(size_t)pair * F + n] = from_f32<act_t>(square_of_relu(u));
      continue;
    }
    const act_t* gr = wg + (size_t)n * W;
    const act_t* ur = wg + (size_t)(F + n) * W;
    const float g = row_dot(gr, xs, W, lane), u = row_dot(ur, xs, W, lane);
    if (lane == 0) y[(size_t)pair * F + n] = from_f32<act_t>(expert_act(g, u, limit, act));
  }
}

// What a shared layer adds to a row's sum: ``add`` [T, W] (may be null), times the sigmoid of the row's number in
// ``gate`` (may be null).
struct SharedRows {
  const float* add;
  const float* gate;
  int gate_ld;
  __device__ __forceinline__ float factor(int t) const {
    return (add && gate) ? 1.0f / (1.0f + expf(-gate[(size_t)t * gate_ld])) : 1.0f;
  }
};

// out[t, n] = sum_k Wd[e_k][n] . y[(t, k)], an identity expert's term s_k x[t, n], plus the shared layer's row
__global__ __launch_bounds__(256) void moe_down_kernel(const act_t* __restrict__ y, const int* __restrict__ ids,
                                                       const act_t* __restrict__ w_down, float* __restrict__ out,
                                                       int top, int W, int F, int rows_per_block,
                                                       const float* __restrict__ wts, int on_out,
                                                       const act_t* __restrict__ x, int experts, SharedRows shared) {
  extern __shared__ float ys[];                   // [top][F]
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int i = tid; i < top * F; i += 256)
    ys[i] = ids[(size_t)t * top + i / F] < experts ? to_f32(y[(size_t)t * top * F + i]) : 0.f;
  __syncthreads();
  const int n0 = blockIdx.y * rows_per_block;
  const float sg = shared.factor(t);
  for (int n = n0 + wave; n < min(W, n0 + rows_per_block); n += 4) {
    float total = 0.f;
    for (int k = 0; k < top; k++) {
      const int e = ids[(size_t)t * top + k];
      const float s = wts[(size_t)t * top + k];
      if (e >= experts) {
        total += s * to_f32(x[(size_t)t * W + n]);
        continue;
      }
      const act_t* wr = w_down + ((size_t)e * W + n) * F;
      const float d = row_dot(wr, ys + k * F, F, lane);
      total += on_out ? s * d : d;
    }
    if (lane == 0) out[(size_t)t * W + n] = shared.add ? total + sg * shared.add[(size_t)t * W + n] : total;
  }
}

// ---- a dense layer of the same form: y = act(gu[:, :F], gu[:, F:])
__global__ void clamped_glu_kernel(const act_t* __restrict__ gu, act_t* __restrict__ y, int F, float limit) {
  const int t = blockIdx.y;
  const int n = blockIdx.x * blockDim.x + threadIdx.x;
  if (n >= F) return;
  const act_t* row = gu + (size_t)t * 2 * F;
  y[(size_t)t * F + n] = from_f32<act_t>(clamped_swiglu(to_f32(row[n]), to_f32(row[F + n]), limit));
}

// ---- many tokens: sort the pairs by expert
// One block.  order[i] = the pair at sorted place i, place[] the reverse; first[e] = the first place of
// expert e (first[E] = pairs).  Which place among its expert's a pair gets is left to chance: a row's
// result does not depend on its place.
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int* __restrict__ ids, int pairs, int E,
                                                        int* __restrict__ first, int* __restrict__ order,
                                                       int* __restrict__ place) {
  __shared__ int count[MOE_MAX_EXPERTS + 1];
  __shared__ int cursor[MOE_MAX_EXPERTS];
  const int tid = threadIdx.x;
  for (int e = tid; e <= E; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = tid; i < pairs; i += 1024) atomicAdd(&count[ids[i] + 1], 1);
  __syncthreads();
  if (tid == 0) {
    for (int e = 0; e < E; e++) count[e + 1] += count[e];
  }
  __syncthreads();
  for (int e = tid; e <= E; e += 1024) first[e] = count[e];
  for (int e = tid; e < E; e += 1024) cursor[e] = count[e];
  __syncthreads();
  for (int i = tid; i < pairs; i += 1024) {
    const int at = atomicAdd(&cursor[ids[i]], 1);
    order[at] = i;
    place[i] = at;
  }
}

// the rows times their weights, in sorted order (weights that multiply the inputs)
__global__ void moe_gather_kernel(const act_t* __restrict__ x, const int* __restrict__ order,
                                  const float* __restrict__ wts, act_t* __restrict__ xg, int top, int W,
                                  const int* __restrict__ ids, int experts) {
  const int i = blockIdx.x;
  const int pair = order[i];
  if (ids[pair] >= experts) return;                       // sorted behind every expert's rows, never multiplied
  const float s = wts[pair];
  const act_t* xr = x + (size_t)(pair / top) * W;
  for (int c = threadIdx.x; c < W; c += blockDim.x) xg[(size_t)i * W + c] = from_f32<act_t>(s * to_f32(xr[c]));
}

#if ZSE_ACT_BF16
// Grouped product on the matrix cores: C[i, n] = sum_k A[i, k] B[e(i)][n, k] over rows sorted by
// expert.  A block takes TM rows of one expert and 64 columns (or NB times 64); which expert and which
// rows it finds in first[] (tiles never span two experts; a tile past the last one ends at once).
// Four waves, each TM / 2 rows by 32 of every 64 columns, 32 x 32 x 16 products.  Operands pass through
// local memory in steps of TK channels, two buffers; DEPTH steps are on their way in registers while one is
// multiplied, their loads without conditions (rows and columns past the end read the last one and are not
// stored, channels past the end are replaced by zeros).
//
// order (may be null): the sorted row i is row order[i] / top of A; without it A is sorted itself.
// mode 0: C = act(gate, up) with B = [E][2F][K], stores y[i, n] (n < F), the 64 columns' gate rows and up
// rows in the two halves of a B tile; mode 1: plain product with B = [E][N][K], stores float
// rows; mode 2: the square of relu of that product, stores y.
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx16 __attribute__((ext_vector_type(16)));

template <int MODE, int TM, int NB, int TK, int DEPTH>
__global__ __launch_bounds__(256) void moe_grouped_kernel(const __bf16* __restrict__ A, const int* __restrict__ order, int top,
                                                          const __bf16* __restrict__ B, const int* __restrict__ first, int E,
                                                          int N, int K, __bf16* __restrict__ y, float* __restrict__ out_rows,
                                                          float limit, int act) {
  static_assert(MODE != 0 || NB == 2, "a gate tile and an up tile");
  constexpr int LD = TK + 8, CPR = TK / 8, TN = NB * 64, MI = TM / 64;
  constexpr int APT = TM * CPR / 256, BPT = TN * CPR / 256;          // 16-byte pieces a thread moves
  constexpr int COLS = MODE == 0 ? 64 : TN;                          // columns of the result a block makes
  extern __shared__ __attribute__((aligned(16))) unsigned char grouped_raw[];
  __bf16* As = (__bf16*)grouped_raw;             // [2][TM][LD]
  __bf16* Bs = As + 2 * TM * LD;                 // [2][TN][LD]
  __shared__ int tile_e, tile_row, tile_end;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  if (wave == 0) {
    // the blockIdx.y-th tile of rows, counting each expert's rows in whole tiles, 64 experts a turn
    int left = blockIdx.y;
    bool found = false;
    for (int e0 = 0; e0 < E && !found; e0 += 64) {
      const int e = e0 + lane;
      const int lo = first[min(e, E)], hi = first[min(e + 1, E)];
      const int tiles = (hi - lo + TM - 1) / TM;
      int sum = tiles;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int other = __shfl_up(sum, o, 64);
        if (lane >= o) sum += other;
      }
      const bool mine = left < sum && left >= sum - tiles;
      if (mine) {
        tile_e = e;
        tile_row = lo + (left - (sum - tiles)) * TM;
        tile_end = hi;
      }
      found = __any(mine);
      left -= __shfl(sum, 63, 64);
    }
    if (!found && lane == 0) tile_row = -1;
  }
  __syncthreads();
  if (tile_row < 0) return;
  const int e = tile_e, row0 = tile_row, rows = min(TM, tile_end - tile_row);
  const int n0 = blockIdx.x * COLS;
  const int wm = (wave & 1) * (TM / 2), wn = (wave >> 1) * 32;
  const __bf16* Be = B + (size_t)e * (MODE == 0 ? 2 : 1) * N * K;
  // the thread's pieces: their rows' beginnings, their place in a step of TK channels and in local memory
  const __bf16* arow[APT];
  const __bf16* brow[BPT];
#pragma unroll
  for (int j = 0; j < APT; j++) {
    const int i = row0 + min((tid + 256 * j) / CPR, rows - 1);
    arow[j] = A + (size_t)(order ? order[i] / top : i) * K;
  }
#pragma unroll
  for (int j = 0; j < BPT; j++) {
    const int r = (tid + 256 * j) / CPR;
    brow[j] = Be + (size_t)(MODE == 0 ? (r >> 6) * N + min(n0 + (r & 63), N - 1) : min(n0 + r, N - 1)) * K;
  }
  const int lc = (tid % CPR) * 8;                // 256 is a multiple of CPR: the same for all of a thread's pieces
  bf16x8 ra[DEPTH][APT], rb[DEPTH][BPT];
  auto load = [&](int k0, bf16x8 (&a)[APT], bf16x8 (&b)[BPT]) {
    const int k = min(k0 + lc, K - 8);           // K is a multiple of 8
#pragma unroll
    for (int j = 0; j < APT; j++) a[j] = *(const bf16x8*)(arow[j] + k);
#pragma unroll
    for (int j = 0; j < BPT; j++) b[j] = *(const bf16x8*)(brow[j] + k);
  };
  floatx16 acc[MI][NB];
#pragma unroll
  for (int mi = 0; mi < MI; mi++)
#pragma unroll
    for (int nb = 0; nb < NB; nb++) acc[mi][nb] = floatx16{0};
#pragma unroll
  for (int d = 0; d < DEPTH; d++) load(d * TK, ra[d], rb[d]);
  int buf = 0;
  for (int k0 = 0; k0 < K; k0 += DEPTH * TK) {
#pragma unroll
    for (int d = 0; d < DEPTH; d++) {
      const int kd = k0 + d * TK;
      const bool in = kd + lc < K;
      __bf16* as = As + buf * TM * LD;
      __bf16* bs = Bs + buf * TN * LD;
#pragma unroll
      for (int j = 0; j < APT; j++) *(bf16x8*)(as + ((tid + 256 * j) / CPR) * LD + lc) = in ? ra[d][j] : bf16x8{0};
#pragma unroll
      for (int j = 0; j < BPT; j++) *(bf16x8*)(bs + ((tid + 256 * j) / CPR) * LD + lc) = in ? rb[d][j] : bf16x8{0};
      load(kd + DEPTH * TK, ra[d], rb[d]);
      __syncthreads();
      // (a wave whose rows are all past the tile's end has nothing to multiply)
      if (wm < rows) {
#pragma unroll
        for (int kk = 0; kk < TK; kk += 16) {
          bf16x8 av[MI];
#pragma unroll
          for (int mi = 0; mi < MI; mi++)
            av[mi] = *(const bf16x8*)(as + (wm + mi * 32 + (lane & 31)) * LD + kk + (lane >> 5) * 8);
#pragma unroll
          for (int nb = 0; nb < NB; nb++) {
            const bf16x8 bv = *(const bf16x8*)(bs + (nb * 64 + wn + (lane & 31)) * LD + kk + (lane >> 5) * 8);
#pragma unroll
            for (int mi = 0; mi < MI; mi++) acc[mi][nb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(av[mi], bv, acc[mi][nb], 0, 0, 0);
          }
        }
      }
      buf ^= 1;
    }
  }
  // element i of an accumulator: row (i / 4) * 8 + (lane / 32) * 4 + i % 4, column lane % 32
#pragma unroll
  for (int mi = 0; mi < MI; mi++)
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const int r = wm + mi * 32 + (i / 4) * 8 + (lane >> 5) * 4 + (i % 4);
      if (r >= rows) continue;
      if (MODE == 0) {
        const int col = n0 + wn + (lane & 31);
        if (col < N) y[(size_t)(row0 + r) * N + col] = (__bf16)expert_act(acc[mi][0][i], acc[mi][NB - 1][i], limit, act);
      } else {
#pragma unroll
        for (int nb = 0; nb < NB; nb++) {
          const int col = n0 + nb * 64 + wn + (lane & 31);
          if (col >= N) continue;
          if (MODE == 2) y[(size_t)(row0 + r) * N + col] = (__bf16)square_of_relu(acc[mi][nb][i]);
          else out_rows[(size_t)(row0 + r) * N + col] = acc[mi][nb][i];
        }
      }
    }
}

template <int MODE, int TM, int NB, int TK, int DEPTH>
static int launch_grouped(const void* A, const int* order, int top, const void* B, const int* first, int pairs, int E, int N, int K,
                          void* y, float* out_rows, float limit, int act, hipStream_t st) {
  constexpr size_t lds = (size_t)2 * (TM + NB * 64) * (TK + 8) * sizeof(__bf16);
  static bool raised = false;
  if (!raised) {
    if (lds > 64 * 1024 && hipFuncSetAttribute((const void*)moe_grouped_kernel<MODE, TM, NB, TK, DEPTH>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return zk_fail("zk_moe_experts_grouped: the local memory was refused");
    raised = true;
  }
  constexpr int cols = MODE == 0 ? 64 : NB * 64;
  const dim3 grid((N + cols - 1) / cols, (pairs + TM - 1) / TM + E);       // each expert may end in a tile that is not full
  moe_grouped_kernel<MODE, TM, NB, TK, DEPTH><<<grid, 256, lds, st>>>((const __bf16*)A, order, top, (const __bf16*)B, first, E, N, K,
                                                                      (__bf16*)y, out_rows, limit, act);
  return zk_launch_status("zk_moe_experts_grouped");
}

// out[t, :] = sum over t's choices, in their order, of the sorted rows' results (of s x[t, :] for an identity expert),
// plus the shared layer's row.  A thread takes four columns (W is a multiple of 8).
__global__ __launch_bounds__(256) void moe_combine_kernel(const float* __restrict__ rows, const int* __restrict__ place,
                                                          float* __restrict__ out, int top, int W, const float* __restrict__ wts,
                                                          int on_out, const int* __restrict__ ids, const __bf16* __restrict__ x,
                                                          int experts, SharedRows shared) {
  typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
  const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (c >= W) return;
  float4 sum = make_float4(0.f, 0.f, 0.f, 0.f), add = sum;
  if (shared.add) add = *(const float4*)(shared.add + (size_t)t * W + c);
  for (int k = 0; k < top; k++) {
    const size_t pair = (size_t)t * top + k;
    const bool identity = ids[pair] >= experts;
    const float s = (identity || on_out) ? wts[pair] : 1.f;
    float4 v;
    if (identity) {
      const bf16x4 xv = *(const bf16x4*)(x + (size_t)t * W + c);
      v = make_float4((float)xv[0], (float)xv[1], (float)xv[2], (float)xv[3]);
    } else {
      v = *(const float4*)(rows + (size_t)place[pair] * W + c);
    }
    sum.x += s * v.x;
    sum.y += s * v.y;
    sum.z += s * v.z;
    sum.w += s * v.w;
  }
  if (shared.add) {
    const float g = shared.factor(t);
    sum.x += g * add.x;
    sum.y += g * add.y;
    sum.z += g * add.z;
    sum.w += g * add.w;
  }
  *(float4*)(out + (size_t)t * W + c) = sum;
}
#endif

extern "C" {

// logits: float [T, E] -> ids int32 [T, top], wts float [T, top] (the scores themselves).
// (device memory that a kernel writes is passed as void*: an ``int*`` argument means a result the
// host reads, which a launch list replaces)
// ld: the distance between rows of logits (>= E; a row may hold more than the experts' logits).
// softmax: the scores are exp(z) / sum over all experts instead of sigmoid(z).
int zk_moe_route_ext(const float* logits, int ld, void* ids, float* wts, int T, int E, int top, int softmax, void* stream) {
  ZK_REQUIRE(T >= 0 && E > 0 && top > 0 && top <= E && ld >= E, "zk_moe_route: bad sizes");
  ZK_REQUIRE(E <= MOE_MAX_EXPERTS && top <= MOE_MAX_TOP, "zk_moe_route: up to 1024 experts and 16 choices");
  if (T == 0) return 0;
  moe_route_kernel<<<T, 64, 0, (hipStream_t)stream>>>(logits, ld, E, top, (int*)ids, wts, softmax);
  return zk_launch_status("zk_moe_route");
}

int zk_moe_route(const float* logits, void* ids, float* wts, int T, int E, int top, void* stream) {
  return zk_moe_route_ext(logits, E, ids, wts, T, E, top, 0, stream);
}

// As zk_moe_route_ext with a correction per expert (float [E], may be null: 0) that counts in the choice
// alone, ``groups`` groups of neighbours of which ``keep`` stay (groups <= 1: none), and weights that are
// divided by their sum (normalise) and times ``scale``.  group_best: a group is judged by the sum of its that
// many (1 or 2) largest choice scores.
int zk_moe_route_best(const float* logits, int ld, const float* correction, void* ids, float* wts, int T, int E, int top,
                      int groups, int keep, int softmax, int normalise, float scale, int group_best, void* stream) {
  ZK_REQUIRE(group_best == 1 || group_best == 2, "zk_moe_route_groups: a group is judged by its one or two best");
  ZK_REQUIRE(T >= 0 && E > 0 && top > 0 && top <= E && ld >= E, "zk_moe_route_groups: bad sizes");
  ZK_REQUIRE(E <= MOE_MAX_EXPERTS && top <= MOE_MAX_TOP, "zk_moe_route_groups: up to 1024 experts and 16 choices");
  ZK_REQUIRE(groups <= 1 || (E % groups == 0 && keep >= 1 && keep <= groups && keep * (E / groups) >= top),
             "zk_moe_route_groups: equal groups, of which enough stay for the choices");
  if (T == 0) return 0;
  moe_route_groups_kernel<<<T, 64, 0, (hipStream_t)stream>>>(logits, ld, correction, E, top, groups, keep, softmax, normalise,
                                                            scale, group_best, (int*)ids, wts);
  return zk_launch_status("zk_moe_route_groups");
}

int zk_moe_route_groups(const float* logits, int ld, const float* correction, void* ids, float* wts, int T, int E, int top,
                        int groups, int keep, int softmax, int normalise, float scale, void* stream) {
  return zk_moe_route_best(logits, ld, correction, ids, wts, T, E, top, groups, keep, softmax, normalise, scale, 2, stream);
}

// x: [T, W]; w_gu: [E][2F][W], an expert's gate rows, then its up rows; w_down: [E][W][F].
// y: scratch [T * top, F] activations; out: float [T, W].
// act: 0 the clamped form, 1 silu(gate) up, 2 the square of relu(up) without a gate (w_gu is then
// [E][F][W]).  on_out: the weight multiplies the expert's output.  experts: numbers below it have weights,
// numbers from it on are identity experts.  add (may be null): float [T, W], added to every row's sum, times
// sigmoid(gate[t * gate_ld]) where a gate is given.
int zk_moe_experts_identity(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down, void* y,
                            float* out, int T, int top, int W, int F, float limit, int act, int on_out, int experts,
                            const float* add, const float* gate, int gate_ld, void* stream) {
  ZK_REQUIRE(experts > 0, "zk_moe_experts: no experts");
  ZK_REQUIRE(T >= 0 && top > 0 && top <= MOE_MAX_TOP && W > 0 && F > 0, "zk_moe_experts: bad sizes");
  ZK_REQUIRE(T <= 65535 && (size_t)T * top <= 0x7fffffff, "zk_moe_experts: more than 65535 rows");
  ZK_REQUIRE((size_t)W * 4 <= 64 * 1024 && (size_t)top * F * 4 <= 64 * 1024, "zk_moe_experts: rows too wide for local memory");
  if (T == 0) return 0;
  const int rpb = 32;
  static bool raised = false;
  if (!raised) {
    hipFuncSetAttribute((const void*)moe_gate_up_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
    hipFuncSetAttribute((const void*)moe_down_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
    raised = true;
  }
  dim3 grid_up(T * top, (F + rpb - 1) / rpb);
  moe_gate_up_kernel<<<grid_up, 256, (size_t)W * 4, (hipStream_t)stream>>>((const act_t*)x, ids, wts, (const act_t*)w_gu,
                                                                          (act_t*)y, top, W, F, limit, rpb, act, on_out, experts);
  dim3 grid(T, (W + rpb - 1) / rpb);
  moe_down_kernel<<<grid, 256, (size_t)top * F * 4, (hipStream_t)stream>>>((const act_t*)y, ids, (const act_t*)w_down, out, top,
                                                                         W, F, rpb, wts, on_out, (const act_t*)x, experts,
                                                                         SharedRows{add, gate, gate_ld});
  return zk_launch_status("zk_moe_experts");
}

int zk_moe_experts_ext(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down, void* y,
                       float* out, int T, int top, int W, int F, float limit, int act, int on_out, void* stream) {
  return zk_moe_experts_identity(x, ids, wts, w_gu, w_down, y, out, T, top, W, F, limit, act, on_out, 0x7fffffff, nullptr,
                                 nullptr, 0, stream);
}

int zk_moe_experts(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down, void* y,
                   float* out, int T, int top, int W, int F, float limit, void* stream) {
  return zk_moe_experts_ext(x, ids, wts, w_gu, w_down, y, out, T, top, W, F, limit, 0, 0, stream);
}

// gu: [T, 2F] -> y [T, F]
int zk_clamped_glu(const void* gu, void* y, int T, int F, float limit, void* stream) {
  ZK_REQUIRE(T >= 0 && T <= 65535 && F > 0, "zk_clamped_glu: bad sizes");
  if (T == 0) return 0;
  dim3 grid((F + 255) / 256, T);
  clamped_glu_kernel<<<grid, 256, 0, (hipStream_t)stream>>>((const act_t*)gu, (act_t*)y, F, limit);
  return zk_launch_status("zk_clamped_glu");
}

#if ZSE_ACT_BF16
// The same through the grouped matrix-core product, with ``identity`` numbers behind the E experts'.  work: int32
// [E + identity + 1 + 2 * T * top] (first, order, place); xg: [T * top, W] (used only where the weights multiply the
// inputs, may be null otherwise) and y: [T * top, F] bfloat16; rows: float [T * top, W].
int zk_moe_experts_grouped_identity(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down,
                                    void* work, void* xg, void* y, float* rows, float* out, int T, int E, int top, int W,
                                    int F, float limit, int act, int on_out, int identity, const float* add,
                                    const float* gate, int gate_ld, void* stream) {
  ZK_REQUIRE(T >= 0 && top > 0 && top <= MOE_MAX_TOP && W > 0 && F > 0 && E > 0 && identity >= 0 &&
                 E + identity <= MOE_MAX_EXPERTS,
             "zk_moe_experts_grouped: bad sizes");
  ZK_REQUIRE(W % 8 == 0 && F % 8 == 0, "zk_moe_experts_grouped: widths in whole groups of eight");
  ZK_REQUIRE(((uintptr_t)x | (uintptr_t)y | (uintptr_t)xg | (uintptr_t)w_gu | (uintptr_t)w_down | (uintptr_t)rows | (uintptr_t)out |
              (uintptr_t)add) % 16 == 0, "zk_moe_experts_grouped: operands must be 16-byte aligned");
  ZK_REQUIRE(T <= 65535, "zk_moe_experts_grouped: more than 65535 rows");
  if (T == 0) return 0;
  const int pairs = T * top;
  int* first = (int*)work;
  int* order = first + E + identity + 1;
  int* place = order + pairs;
  hipStream_t st = (hipStream_t)stream;
  moe_sort_kernel<<<1, 1024, 0, st>>>(ids, pairs, E + identity, first, order, place);
  const void* in = x;
  const int* map = order;
  if (!on_out) {
    ZK_REQUIRE(xg != nullptr, "zk_moe_experts_grouped: no room for the scaled rows");
    moe_gather_kernel<<<pairs, 256, 0, st>>>((const act_t*)x, order, wts, (act_t*)xg, top, W, ids, E);
    in = xg;
    map = nullptr;
  }
  // few rows an expert: tiles of 64 rows, long steps, so that much of the weights is on its way at a time; many: 128 rows
  const bool few = pairs <= 32 * E;
  int rc;
#define ZK_GROUPED(MODE, ...) (few ? launch_grouped<MODE, 64, MODE == 0 ? 2 : 1, 128, 2>(__VA_ARGS__) \
                                   : launch_grouped<MODE, 128, 2, 64, 2>(__VA_ARGS__))
  if (act == MOE_NO_GATE) rc = ZK_GROUPED(2, in, map, top, w_gu, first, pairs, E, F, W, y, nullptr, limit, act, st);
  else rc = ZK_GROUPED(0, in, map, top, w_gu, first, pairs, E, F, W, y, nullptr, limit, act, st);
  if (rc) return rc;
  rc = ZK_GROUPED(1, y, nullptr, top, w_down, first, pairs, E, W, F, nullptr, rows, 0.f, 0, st);
#undef ZK_GROUPED
  if (rc) return rc;
  moe_combine_kernel<<<dim3(T, (W / 4 + 255) / 256), 256, 0, st>>>(rows, place, out, top, W, wts, on_out, ids, (const __bf16*)x, E,
                                                                 SharedRows{add, gate, gate_ld});
  return zk_launch_status("zk_moe_experts_grouped");
}

int zk_moe_experts_grouped_ext(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down,
                               void* work, void* xg, void* y, float* rows, float* out, int T, int E, int top, int W, int F,
                               float limit, int act, int on_out, void* stream) {
  return zk_moe_experts_grouped_identity(x, ids, wts, w_gu, w_down, work, xg, y, rows, out, T, E, top, W, F, limit, act,
                                         on_out, 0, nullptr, nullptr, 0, stream);
}

int zk_moe_experts_grouped(const void* x, const int* ids, const float* wts, const void* w_gu, const void* w_down,
                           void* work, void* xg, void* y, float* rows, float* out, int T, int E, int top, int W, int F,
                           float limit, void* stream) {
  return zk_moe_experts_grouped_ext(x, ids, wts, w_gu, w_down, work, xg, y, rows, out, T, E, top, W, F, limit, 0, 0, stream);
}
#endif

}  // extern "C"

#if ZSE_ACT_BF16
ZK_ENTER(zk_moe_experts_grouped)
ZK_ENTER(zk_moe_experts_grouped_ext)
ZK_ENTER(zk_moe_experts_grouped_identity)
#endif
ZK_ENTER(zk_moe_route_ext)
ZK_ENTER(zk_moe_route_groups)
ZK_ENTER(zk_moe_route_best)
ZK_ENTER(zk_moe_experts_identity)
ZK_ENTER(zk_moe_experts_ext)
ZK_ENTER(zk_moe_route)
ZK_ENTER(zk_moe_experts)
ZK_ENTER(zk_clamped_glu)
