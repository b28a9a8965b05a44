// Paged attention on the matrix cores, bfloat16 in, float softmax.
//
// A wave owns up to 32 query rows: TPW consecutive tokens of one request times the g = nh / nkv
// query heads that share a KV head, so every K and V tile it loads serves the
// whole group (the reference's paged_attention_v2 stages a K/V tile once for
// the heads of a group too, orchestrator/kernels.py:687-854, but is never
// launched; the launched kernels read K and V once per query head and hold one
// score per cached token in shared memory, :524-671, :859-958).
//
// Per tile of 32 keys:
//   S^T[key, row]  = K[key, :] . Q[row, :]        32x32x16 MFMA, hd/16 steps
//   scale, soft cap, mask (key <= pos, pos - key < window), running max / sum
//   O^T[d, row]   += V^T[d, key] * P^T[key, row]  32x32x16 MFMA, 2 per 32 channels
// S^T and O^T both keep a query row in a fixed lane (column = lane % 32), so the
// running maximum, sum and rescale are per-lane scalars, and the probabilities
// a lane holds after the first product are exactly its operand for the second:
// the contraction order over keys is permuted to match (slots e < 4 of lane half
// h are keys 4h + e, slots e >= 4 are keys 8 + 4h + e - 4), and V is read with
// the same permutation.  V is therefore cached transposed, [page][kv head][hd][bs],
// so that four consecutive keys of a channel are one 8-byte load.
//
// Portions have three kernels, chosen by the launch's sizes (zk_attention_bf16): a group of 32
// rows a block, its four waves sharing out the keys (attn_mfma_kernel: few groups); four or
// eight consecutive groups a block with every tile of keys and values fetched once into LDS for
// all of them (attn_shared_kernel: many groups); and the latter with the keys of a block of rows
// cut into ranges over several blocks, joined by attn_portion_join_kernel (few groups with long
// contexts: a portion of a prompt behind thousands of tokens).
//
// Decoded tokens use a split variant: the keys are cut into chunks of 64 (or 32, as
// the caller says) aligned to absolute positions, one wave per chunk writes (max, sum, O)
// and a second kernel joins the chunks in order; the cut is the caller's choice and never
// follows from the batch, so a request's result is the same whoever shares its step.  With
// at most 16 heads a KV head the chunks run on 16x16x32 MFMAs (attn_decode_kernel):
// a single query token fills only g of a tile's columns, and the narrower tile
// halves both the accumulator registers and the wasted work, so two waves fit a SIMD.
//
// A head's values may be half or twice as wide as its keys.  Where a window keeps the sequence's first
// keys in sight, the tiles (or a decoded token's chunks) of those keys come first and are
// followed by the window's.
// The kernels are templates in attention_bf16_kernels.h.
#include "attention_bf16_kernels.h"
#include "packed_call.h"

#include <algorithm>

#if ZSE_ACT_BF16

// Joins the ranges of keys of a portion's rows (attn_shared_kernel, SPLIT), in their order: a
// block of 64 threads per (32 channels of a wave of a block of rows, KV head, request), every
// lane the row and the channels it had in the kernel that wrote the partial results.  The ranges a block of rows
// has follow from its first and last key as there; a range that a row does not see at all (one
// past its position, in a block of rows on the diagonal) has the maximum -inf and weighs nothing.
__global__ __launch_bounds__(64) void attn_portion_join_kernel(AttnParams p, int per_block, int row_blocks, int dts) {
  const int r = p.r_begin + blockIdx.z, kvh = blockIdx.y;
  const int dt = blockIdx.x % dts, ww = blockIdx.x / dts;      // 32 channels of a wave's rows a block
  const int rows_x = ww >> 2, wave = ww & 3;
  const int lane = threadIdx.x, lr = lane & 31, lk = lane >> 5;
  const int qs = p.q_start[r], n = p.q_start[r + 1] - qs;
  if (n <= 0) return;
  const int start = p.ctx_len[r] - n;
  const int bi = (n + per_block - 1) / per_block - 1 - rows_x;
  if (bi < 0) return;
  const int g = p.nh / p.nkv;
  const int t0 = bi * per_block + wave * p.tpw;
  const int ntok = max(0, min(p.tpw, n - t0));
  const int tok = lr / g, hq = lr - tok * g;
  if (tok >= ntok) return;
  const int blk_lo = start + bi * per_block, blk_hi = start + min(n, (bi + 1) * per_block) - 1;
  const int key_lo = first_key(p, blk_lo);
  const int ranges = (KeyTiles(p, key_lo, blk_hi).count - 1) / p.chunk + 1;
  const size_t slot0 = ((((size_t)blockIdx.z * p.nkv + kvh) * row_blocks + rows_x) * p.nchunks) * 4 + wave;
  float m = -INFINITY;
  for (int c = 0; c < ranges; c++) m = fmaxf(m, p.part_ml[(slot0 + (size_t)c * 4) * 128 + lr]);
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; j++) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float l = 0.f;
  for (int c = 0; c < ranges; c++) {
    const size_t slot = slot0 + (size_t)c * 4;
    const float mc = p.part_ml[slot * 128 + lr];
    const float w = mc == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mc - m);
    l += w * p.part_ml[slot * 128 + 32 + lr];
    const f32x4* po = (const f32x4*)p.part_o + slot * ((size_t)dts * 4 * 64) + (size_t)dt * 4 * 64 + lane;
#pragma unroll
    for (int j = 0; j < 4; j++) acc[j] += w * po[j * 64];
  }
  const int row = qs + t0 + tok, head = q_head_of(p, kvh, hq);
  const float inv = row_factor(p, row, head, l, m);
  __bf16* orow = p.out + ((size_t)row * p.nh + head) * p.vd;
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const int d = dt * 32 + 8 * j + 4 * lk;
    if (d < p.vd) {
      bf16x4 w4;
#pragma unroll
      for (int i = 0; i < 4; i++) w4[i] = (__bf16)(acc[j][i] * inv);
      *(bf16x4*)(orow + d) = w4;
    }
  }
}

// Joins the chunks of a decoded token's attention, in chunk order: a block per
// (request, head), a thread per channel; the chunks' weights exp(m_c - m) are computed once.
#define ATT_MAX_CHUNKS 1024
__global__ __launch_bounds__(256) void attn_combine_kernel(const float* __restrict__ part_o,
                                                           const float* __restrict__ part_ml,
                                                           const int* __restrict__ q_start,
                                                           const int* __restrict__ ctx_len,
                                                           __bf16* __restrict__ out, int nh, int hd,
                                                           int window, int r_begin, int nchunks, int span,
                                                           int mask_chunk, int sink, int keep,
                                                           const float* __restrict__ sinks,
                                                           const __bf16* __restrict__ gate, int gate_ld) {
  __shared__ float wgt[ATT_MAX_CHUNKS];
  __shared__ float red[17];
  const int rr = blockIdx.x, head = blockIdx.y;
  const int r = r_begin + rr;
  const int n = q_start[r + 1] - q_start[r];
  if (n <= 0) return;
  const int pos = ctx_len[r] - 1;
  const int lo = mask_chunk > 0 ? pos - pos % mask_chunk : window > 0 ? max(0, pos - window + 1) : 0;
  // the parts of the kept first keys, [0, kept), then those from the window's first on, [c0, c1]
  const int c0 = lo / span, c1 = pos / span, kept = min((keep + span - 1) / span, c0);
  auto part_of = [&](int i) { return i < kept ? i : c0 + i - kept; };
  const size_t base = ((size_t)rr * nh + head) * nchunks;
  const int np = kept + c1 - c0 + 1;
  // the first partial results of the thread's channel are asked for now: they come in while
  // the weights are worked out (a part past the last is read from the last and not used)
  constexpr int PF = 16;
  const int d0 = min((int)threadIdx.x, hd - 1);
  float pf[PF];
  {
    const float* po = part_o + base * hd + d0;
#pragma unroll
    for (int c = 0; c < PF; c++) pf[c] = po[(size_t)part_of(min(c, np - 1)) * hd];
  }
  float m = -INFINITY;
  for (int c = threadIdx.x; c < np; c += 256) m = fmaxf(m, part_ml[(base + part_of(c)) * 2]);
  m = wave_max(m);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = m;
  __syncthreads();
  m = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  __syncthreads();
  float l = 0.f;
  for (int c = threadIdx.x; c < np; c += 256) {
    const size_t at = (base + part_of(c)) * 2;
    const float w = __builtin_amdgcn_exp2f(part_ml[at] - m);
    wgt[c] = w;
    l += part_ml[at + 1] * w;
  }
  l = block_sum(l, red);
  const int row = q_start[r];
  const float inv = gate_factor(gate, gate_ld, row, head) / (l + sink_weight(sinks, sink, head, m));
  __bf16* orow = out + ((size_t)row * nh + head) * hd;
  for (int d = threadIdx.x; d < hd; d += 256) {
    const float* po = part_o + base * hd + d;
    float acc = 0.f;
    int c = 0;
    if (d == d0) {                      // the channel whose first parts are here already
#pragma unroll
      for (int q = 0; q < PF; q++)
        if (q < np) acc += pf[q] * wgt[q];
      c = min(np, PF);
    }
    for (; c + 4 <= np; c += 4) {       // four loads in flight, summed in part order
      const float v0 = po[(size_t)part_of(c) * hd], v1 = po[(size_t)part_of(c + 1) * hd];
      const float v2 = po[(size_t)part_of(c + 2) * hd], v3 = po[(size_t)part_of(c + 3) * hd];
      acc += v0 * wgt[c];
      acc += v1 * wgt[c + 1];
      acc += v2 * wgt[c + 2];
      acc += v3 * wgt[c + 3];
    }
    for (; c < np; c++) acc += po[(size_t)part_of(c) * hd] * wgt[c];
    orow[d] = (__bf16)(acc * inv);
  }
}

static int launch_attn(int what, const AttnParams& p, dim3 grid, hipStream_t s) {
  if (p.vd != p.hd) return attn_launch_uneven(what, p, grid, s);
  switch (p.hd / 16) {
    case 1: return launch_sizes<1, 1>(what, p, grid, s);
    case 2: return launch_sizes<2, 2>(what, p, grid, s);
    case 4: return launch_sizes<4, 4>(what, p, grid, s);
    case 8: return launch_sizes<8, 8>(what, p, grid, s);
    case 16: return launch_sizes<16, 16>(what, p, grid, s);
    default: return zk_fail("zk_attention_bf16: head_dim must be 16, 32, 64, 128 or 256");
  }
}

// Bytes the portions' split variant needs behind the decoded tokens' part of the workspace.
// Per (request, KV head, block of rows, range, wave): the wave's accumulators as they lie in
// its registers (ceil(hd / 32) x 16 floats a lane) and 128 floats of maxima and sums.
static size_t portion_split_bytes(long row_blocks, int nkv, int hd, int ranges) {
  const size_t dt = (size_t)(hd + 31) / 32;
  return (size_t)row_blocks * nkv * ranges * 4 * (dt * 16 * 64 + 128) * sizeof(float);
}

// The ranges of keys for a launch of few blocks of rows: tiles a range (0: do not split) and the
// most ranges a block of rows can have.  Priced for one causal request of max_q_len rows ending
// at max_ctx, window or not: blocks(ct) = sum over the blocks of rows of ceil(tiles / ct), and
// the time goes with ceil(blocks / 256) * ct; of equal times the longer range (fewer partial
// results).  No split unless it at least halves the longest block's tiles; at most
// ATT_MOST_RANGES ranges for the longest block of rows the caller's limits allow (bound_tiles),
// which bounds the workspace.
static int portion_ranges(int max_q_len, int max_ctx, int window, int mask_chunk, int keep, int per_block, int nkv,
                          int r_prefill, int bound_tiles) {
  const int row_blocks = (max_q_len + per_block - 1) / per_block;
  auto tiles_of = [&](int bi) {
    const int lo = max_ctx - max_q_len + bi * per_block, hi = std::min(max_ctx, lo + per_block) - 1;
    const int klo = mask_chunk > 0 ? lo - lo % mask_chunk : window > 0 ? std::max(0, lo - window + 1) : 0;
    return std::min((keep + 31) / 32, klo / 32) + hi / 32 - klo / 32 + 1;
  };
  int longest = 0;
  for (int bi = 0; bi < row_blocks; bi++) longest = std::max(longest, tiles_of(bi));
  static const int cands[] = {32, 24, 16, 12, 10, 8, 6, 4};
  int best = 0;
  long best_cost = (long)((long)row_blocks * nkv * r_prefill + 255) / 256 * (longest + 10);
  for (int ct : cands) {
    if (2 * ct > longest || (bound_tiles + ct - 1) / ct > ATT_MOST_RANGES) continue;
    long blocks = 0;
    for (int bi = 0; bi < row_blocks; bi++) blocks += (tiles_of(bi) + ct - 1) / ct;
    blocks *= (long)nkv * r_prefill;
    const long cost = (blocks + 255) / 256 * (ct + 10) + 6;   // a block's start and end, the joining launch: in tiles' worth
    if (cost < best_cost) { best = ct; best_cost = cost; }
  }
  return best;
}

// 0: the portion kernel is chosen by the sizes; 1: a group of rows a block; 4, 8: shared
// tiles with that many waves a block; 5: shared tiles, four waves, the keys in ranges (as far as
// the workspace allows).  For tests and measurements (process-wide).
static int portion_kernel_mode = 0;

extern "C" {

int zk_attention_bf16_portion_kernel(int mode) {
  const int before = portion_kernel_mode;
  if (mode == 0 || mode == 1 || mode == 4 || mode == 5 || mode == 8) portion_kernel_mode = mode;
  return before;
}

// 1 if the matrix-core kernel takes these sizes, else 0 (the caller then uses the plain kernel).
int zk_attention_bf16_supports(int nh, int nkv, int hd, int bs) {
  if (nkv <= 0 || nh % nkv) return 0;
  const int g = nh / nkv;
  const bool hd_ok = hd == 16 || hd == 32 || hd == 64 || hd == 128 || hd == 256;
  return hd_ok && g <= 32 && bs >= 4 && (bs & (bs - 1)) == 0;
}

// The same for heads whose values have vd channels: as wide as keys, half or twice as wide.
int zk_attention_bf16_supports_values(int nh, int nkv, int hd, int vd, int bs) {
  return zk_attention_bf16_supports(nh, nkv, hd, bs) && (vd == hd || (zk_attention_bf16_supports(nh, nkv, vd, bs) &&
                                                                     (vd == 2 * hd || hd == 2 * vd)));
}

// Bytes of workspace the split variant needs for ``n_decode`` single-token requests.
size_t zk_attention_bf16_workspace(int n_decode, int nh, int hd, int max_ctx) {
  const size_t nchunks = ((size_t)max_ctx + ATT_CHUNK - 1) / ATT_CHUNK;      // an upper bound for both variants
  return (size_t)n_decode * nh * nchunks * (hd + 2) * sizeof(float);
}

// Bytes of workspace that let portions of up to ``max_rows`` rows in all split their keys into
// ranges (a launch of few blocks of rows with long contexts), on top of the decoded tokens'
// part.  A caller that brings less gets the kernels that need none.
size_t zk_attention_bf16_portion_workspace(int max_rows, int nh, int nkv, int hd) {
  if (max_rows <= 0 || nkv <= 0 || nh % nkv || hd <= 0) return 0;
  const int per_block = 4 * std::max(1, 32 / (nh / nkv));
  return portion_split_bytes((max_rows + per_block - 1) / per_block, nkv, hd, ATT_MOST_RANGES) + 256;
}

// Whether decoded tokens of these sizes run on the 16-wide tiles (partial results joined four
// chunks at a time inside a block) or on the 32-wide ones (one partial result a chunk).
static bool decode_on_narrow_tiles(int nh, int nkv, int hd) { return nh / nkv <= 16 && hd % 32 == 0; }

// The longest context the split variant takes for decoded tokens (the joining kernel keeps one
// weight per partial result in LDS).  ``decode_chunk`` as in zk_attention_bf16.
long long zk_attention_bf16_max_context(int nh, int nkv, int hd, int decode_chunk) {
  if (nkv <= 0 || nh % nkv) return 0;
  const int chunk = decode_chunk == 32 ? 32 : ATT_CHUNK;
  const long long span = decode_on_narrow_tiles(nh, nkv, hd) ? 4LL * chunk : ATT_CHUNK;
  return span * ATT_MAX_CHUNKS;
}

// Requests [0, r_prefill) hold portions of more than one token (max_q_len the longest);
// requests [r_prefill, R) hold one token each and use the split variant over max_ctx keys.
// decode_chunk: keys a wave of the split variant takes on the 16-wide tiles, 32 or 64 (0: 64).
// It fixes where the sums over keys are cut, and so the bits of the result: a caller that wants
// a request's result not to depend on the rest of the batch passes the same value in every
// step.  32 gives twice the waves, each with one load from memory in its chain instead of
// two: better for few requests with short contexts, worse for many.
// mask_chunk > 0: a row sees the keys of its own chunk of that many positions (counted from
// position 0) instead of a window; sink: a key of score 0 without a value in every denominator;
// wide_weights: the weights keep 16 bits of mantissa in the product with the values.
// v_shift: 2^v_shift neighbouring key heads read the values of one value head (the value cache
// then holds nkv >> v_shift heads): several maps of keys over the same values.
// vd: channels of a value and of the output's heads (hd, hd / 2 or 2 hd); the workspace functions above
// are asked with vd for their hd.  keep (with a window): a row sees the first ``keep`` keys of its sequence
// beside its window; the caller keeps their pages.
// sinks (may be null; not together with ``sink``): float [nh], exp(sinks[h]) joins head h's denominators.
// gate (may be null): bf16, row t's nh numbers at gate + t * gate_ld; head h's output times sigmoid of the h-th.
int zk_attention_bf16_gated(const void* q, int q_stride, const void* kcache, const void* vcache_t,
                           const int* block_table, int max_blocks, const int* q_start, const int* ctx_len,
                           void* out, int R, int r_prefill, int max_q_len, int max_ctx, int nh, int nkv,
                           int hd, int bs, float scale, float softcap, int window, int decode_chunk,
                           void* workspace, size_t workspace_bytes, int mask_chunk, int sink, int wide_weights,
                           int v_shift, int vd, int keep, const float* sinks, const void* gate, int gate_ld,
                           void* stream) {
  ZK_REQUIRE(!sink || sinks == nullptr, "zk_attention_bf16: a unit sink or learned sinks, not both");
  ZK_REQUIRE(gate == nullptr || gate_ld >= nh, "zk_attention_bf16: gate rows hold a number per head");
  ZK_REQUIRE(keep >= 0 && (keep == 0 || window > 0), "zk_attention_bf16: first keys are kept beside a window");
  ZK_REQUIRE(v_shift >= 0 && v_shift <= 4 && nkv % (1 << v_shift) == 0, "zk_attention_bf16: key heads in whole groups of a value head");
  ZK_REQUIRE(mask_chunk >= 0 && (mask_chunk == 0 || window == 0), "zk_attention_bf16: a window or a chunk, not both");
  ZK_REQUIRE(R >= 0 && r_prefill >= 0 && r_prefill <= R, "zk_attention_bf16: bad request counts");
  ZK_REQUIRE(zk_attention_bf16_supports_values(nh, nkv, hd, vd, bs), "zk_attention_bf16: sizes not supported "
             "(head_dim 16/32/64/128/256, values as wide, half or twice as wide, at most 32 heads a KV head, page size a power of "
             "two from 4)");
  ZK_REQUIRE(q_stride >= nh * hd && q_stride % 8 == 0 && ((uintptr_t)q % 16 == 0),
             "zk_attention_bf16: q rows must be 16-byte aligned");
  ZK_REQUIRE(max_blocks > 0 && nkv <= 65535 && R <= 65535, "zk_attention_bf16: grid too large");
  ZK_REQUIRE(decode_chunk == 0 || decode_chunk == 32 || decode_chunk == 64,
             "zk_attention_bf16: decode_chunk must be 32 or 64");
  if (R == 0) return 0;
  // everything that can refuse is checked before the first launch
  if (R - r_prefill > 0) {
    ZK_REQUIRE(max_ctx > 0, "zk_attention_bf16: max_ctx must be positive");
    ZK_REQUIRE(max_ctx <= zk_attention_bf16_max_context(nh, nkv, hd, decode_chunk),
               "zk_attention_bf16: context too long for the split variant");
    ZK_REQUIRE(zk_attention_bf16_workspace(R - r_prefill, nh, vd, max_ctx) <= workspace_bytes,
               "zk_attention_bf16: workspace too small for the split partial results");
  }
  if (r_prefill > 0) ZK_REQUIRE(max_q_len > 0, "zk_attention_bf16: max_q_len must be positive");
  hipStream_t s = (hipStream_t)stream;
  AttnParams p;
  p.q = (const __bf16*)q; p.q_stride = q_stride;
  p.kcache = (const __bf16*)kcache; p.vcache = (const __bf16*)vcache_t; p.v_shift = v_shift;
  p.block_table = block_table; p.max_blocks = max_blocks;
  p.q_start = q_start; p.ctx_len = ctx_len; p.out = (__bf16*)out;
  p.nh = nh; p.nkv = nkv; p.hd = hd; p.vd = vd; p.bs = bs; p.keep = keep;
  p.scale = scale; p.softcap = softcap; p.window = window;
  p.from_window = 0;
  p.mask_chunk = mask_chunk; p.sink = sink ? 1 : 0; p.wide_weights = wide_weights ? 1 : 0;
  p.sinks = sinks; p.gate = (const __bf16*)gate; p.gate_ld = gate_ld;
  p.bs_shift = 0;
  while ((1 << p.bs_shift) < bs) p.bs_shift++;
  const float log2e = 1.4426950408889634f;
  p.k1 = scale * log2e;
  p.k2 = softcap > 0.f ? 2.f * scale / softcap * log2e : 0.f;
  p.c2 = softcap * log2e;
  const int g = nh / nkv, wide = std::max(hd, vd);
  if (r_prefill > 0) {
    p.tpw = 32 / g; p.r_begin = 0; p.nchunks = 1; p.part_o = nullptr; p.part_ml = nullptr;
    const int groups = (max_q_len + p.tpw - 1) / p.tpw;
    // one block a group; two groups a block when that lets every block run at once (256 CUs,
    // one block each) where single groups would need a second round
    const long long single = (long long)groups * nkv * r_prefill, paired = (long long)((groups + 1) / 2) * nkv * r_prefill;
    int rc;
    // Many groups: tiles shared by the four or eight groups of a block, where that still gives
    // every CU a block (four) or two (eight; head sizes up to 128, whose registers let two
    // waves share a SIMD).  Measured at 8 to 32 heads of 128 and 256 with 512 to 8,192 rows:
    // with fewer than about 768 groups the kernel of one group a block is faster (2,048 rows of
    // 8 heads of 256, 512 groups: 75 us against 111; 768 groups: a tie), with more the shared
    // tiles are (8 portions of 512 rows behind 7,680 tokens, 32 heads of 128: 1,630 -> 780 us;
    // 16 heads of 256: 1,560 -> 845 us; 8,192 rows of 8 heads of 256: 877 -> 463 us).
    int shared_waves = 0;
    if (bs >= 8 && portion_kernel_mode != 1) {
      if (portion_kernel_mode > 1) shared_waves = portion_kernel_mode;
      else if (single >= 4096 && wide <= 128) shared_waves = 8;
      else if (single >= 768) shared_waves = 4;
      if (shared_waves == 8 && wide > 128) shared_waves = 4;       // no room for two waves a SIMD
    }
    // Few blocks of rows with many keys each (a portion of a few hundred rows behind thousands of
    // tokens): four groups a block and the keys in ranges, where the workspace behind the decoded
    // tokens' part holds the ranges' partial results.  512 rows behind 3,584 tokens, 8 heads of
    // 256: 111 -> 52 us; behind 7,680: 209 -> 79 us; 16 heads of 256: 118 -> 76 us; 32 heads of
    // 128: 100 -> 73 us.  A whole prompt from its first token, 8 heads of 256: 2,048 rows 74 -> 62
    // us, 1,024 rows the same time either way (its blocks of rows are many and short already).
    int range_tiles = 0, most_ranges = 0;
    size_t split_at = 0;
    if (bs >= 8 && (portion_kernel_mode == 5 || (portion_kernel_mode == 0 && !shared_waves))) {
      const int per_block = 4 * p.tpw;
      // no block of rows has more tiles than this, whatever its request's length
      int bound = (max_ctx + 31) / 32;
      // (a chunk's rows see no more keys than a window of its size would show them)
      const int reach = mask_chunk > 0 ? mask_chunk : window;
      if (reach > 0) bound = std::min(bound, (reach + per_block + 31) / 32 + 1 + (keep + 31) / 32);
      range_tiles = portion_ranges(max_q_len, max_ctx, window, mask_chunk, keep, per_block, nkv, r_prefill, bound);
      if (range_tiles) {
        most_ranges = (bound + range_tiles - 1) / range_tiles;
        if (R - r_prefill > 0) split_at = (zk_attention_bf16_workspace(R - r_prefill, nh, vd, max_ctx) + 255) / 256 * 256;
        const size_t need = portion_split_bytes((long)r_prefill * ((max_q_len + per_block - 1) / per_block), nkv, vd,
                                                most_ranges);
        if (workspace == nullptr || (uintptr_t)workspace % 16 != 0 || split_at + need > workspace_bytes)
          range_tiles = 0;
      }
    }
    if (range_tiles) {
      const int per_block = 4 * p.tpw;
      AttnParams ps = p;
      ps.chunk = range_tiles;
      ps.nchunks = most_ranges;
      const int row_blocks = (max_q_len + per_block - 1) / per_block;
      const size_t slots = (size_t)r_prefill * nkv * row_blocks * most_ranges * 4;
      const int dts = (vd + 31) / 32;
      ps.part_o = (float*)((char*)workspace + split_at);
      ps.part_ml = ps.part_o + slots * dts * 16 * 64;
      dim3 grid(row_blocks * most_ranges, nkv, r_prefill);
      rc = launch_attn(ATT_RANGES, ps, grid, s);
      if (rc) return rc;
      attn_portion_join_kernel<<<dim3(row_blocks * 4 * dts, nkv, r_prefill), 64, 0, s>>>(ps, per_block, row_blocks, dts);
      rc = zk_launch_status("zk_attention_bf16 (join of the portions' ranges)");
    } else if (shared_waves) {
      if (shared_waves == 5) shared_waves = 4;
      dim3 grid((groups + shared_waves - 1) / shared_waves, nkv, r_prefill);
      rc = launch_attn(shared_waves == 4 ? ATT_SHARED4 : ATT_SHARED8, p, grid, s);
    } else if (single > 256 && paired <= 256) rc = launch_attn(ATT_PAIRS, p, dim3((groups + 1) / 2, nkv, r_prefill), s);
    else rc = launch_attn(ATT_GROUPS, p, dim3(groups, nkv, r_prefill), s);
    if (rc) return rc;
  }
  const int n_dec = R - r_prefill;
  if (n_dec > 0) {
    const int nchunks = (max_ctx + ATT_CHUNK - 1) / ATT_CHUNK;
    p.tpw = 1; p.r_begin = r_prefill; p.nchunks = nchunks;
    p.part_o = (float*)workspace;
    p.part_ml = (float*)workspace + (size_t)n_dec * nh * nchunks * vd;
    dim3 grid((nchunks + 3) / 4, nkv, n_dec);
    int rc = 0;
    int span = ATT_CHUNK;        // keys one partial result covers
    p.chunk = ATT_CHUNK;
    if (decode_on_narrow_tiles(nh, nkv, hd)) {
      if (decode_chunk == 32) {
        p.chunk = ATT_CHUNK / 2;
        grid.x = (2 * nchunks + 3) / 4;
      }
      // the block joins its four chunks: one partial result per 4 chunks of keys
      span = 4 * p.chunk;
      p.nchunks = grid.x;
      // a window covers at most ceil(window / span) + 1 blocks of span keys
      const int reach = mask_chunk > 0 ? mask_chunk : window;
      const int window_blocks = reach > 0 ? (reach + span - 1) / span + 1 + (keep + span - 1) / span : 0;
      if (reach > 0 && window_blocks < (int)grid.x) {
        p.from_window = 1;
        grid.x = window_blocks;
      }
      p.part_ml = (float*)workspace + (size_t)n_dec * nh * p.nchunks * vd;
      rc = launch_attn(ATT_DECODE, p, grid, s);
    } else {
      rc = launch_attn(ATT_DECODE_WIDE, p, grid, s);
    }
    if (rc) return rc;
    dim3 cgrid(n_dec, nh);
    attn_combine_kernel<<<cgrid, 256, 0, s>>>(p.part_o, p.part_ml, q_start, ctx_len, (__bf16*)out, nh, vd,
                                              window, r_prefill, p.nchunks, span, mask_chunk, sink, keep, sinks,
                                              (const __bf16*)gate, gate_ld);
    return zk_launch_status("zk_attention_bf16 (combine)");
  }
  return 0;
}

int zk_attention_bf16_sized(const void* q, int q_stride, const void* kcache, const void* vcache_t,
                           const int* block_table, int max_blocks, const int* q_start, const int* ctx_len,
                           void* out, int R, int r_prefill, int max_q_len, int max_ctx, int nh, int nkv,
                           int hd, int bs, float scale, float softcap, int window, int decode_chunk,
                           void* workspace, size_t workspace_bytes, int mask_chunk, int sink, int wide_weights,
                           int v_shift, int vd, int keep, void* stream) {
  return zk_attention_bf16_gated(q, q_stride, kcache, vcache_t, block_table, max_blocks, q_start, ctx_len, out, R,
                                 r_prefill, max_q_len, max_ctx, nh, nkv, hd, bs, scale, softcap, window, decode_chunk,
                                 workspace, workspace_bytes, mask_chunk, sink, wide_weights, v_shift, vd, keep, nullptr,
                                 nullptr, 0, stream);
}

int zk_attention_bf16_maps(const void* q, int q_stride, const void* kcache, const void* vcache_t,
                           const int* block_table, int max_blocks, const int* q_start, const int* ctx_len,
                           void* out, int R, int r_prefill, int max_q_len, int max_ctx, int nh, int nkv,
                           int hd, int bs, float scale, float softcap, int window, int decode_chunk,
                           void* workspace, size_t workspace_bytes, int mask_chunk, int sink, int wide_weights,
                           int v_shift, void* stream) {
  return zk_attention_bf16_sized(q, q_stride, kcache, vcache_t, block_table, max_blocks, q_start, ctx_len, out, R,
                                 r_prefill, max_q_len, max_ctx, nh, nkv, hd, bs, scale, softcap, window, decode_chunk,
                                 workspace, workspace_bytes, mask_chunk, sink, wide_weights, v_shift, hd, 0, stream);
}

int zk_attention_bf16_masked(const void* q, int q_stride, const void* kcache, const void* vcache_t,
                             const int* block_table, int max_blocks, const int* q_start, const int* ctx_len,
                             void* out, int R, int r_prefill, int max_q_len, int max_ctx, int nh, int nkv,
                             int hd, int bs, float scale, float softcap, int window, int decode_chunk,
                             void* workspace, size_t workspace_bytes, int mask_chunk, int sink, int wide_weights,
                             void* stream) {
  return zk_attention_bf16_maps(q, q_stride, kcache, vcache_t, block_table, max_blocks, q_start, ctx_len, out, R,
                                r_prefill, max_q_len, max_ctx, nh, nkv, hd, bs, scale, softcap, window, decode_chunk,
                                workspace, workspace_bytes, mask_chunk, sink, wide_weights, 0, stream);
}

int zk_attention_bf16(const void* q, int q_stride, const void* kcache, const void* vcache_t,
                      const int* block_table, int max_blocks, const int* q_start, const int* ctx_len,
                      void* out, int R, int r_prefill, int max_q_len, int max_ctx, int nh, int nkv,
                      int hd, int bs, float scale, float softcap, int window, int decode_chunk,
                      void* workspace, size_t workspace_bytes, void* stream) {
  return zk_attention_bf16_masked(q, q_stride, kcache, vcache_t, block_table, max_blocks, q_start, ctx_len, out, R,
                                  r_prefill, max_q_len, max_ctx, nh, nkv, hd, bs, scale, softcap, window, decode_chunk,
                                  workspace, workspace_bytes, 0, 0, 0, stream);
}

}  // extern "C"

extern "C" int zk_steplist_register(const char* name, int nargs, void* fn);
static const int zk_attention_bf16_masked_entered = zk_steplist_register(
    "zk_attention_bf16_masked", zk_packed::Call<zk_attention_bf16_masked>::nargs,
    (void*)zk_packed::Call<zk_attention_bf16_masked>::call);

static const int zk_attention_bf16_gated_entered = zk_steplist_register(
    "zk_attention_bf16_gated", zk_packed::Call<zk_attention_bf16_gated>::nargs,
    (void*)zk_packed::Call<zk_attention_bf16_gated>::call);

static const int zk_attention_bf16_sized_entered = zk_steplist_register(
    "zk_attention_bf16_sized", zk_packed::Call<zk_attention_bf16_sized>::nargs,
    (void*)zk_packed::Call<zk_attention_bf16_sized>::call);

static const int zk_attention_bf16_maps_entered = zk_steplist_register(
    "zk_attention_bf16_maps", zk_packed::Call<zk_attention_bf16_maps>::nargs,
    (void*)zk_packed::Call<zk_attention_bf16_maps>::call);

#endif  // ZSE_ACT_BF16
