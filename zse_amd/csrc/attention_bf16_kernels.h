// The kernels of attention_bf16.hip as templates over the sizes of a head's keys (HD16 sixteens) and of
// its values (VD16), and what launches them for one pair of sizes.  attention_bf16.hip holds those whose
// sizes are equal, attention_bf16_uneven.hip those of values half or twice as wide as keys, so
// that the two compile side by side.
#pragma once
#include "common.h"

#include <type_traits>

#if ZSE_ACT_BF16

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

#define ATT_CHUNK 64
#define ATT_MOST_RANGES 8      // ranges of keys a block of rows of a portion is cut into, at most

struct AttnParams {
  const __bf16* q;
  int q_stride;
  const __bf16* kcache;   // [page][nkv][bs][hd]
  const __bf16* vcache;   // [page][nkv >> v_shift][vd][bs]
  int v_shift;            // 2^v_shift neighbouring key heads share one value head (0: a value head per key head)
  const int* block_table;
  int max_blocks;
  const int* q_start;     // [R + 1]
  const int* ctx_len;     // [R]
  __bf16* out;            // [T][nh][vd]
  float* part_o;          // split: [slot][vd]
  float* part_ml;         // split: [slot][2]
  int nh, nkv, hd, bs;
  int vd;                 // channels of a value (and of the output's heads); hd: of a query or key
  int bs_shift;           // page size is 1 << bs_shift in the tuned kernels
  float scale, softcap;
  // scores in the log2 domain: with a cap c,  s2 = c2 * tanh(k2 * dot / 2)  computed as
  // c2 * (1 - 2 / (exp2(k2 * dot) + 1)),  k2 = 2 * scale / c * log2(e),  c2 = c * log2(e);
  // without a cap  s2 = k1 * dot,  k1 = scale * log2(e).  Probabilities are exp2(s2 - m2).
  float k1, k2, c2;
  int window;
  int tpw;                // tokens a wave owns
  int r_begin;            // first request of this launch
  int nchunks;            // split: chunks the grid covers
  int from_window;        // decode: block 0 of a request is the one its window begins in
  int chunk;              // decoded tokens on 16-wide tiles: keys a wave takes, 32 or 64
  int mask_chunk;         // > 0: a row sees the keys of its own chunk of this many positions only (no window then)
  int keep;               // beside its window a row sees the first ``keep`` keys of its sequence
  int sink;               // 1: a key of score 0 without a value joins every row's denominator
  const float* sinks;     // [nh] (may be null): exp(sinks[h]) joins head h's denominator, with no key and no value
  const __bf16* gate;     // (may be null) row t's numbers per head at gate + t * gate_ld; head h's output is
  int gate_ld;            // multiplied by the sigmoid of the h-th
  int wide_weights;       // 1: a weight meets the values as two bf16 numbers, its rounded value and what the
                          // rounding left (16 bits of mantissa instead of 8; one more product a tile)
};

// The query head that is the hq-th of key head kvh.  Without shared values: kvh * g + hq.  With
// 2^v_shift maps of keys over one value head, key head (v, m) serves map m of the g query heads
// of value head v, and a query head's maps lie side by side: ((v * g + hq) << v_shift) + m.
__device__ __forceinline__ int q_head_of(const AttnParams& p, int kvh, int hq) {
  const int g = p.nh / p.nkv;
  return (((kvh >> p.v_shift) * g + hq) << p.v_shift) | (kvh & ((1 << p.v_shift) - 1));
}

// The first key a row at position ``pos`` sees.  It never decreases as pos grows, which is all
// the kernels' bounds over groups and blocks of rows rest on.
__device__ __forceinline__ int first_key(const AttnParams& p, int pos) {
  if (p.mask_chunk > 0) return pos - pos % p.mask_chunk;
  return p.window > 0 ? max(0, pos - p.window + 1) : 0;
}

// The tiles of 32 keys that rows whose first key (but for the kept ones) is key_lo walk up to key_hi: those
// of the kept first keys, then from key_lo's on.  Tile i begins at key_of(i), 0 <= i < count.
struct KeyTiles {
  int kept, lo, count;
  __device__ __forceinline__ KeyTiles(const AttnParams& p, int key_lo, int key_hi) {
    lo = key_lo / 32;
    kept = min((p.keep + 31) / 32, lo);
    count = key_hi < 0 ? 0 : kept + key_hi / 32 - lo + 1;
  }
  __device__ __forceinline__ int key_of(int i) const { return 32 * (i < kept ? i : lo + i - kept); }
};

// What a head's sink adds to a row's sum of weights: 2^(sink - m), scores and maximum in the log2 domain.
__device__ __forceinline__ float sink_weight(const float* sinks, int unit_sink, int head, float m) {
  if (sinks) return __builtin_amdgcn_exp2f(sinks[head] * 1.4426950408889634f - m);
  return unit_sink ? __builtin_amdgcn_exp2f(-m) : 0.f;
}

// The sigmoid of a row's gate for a head.
__device__ __forceinline__ float gate_factor(const __bf16* gate, int gate_ld, int row, int head) {
  if (!gate) return 1.f;
  return 1.f / (1.f + __expf(-(float)gate[(size_t)row * gate_ld + head]));
}

// What a row's sum of weighted values is multiplied by: 1 over the sum of its weights, and its gate.
__device__ __forceinline__ float row_factor(const AttnParams& p, int row, int head, float l, float m) {
  return gate_factor(p.gate, p.gate_ld, row, head) / (l + sink_weight(p.sinks, p.sink, head, m));
}

__device__ __forceinline__ float score_log2(const AttnParams& p, float dot) {
  if (p.softcap > 0.f) {
    const float e = __builtin_amdgcn_exp2f(p.k2 * dot);
    return p.c2 * (1.f - 2.f * __builtin_amdgcn_rcpf(e + 1.f));
  }
  return p.k1 * dot;
}

// Portions: which (group, KV head) a block takes.  Blocks go to the 8 XCDs in turn by their
// number, and every XCD has an L2 of its own; blocks that read the same keys and values (those
// of one KV head) are therefore given to as few XCDs as possible, so that what one of them has
// fetched is in the L2 for the others instead of crossing from the memory side once per block.
__device__ __forceinline__ void portion_block(int& bx, int& by) {
  const int gx = gridDim.x, gy = gridDim.y;
  bx = blockIdx.x;
  by = blockIdx.y;
  const int total = gx * gy;
  if (total % 8) return;
  const int lin = blockIdx.x + gx * blockIdx.y, xcd = lin & 7, slot = lin >> 3;
  if (gy <= 8 && 8 % gy == 0) {            // 8 / gy XCDs a head
    const int per = 8 / gy;
    by = xcd % gy;
    bx = slot * per + xcd / gy;
  } else if (gy % 8 == 0) {                // gy / 8 heads an XCD
    const int heads = gy / 8;
    by = xcd + 8 * (slot % heads);
    bx = slot / heads;
  }
}

template <int HD16, int VD16, bool SPLIT, bool PAIR>
__global__ __launch_bounds__(256, (HD16 <= 8 && VD16 <= 8 && !PAIR) ? 2 : 1) void attn_mfma_kernel(AttnParams p) {
  constexpr int DT = (VD16 + 1) / 2;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lr = lane & 31, lk = lane >> 5;
  const int r = p.r_begin + blockIdx.z;
  int block_x = blockIdx.x, kvh = blockIdx.y;
  if (!SPLIT) portion_block(block_x, kvh);
  const int qs = p.q_start[r], n = p.q_start[r + 1] - qs;
  if (n <= 0) return;
  const int start = p.ctx_len[r] - n;
  // portions: a block owns one group of rows and its four waves take every fourth tile of
  // keys (their results are joined at the end).  Or (PAIR, for portions whose groups would
  // need a second, half-empty round of blocks) two groups: one from the end of the portion,
  // which sees many keys, and its mirror from the start, which sees few, so that every block
  // has about the same work; the four waves are shared out between the two by their numbers
  // of key tiles (3 + 1, 2 + 2 or 1 + 3), a group's waves taking its tiles in turn.
  // Decoded tokens: a wave owns one chunk of keys.
  int gi = 0, phase = wave, nphase = 4, first_wave = 0;        // group, and the wave's place among its waves
  int na_block = 4;                                            // waves of the block's first group
  // single groups: the last group of a portion sees the most keys and goes first, so that the
  // blocks still running at the end are the short ones
  if (!SPLIT && !PAIR) gi = (n + p.tpw - 1) / p.tpw - 1 - block_x;
  if (PAIR) {
    const int groups = (n + p.tpw - 1) / p.tpw;
    if (block_x >= (groups + 1) / 2) return;           // the whole block is past the portion
    const int ga = groups - 1 - block_x, gb = block_x;
    if (ga != gb) {
      auto tiles_of = [&](int gr) {
        const int lo = start + gr * p.tpw, hi = start + min(n, (gr + 1) * p.tpw) - 1;
        return KeyTiles(p, first_key(p, lo), hi).count;
      };
      const int ta = tiles_of(ga), tb = tiles_of(gb);
      const int na = min(3, max(1, (4 * ta + (ta + tb) / 2) / (ta + tb)));
      na_block = na;
      if (wave < na) { gi = ga; phase = wave; nphase = na; }
      else { gi = gb; phase = wave - na; nphase = 4 - na; first_wave = na; }
    } else {
      gi = ga;
    }
  }
  const int chunk = SPLIT ? block_x * 4 + wave : 0;
  const int t0 = gi * p.tpw;
  if (!PAIR && (gi < 0 || t0 >= n)) return;
  const int g = p.nh / p.nkv;
  const int tok = lr / g, hq = lr - tok * g;
  const int ntok = min(p.tpw, n - t0);
  const bool row_ok = tok < ntok;
  const int trow = qs + t0 + (row_ok ? tok : 0);
  const int pos = start + t0 + (row_ok ? tok : 0);
  const int head = q_head_of(p, kvh, row_ok ? hq : 0);
  const int pos_lo = start + t0, pos_hi = start + t0 + ntok - 1;
  int key_lo = first_key(p, pos_lo);
  int key_hi = pos_hi;
  if (SPLIT) {
    key_lo = chunk * ATT_CHUNK < p.keep ? chunk * ATT_CHUNK : max(key_lo, chunk * ATT_CHUNK);
    key_hi = min(key_hi, chunk * ATT_CHUNK + ATT_CHUNK - 1);
  }
  if (SPLIT && key_lo > key_hi) return;
  const int row_lo = first_key(p, pos);
  const int* table = p.block_table + (size_t)r * p.max_blocks;
  const int hd = p.hd, vd = p.vd, bsh = p.bs_shift, bmask = p.bs - 1, nkv = p.nkv;

  bf16x8 qf[HD16];
  {
    const __bf16* qr = p.q + (size_t)trow * p.q_stride + (size_t)head * hd + lk * 8;
#pragma unroll
    for (int ks = 0; ks < HD16; ks++) {
      if (row_ok) qf[ks] = *(const bf16x8*)(qr + ks * 16);
      else
#pragma unroll
        for (int e = 0; e < 8; e++) qf[ks][e] = (__bf16)0.f;
    }
  }
  f32x16 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; dt++)
#pragma unroll
    for (int e = 0; e < 16; e++) o[dt][e] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;
  // where the lane's channels dt * 32 + lr lie in a (page, kv head) block of the transposed V cache
  int vrow[DT];
#pragma unroll
  for (int dt = 0; dt < DT; dt++) vrow[dt] = min(dt * 32 + lr, vd - 1) << bsh;
  const bool capped = p.softcap > 0.f;
  // keys every row of the group sees (none beyond the first row's position, none before the
  // last row's window; no range at all unless every lane holds a row): tiles inside this range
  // need no mask
  const int all_hi = ntok * g == 32 ? pos_lo : -1;
  const int all_lo = first_key(p, pos_hi);

  // The pages of a tile are looked up a tile ahead as well, so that no load waits for a table
  // entry: the lane's key row, and the four places its V pieces come from.
  struct TilePages { int k, va[2], vb[2]; };
  auto look_up = [&](int key0, TilePages& pg) {
    pg.k = table[min(key0 + lr, key_hi) >> bsh];
#pragma unroll
    for (int h = 0; h < 2; h++) {
      pg.va[h] = table[min(key0 + h * 16 + 4 * lk, key_hi & ~3) >> bsh];
      pg.vb[h] = table[min(key0 + h * 16 + 8 + 4 * lk, key_hi & ~3) >> bsh];
    }
  };
  auto load_k = [&](int key0, int page, bf16x8 (&kf)[HD16]) {
    const int kk = min(key0 + lr, key_hi);
    const __bf16* kr = p.kcache + ((((size_t)max(page, 0) * nkv + kvh) << bsh) + (kk & bmask)) * hd + lk * 8;
#pragma unroll
    for (int ks = 0; ks < HD16; ks++) kf[ks] = *(const bf16x8*)(kr + ks * 16);
  };
  auto tile = [&](int key0, const TilePages& pg, int knext, TilePages& pn) {
    bf16x8 kf[HD16];
    load_k(key0, pg.k, kf);
    look_up(knext, pn);
    // ---- S^T = K Q^T
    f32x16 s;
#pragma unroll
    for (int e = 0; e < 16; e++) s[e] = 0.f;
#pragma unroll
    for (int ks = 0; ks < HD16; ks++) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[ks], qf[ks], s, 0, 0, 0);
    // ---- V^T pieces for this tile (issued early; used after the softmax)
    bf16x8 vf[DT][2];
#pragma unroll
    for (int h = 0; h < 2; h++) {
      const int ka = min(key0 + h * 16 + 4 * lk, key_hi & ~3), kb = min(key0 + h * 16 + 8 + 4 * lk, key_hi & ~3);
      const int pa = max(pg.va[h], 0), pb = max(pg.vb[h], 0);
      const __bf16* vpa = p.vcache + ((((size_t)pa * (nkv >> p.v_shift) + (kvh >> p.v_shift)) * vd) << bsh) + (ka & bmask);
      const __bf16* vpb = p.vcache + ((((size_t)pb * (nkv >> p.v_shift) + (kvh >> p.v_shift)) * vd) << bsh) + (kb & bmask);
#pragma unroll
      for (int dt = 0; dt < DT; dt++) {
        const bf16x4 va = *(const bf16x4*)(vpa + vrow[dt]);
        const bf16x4 vb = *(const bf16x4*)(vpb + vrow[dt]);
#pragma unroll
        for (int e = 0; e < 4; e++) {
          vf[dt][h][e] = va[e];
          vf[dt][h][4 + e] = vb[e];
        }
      }
    }
    // ---- scale, cap, mask, running softmax (one query row per lane)
    float mt = -INFINITY;
    if (capped) {
#pragma unroll
      for (int e = 0; e < 16; e++) {
        const float ex = __builtin_amdgcn_exp2f(p.k2 * s[e]);
        s[e] = p.c2 * (1.f - 2.f * __builtin_amdgcn_rcpf(ex + 1.f));
      }
    } else {
#pragma unroll
      for (int e = 0; e < 16; e++) s[e] *= p.k1;
    }
    if (key0 < all_lo || key0 + 31 > all_hi || key0 < key_lo || key0 + 31 > key_hi) {
#pragma unroll
      for (int j = 0; j < 4; j++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int key = key0 + 8 * j + 4 * lk + i;
          const bool ok = row_ok && (key >= row_lo || key < p.keep) && key <= pos && key <= key_hi;
          s[4 * j + i] = ok ? s[4 * j + i] : -INFINITY;
        }
    }
#pragma unroll
    for (int e = 0; e < 16; e++) mt = fmaxf(mt, s[e]);
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    const float m_new = mt > m_run + 8.f ? mt : m_run;      // the reference follows the maximum lazily
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const bool moved = m_new > m_run;
    const float corr = moved ? __builtin_amdgcn_exp2f(m_run - m_use) : 1.f;
    float rs = 0.f;
#pragma unroll
    for (int e = 0; e < 16; e++) {
      const float pe = __builtin_amdgcn_exp2f(s[e] - m_use);
      s[e] = pe;
      rs += pe;
    }
    rs += __shfl_xor(rs, 32, 64);
    l_run = l_run * corr + rs;
    m_run = m_new;
    bf16x8 pb[2];
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int e = 0; e < 8; e++) pb[h][e] = (__bf16)s[8 * h + e];
    // ---- O^T = corr * O^T + V^T P^T  (the maximum rarely rises by the threshold after a
    // row's first tiles; said so, the compiler keeps the accumulators where the products
    // want them instead of moving all of them on every tile)
    if (__builtin_expect(__any(moved), 0)) {
      // in the accumulation registers, where the products keep them: written so, the compiler
      // does not copy all of them to ordinary registers on every tile for this rare path
#pragma unroll
      for (int dt = 0; dt < DT; dt++)
#pragma unroll
        for (int e = 0; e < 16; e++) {
          float t;
          asm volatile("v_accvgpr_read_b32 %1, %0\n\tv_mul_f32 %1, %1, %2\n\ts_nop 0\n\tv_accvgpr_write_b32 %0, %1"
                       : "+a"(o[dt][e]), "=&v"(t)
                       : "v"(corr));
        }
    }
#pragma unroll
    for (int dt = 0; dt < DT; dt++) {
      o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[dt][0], pb[0], o[dt], 0, 0, 0);
      o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[dt][1], pb[1], o[dt], 0, 0, 0);
    }
    if (p.wide_weights) {
#pragma unroll
      for (int h = 0; h < 2; h++)
#pragma unroll
        for (int e = 0; e < 8; e++) pb[h][e] = (__bf16)(s[8 * h + e] - (float)pb[h][e]);
#pragma unroll
      for (int dt = 0; dt < DT; dt++) {
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[dt][0], pb[0], o[dt], 0, 0, 0);
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[dt][1], pb[1], o[dt], 0, 0, 0);
      }
    }
  
  };
  {
    // (a chunk of a decoded token has its tiles one behind the other, kept keys among them or not)
    KeyTiles ts(p, key_lo, key_hi);
    if (SPLIT) {
      ts.kept = 0;
      ts.count = key_hi / 32 - ts.lo + 1;
    }
    const int step = SPLIT ? 1 : nphase;
    int i = SPLIT ? 0 : phase;
    TilePages p0, p1;
    if (i < ts.count) look_up(ts.key_of(i), p0);
    for (; i < ts.count; i += 2 * step) {
      tile(ts.key_of(i), p0, ts.key_of(i + step), p1);
      if (i + step >= ts.count) break;
      tile(ts.key_of(i + step), p1, ts.key_of(i + 2 * step), p0);
    }
  }
  if (SPLIT) {
    if (!row_ok) return;
    const size_t slot = ((size_t)(r - p.r_begin) * p.nh + head) * p.nchunks + chunk;
    if (lk == 0) {
      p.part_ml[slot * 2] = m_run;
      p.part_ml[slot * 2 + 1] = l_run;
    }
    float* po = p.part_o + slot * vd;
#pragma unroll
    for (int dt = 0; dt < DT; dt++)
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int d = dt * 32 + 8 * j + 4 * lk;
        if (d < vd) *(f32x4*)(po + d) = f32x4{o[dt][4 * j], o[dt][4 * j + 1], o[dt][4 * j + 2], o[dt][4 * j + 3]};
      }
  } else {
    // join a group's waves: common maximum and sum per row, then the accumulators of the
    // group's other waves reach its first wave through LDS, one wave a round (a slot a group)
    extern __shared__ float dyn[];
    float* sm_ml = dyn;                          // [4][32][2]
    float* sm_o = dyn + 4 * 32 * 2;              // [2][DT * 16][64]
    if (lk == 0) {
      sm_ml[(wave * 32 + lr) * 2] = m_run;
      sm_ml[(wave * 32 + lr) * 2 + 1] = l_run;
    }
    __syncthreads();
    float m_all = -INFINITY;
    for (int w = first_wave; w < first_wave + nphase; w++) m_all = fmaxf(m_all, sm_ml[(w * 32 + lr) * 2]);
    float l_all = 0.f;
    for (int w = first_wave; w < first_wave + nphase; w++) {
      const float mw = sm_ml[(w * 32 + lr) * 2];
      l_all += mw == -INFINITY ? 0.f : sm_ml[(w * 32 + lr) * 2 + 1] * __builtin_amdgcn_exp2f(mw - m_all);
    }
    const float f = m_run == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m_run - m_all);
#pragma unroll
    for (int dt = 0; dt < DT; dt++)
#pragma unroll
      for (int e = 0; e < 16; e++) o[dt][e] *= f;
    float* slot = sm_o + (size_t)(first_wave ? 1 : 0) * DT * 16 * 64;
    const int rounds = max(na_block, 4 - na_block) - 1;
    for (int step = 1; step <= rounds; step++) {
      if (phase == step) {
#pragma unroll
        for (int dt = 0; dt < DT; dt++)
#pragma unroll
          for (int e = 0; e < 16; e++) slot[(dt * 16 + e) * 64 + lane] = o[dt][e];
      }
      __syncthreads();
      if (phase == 0 && step < nphase) {
#pragma unroll
        for (int dt = 0; dt < DT; dt++)
#pragma unroll
          for (int e = 0; e < 16; e++) o[dt][e] += slot[(dt * 16 + e) * 64 + lane];
      }
      __syncthreads();
    }
    if (phase != 0 || !row_ok) return;
    const float inv = row_factor(p, trow, head, l_all, m_all);
    __bf16* orow = p.out + ((size_t)trow * p.nh + head) * vd;
#pragma unroll
    for (int dt = 0; dt < DT; dt++)
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int d = dt * 32 + 8 * j + 4 * lk;
        if (d < vd) {
          bf16x4 w;
#pragma unroll
          for (int i = 0; i < 4; i++) w[i] = (__bf16)(o[dt][4 * j + i] * inv);
          *(bf16x4*)(orow + d) = w;
        }
      }
  }
}

// Long portions.  A block of NW waves owns NW groups of rows that follow each other in one
// request (NW * tpw tokens times the g heads of a KV head), every wave one group, and all of
// them walk the same keys: a tile of 32 keys and its values come from the cache once a block,
// wait in LDS and serve every wave (attn_mfma_kernel fetches them once a group of 32 rows:
// with many groups the way from L2 to the CUs then sets the time).  No join: a wave sees all
// the keys of its rows.  Two buffers: the loads of the next tile are in flight while the
// current one is multiplied, and one barrier a tile suffices.
//   sK [2][32 keys][hd + 8]       a lane's piece for the first product is 16 bytes of a key's row
//   sV [2][vd][32 + 8]            a channel's 32 keys in the order the second product wants:
//                                 piece 2h + lk = keys 16h + 4lk + (0..3), 16h + 8 + 4lk + (0..3)
// The padding of 16 bytes a row keeps the 16-byte reads of 16 lanes on different banks.
// Pages of at least 8 keys (a 16-byte piece of the transposed V holds 8 keys of one page).
//
// SPLIT: a launch of few blocks with many keys each (a prompt of a few thousand tokens and few
// heads) cuts the keys of a block of rows into ranges of p.chunk tiles, counted from the
// block's first tile; blockIdx.x is (block of rows) * p.nchunks + range.  A block then leaves
// (max, sum, O) of its range for every row, as the chunks of a decoded token do, and
// attn_portion_join_kernel joins a row's ranges in their order.
template <int HD16, int VD16, int NW, bool SPLIT>
__global__ __launch_bounds__(NW * 64, (HD16 <= 8 && VD16 <= 8 && NW <= 4) ? 2 : 1) void attn_shared_kernel(AttnParams p) {
  constexpr int HD = HD16 * 16, VD = VD16 * 16, DT = (VD16 + 1) / 2;
  constexpr int KLD = HD + 8, VLD = 32 + 8;
  constexpr int NT = NW * 64;
  constexpr int PIECES = 4 * HD, V_PIECES = 4 * VD;     // 16-byte pieces of a K tile, and of a V tile
  constexpr int PPT = (PIECES + NT - 1) / NT, VPT = (V_PIECES + NT - 1) / NT;           // pieces of each a thread moves
  constexpr int CPK = HD / 8;                           // pieces of a key's row
  extern __shared__ __attribute__((aligned(16))) unsigned char shared_raw[];
  __bf16* sK = (__bf16*)shared_raw;                     // [2][32][KLD]
  __bf16* sV = sK + 2 * 32 * KLD;                       // [2][VD][VLD]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lr = lane & 31, lk = lane >> 5;
  const int r = p.r_begin + blockIdx.z;
  int block_x, kvh;
  portion_block(block_x, kvh);
  const int qs = p.q_start[r], n = p.q_start[r + 1] - qs;
  if (n <= 0) return;
  const int start = p.ctx_len[r] - n;
  const int per_block = NW * p.tpw;
  // the last rows of a portion see the most keys and go first
  const int rows_x = SPLIT ? block_x / p.nchunks : block_x;
  const int range = SPLIT ? block_x - rows_x * p.nchunks : 0;
  const int bi = (n + per_block - 1) / per_block - 1 - rows_x;
  if (bi < 0) return;
  const int g = p.nh / p.nkv;
  // the block's keys: from the window of its first row to its last row
  const int blk_lo = start + bi * per_block, blk_hi = start + min(n, (bi + 1) * per_block) - 1;
  const int key_lo = first_key(p, blk_lo), key_hi = blk_hi;
  const KeyTiles ts(p, key_lo, key_hi);
  int tile_i = 0, tile_end = ts.count;
  if (SPLIT) {
    tile_i = range * p.chunk;
    if (tile_i >= ts.count) return;                    // the block of rows has fewer ranges
    tile_end = min(ts.count, tile_i + p.chunk);
  }
  // the wave's rows
  const int t0 = bi * per_block + wave * p.tpw;
  const int ntok = max(0, min(p.tpw, n - t0));
  const int tok = lr / g, hq = lr - tok * g;
  const bool row_ok = tok < ntok;
  const int trow = qs + (row_ok ? t0 + tok : 0);
  const int pos = start + (row_ok ? t0 + tok : 0);
  const int head = q_head_of(p, kvh, row_ok ? hq : 0);
  const int pos_lo = start + t0, pos_hi = start + t0 + ntok - 1;          // ntok == 0: no keys at all
  const int row_lo = first_key(p, pos);
  const int all_hi = ntok * g == 32 ? pos_lo : -1;
  const int all_lo = first_key(p, pos_hi);
  const int* table = p.block_table + (size_t)r * p.max_blocks;
  const int bsh = p.bs_shift, bmask = p.bs - 1, nkv = p.nkv;

  bf16x8 qf[HD16];
  {
    const __bf16* qr = p.q + (size_t)trow * p.q_stride + (size_t)head * HD + lk * 8;
#pragma unroll
    for (int ks = 0; ks < HD16; ks++) {
      if (row_ok) qf[ks] = *(const bf16x8*)(qr + ks * 16);
      else
#pragma unroll
        for (int e = 0; e < 8; e++) qf[ks][e] = (__bf16)0.f;
    }
  }
  f32x16 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; dt++)
#pragma unroll
    for (int e = 0; e < 16; e++) o[dt][e] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;

  // The thread's pieces of a tile.  K: piece q is 8 channels (q % CPK) of key q / CPK.  V: the
  // pieces of a page's part of the tile lie one behind the other in the cache, channel by
  // channel: with tk = min(page size, 32) keys of a page in the tile, piece q is the keys
  // [8c, 8c + 8) of channel d in part q / (HD tk / 8), d = (q / (tk / 8)) % HD, c = q % (tk / 8).
  const int tk_shift = min(bsh, 5);                     // log2 of a page's keys in a tile
  const int cpp_shift = tk_shift - 3;                   // log2 of the pieces of a channel in a page's part
  // What does not change from tile to tile is worked out here, per piece: its place in the page
  // table relative to the tile's first entry, its offset inside a page's block of the cache (the
  // KV head, the key's place in the page, the channels) and its place in LDS.  A tile then costs
  // a piece one table entry and one multiply-add.  (Tiles start at multiples of 32 keys: with
  // pages of up to 32 keys a key's place in its page does not depend on the tile, with larger
  // pages the whole tile lies in one page and the tile's offset in it is the same for all.)
  int k_idx[PPT], v_idx[VPT], k_lds[PPT], v_lds[VPT];
  unsigned k_off[PPT], v_off[VPT];
#pragma unroll
  for (int j = 0; j < PPT; j++) {
    const int q = min(tid + j * NT, PIECES - 1);
    const int kk = q / CPK, col = (q % CPK) * 8;
    k_idx[j] = kk >> bsh;
    k_off[j] = (unsigned)(((kvh << bsh) + (kk & bmask)) * HD + col);
    k_lds[j] = kk * KLD + col;
  }
#pragma unroll
  for (int j = 0; j < VPT; j++) {
    const int q = min(tid + j * NT, V_PIECES - 1);
    const int part = q / (VD << cpp_shift), rem = q - part * (VD << cpp_shift);
    const int d = rem >> cpp_shift;
    const int vk = (part << tk_shift) + ((rem & ((1 << cpp_shift) - 1)) << 3);
    v_idx[j] = vk >> bsh;
    v_off[j] = (unsigned)((((kvh >> p.v_shift) * VD + d) << bsh) + (vk & bmask));
    // keys 8c + (0..3) go to piece 2h of the channel, keys 8c + 4 + (0..3) to piece 2h + 1,
    // both at slot 4 (c % 2), with h = c / 2
    const int c = vk >> 3;
    v_lds[j] = d * VLD + (c >> 1) * 16 + (c & 1) * 4;
  }
  const size_t page_elems = ((size_t)nkv * HD) << bsh;        // of a page of K
  const size_t v_page_elems = ((size_t)(nkv >> p.v_shift) * VD) << bsh;
  const int last_entry = p.max_blocks - 1;
  struct Pages { int k[PPT], v[VPT]; };
  struct Stage { bf16x8 k[PPT], v[VPT]; };
  // A key past the request's last (in its last tile, or in the tile fetched after the last) is
  // read from wherever its table entry points, page 0 where there is none.  It is masked, but
  // its value still meets a weight of 0 in the second product, and 0 x NaN is NaN: the caller
  // keeps page 0 cleared and clears a page before a request first writes to part of it, so
  // what is read here is the request's own or zero, never what another request left.
  auto look_up = [&](int key0, Pages& pg) {
    const int first = key0 >> bsh;
#pragma unroll
    for (int j = 0; j < PPT; j++) pg.k[j] = table[min(first + k_idx[j], last_entry)];
#pragma unroll
    for (int j = 0; j < VPT; j++) pg.v[j] = table[min(first + v_idx[j], last_entry)];
  };
  auto fetch = [&](int key0, const Pages& pg, Stage& st) {
    const unsigned in_page = (unsigned)(key0 & bmask);
#pragma unroll
    for (int j = 0; j < PPT; j++)
      st.k[j] = *(const bf16x8*)(p.kcache + ((size_t)max(pg.k[j], 0) * page_elems + (k_off[j] + in_page * HD)));
#pragma unroll
    for (int j = 0; j < VPT; j++)
      st.v[j] = *(const bf16x8*)(p.vcache + ((size_t)max(pg.v[j], 0) * v_page_elems + (v_off[j] + in_page)));
  };
  auto stash = [&](int buf, const Stage& st) {
    __bf16* kb = sK + buf * 32 * KLD;
    __bf16* vb = sV + buf * VD * VLD;
#pragma unroll
    for (int j = 0; j < PPT; j++)
      if (PIECES % NT == 0 || tid + j * NT < PIECES) *(bf16x8*)(kb + k_lds[j]) = st.k[j];
#pragma unroll
    for (int j = 0; j < VPT; j++) {
      if (V_PIECES % NT == 0 || tid + j * NT < V_PIECES) {
        __bf16* vrow = vb + v_lds[j];
        bf16x4 lo4, hi4;
#pragma unroll
        for (int e = 0; e < 4; e++) {
          lo4[e] = st.v[j][e];
          hi4[e] = st.v[j][4 + e];
        }
        *(bf16x4*)vrow = lo4;
        *(bf16x4*)(vrow + 8) = hi4;
      }
    }
  };
  const bool capped = p.softcap > 0.f;
  auto tile = [&](int buf, int key0) {
    const __bf16* kb = sK + buf * 32 * KLD + lr * KLD + lk * 8;
    const __bf16* vb = sV + buf * VD * VLD + lk * 8;
    // ---- S^T = K Q^T
    f32x16 s;
#pragma unroll
    for (int e = 0; e < 16; e++) s[e] = 0.f;
#pragma unroll
    for (int ks = 0; ks < HD16; ks++)
      s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8*)(kb + ks * 16), qf[ks], s, 0, 0, 0);
    // ---- scale, cap, mask, running softmax (one query row per lane)
    float mt = -INFINITY;
    if (capped) {
#pragma unroll
      for (int e = 0; e < 16; e++) {
        const float ex = __builtin_amdgcn_exp2f(p.k2 * s[e]);
        s[e] = p.c2 * (1.f - 2.f * __builtin_amdgcn_rcpf(ex + 1.f));
      }
    } else {
#pragma unroll
      for (int e = 0; e < 16; e++) s[e] *= p.k1;
    }
    if (key0 < all_lo || key0 + 31 > all_hi) {
#pragma unroll
      for (int j = 0; j < 4; j++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int key = key0 + 8 * j + 4 * lk + i;
          const bool ok = row_ok && (key >= row_lo || key < p.keep) && key <= pos;
          s[4 * j + i] = ok ? s[4 * j + i] : -INFINITY;
        }
    }
#pragma unroll
    for (int e = 0; e < 16; e++) mt = fmaxf(mt, s[e]);
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    const float m_new = mt > m_run + 8.f ? mt : m_run;      // the maximum is followed lazily
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const bool moved = m_new > m_run;
    const float corr = moved ? __builtin_amdgcn_exp2f(m_run - m_use) : 1.f;
    float rs = 0.f;
#pragma unroll
    for (int e = 0; e < 16; e++) {
      const float pe = __builtin_amdgcn_exp2f(s[e] - m_use);
      s[e] = pe;
      rs += pe;
    }
    rs += __shfl_xor(rs, 32, 64);
    l_run = l_run * corr + rs;
    m_run = m_new;
    bf16x8 pb[2];
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int e = 0; e < 8; e++) pb[h][e] = (__bf16)s[8 * h + e];
    // ---- O^T = corr O^T + V^T P^T
    if (__builtin_expect(__any(moved), 0)) {
      // in the accumulation registers, where the products keep them
#pragma unroll
      for (int dt = 0; dt < DT; dt++)
#pragma unroll
        for (int e = 0; e < 16; e++) {
          float t;
          asm volatile("v_accvgpr_read_b32 %1, %0\n\tv_mul_f32 %1, %1, %2\n\ts_nop 0\n\tv_accvgpr_write_b32 %0, %1"
                       : "+a"(o[dt][e]), "=&v"(t)
                       : "v"(corr));
        }
    }
#pragma unroll
    for (int dt = 0; dt < DT; dt++) {
      const __bf16* vr = vb + min(dt * 32 + lr, VD - 1) * VLD;
      o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8*)vr, pb[0], o[dt], 0, 0, 0);
      o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8*)(vr + 16), pb[1], o[dt], 0, 0, 0);
    }
    if (p.wide_weights) {
#pragma unroll
      for (int h = 0; h < 2; h++)
#pragma unroll
        for (int e = 0; e < 8; e++) pb[h][e] = (__bf16)(s[8 * h + e] - (float)pb[h][e]);
#pragma unroll
      for (int dt = 0; dt < DT; dt++) {
        const __bf16* vr = vb + min(dt * 32 + lr, VD - 1) * VLD;
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8*)vr, pb[0], o[dt], 0, 0, 0);
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8*)(vr + 16), pb[1], o[dt], 0, 0, 0);
      }
    }
  };

  // Every wave takes every tile of the block, also the few near the diagonal (or before its
  // window) that none of its rows sees: masked, such a tile adds nothing, and a loop without a
  // branch around the products lets the compiler leave the accumulators where they are (with
  // the branch it copied all of them to ordinary registers on every turn: 852 instead of 1,135 us
  // at 16 heads of 256).  The turn after the last tile fetches that tile again and leaves it
  // unused.
  {
    Pages pg, pn;
    Stage st;
    look_up(ts.key_of(tile_i), pg);
    fetch(ts.key_of(tile_i), pg, st);
    look_up(ts.key_of(tile_i + 1), pn);
    stash(0, st);
    __syncthreads();
    for (int buf = 0; tile_i < tile_end; tile_i++, buf ^= 1) {
      fetch(ts.key_of(tile_i + 1), pn, st);
      look_up(ts.key_of(tile_i + 2), pn);
      tile(buf, ts.key_of(tile_i));
      stash(buf ^ 1, st);
      __syncthreads();
    }
  }
  if (!SPLIT && !row_ok) return;
  if (SPLIT) {
    // A wave's results of its range, as they lie in its registers: 16 bytes a lane, a wave's 64
    // lanes one contiguous KB per (dt, j), so every store is whole lines.  The joining kernel
    // reads them back with the same lanes.  Every lane stores, rows or not.
    const size_t slot = ((((size_t)blockIdx.z * p.nkv + kvh) * (gridDim.x / p.nchunks) + rows_x) * p.nchunks + range) * NW + wave;
    p.part_ml[slot * 128 + lane] = lk == 0 ? m_run : l_run;
    f32x4* po = (f32x4*)p.part_o + slot * (DT * 4 * 64) + lane;
#pragma unroll
    for (int dt = 0; dt < DT; dt++)
#pragma unroll
      for (int j = 0; j < 4; j++)
        po[(dt * 4 + j) * 64] = f32x4{o[dt][4 * j], o[dt][4 * j + 1], o[dt][4 * j + 2], o[dt][4 * j + 3]};
    return;
  }
  const float inv = row_factor(p, trow, head, l_run, m_run);
  __bf16* orow = p.out + ((size_t)trow * p.nh + head) * VD;
#pragma unroll
  for (int dt = 0; dt < DT; dt++)
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const int d = dt * 32 + 8 * j + 4 * lk;
      if (d < VD) {
        bf16x4 w;
#pragma unroll
        for (int i = 0; i < 4; i++) w[i] = (__bf16)(o[dt][4 * j + i] * inv);
        *(bf16x4*)(orow + d) = w;
      }
    }
}

// One wave per (request, KV head, chunk of 64 keys) for requests that bring one token.
// Columns of every tile are the g query heads of the KV head (col = lane % 16), rows are
// keys (first product) or channels (second product).
template <int HD32, int VD16>
__global__ __launch_bounds__(256, 2) void attn_decode_kernel(AttnParams p) {
  constexpr int KS = HD32;       // 32-wide steps over head_dim
  constexpr int DT = VD16;       // 16-channel output tiles
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, kq = lane >> 4;
  const int r = p.r_begin + blockIdx.z;
  const int kvh = blockIdx.y;
  // Where the window is much shorter than the longest context, the grid covers a window's
  // blocks only and counts them from the block the request's window begins in.
  int block_x = blockIdx.x;
  // In front of them come the blocks of the kept first keys, which every request has.
  const int kept_blocks = (p.keep + 4 * p.chunk - 1) / (4 * p.chunk);
  if (p.from_window && block_x >= kept_blocks)
    block_x += max(first_key(p, max(p.ctx_len[r] - 1, 0)) / (4 * p.chunk), kept_blocks) - kept_blocks;
  const int chunk = block_x * 4 + wave;
  const int* table = p.block_table + (size_t)r * p.max_blocks;
  const int hd = p.hd, vd = p.vd, bsh = p.bs_shift, bmask = p.bs - 1, nkv = p.nkv;
  // The pages of the chunk's (up to two) tiles are asked for before the request's length is
  // known, beside it: where a key lies follows from the chunk alone.  A key past the context is
  // masked below; a hole in the table reads page 0, which the caller keeps cleared, and the
  // places of a request's last page behind its last token are cleared too (a masked value
  // still meets a weight of 0 in the second product, and 0 x NaN is NaN).
  int kpage[2][2], vpage[2][2];
#pragma unroll
  for (int i = 0; i < 2; i++) {
    const int k0 = chunk * p.chunk + 32 * i;
#pragma unroll
    for (int t = 0; t < 2; t++) {
      kpage[i][t] = table[min((k0 + 16 * t + col) >> bsh, p.max_blocks - 1)];
      vpage[i][t] = table[min((k0 + 16 * t + 4 * kq) >> bsh, p.max_blocks - 1)];
    }
  }
  const int n = p.q_start[r + 1] - p.q_start[r];
  if (n <= 0) return;
  const int pos = p.ctx_len[r] - 1;
  const int row_lo = first_key(p, pos);
  // a block whose four chunks all lie past the context or before the window ends here, all
  // its waves alike: the grid is sized for the longest context the caller allows
  const int first_chunk = block_x * 4;
  if (first_chunk * p.chunk > pos ||
      (first_chunk * p.chunk + 4 * p.chunk - 1 < row_lo && first_chunk * p.chunk >= p.keep)) return;
  const int key_lo = chunk * p.chunk < p.keep ? chunk * p.chunk : max(row_lo, chunk * p.chunk);
  const int key_hi = min(pos, chunk * p.chunk + p.chunk - 1);
  const bool active = key_lo <= key_hi;          // a wave without keys still meets the others at the barrier
  const int g = p.nh / p.nkv;
  const bool col_ok = col < g;
  const int head = q_head_of(p, kvh, col_ok ? col : 0);
  const int trow = p.q_start[r];

  // the query operand waits in LDS (one 16-byte piece per lane and step), not in registers
  __shared__ bf16x8 sq[4][KS][64];
  {
    const __bf16* qr = p.q + (size_t)trow * p.q_stride + (size_t)head * hd + kq * 8;
#pragma unroll
    for (int ks = 0; ks < KS; ks++) {
      bf16x8 t;
      if (col_ok) t = *(const bf16x8*)(qr + ks * 32);
      else
#pragma unroll
        for (int e = 0; e < 8; e++) t[e] = (__bf16)0.f;
      sq[wave][ks][lane] = t;
    }
  }
  f32x4 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; dt++) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;

#pragma unroll
  for (int i = 0; i < 2; i++) {
    const int key0 = chunk * p.chunk + 32 * i;
    if (!active || 32 * i >= p.chunk || key0 > key_hi || key0 + 31 < key_lo) continue;
    bf16x8 kf[2][KS];
#pragma unroll
    for (int t = 0; t < 2; t++) {
      const int kk = key0 + 16 * t + col;
      const int page = max(kpage[i][t], 0);
      const __bf16* kr = p.kcache + ((((size_t)page * nkv + kvh) << bsh) + (kk & bmask)) * hd + kq * 8;
#pragma unroll
      for (int ks = 0; ks < KS; ks++) kf[t][ks] = *(const bf16x8*)(kr + ks * 32);
    }
    bf16x8 vf[DT];
    {
      const int ka = key0 + 4 * kq, kb = key0 + 16 + 4 * kq;
      const int pa = max(vpage[i][0], 0), pb = max(vpage[i][1], 0);
      const __bf16* va_base = p.vcache + ((((size_t)pa * (nkv >> p.v_shift) + (kvh >> p.v_shift)) * vd) << bsh) + (ka & bmask);
      const __bf16* vb_base = p.vcache + ((((size_t)pb * (nkv >> p.v_shift) + (kvh >> p.v_shift)) * vd) << bsh) + (kb & bmask);
#pragma unroll
      for (int dt = 0; dt < DT; dt++) {
        const int d = dt * 16 + col;
        const bf16x4 va = *(const bf16x4*)(va_base + ((size_t)d << bsh));
        const bf16x4 vb = *(const bf16x4*)(vb_base + ((size_t)d << bsh));
#pragma unroll
        for (int e = 0; e < 4; e++) {
          vf[dt][e] = va[e];
          vf[dt][4 + e] = vb[e];
        }
      }
    }
    f32x4 s[2];
#pragma unroll
    for (int t = 0; t < 2; t++) {
      s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ks++) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][ks], sq[wave][ks][lane], s[t], 0, 0, 0);
    }
    float mt = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int key = key0 + 16 * t + 4 * kq + i;
        float v = score_log2(p, s[t][i]);
        v = (col_ok && (key >= row_lo || key < p.keep) && key <= key_hi) ? v : -INFINITY;
        s[t][i] = v;
        mt = fmaxf(mt, v);
      }
    mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    const float m_new = fmaxf(m_run, mt);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float corr = __builtin_amdgcn_exp2f(m_run - m_use);
    float rs = 0.f;
    bf16x8 pb8;
#pragma unroll
    for (int t = 0; t < 2; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float pe = __builtin_amdgcn_exp2f(s[t][i] - m_use);
        rs += pe;
        pb8[4 * t + i] = (__bf16)pe;
        s[t][i] = pe;
      }
    rs += __shfl_xor(rs, 16, 64);
    rs += __shfl_xor(rs, 32, 64);
    l_run = l_run * corr + rs;
    m_run = m_new;
#pragma unroll
    for (int dt = 0; dt < DT; dt++) {
      o[dt] *= corr;
      o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[dt], pb8, o[dt], 0, 0, 0);
    }
    if (p.wide_weights) {
#pragma unroll
      for (int t = 0; t < 2; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) pb8[4 * t + i] = (__bf16)(s[t][i] - (float)pb8[4 * t + i]);
#pragma unroll
      for (int dt = 0; dt < DT; dt++) o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[dt], pb8, o[dt], 0, 0, 0);
    }
  }
  // the block's four chunks are joined here, in chunk order: one partial result per 256 keys
  extern __shared__ float dyn[];
  float* sm_ml = dyn;                 // [4][16][2]
  float* sm_o = dyn + 4 * 16 * 2;     // [4][g][vd]
  if (col_ok) {
    if (kq == 0) {
      sm_ml[(wave * 16 + col) * 2] = m_run;
      sm_ml[(wave * 16 + col) * 2 + 1] = l_run;
    }
    float* so = sm_o + ((size_t)wave * g + col) * vd;
#pragma unroll
    for (int dt = 0; dt < DT; dt++) *(f32x4*)(so + dt * 16 + 4 * kq) = o[dt];
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < g * vd; idx += 256) {
    const int c = idx / vd, d = idx - c * vd;
    float mw[4], m = -INFINITY;
#pragma unroll
    for (int w = 0; w < 4; w++) {
      mw[w] = sm_ml[(w * 16 + c) * 2];
      m = fmaxf(m, mw[w]);
    }
    float acc = 0.f, l = 0.f;
#pragma unroll
    for (int w = 0; w < 4; w++) {
      const float e = mw[w] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mw[w] - m);
      acc += e * sm_o[((size_t)w * g + c) * vd + d];
      l += e * sm_ml[(w * 16 + c) * 2 + 1];
    }
    const size_t slot = ((size_t)(r - p.r_begin) * p.nh + q_head_of(p, kvh, c)) * p.nchunks + block_x;
    p.part_o[slot * vd + d] = acc;
    if (d == 0) {
      p.part_ml[slot * 2] = m;
      p.part_ml[slot * 2 + 1] = l;
    }
  }
}

// One pair of sizes.  what: 0 decoded tokens on 32-wide tiles, 1 pairs of groups a block, 2 a group a block,
// 3 shared tiles with four waves, 4 with eight, 5 with four and the keys in ranges, 6 decoded tokens
// on 16-wide tiles (keys in whole 32s).
enum AttnWhat { ATT_DECODE_WIDE, ATT_PAIRS, ATT_GROUPS, ATT_SHARED4, ATT_SHARED8, ATT_RANGES, ATT_DECODE };

template <int HD16, int VD16, int NW, bool SPLIT>
static int launch_shared_one(const AttnParams& p, dim3 grid, hipStream_t s) {
  constexpr int HD = HD16 * 16, VD = VD16 * 16;
  constexpr size_t lds = ((size_t)2 * 32 * (HD + 8) + (size_t)2 * VD * (32 + 8)) * sizeof(__bf16);
  static bool prepared = false;
  if (!prepared) {
    if (lds > 64 * 1024 && hipFuncSetAttribute((const void*)attn_shared_kernel<HD16, VD16, NW, SPLIT>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return zk_fail("zk_attention_bf16: the shared-tile kernel's LDS buffers were refused");
    prepared = true;
  }
  attn_shared_kernel<HD16, VD16, NW, SPLIT><<<grid, NW * 64, lds, s>>>(p);
  return zk_launch_status("zk_attention_bf16 (shared tiles)");
}

template <int HD16, int VD16>
static int launch_sizes(int what, const AttnParams& p, dim3 grid, hipStream_t s) {
  // the join of a portion's four waves needs [4][32][2] + [2][ceil(vd/32) * 16][64] floats of LDS
  const size_t join = (4 * 32 * 2 + (size_t)2 * ((p.vd + 31) / 32) * 16 * 64) * sizeof(float);
  switch (what) {
    case ATT_DECODE_WIDE: attn_mfma_kernel<HD16, VD16, true, false><<<grid, 256, 0, s>>>(p); break;
    case ATT_PAIRS: attn_mfma_kernel<HD16, VD16, false, true><<<grid, 256, join, s>>>(p); break;
    case ATT_GROUPS: attn_mfma_kernel<HD16, VD16, false, false><<<grid, 256, join, s>>>(p); break;
    case ATT_SHARED4: return launch_shared_one<HD16, VD16, 4, false>(p, grid, s);
    case ATT_SHARED8:
      if constexpr (HD16 <= 8 && VD16 <= 8) return launch_shared_one<HD16, VD16, 8, false>(p, grid, s);
      else return zk_fail("zk_attention_bf16: eight waves a block take head sizes up to 128");
    case ATT_RANGES: return launch_shared_one<HD16, VD16, 4, true>(p, grid, s);
    case ATT_DECODE:
      if constexpr (HD16 % 2 == 0) {
        const size_t lds = (4 * 16 * 2 + (size_t)4 * (p.nh / p.nkv) * p.vd) * sizeof(float);
        attn_decode_kernel<HD16 / 2, VD16><<<grid, 256, lds, s>>>(p);
        break;
      } else {
        return zk_fail("zk_attention_bf16: the narrow tiles take keys in whole 32s");
      }
    default: return zk_fail("zk_attention_bf16: unknown kernel");
  }
  return zk_launch_status("zk_attention_bf16");
}

// attention_bf16_uneven.hip
int attn_launch_uneven(int what, const AttnParams& p, dim3 grid, hipStream_t s);

#endif  // ZSE_ACT_BF16
