// Matrix-core windowed attention over the paged cache: device code shared by the translation units that instantiate it
// (attn_window.hip: windows, blocks, causal; attn_pool.hip: the same with pooled blocks behind the window, capped scores and a norm
// over the whole query projection).
#pragma once
#include "seq_common.h"

// everything a call of the attention kernels needs (device pointers unless said otherwise; see include/nvl_seq.h)
struct WindowAttnArgs {
  const void *q, *qnorm, *gate, *k_cache, *v_cache;
  void* out;
  const int32_t *block_tables, *cu_q, *ctx0, *tseq;
  const float *rot_freq, *sink;
  int64_t q_stride, gate_stride, bt_stride, n;
  int gate_w, block_size, nseq, H, G, d, dv, window, chunk, rot_dims, qt_every;
  float eps, scale, qt_coef;
  int bs_shift, hw;                       // set by the launcher
  int no_lds, packed_heads;               // tests / A-B: own operand loads per wavefront; heads in the query tiles of single-token steps
  // what only the extended form reads
  const float* q_row;                     // [n]: factor of every query row (then qnorm has H * d weights)
  const void *pool_k, *pool_v;            // means over blocks of `pool` tokens
  int pool;
  float softcap;
};

// first key position the query at position p sees (both masks are monotone in p, which the tile bounds below rely on)
__device__ __forceinline__ int vis_lo(int p, int window, int chunk) {
  if (window > 0) return p - window + 1 > 0 ? p - window + 1 : 0;
  if (chunk > 0) return p - p % chunk;
  return 0;
}

// factor on the query at position p: 1 + coef * ln(floor((p + 1) / every) + 1) — a temperature that grows with the logarithm of the
// position, in steps of `every` positions (every == 0: none)
// (positions are below 2^24, so p + 1 and `every` are exact in 32-bit floats and the correctly rounded quotient has the integer
// quotient's floor: a float division instead of the long expansion of an integer one)
__device__ __forceinline__ float query_temp(int p, float coef, int every) {
  if (every <= 0) return 1.f;
  return 1.f + coef * logf(floorf((float)(p + 1) / (float)every) + 1.f);
}

// Pooled blocks. Block b is the mean of the tokens b P .. b P + P - 1 and is seen from position p if all of them lie before p's
// window: (b + 1) P <= p - window + 1.
__device__ __forceinline__ int seen_blocks(int p, int window, int pool) {
  const int before = p - window + 1;                // tokens before the window
  return pool > 0 && before > 0 ? before / pool : 0;
}
// Blocks are kept in units of 8 (values transposed inside a unit). Unit u lives in the page of the LAST token of its first block,
// position 8 u P + P - 1, so a page of B tokens has room for ceil(B / (8 P)) units and nothing beside the page tables is needed.
__device__ __forceinline__ int pool_unit(int u, int pool, int block_size, const int32_t* __restrict__ bt) {
  const int page = (8 * u * pool + pool - 1) / block_size;
  const int first = page * block_size < pool ? 0 : (page * block_size - pool + 8 * pool) / (8 * pool);   // the page's first unit
  return bt[page] * ((block_size + 8 * pool - 1) / (8 * pool)) + (u - first);
}

// cap * tanh(s / cap) from one exponential (absolute error a few ulp of cap)
__device__ __forceinline__ float capped(float s, float cap) {
  const float e = __expf(2.f * (s / cap));
  return cap * (1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e));
}

namespace {

// ---- bf16 matrix-core form ------------------------------------------------------------------------------------------
// One wavefront per (16 consecutive queries of a portion, query head); four query tiles per workgroup, no LDS. Everything
// is computed transposed so that each lane owns ONE query (column l & 15) and the softmax statistics need two shuffles:
//   S^T[keys x queries] = K Q^T   v_mfma_f32_16x16x32_bf16, A = 16 key rows x 32 of d (16-byte loads from the K cache),
//                                 B = Q^T (normed, scaled, held in registers for the whole tile)
//   O^T[dv x queries]  += V^T P^T A = 16 value columns x 32 tokens: 16-byte loads from the page-transposed V cache,
//                                 B = P^T straight from the S^T accumulators of two key blocks
// The MFMA's contraction index may be permuted freely as long as both operands agree; the key rows of block kb are the
// tokens base + 32 (kb / 2) + 8 (i / 4) + 4 (kb % 2) + i % 4, which makes the 8 weights a lane holds after two key blocks
// the 8 CONSECUTIVE tokens its V load covers. Scores, maxima, sums and O stay 32-bit; the weights enter the second product
// as bf16, like V. d % 8 == 0, block_size % 8 == 0; d and dv are padded to the template's sizes with zero operands.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4_t;
// d <= 32 DK, dv <= 16 DVB, QT tiles of 16 queries per wavefront (they share every K / V load)
template <int DK, int DVB, int QT>
__global__ __launch_bounds__(256) void window_attn_mfma_kernel(const WindowAttnArgs A) {
  const bf16_t* __restrict__ q = (const bf16_t*)A.q;
  const bf16_t* __restrict__ qnorm = (const bf16_t*)A.qnorm;
  const bf16_t* __restrict__ gate = (const bf16_t*)A.gate;
  const bf16_t* __restrict__ k_cache = (const bf16_t*)A.k_cache;
  const bf16_t* __restrict__ v_cache = (const bf16_t*)A.v_cache;
  bf16_t* __restrict__ out = (bf16_t*)A.out;
  const int32_t* __restrict__ block_tables = A.block_tables;
  const int32_t* __restrict__ cu_q = A.cu_q;
  const int32_t* __restrict__ ctx0 = A.ctx0;
  const float* __restrict__ rot_freq = A.rot_freq;
  const float* __restrict__ sink = A.sink;
  const int64_t q_stride = A.q_stride, gate_stride = A.gate_stride, bt_stride = A.bt_stride;
  const int gate_w = A.gate_w, block_size = A.block_size, nseq = A.nseq, H = A.H, G = A.G, d = A.d, dv = A.dv, window = A.window, chunk = A.chunk,
            rot_dims = A.rot_dims, qt_every = A.qt_every, bs_shift = A.bs_shift;
  const float eps = A.eps, scale = A.scale, qt_coef = A.qt_coef;
  constexpr int QW = 16 * QT;                       // queries per wavefront
  const int lane = threadIdx.x & 63, qi = lane & 15, gq = lane >> 4;
  int tile = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int h = blockIdx.y, g = h / (H / G);
  int s = 0, len = 0;
  for (; s < nseq; ++s) {
    len = cu_q[s + 1] - cu_q[s];
    const int tiles = (len + QW - 1) / QW;
    if (tile < tiles) break;
    tile -= tiles;
  }
  if (s >= nseq) return;                            // (no workgroup barrier below: a wavefront may leave alone)
  // positions fit 32 bits (the engine's tables do); page and offset of a token by shift and mask when pages are a power of two
  const int c0 = ctx0[s];
  const int p_first = c0 + tile * QW;
  const int p_last = c0 + (tile * QW + QW - 1 < len ? tile * QW + QW - 1 : len - 1);
  const int bs_mask = block_size - 1;

  // Q^T operands: lane holds d elements [32 c + 8 gq, + 8) of query qi of each tile, normed and scaled
  bf16x8_t qb[QT][DK];
  bool valid_q[QT];
  int64_t row[QT];
  int pos[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int rel = tile * QW + t * 16 + qi;
    valid_q[t] = rel < len;
    row[t] = (int64_t)cu_q[s] + (valid_q[t] ? rel : len - 1);
    pos[t] = c0 + rel;
    float qv[DK][8];
    float ss = 0.f;
    const bf16_t* qp = q + row[t] * q_stride + (int64_t)h * d;
#pragma unroll
    for (int c = 0; c < DK; ++c)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int col = c * 32 + gq * 8 + e;
        qv[c][e] = col < d ? (float)qp[col] : 0.f;
        ss += qv[c][e] * qv[c][e];
      }
    float r = scale * query_temp(pos[t], qt_coef, qt_every);
    if (qnorm) {
      ss += __shfl_xor(ss, 16, 64);
      ss += __shfl_xor(ss, 32, 64);
      r *= rsqrtf(ss / (float)d + eps);
    }
#pragma unroll
    for (int c = 0; c < DK; ++c)
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const int col = c * 32 + gq * 8 + e;
        const float w0 = (qnorm && col < d) ? (float)qnorm[col] : 1.f;
        const float w1 = (qnorm && col + 1 < d) ? (float)qnorm[col + 1] : 1.f;
        float a = qv[c][e] * r * w0, b = qv[c][e + 1] * r * w1;
        if (col < rot_dims) {                        // the pair (2i, 2i+1) turns by pos * freq[i]; both halves are this lane's
          float sn, cs;
          sincosf((float)pos[t] * rot_freq[col >> 1], &sn, &cs);
          const float a2 = a * cs - b * sn;
          b = b * cs + a * sn;
          a = a2;
        }
        qb[t][c][e] = (bf16_t)a;
        qb[t][c][e + 1] = (bf16_t)b;
      }
  }
  const int lo = vis_lo(p_first, window, chunk);
  const int lo_hi = vis_lo(c0 + tile * QW + QW - 1, window, chunk);      // the tile's last query sees the least far back
  const int32_t* bt = block_tables + (int64_t)s * bt_stride;
  const float sink_m = sink ? sink[h] : -1e30f, sink_l = sink && gq == 0 ? 1.f : 0.f;      // (see the LDS form below)
  float m[QT], lsum[QT];
  f32x4_t oacc[QT][DVB];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    m[t] = sink_m;
    lsum[t] = sink_l;
#pragma unroll
    for (int db = 0; db < DVB; ++db) oacc[t][db] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const bf16x8_t zero8 = __builtin_bit_cast(bf16x8_t, u32x4_t{0u, 0u, 0u, 0u});

  for (int j0 = lo & ~31; j0 <= p_last; j0 += 64) {
    // every query of the wavefront sees all 64 tokens of the round: no masks (most rounds of a long window)
    const bool interior = j0 + 63 <= p_first && j0 >= lo_hi;
    // ---- S^T for 64 tokens: 4 key blocks, every K fragment feeds all QT tiles
    f32x4_t sacc[QT][4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
      for (int t = 0; t < QT; ++t) sacc[t][kb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const int j = j0 + (kb >> 1) * 32 + (qi >> 2) * 8 + (kb & 1) * 4 + (qi & 3);          // the token of this lane's A row
      const bool have = j <= p_last;
      const bf16_t* kp = k_cache;
      if (have) {
        const int pg = bs_shift >= 0 ? j >> bs_shift : j / block_size;
        const int off = bs_shift >= 0 ? j & bs_mask : j - pg * block_size;
        kp += (((int64_t)bt[pg] * block_size + off) * G + g) * d + gq * 8;
      }
#pragma unroll
      for (int c = 0; c < DK; ++c) {
        bf16x8_t a = zero8;
        if (have && c * 32 + gq * 8 < d) a = *(const bf16x8_t*)(kp + c * 32);
#pragma unroll
        for (int t = 0; t < QT; ++t) sacc[t][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qb[t][c], sacc[t][kb], 0, 0, 0);
      }
    }
    // ---- mask, running maximum, weights (this lane: query qi of tile t, tokens 32 (kb/2) + 8 gq + 4 (kb%2) + r)
    bf16x8_t pb[QT][2];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float mx = m[t];
      unsigned okbits = 0xffffu;                     // bit 4 kb + r: the token is visible to this lane's query
      if (!interior) {
        okbits = 0u;
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = j0 + (kb >> 1) * 32 + gq * 8 + (kb & 1) * 4 + r;
            const bool ok = valid_q[t] && j <= pos[t] && j >= vis_lo(pos[t], window, chunk);
            okbits |= ok ? (1u << (kb * 4 + r)) : 0u;
          }
      }
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (okbits & (1u << (kb * 4 + r))) mx = fmaxf(mx, sacc[t][kb][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float alpha = __expf(m[t] - mx);
      m[t] = mx;
      float ls = lsum[t] * alpha;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = (okbits & (1u << (kb * 4 + r))) ? __expf(sacc[t][kb][r] - mx) : 0.f;
          ls += p;
          pb[t][kb >> 1][(kb & 1) * 4 + r] = (bf16_t)p;
        }
      lsum[t] = ls;
      if (__ballot(alpha != 1.f) != 0ull) {          // the maximum moved for some query of the tile
#pragma unroll
        for (int db = 0; db < DVB; ++db) oacc[t][db] *= alpha;
      }
    }
    // ---- O^T += V^T P^T: two groups of 32 tokens, every V fragment feeds all QT tiles
#pragma unroll
    for (int mg = 0; mg < 2; ++mg) {
      const int jb = j0 + mg * 32 + gq * 8;                                                 // 8 consecutive tokens, one page
      const bool have = jb <= p_last;
      const bf16_t* vp = v_cache;
      if (have) {
        const int pg = bs_shift >= 0 ? jb >> bs_shift : jb / block_size;
        const int off = bs_shift >= 0 ? jb & bs_mask : jb - pg * block_size;
        vp += (((int64_t)bt[pg] * G + g) * dv) * block_size + off;
      }
#pragma unroll
      for (int db = 0; db < DVB; ++db) {
        const int col = db * 16 + qi;
        bf16x8_t a = zero8;
        if (have && col < dv) a = *(const bf16x8_t*)(vp + (int64_t)col * block_size);
#pragma unroll
        for (int t = 0; t < QT; ++t) oacc[t][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb[t][mg], oacc[t][db], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float ls = lsum[t];
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (!valid_q[t]) continue;
    const float inv = 1.f / ls;
    bf16_t* op = out + ((int64_t)row[t] * H + h) * dv;
    const bf16_t* gp = gate ? gate + row[t] * gate_stride + (int64_t)h * gate_w : nullptr;
#pragma unroll
    for (int db = 0; db < DVB; ++db)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = db * 16 + gq * 4 + r;
        if (c < dv) {
          float o = oacc[t][db][r] * inv;
          if (gp) o *= 1.f / (1.f + expf(-(float)gp[gate_w == 1 ? 0 : c]));
          op[c] = (bf16_t)o;
        }
      }
  }
}

// ---- the same, with the K / V tiles of a round shared through LDS ------------------------------------------------------
// A workgroup of four wavefronts serves ONE kv head: `hw` query heads of its group times 4 / hw query tiles, so every K / V
// byte is fetched from the caches once per workgroup and round instead of once per wavefront (4x less traffic; with grouped
// query heads the sharing is across heads, which also holds when every portion is a single decoded token). All threads load
// the round's 64 tokens with coalesced 16-byte loads — the NEXT round's loads are issued before the current round is
// computed — K as [token][d], V as [column][token]; the MFMA operands are 16-byte LDS reads. Softmax, masks and the token
// permutation are those of the kernel above.
template <int DK, int DVB, int QT, bool EXT>
__global__ __launch_bounds__(256) void window_attn_mfma_lds_kernel(const WindowAttnArgs A) {
  const bf16_t* __restrict__ q = (const bf16_t*)A.q;
  const bf16_t* __restrict__ qnorm = (const bf16_t*)A.qnorm;
  const bf16_t* __restrict__ gate = (const bf16_t*)A.gate;
  const bf16_t* __restrict__ k_cache = (const bf16_t*)A.k_cache;
  const bf16_t* __restrict__ v_cache = (const bf16_t*)A.v_cache;
  bf16_t* __restrict__ out = (bf16_t*)A.out;
  const int32_t* __restrict__ block_tables = A.block_tables;
  const int32_t* __restrict__ cu_q = A.cu_q;
  const int32_t* __restrict__ ctx0 = A.ctx0;
  const float* __restrict__ rot_freq = A.rot_freq;
  const float* __restrict__ sink = A.sink;
  const int64_t q_stride = A.q_stride, gate_stride = A.gate_stride, bt_stride = A.bt_stride;
  const int gate_w = A.gate_w, block_size = A.block_size, nseq = A.nseq, H = A.H, G = A.G, d = A.d, dv = A.dv, window = A.window, chunk = A.chunk,
            rot_dims = A.rot_dims, qt_every = A.qt_every, bs_shift = A.bs_shift;
  const float eps = A.eps, scale = A.scale, qt_coef = A.qt_coef;
  const int hw = A.hw;
  const bf16_t* __restrict__ pool_k = (const bf16_t*)A.pool_k;
  const bf16_t* __restrict__ pool_v = (const bf16_t*)A.pool_v;
  const int pool = EXT ? A.pool : 0;
  constexpr int QW = 16 * QT, KP = 32 * DK + 8, VP = 64 + 8, VU = DVB / 2;
  __shared__ __attribute__((aligned(16))) bf16_t Ks[64][KP];
  __shared__ __attribute__((aligned(16))) bf16_t Vs[16 * DVB][VP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, qi = lane & 15, gq = lane >> 4;
  // hw == 0 ("packed", QT == 1): the workgroup serves ONE token and the rows of a wavefront's query tile are 16 HEADS of the kv
  // group at that token (64 heads per workgroup) — for steps of single tokens with many query heads per kv head, where a
  // tile of 16 consecutive positions would hold one query.
  const bool packed = hw == 0;
  const int hpg = H / G, chunks = packed ? (hpg + 63) / 64 : hpg / hw;
  const int g = blockIdx.y / chunks;
  const int hl0 = packed ? (blockIdx.y % chunks) * 64 + wave * 16 : (blockIdx.y % chunks) * hw + (wave % hw);   // the wavefront's first head in the group
  const int BQ = packed ? 1 : (4 / hw) * QW;       // queries (positions) of the workgroup
  int btile = blockIdx.x, s = 0, len = 0;
  for (; s < nseq; ++s) {
    len = cu_q[s + 1] - cu_q[s];
    const int tiles = (len + BQ - 1) / BQ;
    if (btile < tiles) break;
    btile -= tiles;
  }
  if (s >= nseq) return;                            // the whole workgroup leaves
  const int c0 = ctx0[s];
  const int rel0 = packed ? btile : btile * BQ + (wave / hw) * QW;   // this wavefront's first query inside the portion (may lie beyond its end)
  const int p_first = c0 + rel0, p_hi = packed ? p_first : c0 + rel0 + QW - 1;
  const bool idle = packed ? hl0 >= hpg : rel0 >= len;               // a wavefront without queries only helps to load
  const int b_first = c0 + btile * BQ;
  const int b_last = c0 + (btile * BQ + BQ - 1 < len ? btile * BQ + BQ - 1 : len - 1);
  const int bs_mask = block_size - 1;
  const int32_t* bt = block_tables + (int64_t)s * bt_stride;

  bf16x8_t qb[QT][DK];
  bool valid_q[QT];
  int64_t row[QT];
  int pos[QT], hq[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int rel = packed ? rel0 : rel0 + t * 16 + qi;
    const int hl = packed ? hl0 + qi : hl0;
    valid_q[t] = rel < len && hl < hpg;
    hq[t] = g * hpg + (hl < hpg ? hl : hpg - 1);
    row[t] = (int64_t)cu_q[s] + (rel < len ? rel : len - 1);
    pos[t] = c0 + rel;
    float qv[DK][8];
    float ss = 0.f;
    const bf16_t* qp = q + row[t] * q_stride + (int64_t)hq[t] * d;
#pragma unroll
    for (int c = 0; c < DK; ++c)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int col = c * 32 + gq * 8 + e;
        qv[c][e] = col < d ? (float)qp[col] : 0.f;
        ss += qv[c][e] * qv[c][e];
      }
    float r = scale * query_temp(pos[t], qt_coef, qt_every);
    const bf16_t* qw = qnorm;
    if (EXT && A.q_row) {                            // norm over the whole projection: one factor per token, weights of every head
      r *= A.q_row[row[t]];
      qw = qnorm + hq[t] * d;
    } else if (qnorm) {
      ss += __shfl_xor(ss, 16, 64);
      ss += __shfl_xor(ss, 32, 64);
      r *= rsqrtf(ss / (float)d + eps);
    }
#pragma unroll
    for (int c = 0; c < DK; ++c)
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const int col = c * 32 + gq * 8 + e;
        const float w0 = (qw && col < d) ? (float)qw[col] : 1.f;
        const float w1 = (qw && col + 1 < d) ? (float)qw[col + 1] : 1.f;
        float a = qv[c][e] * r * w0, b = qv[c][e + 1] * r * w1;
        if (col < rot_dims) {                        // the pair (2i, 2i+1) turns by pos * freq[i]; both halves are this lane's
          float sn, cs;
          sincosf((float)pos[t] * rot_freq[col >> 1], &sn, &cs);
          const float a2 = a * cs - b * sn;
          b = b * cs + a * sn;
          a = a2;
        }
        qb[t][c][e] = (bf16_t)a;
        qb[t][c][e + 1] = (bf16_t)b;
      }
  }
  // a sink: a score in the denominator without a value; the running maximum and sum start from it (the sum once per query: in
  // the lanes with gq 0). All tiles of a wavefront belong to one head, except in the packed form, which has one tile.
  const float sink_m = sink ? sink[hq[0]] : -1e30f, sink_l = sink && gq == 0 ? 1.f : 0.f;
  float m[QT], lsum[QT];
  f32x4_t oacc[QT][DVB];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    m[t] = sink_m;
    lsum[t] = sink_l;
#pragma unroll
    for (int db = 0; db < DVB; ++db) oacc[t][db] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const u32x4_t zero4 = u32x4_t{0u, 0u, 0u, 0u};
  // staging: thread -> DK 16-byte units of K (token, 8 of d) and VU units of V (column, 8 tokens)
  u32x4_t kf[DK], vf[VU];
  // page ids are looked up one round ahead of the loads that use them: a round's loads then depend on nothing in flight
  int pgk[DK], pgv;
  // EXT: rounds [0, npr) hold 64 pooled blocks each (a causal list of blocks: block b is seen by the queries with seen_blocks > b),
  // the rounds after them 64 tokens of the window. A pooled round's unit of 8 blocks takes the place of a page of 8 tokens.
  const int lo = vis_lo(b_first, window, chunk);
  const int lo_first = vis_lo(p_first, window, chunk), lo_hi = vis_lo(p_hi, window, chunk);
  const int nb_last = EXT ? seen_blocks(b_last, window, pool) : 0, npr = EXT ? (nb_last + 63) >> 6 : 0;
  const int nb_first = EXT ? seen_blocks(p_first, window, pool) : 0, nb_hi = EXT ? seen_blocks(p_hi, window, pool) : 0;
  const int jt = (lo & ~31) - npr * 64;             // a token round's first token is jt + 64 * (its number)
  auto lookup = [&](int it) {
    if (EXT && it < npr) {
#pragma unroll
      for (int i = 0; i < DK; ++i) {
        const int b = it * 64 + (tid + i * 256) / (4 * DK);
        pgk[i] = b < nb_last ? pool_unit(b >> 3, pool, block_size, bt) : 0;
      }
      const int b = it * 64 + (tid & 7) * 8;
      pgv = b < nb_last ? pool_unit(b >> 3, pool, block_size, bt) : 0;
      return;
    }
    const int j0 = jt + it * 64;
#pragma unroll
    for (int i = 0; i < DK; ++i) {
      const int j = j0 + (tid + i * 256) / (4 * DK);
      pgk[i] = j <= b_last ? bt[bs_shift >= 0 ? j >> bs_shift : j / block_size] : 0;
    }
    const int j = j0 + (tid & 7) * 8;
    pgv = j <= b_last ? bt[bs_shift >= 0 ? j >> bs_shift : j / block_size] : 0;
  };
  auto fetch = [&](int it) {
    if (EXT && it < npr) {
#pragma unroll
      for (int i = 0; i < DK; ++i) {
        const int u = tid + i * 256, tok = u / (4 * DK), part = u - tok * (4 * DK);
        const int b = it * 64 + tok;
        kf[i] = zero4;
        if (b < nb_last && part * 8 < d) kf[i] = *(const u32x4_t*)(pool_k + (((int64_t)pgk[i] * 8 + (b & 7)) * G + g) * d + part * 8);
      }
#pragma unroll
      for (int i = 0; i < VU; ++i) {
        const int u = tid + i * 256, col = u >> 3, b = it * 64 + (u & 7) * 8;
        vf[i] = zero4;
        if (b < nb_last && col < dv) vf[i] = *(const u32x4_t*)(pool_v + (((int64_t)pgv * G + g) * dv + col) * 8);
      }
      return;
    }
    const int j0 = jt + it * 64;
#pragma unroll
    for (int i = 0; i < DK; ++i) {
      const int u = tid + i * 256, tok = u / (4 * DK), part = u - tok * (4 * DK);
      const int j = j0 + tok;
      kf[i] = zero4;
      if (j <= b_last && part * 8 < d) {
        const int off = bs_shift >= 0 ? j & bs_mask : j % block_size;
        kf[i] = *(const u32x4_t*)(k_cache + (((int64_t)pgk[i] * block_size + off) * G + g) * d + part * 8);
      }
    }
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int u = tid + i * 256, col = u >> 3, grp = u & 7;
      const int j = j0 + grp * 8;
      vf[i] = zero4;
      if (j <= b_last && col < dv) {
        const int off = bs_shift >= 0 ? j & bs_mask : j % block_size;
        vf[i] = *(const u32x4_t*)(v_cache + (((int64_t)pgv * G + g) * dv + col) * block_size + off);
      }
    }
  };
  const int rounds = npr + ((b_last - (lo & ~31)) >> 6) + 1;
  lookup(0);
  fetch(0);
  lookup(1);
  for (int it = 0; it < rounds; ++it) {
    const bool pooled = EXT && it < npr;
    const int j0 = pooled ? it * 64 : jt + it * 64;           // the round's first block or token
    __syncthreads();                                // the previous round's readers are done
#pragma unroll
    for (int i = 0; i < DK; ++i) {
      const int u = tid + i * 256, tok = u / (4 * DK), part = u - tok * (4 * DK);
      *(u32x4_t*)&Ks[tok][part * 8] = kf[i];
    }
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int u = tid + i * 256, col = u >> 3, grp = u & 7;
      *(u32x4_t*)&Vs[col][grp * 8] = vf[i];
    }
    __syncthreads();
    if (it + 1 < rounds) {
      fetch(it + 1);
      lookup(it + 2);
    }
    // a wavefront whose queries all lie before the round's tokens (or beyond the portion) has nothing to add
    if (idle || (pooled ? j0 >= nb_hi : (j0 > p_hi || j0 + 63 < lo_first))) continue;
    const bool interior = pooled ? j0 + 63 < nb_first : j0 + 63 <= p_first && j0 >= lo_hi;
    f32x4_t sacc[QT][4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
      for (int t = 0; t < QT; ++t) sacc[t][kb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const int tok = (kb >> 1) * 32 + (qi >> 2) * 8 + (kb & 1) * 4 + (qi & 3);
#pragma unroll
      for (int c = 0; c < DK; ++c) {
        const bf16x8_t a = *(const bf16x8_t*)&Ks[tok][c * 32 + gq * 8];
#pragma unroll
        for (int t = 0; t < QT; ++t) sacc[t][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qb[t][c], sacc[t][kb], 0, 0, 0);
      }
    }
    bf16x8_t pb[QT][2];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float mx = m[t];
      if (EXT && A.softcap > 0.f) {
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int r = 0; r < 4; ++r) sacc[t][kb][r] = capped(sacc[t][kb][r], A.softcap);
      }
      unsigned okbits = 0xffffu;
      if (!interior) {
        okbits = 0u;
        const int nb = EXT && pooled ? seen_blocks(pos[t], window, pool) : 0, lo_t = vis_lo(pos[t], window, chunk);
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = j0 + (kb >> 1) * 32 + gq * 8 + (kb & 1) * 4 + r;
            const bool ok = valid_q[t] && (pooled ? j < nb : (j <= pos[t] && j >= lo_t));
            okbits |= ok ? (1u << (kb * 4 + r)) : 0u;
          }
      }
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (okbits & (1u << (kb * 4 + r))) mx = fmaxf(mx, sacc[t][kb][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float alpha = __expf(m[t] - mx);
      m[t] = mx;
      float ls = lsum[t] * alpha;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = (okbits & (1u << (kb * 4 + r))) ? __expf(sacc[t][kb][r] - mx) : 0.f;
          ls += p;
          pb[t][kb >> 1][(kb & 1) * 4 + r] = (bf16_t)p;
        }
      lsum[t] = ls;
      if (__ballot(alpha != 1.f) != 0ull) {
#pragma unroll
        for (int db = 0; db < DVB; ++db) oacc[t][db] *= alpha;
      }
    }
#pragma unroll
    for (int mg = 0; mg < 2; ++mg)
#pragma unroll
      for (int db = 0; db < DVB; ++db) {
        const bf16x8_t a = *(const bf16x8_t*)&Vs[db * 16 + qi][mg * 32 + gq * 8];
#pragma unroll
        for (int t = 0; t < QT; ++t) oacc[t][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb[t][mg], oacc[t][db], 0, 0, 0);
      }
  }
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float ls = lsum[t];
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (!valid_q[t]) continue;
    const float inv = 1.f / ls;
    bf16_t* op = out + ((int64_t)row[t] * H + hq[t]) * dv;
    const bf16_t* gp = gate ? gate + row[t] * gate_stride + (int64_t)hq[t] * gate_w : nullptr;
#pragma unroll
    for (int db = 0; db < DVB; ++db)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = db * 16 + gq * 4 + r;
        if (c < dv) {
          float o = oacc[t][db][r] * inv;
          if (gp) o *= 1.f / (1.f + expf(-(float)gp[gate_w == 1 ? 0 : c]));
          op[c] = (bf16_t)o;
        }
      }
  }
}

template <int DK, int DVB, int QT, bool EXT>
void launch_mfma_qt(WindowAttnArgs a, hipStream_t stream) {
  a.bs_shift = -1;
  for (int b = 0; b < 31; ++b)
    if ((1 << b) == a.block_size) a.bs_shift = b;
  const int hpg = a.H / a.G;
  if (EXT || !a.no_lds) {                           // (every size fits: gfx950 has 160 KB of LDS per CU)
    if constexpr (QT == 1) {
      // steps of (mostly) single tokens with many query heads per kv head: heads, not positions, fill the query tiles
      if (hpg >= 8 && 4 * a.n <= (int64_t)a.nseq * hpg && a.packed_heads) {
        a.hw = 0;
        window_attn_mfma_lds_kernel<DK, DVB, 1, EXT><<<dim3((unsigned)a.n, (unsigned)(a.G * ((hpg + 63) / 64))), dim3(256), 0, stream>>>(a);
        return;
      }
    }
    a.hw = hpg % 4 == 0 ? 4 : (hpg % 2 == 0 ? 2 : 1);
    const int bq = (4 / a.hw) * 16 * QT;
    const int64_t btiles = a.n / bq + a.nseq;       // an upper bound: every portion may end with a partial tile
    window_attn_mfma_lds_kernel<DK, DVB, QT, EXT><<<dim3((unsigned)btiles, (unsigned)(a.G * (hpg / a.hw))), dim3(256), 0, stream>>>(a);
    return;
  }
  if constexpr (!EXT) {
    const int64_t tiles = a.n / (16 * QT) + a.nseq;
    window_attn_mfma_kernel<DK, DVB, QT><<<dim3((unsigned)((tiles + 3) / 4), a.H), dim3(256), 0, stream>>>(a);
  }
}

// Long portions (prefill) put two tiles of 16 queries on a wavefront: half the K / V bytes through the vector cache per
// MFMA; steps of short portions (decoding) keep one tile, which gives more wavefronts.
template <int DK, int DVB, bool EXT>
void launch_mfma(const WindowAttnArgs& a, hipStream_t stream) {
  if (a.n >= 32ll * a.nseq) launch_mfma_qt<DK, DVB, 2, EXT>(a, stream);
  else launch_mfma_qt<DK, DVB, 1, EXT>(a, stream);
}

// the template sizes that cover (d, dv): d <= 256 and dv <= 256
template <bool EXT>
void launch_mfma_sizes(const WindowAttnArgs& a, hipStream_t stream) {
  const int dk = a.d <= 64 ? 2 : (a.d <= 128 ? 4 : 8), dvb = a.dv <= 64 ? 4 : (a.dv <= 128 ? 8 : (a.dv <= 192 && a.d > 128 ? 12 : 16));
#define NVS_MFMA_CASE(DK, DVB) \
  if (dk == DK && dvb == DVB) launch_mfma<DK, DVB, EXT>(a, stream);
  NVS_MFMA_CASE(2, 4) NVS_MFMA_CASE(2, 8) NVS_MFMA_CASE(2, 16) NVS_MFMA_CASE(4, 4) NVS_MFMA_CASE(4, 8) NVS_MFMA_CASE(4, 16)
  NVS_MFMA_CASE(8, 4) NVS_MFMA_CASE(8, 8) NVS_MFMA_CASE(8, 12) NVS_MFMA_CASE(8, 16)
#undef NVS_MFMA_CASE
}
}  // namespace
