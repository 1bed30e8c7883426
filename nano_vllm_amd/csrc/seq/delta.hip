// The gated delta rule (see nvs_delta_scan in include/nvl_seq.h): a matrix state per head whose write is the ERROR of what the
// state already answers for the key. Everything from the unit norms on is 32-bit.
#include "seq_common.h"

namespace {

struct DeltaArgs {
  const void *qkv, *gates, *decays;
  const float *A_log, *dt_bias;
  const int32_t *cu_q, *ctx0, *slot;
  float *S, *y;
  int64_t qkv_stride, gates_stride, b_col, a_col, decays_stride;
  int heads, G, dk, dv;
  float q_scale;
};

constexpr float UNIT_EPS = 1e-6f;

// ---- token by token ---------------------------------------------------------------------------------------------------
// The columns of S (one per value channel) do not interact: u_p = beta (v_p - (g S_p) . k), S_p <- g S_p + k u_p. A workgroup takes
// `cols` columns of one (portion, head); NG neighbouring lanes share a column, lane g of them holding the 16 entries
// 4 (g + NG j) + 0..3, j < 4, of PP columns in registers. Both products of a token, (g S) . k and (g S) . q, are taken from the state
// BEFORE the write — o = (g S) . q + (k . q) u — so a token costs one round of lane shuffles, not two. Tokens go in rounds of WALK_TB,
// whose unit vectors, decays and step sizes are staged in LDS a token per wavefront.
constexpr int WALK_R = 16, WALK_TB = 8;

template <typename T, int PP, bool CH>
__global__ __launch_bounds__(256) void delta_walk_kernel(const DeltaArgs A, int NG, int cols) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int s = blockIdx.y, h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int64_t q0 = A.cu_q[s], q1 = A.cu_q[s + 1];
  if (q1 <= q0) return;
  const int dk = A.dk, dv = A.dv, NP = NG * WALK_R, grp = h / (A.heads / A.G);
  const int c0 = blockIdx.z * cols, nc = dv - c0 < cols ? dv - c0 : cols;        // this workgroup's columns
  // per token: k | q (per_channel: k | g | g k | g q), values, then beta, decay, k . q
  const int vecs = CH ? 4 : 2, vat = vecs * NP, per = vat + ((cols + 3) & ~3) + 4;
  const int g = tid & (NG - 1), p = (tid / NG) * PP;                              // first of this thread's columns in the slice
  const bool fresh = A.ctx0[s] == 0, vec = (dk & 3) == 0;
  float* Sh = A.S + (((int64_t)A.slot[s] * A.heads + h) * dv + c0 + p) * dk;
  float st[PP][WALK_R];
#pragma unroll
  for (int i = 0; i < PP; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = 4 * (g + NG * j);
#pragma unroll
      for (int e = 0; e < 4; ++e) st[i][4 * j + e] = 0.f;
      if (!fresh && p + i < nc) {
        const float* src = Sh + (int64_t)i * dk + c;
        if (vec) {
          if (c < dk) {
            const float4 f = *(const float4*)src;
            st[i][4 * j] = f.x, st[i][4 * j + 1] = f.y, st[i][4 * j + 2] = f.z, st[i][4 * j + 3] = f.w;
          }
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e < dk) st[i][4 * j + e] = src[e];
        }
      }
    }
  const T* qp = (const T*)A.qkv + (int64_t)grp * dk;
  const T* kp = (const T*)A.qkv + (int64_t)(A.G + grp) * dk;
  const T* vp = (const T*)A.qkv + (int64_t)2 * A.G * dk + (int64_t)h * dv + c0;
  const T* bp = (const T*)A.gates + A.b_col + h;
  const T* ap = CH ? (const T*)A.decays + A.a_col + (int64_t)h * dk : (const T*)A.gates + A.a_col + h;
  const float* dtb = A.dt_bias + (CH ? (int64_t)h * dk : h);
  const float rate = -expf(A.A_log[h]);
  for (int64_t tb = q0; tb < q1; tb += WALK_TB) {
    const int cnt = (int)(q1 - tb < WALK_TB ? q1 - tb : WALK_TB);
    __syncthreads();                                // the previous round's readers are done
    for (int k = wave; k < cnt; k += nw) {
      const int64_t row = (tb + k) * A.qkv_stride;
      float* tp = lds + k * per;
      float sk = 0.f, sq = 0.f, kq = 0.f;
      for (int c = lane; c < dk; c += 64) {
        const float kv = ldf(kp + row + c), qv = ldf(qp + row + c);
        sk += kv * kv, sq += qv * qv, kq += kv * qv;
      }
      const float rk = 1.f / sqrtf(wave_sum(sk) + UNIT_EPS), rq = A.q_scale / sqrtf(wave_sum(sq) + UNIT_EPS);
      kq = wave_sum(kq) * rk * rq;
      for (int c = lane; c < NP; c += 64) {
        const bool in = c < dk;
        const float kv = in ? ldf(kp + row + c) * rk : 0.f, qv = in ? ldf(qp + row + c) * rq : 0.f;
        tp[c] = kv;
        if (CH) {
          const float gv = in ? expf(rate * softplusf_(ldf(ap + (tb + k) * A.decays_stride + c) + dtb[c])) : 0.f;
          tp[NP + c] = gv;
          tp[2 * NP + c] = gv * kv;
          tp[3 * NP + c] = gv * qv;
        } else {
          tp[NP + c] = qv;
        }
      }
      for (int c = lane; c < nc; c += 64) tp[vat + c] = ldf(vp + row + c);
      if (lane == 0) {
        float* sp = tp + per - 4;
        sp[0] = 1.f / (1.f + expf(-ldf(bp + (tb + k) * A.gates_stride)));
        if (!CH) sp[1] = expf(rate * softplusf_(ldf(ap + (tb + k) * A.gates_stride) + dtb[0]));
        sp[2] = kq;
      }
    }
    __syncthreads();
    for (int k = 0; k < cnt; ++k) {
      const float* tp = lds + k * per;
      const float beta = tp[per - 4], gs = CH ? 1.f : tp[per - 3], kq = tp[per - 2];
      float dk_[PP], dq_[PP];
#pragma unroll
      for (int i = 0; i < PP; ++i) dk_[i] = dq_[i] = 0.f;
      float kv[WALK_R], gv[WALK_R];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = 4 * (g + NG * j);
        const float4 k4 = *(const float4*)(tp + c);
        kv[4 * j] = k4.x, kv[4 * j + 1] = k4.y, kv[4 * j + 2] = k4.z, kv[4 * j + 3] = k4.w;
        float4 a4 = k4, b4;
        if (CH) {
          const float4 g4 = *(const float4*)(tp + NP + c);
          gv[4 * j] = g4.x, gv[4 * j + 1] = g4.y, gv[4 * j + 2] = g4.z, gv[4 * j + 3] = g4.w;
          a4 = *(const float4*)(tp + 2 * NP + c);
          b4 = *(const float4*)(tp + 3 * NP + c);
        } else {
          b4 = *(const float4*)(tp + NP + c);
        }
#pragma unroll
        for (int i = 0; i < PP; ++i) {
          dk_[i] += a4.x * st[i][4 * j] + a4.y * st[i][4 * j + 1] + a4.z * st[i][4 * j + 2] + a4.w * st[i][4 * j + 3];
          dq_[i] += b4.x * st[i][4 * j] + b4.y * st[i][4 * j + 1] + b4.z * st[i][4 * j + 2] + b4.w * st[i][4 * j + 3];
        }
      }
      for (int o = NG >> 1; o > 0; o >>= 1) {
#pragma unroll
        for (int i = 0; i < PP; ++i) {
          dk_[i] += __shfl_xor(dk_[i], o, 64);
          dq_[i] += __shfl_xor(dq_[i], o, 64);
        }
      }
#pragma unroll
      for (int i = 0; i < PP; ++i) {
        const float v = p + i < nc ? tp[vat + p + i] : 0.f;
        const float u = beta * (v - gs * dk_[i]);
#pragma unroll
        for (int r = 0; r < WALK_R; ++r) st[i][r] = (CH ? gv[r] : gs) * st[i][r] + kv[r] * u;
        if (g == 0 && p + i < nc) A.y[((tb + k) * A.heads + h) * dv + c0 + p + i] = gs * dq_[i] + kq * u;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < PP; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = 4 * (g + NG * j);
      if (p + i < nc) {
        float* dst = Sh + (int64_t)i * dk + c;
        if (vec) {
          if (c < dk) *(float4*)dst = make_float4(st[i][4 * j], st[i][4 * j + 1], st[i][4 * j + 2], st[i][4 * j + 3]);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e < dk) dst[e] = st[i][4 * j + e];
        }
      }
    }
}

template <typename T, bool CH>
void launch_walk(const DeltaArgs& A, int nseq, hipStream_t stream) {
  int ng = 1;
  while (ng * WALK_R < A.dk) ng <<= 1;
  const int pp = A.dv % 2 == 0 ? 2 : 1;
  int cols = 256 / ng * pp;                         // columns of a workgroup of 256 threads
  if (cols > A.dv) cols = A.dv;
  const int threads = ((cols + pp - 1) / pp * ng + 63) & ~63;
  const int per = (CH ? 4 : 2) * ng * WALK_R + ((cols + 3) & ~3) + 4;
  const size_t lds = (size_t)WALK_TB * per * sizeof(float);
  const dim3 grid(A.heads, (unsigned)nseq, (unsigned)((A.dv + cols - 1) / cols));
  if (pp == 2) {
    if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)delta_walk_kernel<T, 2, CH>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    delta_walk_kernel<T, 2, CH><<<grid, dim3(threads), lds, stream>>>(A, ng, cols);
  } else {
    if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)delta_walk_kernel<T, 1, CH>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    delta_walk_kernel<T, 1, CH><<<grid, dim3(threads), lds, stream>>>(A, ng, cols);
  }
}

// ---- in chunks of 16 tokens -------------------------------------------------------------------------------------------
// With G_t the product of a chunk's decays up to token t (inclusive) and S the state before the chunk, the chunk's writes u_t solve a
// unit lower triangular system, and outputs and the next state are plain products:
//   u_t + beta_t sum_{j<t} A_tj u_j = beta_t (v_t - (G_t k_t) . S),   A_tj = sum_c k_tc k_jc (G_t / G_j)_c
//   o_t = (G_t q_t) . S + sum_{j<=t} M_tj u_j,                         M_tj = sum_c q_tc k_jc (G_t / G_j)_c
//   S  <- G_C S + sum_j (G_C / G_j k_j) u_j^T
// All products run on v_mfma_f32_16x16x4_f32. A workgroup serves one (portion, head) and up to 8 x 16 value columns: four wavefronts
// prepare chunk n + 1 (unit vectors, decays, A, M, the inverse T of the system) while the others, 16 columns each with their dk x 16
// piece of the state in accumulators, work on chunk n. The state piece is a B operand as it stands — an accumulator register r holds
// rows 4 (lane / 16) + r of its tile, so contraction step r of a tile takes A's column 4 (lane / 16) + r — and so are u and the
// output, so nothing is ever exchanged between lanes. Four phases per chunk, a workgroup barrier after each:
//   columns:  O = Q S | U = T (V - P), O += M U, store | S = G_C S + K^T U | P = K S of the next chunk
//   prepare:  unit vectors, decays | decay products, G k, G q | A, M | T; K^T, G_C
// Decay products are multiplied up (no exponential of a difference). Per-channel decays: A and M are products of G k with k / G as
// long as no channel decays by more than 1e-30 within the chunk; otherwise every pair (j, t) is walked with the product G_t / G_j
// carried along. A partial chunk is filled with tokens that change nothing (k = q = v = 0, beta = 0, decay 1).
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
constexpr int CHUNK = 16, PREP = 256, MST = 20;      // MST: row stride of the 16 x 16 matrices in LDS (float4-aligned)

__device__ __forceinline__ f32x4_t mfma4(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// A barrier for data in LDS only: __syncthreads would also wait for every global load in flight, and the next chunk's loads are
// meant to stay in flight across the barriers of this one.
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// softplus from the hardware exponential and logarithm; the error of the decay's exponent stays at a few 1e-8 (log(1 + e) by its
// series where e is small)
__device__ __forceinline__ float softplus_fast(float x) {
  const float e = __expf(-fabsf(x));
  return fmaxf(x, 0.f) + (e < 0.02f ? e * (1.f - e * (0.5f - e * (0.33333333f - 0.25f * e))) : __logf(1.f + e));
}

// N consecutive elements kept as they were loaded: turning them into floats waits for the load, so that is left to the use.
template <typename T, int N>
struct RawRun {
  static constexpr int WORDS = N * (int)sizeof(T) / 4;
  uint32_t w[WORDS];
  __device__ __forceinline__ void clear() {
#pragma unroll
    for (int i = 0; i < WORDS; ++i) w[i] = 0u;
  }
  // in one piece (aligned to the piece, or to 16 bytes)
  __device__ __forceinline__ void load(const T* p) {
    constexpr int M = WORDS < 4 ? WORDS : 4;
    typedef __attribute__((ext_vector_type(M))) uint32_t vec_t;
#pragma unroll
    for (int i = 0; i < WORDS; i += M) {
      const vec_t f = *(const vec_t*)((const uint32_t*)p + i);
#pragma unroll
      for (int e = 0; e < M; ++e) w[i + e] = f[e];
    }
  }
  // the first `count` elements, one at a time, zeros behind them
  __device__ __forceinline__ void load_some(const T* p, int count) {
    clear();
#pragma unroll
    for (int e = 0; e < N; ++e) {
      if (e < count) {
        if constexpr (sizeof(T) == 4) w[e] = __builtin_bit_cast(uint32_t, p[e]);
        else w[e / 2] |= (uint32_t)__builtin_bit_cast(uint16_t, p[e]) << (16 * (e & 1));
      }
    }
  }
  __device__ __forceinline__ float get(int e) const {
    if constexpr (sizeof(T) == 4) return __builtin_bit_cast(float, w[e]);
    else return __builtin_bit_cast(float, (e & 1) ? w[e / 2] & 0xffff0000u : w[e / 2] << 16);
  }
};

// one element, likewise
__device__ __forceinline__ uint32_t raw_one(const float* p) { return *(const uint32_t*)p; }
__device__ __forceinline__ uint32_t raw_one(const bf16_t* p) { return *(const uint16_t*)p; }
template <typename T>
__device__ __forceinline__ float raw_value(uint32_t w) { return __builtin_bit_cast(float, sizeof(T) == 4 ? w : w << 16); }

// sum over the 16 lanes of a row, in every lane (rotations inside the row: plain VALU moves, no LDS)
__device__ __forceinline__ float row16_sum(float v) {
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x128, 0xf, 0xf, false));      // row_ror:8
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x124, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x122, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x121, 0xf, 0xf, false));
  return v;
}

template <int DKT, bool CH>
struct ChunkLds {
  static constexpr int DKP = 16 * DKT, LD = DKP + 4;
  float kg[CHUNK][LD], qg[CHUNK][LD];               // G k, G q
  float kn[CHUNK][LD], qn[CHUNK][LD];               // unit vectors
  float g[CH ? CHUNK : 1][LD];                      // decays per channel, or [0][t] per token
  float ki[CH ? CHUNK : 1][LD];                     // k / G
  float kt[DKP][MST];                               // (G_C / G_j k_j) transposed: channel, token
  float gc[DKP];                                    // G_C
  float part[4][CHUNK][MST];                        // A (0, 1) and M (2, 3) in two halves of the channels each
  float ratio[CH ? 1 : CHUNK][MST];                 // G_t / G_j of per-head decays
  float T[CHUNK][MST], M[CHUNK][MST];
  float beta[CHUNK];
  int strong;                                       // chunk number + 1 of the last chunk with a channel below the limit
};

template <typename T, int DKT, bool CH>
__global__ __launch_bounds__(768) void delta_chunk_kernel(const DeltaArgs A) {
  typedef ChunkLds<DKT, CH> Lds;
  constexpr int DKP = Lds::DKP;
  extern __shared__ __attribute__((aligned(16))) char chunk_lds[];
  Lds& W = *(Lds*)chunk_lds;
  const int s = blockIdx.y, h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int64_t q0 = A.cu_q[s], q1 = A.cu_q[s + 1];
  if (q1 <= q0) return;
  const int dk = A.dk, dv = A.dv, grp = h / (A.heads / A.G);
  const int li = lane & 15, lq = lane >> 4;
  const bool prep = wave < 4;
  const int nch = (int)((q1 - q0 + CHUNK - 1) / CHUNK);
  if (tid == 0) W.strong = 0;

  // ---- prepare: thread (token pt, lane pl of 16) holds the DKT channels from pl DKT on of its token
  const int pt = (tid >> 4) & 15, pl = tid & 15;
  const T* qp = (const T*)A.qkv + (int64_t)grp * dk;
  const T* kp = (const T*)A.qkv + (int64_t)(A.G + grp) * dk;
  const T* ap = CH ? (const T*)A.decays + A.a_col + (int64_t)h * dk : (const T*)A.gates + A.a_col + h;
  const T* bp = (const T*)A.gates + A.b_col + h;
  const float* dtb = A.dt_bias + (CH ? (int64_t)h * dk : h);
  const float rate = -expf(A.A_log[h]);
  RawRun<T, DKT> rk_, rq_, ra_;                     // (ra_: per-channel decays only)
  uint32_t ra1 = 0u, rb = 0u;
  const int64_t rows_al = A.qkv_stride | dk | (CH ? A.decays_stride | A.a_col : 0);
  const bool runs = rows_al % DKT == 0 && ((uintptr_t)A.qkv | (uintptr_t)(CH ? A.decays : A.qkv)) % 16 == 0;      // whole runs, aligned
  const int pc = pl * DKT;
  float dtc[CH ? DKT : 1];
  if (CH) {
#pragma unroll
    for (int e = 0; e < DKT; ++e) dtc[e] = pc + e < dk ? dtb[pc + e] : 0.f;
  } else {
    dtc[0] = dtb[0];
  }
  auto load = [&](int n) {
    const int64_t t = q0 + (int64_t)n * CHUNK + pt;
    const bool in = t < q1;
    if (in && runs && pc < dk) {
      rk_.load(kp + t * A.qkv_stride + pc);
      rq_.load(qp + t * A.qkv_stride + pc);
      if constexpr (CH) ra_.load(ap + t * A.decays_stride + pc);
    } else {
      const int count = in && !runs ? dk - pc : 0;
      rk_.load_some(kp + t * A.qkv_stride + pc, count);
      rq_.load_some(qp + t * A.qkv_stride + pc, count);
      if constexpr (CH) ra_.load_some(ap + t * A.decays_stride + pc, count);
    }
    if (in) {
      rb = raw_one(bp + t * A.gates_stride);
      if constexpr (!CH) ra1 = raw_one(ap + t * A.gates_stride);
    }
  };
  auto stage = [&](int n) {
    const bool in = q0 + (int64_t)n * CHUNK + pt < q1;
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int e = 0; e < DKT; ++e) sk += rk_.get(e) * rk_.get(e), sq += rq_.get(e) * rq_.get(e);
    const float fk = 1.f / sqrtf(row16_sum(sk) + UNIT_EPS), fq = A.q_scale / sqrtf(row16_sum(sq) + UNIT_EPS);
#pragma unroll
    for (int e = 0; e < DKT; ++e) {
      W.kn[pt][pc + e] = rk_.get(e) * fk;
      W.qn[pt][pc + e] = rq_.get(e) * fq;
      if constexpr (CH) W.g[pt][pc + e] = in && pc + e < dk ? __expf(rate * softplus_fast(ra_.get(e) + dtc[e])) : 1.f;
    }
    if (pl == 0) {
      if constexpr (!CH) W.g[0][pt] = in ? __expf(rate * softplus_fast(raw_value<T>(ra1) + dtc[0])) : 1.f;
      W.beta[pt] = in ? 1.f / (1.f + __expf(-raw_value<T>(rb))) : 0.f;
    }
  };
  auto products = [&](int n) {                       // G k, G q, k / G: a channel per thread, K and Q parts apart
    for (int w = tid; w < 2 * DKP; w += PREP) {
      const int c = w & (DKP - 1);
      float G = 1.f;
      if (w < DKP) {
#pragma unroll
        for (int t = 0; t < CHUNK; ++t) {
          G *= CH ? W.g[t][c] : W.g[0][t];
          const float k = W.kn[t][c];
          W.kg[t][c] = G * k;
          if (CH) W.ki[t][c] = k * __builtin_amdgcn_rcpf(G);
        }
        if (CH && G < 1e-30f) W.strong = n + 1;
      } else {
#pragma unroll
        for (int t = 0; t < CHUNK; ++t) {
          G *= CH ? W.g[t][c] : W.g[0][t];
          W.qg[t][c] = G * W.qn[t][c];
        }
      }
    }
    if (!CH) {
      float r = 1.f;
#pragma unroll
      for (int i = 1; i < CHUNK; ++i) r *= i > pl && i <= pt ? W.g[0][i] : 1.f;
      W.ratio[pt][pl] = r;
    }
  };
  auto matrices = [&](int n) {
    if (CH && W.strong == n + 1) {
      // pair by pair: thread (token j = pt, lane pl) carries its channels of k_j times the decays since j through the later tokens
      float w[DKT];
#pragma unroll
      for (int e = 0; e < DKT; ++e) w[e] = W.kn[pt][pc + e];
#pragma unroll 4
      for (int t = 0; t < CHUNK; ++t) {
        float a = 0.f, m = 0.f;
#pragma unroll
        for (int e = 0; e < DKT; ++e) {
          w[e] *= t > pt ? W.g[t][pc + e] : 1.f;
          a += W.kn[t][pc + e] * w[e];
          m += W.qn[t][pc + e] * w[e];
        }
        a = row16_sum(a), m = row16_sum(m);          // (entries above the diagonal are not looked at)
        if (pl == 0) W.part[0][t][pt] = a, W.part[1][t][pt] = 0.f, W.part[2][t][pt] = m, W.part[3][t][pt] = 0.f;
      }
      return;
    }
    const int half = wave & 1;
    const auto& left = wave < 2 ? (CH ? W.kg : W.kn) : (CH ? W.qg : W.qn);
    const auto& right = *(const float(*)[CHUNK][Lds::LD])(CH ? &W.ki[0][0] : &W.kn[0][0]);
    f32x4_t acc[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int i = 0; i < (DKT + 1) / 2; ++i) {
      const int tt = half * ((DKT + 1) / 2) + i;
      if (tt < DKT) {
        const float4 a = *(const float4*)&left[li][16 * tt + 4 * lq], b = *(const float4*)&right[li][16 * tt + 4 * lq];
        acc[0] = mfma4(a.x, b.x, acc[0]);
        acc[1] = mfma4(a.y, b.y, acc[1]);
        acc[0] = mfma4(a.z, b.z, acc[0]);
        acc[1] = mfma4(a.w, b.w, acc[1]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) W.part[wave][4 * lq + r][li] = acc[0][r] + acc[1][r];
  };
  auto solve = [&]() {
    if (wave == 0) {
      // T = (I + L)^-1, L = beta A below the diagonal, by doubling the blocks whose inverses are known: with T block diagonal (blocks
      // of b) and L_b the entries of L that couple the two halves of a block of 2 b, T <- T - T L_b T. L stays in registers as
      // an A operand; X = L_b T comes out as the B operand that T X needs; T goes through LDS once per step to become an A operand.
      const float4 a0 = *(const float4*)&W.part[0][li][4 * lq], a1 = *(const float4*)&W.part[1][li][4 * lq];
      const float bt = W.beta[li];
      float L[4] = {a0.x + a1.x, a0.y + a1.y, a0.z + a1.z, a0.w + a1.w};
      if (!CH) {
        const float4 r = *(const float4*)&W.ratio[li][4 * lq];
        L[0] *= r.x, L[1] *= r.y, L[2] *= r.z, L[3] *= r.w;
      }
      f32x4_t Tm;
#pragma unroll
      for (int r = 0; r < 4; ++r) Tm[r] = 4 * lq + r == li ? 1.f : 0.f;
#pragma unroll
      for (int b = 1; b < CHUNK; b *= 2) {
        if (b > 1) {
#pragma unroll
          for (int r = 0; r < 4; ++r) W.T[4 * lq + r][li] = Tm[r];
          __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup", "local");
          __builtin_amdgcn_wave_barrier();
        }
        f32x4_t X = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int k = 4 * lq + r;                  // entry (li, k): below the diagonal, other half of the same block of 2 b
          const bool couples = li / (2 * b) == k / (2 * b) && (li & b) && !(k & b);
          X = mfma4(couples ? bt * L[r] : 0.f, Tm[r], X);
        }
        if (b == 1) {                                // (T is the unit matrix)
          Tm -= X;
        } else {
          const float4 t4 = *(const float4*)&W.T[li][4 * lq];
          Tm = mfma4(-t4.x, X[0], Tm);
          Tm = mfma4(-t4.y, X[1], Tm);
          Tm = mfma4(-t4.z, X[2], Tm);
          Tm = mfma4(-t4.w, X[3], Tm);
          __builtin_amdgcn_wave_barrier();
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) W.T[4 * lq + r][li] = Tm[r] * bt;      // times beta of the column: U = T diag(beta) (V - P)
    } else if (wave == 1) {
      const float4 m0 = *(const float4*)&W.part[2][li][4 * lq], m1 = *(const float4*)&W.part[3][li][4 * lq];
      float m[4] = {m0.x + m1.x, m0.y + m1.y, m0.z + m1.z, m0.w + m1.w};
      if (!CH) {
        const float4 r = *(const float4*)&W.ratio[li][4 * lq];
        m[0] *= r.x, m[1] *= r.y, m[2] *= r.z, m[3] *= r.w;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) m[r] = 4 * lq + r <= li ? m[r] : 0.f;
      *(float4*)&W.M[li][4 * lq] = make_float4(m[0], m[1], m[2], m[3]);
    } else {
      for (int c = tid - 128; c < DKP; c += 128) {
        float D = 1.f, col[CHUNK];
#pragma unroll
        for (int t = CHUNK - 1; t >= 0; --t) {
          col[t] = D * W.kn[t][c];
          D *= CH ? W.g[t][c] : W.g[0][t];
        }
#pragma unroll
        for (int t = 0; t < CHUNK; t += 4) *(float4*)&W.kt[c][t] = make_float4(col[t], col[t + 1], col[t + 2], col[t + 3]);
        W.gc[c] = D;
      }
    }
  };

  // the two roles in loops of their own (their registers are then not live together); both meet in the same 1 + 4 (nch + 1) barriers
  if (prep) {
    load(0);
    lds_barrier();
    for (int n = 0; n <= nch; ++n) {                // chunk n is prepared while chunk n - 1 is worked on
      const bool next = n < nch;
      if (next) {
        stage(n);
        if (n + 1 < nch) load(n + 1);
      }
      lds_barrier();
      if (next) products(n);
      lds_barrier();
      if (next) matrices(n);
      lds_barrier();
      if (next) solve();
      lds_barrier();
    }
    return;
  }
  // ---- columns: 16 value columns per wavefront
  const int col = (blockIdx.z * ((blockDim.x >> 6) - 4) + (wave - 4)) * 16 + li;
  const bool own = col < dv;
  float* Sc = A.S + (((int64_t)A.slot[s] * A.heads + h) * dv + (own ? col : 0)) * dk;
  const T* vp = (const T*)A.qkv + (int64_t)2 * A.G * dk + (int64_t)h * dv + col;
  f32x4_t st[DKT], P = {0.f, 0.f, 0.f, 0.f}, O = {0.f, 0.f, 0.f, 0.f}, U = {0.f, 0.f, 0.f, 0.f};
  uint32_t v[4] = {0u, 0u, 0u, 0u};                 // (raw: see RawRun)
#pragma unroll
  for (int i = 0; i < DKT; ++i) st[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (own && A.ctx0[s] != 0) {
#pragma unroll
    for (int i = 0; i < DKT; ++i) {
      const int c = 16 * i + 4 * lq;
      if ((dk & 3) == 0) {
        if (c < dk) st[i] = *(const f32x4_t*)(Sc + c);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c + r < dk) st[i][r] = Sc[c + r];
      }
    }
  }
  auto load_v = [&](int n) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int64_t t = q0 + (int64_t)n * CHUNK + 4 * lq + r;
      v[r] = own && t < q1 ? raw_one(vp + t * A.qkv_stride) : 0u;
    }
  };
  auto times_state = [&](const float (&m)[CHUNK][Lds::LD]) {      // m S, [16 tokens x 16 columns]
    f32x4_t a0 = {0.f, 0.f, 0.f, 0.f}, a1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < DKT; ++i) {
      const float4 a = *(const float4*)&m[li][16 * i + 4 * lq];
      a0 = mfma4(a.x, st[i][0], a0);
      a1 = mfma4(a.y, st[i][1], a1);
      a0 = mfma4(a.z, st[i][2], a0);
      a1 = mfma4(a.w, st[i][3], a1);
    }
    return a0 + a1;
  };
  load_v(0);
  lds_barrier();
  for (int n = -1; n < nch; ++n) {
    const bool next = n + 1 < nch;
    if (n >= 0) O = times_state(W.qg);
    lds_barrier();
    if (n >= 0) {
      f32x4_t X;
#pragma unroll
      for (int r = 0; r < 4; ++r) X[r] = raw_value<T>(v[r]) - P[r];
      if (next) load_v(n + 1);
      const float4 t4 = *(const float4*)&W.T[li][4 * lq], m4 = *(const float4*)&W.M[li][4 * lq];
      U = mfma4(t4.x, X[0], f32x4_t{0.f, 0.f, 0.f, 0.f});
      U = mfma4(t4.y, X[1], U);
      U = mfma4(t4.z, X[2], U);
      U = mfma4(t4.w, X[3], U);
      O = mfma4(m4.x, U[0], O);
      O = mfma4(m4.y, U[1], O);
      O = mfma4(m4.z, U[2], O);
      O = mfma4(m4.w, U[3], O);
      if (own) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int64_t t = q0 + (int64_t)n * CHUNK + 4 * lq + r;
          if (t < q1) A.y[(t * A.heads + h) * dv + col] = O[r];
        }
      }
    }
    lds_barrier();
    if (n >= 0) {
#pragma unroll
      for (int i = 0; i < DKT; ++i) {
        const float4 g4 = *(const float4*)&W.gc[16 * i + 4 * lq], a = *(const float4*)&W.kt[16 * i + li][4 * lq];
        st[i][0] *= g4.x, st[i][1] *= g4.y, st[i][2] *= g4.z, st[i][3] *= g4.w;
        st[i] = mfma4(a.x, U[0], st[i]);
        st[i] = mfma4(a.y, U[1], st[i]);
        st[i] = mfma4(a.z, U[2], st[i]);
        st[i] = mfma4(a.w, U[3], st[i]);
      }
    }
    lds_barrier();
    if (next) P = times_state(W.kg);
    lds_barrier();
  }
  if (own) {
#pragma unroll
    for (int i = 0; i < DKT; ++i) {
      const int c = 16 * i + 4 * lq;
      if ((dk & 3) == 0) {
        if (c < dk) *(f32x4_t*)(Sc + c) = st[i];
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c + r < dk) Sc[c + r] = st[i][r];
      }
    }
  }
}

template <typename T, int DKT, bool CH>
void launch_chunk_size(const DeltaArgs& A, int nseq, hipStream_t stream) {
  const int tiles = (A.dv + 15) / 16;
  // column wavefronts per workgroup: all columns of a head together (they share the preparation, which bounds a chunk's time), fewer
  // of them while the workgroups do not even fill half the chip (measured, 128 x 128 heads, 2,048 tokens: 256 pairs 780 us with 8
  // wavefronts, 900 with 4, 1,690 with 2; 64 pairs 770 / 590 / 580)
  int ncw = tiles < 8 ? tiles : 8;
  while (ncw > 1 && (int64_t)A.heads * nseq * ((tiles + ncw - 1) / ncw) < 128) ncw = (ncw + 1) / 2;
  const size_t lds = sizeof(ChunkLds<DKT, CH>);
  if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)delta_chunk_kernel<T, DKT, CH>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  delta_chunk_kernel<T, DKT, CH><<<dim3(A.heads, (unsigned)nseq, (unsigned)((tiles + ncw - 1) / ncw)), dim3(64 * (4 + ncw)), lds, stream>>>(A);
}

template <typename T, bool CH>
void launch_chunk(const DeltaArgs& A, int nseq, hipStream_t stream) {
  if (A.dk <= 32) launch_chunk_size<T, 2, CH>(A, nseq, stream);
  else if (A.dk <= 64) launch_chunk_size<T, 4, CH>(A, nseq, stream);
  else if (A.dk <= 128) launch_chunk_size<T, 8, CH>(A, nseq, stream);
  else launch_chunk_size<T, 16, CH>(A, nseq, stream);
}

int g_delta_mode = 0;

}  // namespace

extern "C" void nvs_delta_force(int mode) { g_delta_mode = mode; }

extern "C" int nvs_delta_scan(const void* qkv, int64_t qkv_stride, const void* gates, int64_t gates_stride, int64_t b_col, int64_t a_col,
                              const void* decays, int64_t decays_stride, int dtype, const float* A_log, const float* dt_bias, float q_scale,
                              int per_channel, int heads, int G, int dk, int dv, const int32_t* cu_q, const int32_t* ctx0,
                              const int32_t* slot, int nseq, int64_t n, int64_t max_q, float* S, float* y, void* stream) {
  NVS_REQUIRE(qkv && gates && A_log && dt_bias && cu_q && ctx0 && slot && S && y && (!per_channel || decays), "nvs_delta_scan: null argument");
  NVS_REQUIRE(heads > 0 && heads <= 65535 && G > 0 && heads % G == 0 && dk > 0 && dk <= 512 && dv > 0 && dv <= 1024 && nseq >= 0 && nseq <= 65535,
              "nvs_delta_scan: heads %d groups %d key size %d (up to 512) value size %d (up to 1024)", heads, G, dk, dv);
  NVS_REQUIRE(qkv_stride >= 2ll * G * dk + (int64_t)heads * dv && b_col >= 0 && b_col + heads <= gates_stride && a_col >= 0 &&
                  (per_channel ? a_col + (int64_t)heads * dk <= decays_stride : a_col + heads <= gates_stride),
              "nvs_delta_scan: columns beyond a row stride");
  if (n == 0 || nseq == 0) return NVS_OK;
  DeltaArgs A = {qkv, gates, decays, A_log, dt_bias, cu_q, ctx0, slot, S, y, qkv_stride, gates_stride, b_col, a_col, decays_stride,
                 heads, G, dk, dv, q_scale};
  const bool chunks = dk <= 256 && (g_delta_mode == 2 || (g_delta_mode == 0 && n > nseq && max_q >= CHUNK));
  if (chunks) {
    if (per_channel) {
      NVS_DISPATCH(dtype, launch_chunk<T, true>(A, nseq, (hipStream_t)stream));
    } else {
      NVS_DISPATCH(dtype, launch_chunk<T, false>(A, nseq, (hipStream_t)stream));
    }
  } else if (per_channel) {
    NVS_DISPATCH(dtype, launch_walk<T, true>(A, nseq, (hipStream_t)stream));
  } else {
    NVS_DISPATCH(dtype, launch_walk<T, false>(A, nseq, (hipStream_t)stream));
  }
  return nvs_check_launch("nvs_delta_scan");
}
