// The gated delta rule (see nvs_delta_scan in include/nvl_seq.h): a matrix state per head whose write is the ERROR of what the
// state already answers for the key. Everything from the unit norms on is 32-bit.
#include "seq_common.h"
#include <stdlib.h>

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
  if (per_channel) {
    NVS_DISPATCH(dtype, launch_walk<T, true>(A, nseq, (hipStream_t)stream));
  } else {
    NVS_DISPATCH(dtype, launch_walk<T, false>(A, nseq, (hipStream_t)stream));
  }
  return nvs_check_launch("nvs_delta_scan");
}
