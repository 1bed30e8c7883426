// Paged attention with a local mask for any head size: key norm / rotation + K/V store, and the attention itself (one wavefront
// per (token row, query head): portions of prompts and single decoded tokens are the same launch). Scores, softmax and the
// output accumulation are 32-bit; the query norm, the rotation of the query and the sigmoid output gate are fused in.
// The mask is one of: a sliding window (the last `window` positions), blocks (`chunk` > 0: a query sees the keys of its own
// block of `chunk` positions, blocks counted from position 0 of the sequence), or plain causal; behind a window the past may be
// kept as means over blocks of positions (attn_pool.hip).
#include "attn_window_core.h"

namespace {

constexpr int MAX_HEAD = 1024;      // scalar kernels (CH = 4 or 16 chunks of 64 entries per head); the matrix-core kernels take up to 256

// one wavefront per (token, kv head)
template <typename T, int CH>
__global__ void knorm_kvstore_kernel(const T* __restrict__ k, const T* __restrict__ v, int64_t stride, const T* __restrict__ knorm,
                                     float eps, int G, int d, int dv, int block_size, const int32_t* __restrict__ slots,
                                     const int64_t* __restrict__ pos, const float* __restrict__ rot_freq, int rot_dims,
                                     T* __restrict__ k_cache, T* __restrict__ v_cache) {
  const int64_t t = blockIdx.x;
  const int g = blockIdx.y, lane = threadIdx.x;
  const int64_t slot = slots[t];
  if (slot < 0) return;
  const T* kp = k + t * stride + (int64_t)g * d;
  float kv[CH];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int c = lane + 64 * i;
    kv[i] = c < d ? ldf(kp + c) : 0.f;
    ss += kv[i] * kv[i];
  }
  float r = 1.f;
  if (knorm) r = rsqrtf(wave_sum(ss) / (float)d + eps);
  T* kc = k_cache + (slot * G + g) * d;
  const float pf = rot_dims > 0 ? (float)pos[t] : 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int c = lane + 64 * i;
    float val = (knorm && c < d) ? kv[i] * r * ldf(knorm + c) : kv[i];
    // rotation of the pair (2i, 2i+1): the partner sits in the neighbouring lane
    const float other = __shfl_xor(val, 1, 64);
    if (c < rot_dims) {
      float sn, cs;
      sincosf(pf * rot_freq[c >> 1], &sn, &cs);
      val = (c & 1) ? val * cs + other * sn : val * cs - other * sn;
    }
    if (c < d) stf(kc + c, val);
  }
  const T* vp = v + t * stride + (int64_t)g * dv;
  // values are kept transposed inside a page, [page][G][dv][block]: the attention kernels read a column's consecutive tokens
  const int64_t page = slot / block_size, off = slot - page * block_size;
  T* vc = v_cache + ((page * G + g) * dv) * block_size + off;
  for (int c = lane; c < dv; c += 64) vc[(int64_t)c * block_size] = vp[c];
}

// one wavefront per (token, query head). Keys go in rounds of 64 (one per lane): score, running maximum, weights into LDS,
// then every lane accumulates its value columns over the round's keys. Pooled blocks are keys like any other, in rounds of their own.
template <typename T, int CH>
__global__ void window_attn_kernel(const WindowAttnArgs A) {
  __shared__ float qs[CH * 64];
  __shared__ float ps[64];
  __shared__ int64_t slot_s[64];                    // element offset of (key, column 0) in its value tensor
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  const int s = A.tseq[t], H = A.H, G = A.G, d = A.d, dv = A.dv, block_size = A.block_size;
  const int64_t pos = (int64_t)A.ctx0[s] + (t - A.cu_q[s]);
  const int g = h / (H / G);
  const T* __restrict__ k_cache = (const T*)A.k_cache;
  const T* __restrict__ v_cache = (const T*)A.v_cache;
  // query (+ norm) into LDS
  {
    const T* qp = (const T*)A.q + t * A.q_stride + (int64_t)h * d;
    const T* qnorm = (const T*)A.qnorm;
    float qv[CH];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = lane + 64 * i;
      qv[i] = c < d ? ldf(qp + c) : 0.f;
      ss += qv[i] * qv[i];
    }
    float r = 1.f;
    if (A.q_row) r = A.q_row[t], qnorm += (int64_t)h * d;      // norm over the whole projection: weights of every head
    else if (qnorm) r = rsqrtf(wave_sum(ss) / (float)d + A.eps);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = lane + 64 * i;
      float val = (qnorm && c < d) ? qv[i] * r * ldf(qnorm + c) : qv[i];
      const float other = __shfl_xor(val, 1, 64);   // rotation of the pair (2i, 2i+1)
      if (c < A.rot_dims) {
        float sn, cs;
        sincosf((float)pos * A.rot_freq[c >> 1], &sn, &cs);
        val = (c & 1) ? val * cs + other * sn : val * cs - other * sn;
      }
      if (c < d) qs[c] = val;
    }
  }
  __syncthreads();
  const int64_t lo = vis_lo((int)pos, A.window, A.chunk);
  const int32_t* bt = A.block_tables + (int64_t)s * A.bt_stride;
  // a sink is a score in the denominator that has no value: the running maximum and sum start from it
  float m = A.sink ? A.sink[h] : -INFINITY, l = A.sink ? 1.f : 0.f;
  const float scale = A.scale * query_temp((int)pos, A.qt_coef, A.qt_every);
  float acc[CH];
#pragma unroll
  for (int i = 0; i < CH; ++i) acc[i] = 0.f;
  // one round: lane's key at kp (live or not), its value column c at vals[voff + c * cstride]; `cnt` lanes from 0 on are live
  auto round = [&](bool live, const T* kp, const T* vals, int64_t voff, int cstride, int cnt) {
    float sc = -INFINITY;
    if (live) {
      float dot = 0.f;
      for (int c = 0; c < d; ++c) dot += qs[c] * ldf(kp + c);
      sc = dot * scale;
      if (A.softcap > 0.f) sc = A.softcap * tanhf(sc / A.softcap);
    }
    const float mn = fmaxf(m, wave_max(sc));          // finite: lane 0 of every round is live
    const float alpha = expf(m - mn);                 // 0 in the first round without a sink (m = -inf)
    const float p = live ? expf(sc - mn) : 0.f;
    l = l * alpha + wave_sum(p);
    m = mn;
    __syncthreads();                                  // the previous round's readers are done
    ps[lane] = p;
    slot_s[lane] = voff;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = lane + 64 * i;
      if (c < dv) {
        float a = acc[i] * alpha;
        for (int jj = 0; jj < cnt; ++jj) a += ps[jj] * ldf(vals + slot_s[jj] + (int64_t)c * cstride);
        acc[i] = a;
      }
    }
  };
  const int nb = seen_blocks((int)pos, A.window, A.pool);
  for (int b0 = 0; b0 < nb; b0 += 64) {
    const int b = b0 + lane;
    const bool live = b < nb;
    const int64_t unit = live ? pool_unit(b >> 3, A.pool, block_size, bt) : 0;
    round(live, (const T*)A.pool_k + ((unit * 8 + (b & 7)) * G + g) * d, (const T*)A.pool_v, ((unit * G + g) * dv) * 8 + (b & 7), 8,
          nb - b0 < 64 ? nb - b0 : 64);
  }
  for (int64_t j0 = lo; j0 <= pos; j0 += 64) {
    const int64_t j = j0 + lane;
    const bool live = j <= pos;
    int64_t page = 0, off = 0;
    if (live) page = bt[j / block_size], off = j % block_size;
    round(live, k_cache + ((page * block_size + off) * G + g) * d, v_cache, ((page * G + g) * dv) * block_size + off, block_size,
          (int)((pos - j0 + 1) < 64 ? (pos - j0 + 1) : 64));
  }
  const float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int c = lane + 64 * i;
    if (c < dv) {
      float o = acc[i] * inv;
      if (A.gate) {
        const float gv = ldf((const T*)A.gate + t * A.gate_stride + (int64_t)h * A.gate_w + (A.gate_w == 1 ? 0 : c));
        o *= 1.f / (1.f + expf(-gv));
      }
      stf((T*)A.out + (t * H + h) * dv + c, o);
    }
  }
}
}  // namespace

void window_attn_extended(const WindowAttnArgs& a, hipStream_t stream);      // attn_pool.hip

static int g_force_scalar = 0, g_no_lds = 0, g_packed_heads = 1;
/* tests: 1 routes bf16 calls through the scalar kernel as well */
extern "C" void nvs_window_attn_force_scalar(int on) {
  g_force_scalar = on == 1;
  g_no_lds = on == 2;
  g_packed_heads = on != 3;
}

extern "C" int nvs_knorm_kvstore(const void* k, const void* v, int64_t stride, int dtype, const void* knorm, float eps, int G, int d,
                                 int dv, int block_size, const int32_t* slots, const int64_t* pos, const float* rot_freq, int rot_dims,
                                 int64_t n, void* k_cache, void* v_cache, void* stream) {
  NVS_REQUIRE(k && v && slots && k_cache && v_cache, "nvs_knorm_kvstore: null argument");
  NVS_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= d && (rot_dims == 0 || (pos && rot_freq)),
              "nvs_knorm_kvstore: rotation of %d of %d dimensions", rot_dims, d);
  NVS_REQUIRE(G > 0 && G <= 65535 && d > 0 && d <= MAX_HEAD && dv > 0 && dv <= MAX_HEAD && n >= 0 && block_size > 0,
              "nvs_knorm_kvstore: G %d d %d dv %d", G, d, dv);
  if (n == 0) return NVS_OK;
  if (d <= 256 && dv <= 256)
    NVS_DISPATCH(dtype, knorm_kvstore_kernel<T, 4><<<dim3((unsigned)n, G), dim3(64), 0, (hipStream_t)stream>>>(
                            (const T*)k, (const T*)v, stride, (const T*)knorm, eps, G, d, dv, block_size, slots, pos, rot_freq, rot_dims,
                            (T*)k_cache, (T*)v_cache));
  else
    NVS_DISPATCH(dtype, knorm_kvstore_kernel<T, 16><<<dim3((unsigned)n, G), dim3(64), 0, (hipStream_t)stream>>>(
                            (const T*)k, (const T*)v, stride, (const T*)knorm, eps, G, d, dv, block_size, slots, pos, rot_freq, rot_dims,
                            (T*)k_cache, (T*)v_cache));
  return nvs_check_launch("nvs_knorm_kvstore");
}

extern "C" int nvs_window_attn(const void* q, int64_t q_stride, const void* qnorm, float eps, const float* q_row, const void* gate,
                               int64_t gate_stride, int gate_per_head, int dtype, const void* k_cache, const void* v_cache,
                               const int32_t* block_tables, int64_t bt_stride, int block_size, const int32_t* cu_q, const int32_t* ctx0,
                               const int32_t* tseq, int nseq, int64_t n, int H, int G, int d, int dv, float scale, float softcap, int window,
                               int chunk, int pool, const void* pool_k, const void* pool_v, const float* rot_freq, int rot_dims,
                               const float* sink, float qt_coef, int qt_every, void* out, void* stream) {
  NVS_REQUIRE(qt_every >= 0, "nvs_window_attn: a query temperature every %d positions", qt_every);
  NVS_REQUIRE(q && k_cache && v_cache && block_tables && cu_q && ctx0 && tseq && out, "nvs_window_attn: null argument");
  NVS_REQUIRE(!(window > 0 && chunk > 0), "nvs_window_attn: a window (%d) and blocks (%d) together", window, chunk);
  NVS_REQUIRE(pool >= 0 && (pool == 0 || (window > 0 && pool_k && pool_v)), "nvs_window_attn: pooled blocks (%d) go behind a window (%d)", pool, window);
  NVS_REQUIRE(!q_row || qnorm, "nvs_window_attn: row factors without norm weights");
  NVS_REQUIRE(softcap >= 0.f, "nvs_window_attn: softcap %g", (double)softcap);
  NVS_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= d && (rot_dims == 0 || rot_freq),
              "nvs_window_attn: rotation of %d of %d dimensions", rot_dims, d);
  NVS_REQUIRE(H > 0 && H <= 65535 && G > 0 && H % G == 0 && d > 0 && d <= MAX_HEAD && dv > 0 && dv <= MAX_HEAD && block_size > 0 && n >= 0,
              "nvs_window_attn: H %d G %d d %d dv %d block %d", H, G, d, dv, block_size);
  if (n == 0 || nseq == 0) return NVS_OK;
  WindowAttnArgs a = {};
  a.q = q, a.qnorm = qnorm, a.gate = gate, a.k_cache = k_cache, a.v_cache = v_cache, a.out = out;
  a.block_tables = block_tables, a.cu_q = cu_q, a.ctx0 = ctx0, a.tseq = tseq, a.rot_freq = rot_freq, a.sink = sink;
  a.q_stride = q_stride, a.gate_stride = gate_stride, a.bt_stride = bt_stride, a.n = n;
  a.gate_w = gate_per_head ? 1 : dv;                 // gate entries per head: one for the whole head, or one per value column
  a.block_size = block_size, a.nseq = nseq, a.H = H, a.G = G, a.d = d, a.dv = dv, a.window = window, a.chunk = chunk;
  a.rot_dims = rot_dims, a.qt_every = qt_every, a.eps = eps, a.scale = scale, a.qt_coef = qt_coef;
  a.no_lds = g_no_lds, a.packed_heads = g_packed_heads;
  a.q_row = q_row, a.pool_k = pool_k, a.pool_v = pool_v, a.pool = pool, a.softcap = softcap;
  if (dtype == NVS_BF16 && d % 8 == 0 && d <= 256 && dv <= 256 && block_size % 8 == 0 && !g_force_scalar) {
    if (q_row || pool > 0 || softcap > 0.f) window_attn_extended(a, (hipStream_t)stream);
    else launch_mfma_sizes<false>(a, (hipStream_t)stream);
    return nvs_check_launch("nvs_window_attn (matrix cores)");
  }
  if (d <= 256 && dv <= 256)
    NVS_DISPATCH(dtype, window_attn_kernel<T, 4><<<dim3((unsigned)n, H), dim3(64), 0, (hipStream_t)stream>>>(a));
  else                                               // heads of up to 1024 entries: the same kernel with 16 entries per lane
    NVS_DISPATCH(dtype, window_attn_kernel<T, 16><<<dim3((unsigned)n, H), dim3(64), 0, (hipStream_t)stream>>>(a));
  return nvs_check_launch("nvs_window_attn");
}
