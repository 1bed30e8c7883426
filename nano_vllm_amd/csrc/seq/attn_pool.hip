// Attention whose past beyond the window is kept as means over blocks of positions: the matrix-core kernels with pooled blocks,
// capped scores and a query norm over the whole projection (instances of attn_window_core.h), the key norm over the whole
// projection with rotation and the paged store, and the means themselves.
#include "attn_window_core.h"

namespace {

constexpr int MAX_HEAD_POOL = 1024;

// The mean of the `pool` cached tokens that end at position p into their block's place (see pool_unit), every kv head: the keys
// (half 0) or the values (half 1), by all threads of the workgroup. Key rows are read a column per thread; values are transposed
// inside a page (and inside a unit of 8 blocks), so there LN neighbouring lanes share a column and read its consecutive tokens.
template <typename T>
__device__ void pool_block(int half, int p, const int32_t* __restrict__ bt, const T* k_cache, const T* v_cache, int G, int d, int dv,
                           int block_size, int pool, T* pool_k, T* pool_v) {
  const int b = p / pool, first = b * pool;
  const int64_t unit = pool_unit(b >> 3, pool, block_size, bt);
  const float inv = 1.f / (float)pool;
  const int nk = G * d, nv = G * dv;
  if (half == 0) {
    for (int c = threadIdx.x; c < nk; c += blockDim.x) {
      float sum = 0.f;
      for (int j = first; j <= p;) {                // a run of tokens inside one page at a time
        const int page = j / block_size, off = j - page * block_size;
        const int run = block_size - off < p + 1 - j ? block_size - off : p + 1 - j;
        const T* src = k_cache + ((int64_t)bt[page] * block_size + off) * nk + c;
#pragma unroll 8
        for (int i = 0; i < run; ++i) sum += ldf(src + (int64_t)i * nk);
        j += run;
      }
      stf(pool_k + (unit * 8 + (b & 7)) * nk + c, sum * inv);
    }
    return;
  }
  int ln = 1;
  while (ln < pool && ln < 16) ln <<= 1;
  const int sub = threadIdx.x & (ln - 1), step = blockDim.x / ln;
  for (int c0 = threadIdx.x / ln; c0 - (int)(threadIdx.x / ln) < nv; c0 += 8 * step) {      // (every thread takes part in the shuffles)
    float sum[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) sum[u] = 0.f;
    for (int j = first + sub; j <= p; j += ln) {
      const int page = j / block_size, off = j - page * block_size;
      const T* src = v_cache + ((int64_t)bt[page] * nv + c0) * block_size + off;
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (c0 + u * step < nv) sum[u] += ldf(src + (int64_t)u * step * block_size);
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      for (int o = ln >> 1; o > 0; o >>= 1) sum[u] += __shfl_xor(sum[u], o, 64);
      const int c = c0 + u * step;
      if (c < nv && sub == 0) stf(pool_v + (unit * nv + c) * 8 + (b & 7), sum[u] * inv);
    }
  }
}

// one workgroup per token: the root mean square of the whole query row (-> q_row) and of the whole key row; the key row times
// its weights, rotated per head, and the value row into the paged cache. finish: the step brings one token per sequence, so a
// block that this token completes has all its other tokens in the cache already and its mean is taken here.
template <typename T>
__global__ __launch_bounds__(256) void qk_rows_kernel(const T* __restrict__ q, int64_t q_stride, int q_cols, int q_vec, const T* __restrict__ k,
                                                      const T* __restrict__ v, int64_t stride, const T* __restrict__ knorm, float eps, int G,
                                                      int d, int dv, int block_size, const int32_t* __restrict__ slots,
                                                      const int64_t* __restrict__ pos, const float* __restrict__ rot_freq, int rot_dims,
                                                      float* __restrict__ q_row, T* k_cache, T* v_cache, int pool, int finish,
                                                      const int32_t* __restrict__ block_tables, int64_t bt_stride,
                                                      const int32_t* __restrict__ tseq, T* pool_k, T* pool_v) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  float ss = 0.f;
  if (q_vec) {
    for (int c = threadIdx.x * 4; c < q_cols; c += blockDim.x * 4) {
      float x[4];
      ldv<4>(q + t * q_stride + c, x);
      ss += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
    }
  } else {
    for (int c = threadIdx.x; c < q_cols; c += blockDim.x) {
      const float x = ldf(q + t * q_stride + c);
      ss += x * x;
    }
  }
  ss = block_sum(ss, red);
  if (threadIdx.x == 0) q_row[t] = 1.f / sqrtf(ss / (float)q_cols + eps);
  if (!k) return;
  const int64_t slot = slots[t];
  if (slot < 0) return;                             // (the whole workgroup)
  const int nk = G * d;
  const T* kp = k + t * stride;
  ss = 0.f;
  for (int c = threadIdx.x; c < nk; c += blockDim.x) {
    const float x = ldf(kp + c);
    ss += x * x;
  }
  const float r = 1.f / sqrtf(block_sum(ss, red) / (float)nk + eps);
  T* kc = k_cache + slot * nk;
  const float pf = (float)pos[t];
  const int hp = (d + 1) >> 1;                      // pairs of a head
  for (int i = threadIdx.x; i < G * hp; i += blockDim.x) {
    const int g = i / hp, pi = i - g * hp, c = g * d + 2 * pi;
    const bool two = 2 * pi + 1 < d;
    float a = ldf(kp + c) * r * ldf(knorm + c), b = two ? ldf(kp + c + 1) * r * ldf(knorm + c + 1) : 0.f;
    if (2 * pi < rot_dims) {
      float sn, cs;
      sincosf(pf * rot_freq[pi], &sn, &cs);
      const float a2 = a * cs - b * sn;
      b = b * cs + a * sn;
      a = a2;
    }
    stf(kc + c, a);
    if (two) stf(kc + c + 1, b);
  }
  const int64_t page = slot / block_size, off = slot - page * block_size;
  const int nv = G * dv;
  for (int c = threadIdx.x; c < nv; c += blockDim.x) v_cache[(page * nv + c) * block_size + off] = v[t * stride + c];
  if (pool > 0 && finish) {
    const int p = (int)pos[t];
    if ((p + 1) % pool != 0) return;
    __syncthreads();                                // this workgroup's stores above are read back
    for (int half = 0; half < 2; ++half)
      pool_block<T>(half, p, block_tables + (int64_t)tseq[t] * bt_stride, k_cache, v_cache, G, d, dv, block_size, pool, pool_k, pool_v);
  }
}

// Two workgroups (keys, values) per token of the step: the block whose last token it is. Workgroups are dealt to the eight XCDs in
// turn and the tokens that end a block are `pool` apart, so tokens are dealt to workgroups in strides of `pool` (`runs` of them):
// neighbouring workgroups then hold the ends of neighbouring blocks, and not one XCD all of them.
template <typename T>
__global__ __launch_bounds__(256) void pool_blocks_kernel(const T* k_cache, const T* v_cache, int G, int d, int dv, int block_size, int pool,
                                                          int64_t n, unsigned runs,
                                                          const int32_t* __restrict__ slots, const int64_t* __restrict__ pos,
                                                          const int32_t* __restrict__ block_tables, int64_t bt_stride,
                                                          const int32_t* __restrict__ tseq, T* pool_k, T* pool_v) {
  const int64_t t = (int64_t)(blockIdx.x % runs) * pool + blockIdx.x / runs;
  if (t >= n) return;
  const int p = (int)pos[t];
  if ((p + 1) % pool != 0 || slots[t] < 0) return;
  pool_block<T>(blockIdx.y, p, block_tables + (int64_t)tseq[t] * bt_stride, k_cache, v_cache, G, d, dv, block_size, pool, pool_k, pool_v);
}

}  // namespace

void window_attn_extended(const WindowAttnArgs& a, hipStream_t stream) { launch_mfma_sizes<true>(a, stream); }

extern "C" int64_t nvs_pool_rows(int block_size, int pool) { return pool > 0 ? (int64_t)((block_size + 8 * pool - 1) / (8 * pool)) * 8 : 0; }

extern "C" int nvs_qk_rows(const void* q, int64_t q_stride, int q_cols, const void* k, const void* v, int64_t stride, int dtype,
                           const void* knorm, float eps, int G, int d, int dv, int block_size, const int32_t* slots, const int64_t* pos,
                           const float* rot_freq, int rot_dims, int64_t n, float* q_row, void* k_cache, void* v_cache, int pool, int finish,
                           const int32_t* block_tables, int64_t bt_stride, const int32_t* tseq, void* pool_k, void* pool_v, void* stream) {
  NVS_REQUIRE(q && q_row && q_cols > 0 && n >= 0, "nvs_qk_rows: null argument");
  NVS_REQUIRE(!k || (v && knorm && slots && pos && k_cache && v_cache && G > 0 && d > 0 && d <= MAX_HEAD_POOL && dv > 0 && dv <= MAX_HEAD_POOL &&
                     block_size > 0 && rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= d && (rot_dims == 0 || rot_freq)),
              "nvs_qk_rows: G %d d %d dv %d block %d rotation %d", G, d, dv, block_size, rot_dims);
  NVS_REQUIRE(pool >= 0 && (!(k && pool > 0 && finish) || (block_tables && tseq && pool_k && pool_v)), "nvs_qk_rows: pooled blocks (%d) without their tensors", pool);
  if (n == 0) return NVS_OK;
  const int q_vec = q_cols % 4 == 0 && q_stride % 4 == 0 && (uintptr_t)q % 16 == 0;
  NVS_DISPATCH(dtype, qk_rows_kernel<T><<<dim3((unsigned)n), dim3(256), 0, (hipStream_t)stream>>>(
                          (const T*)q, q_stride, q_cols, q_vec, (const T*)k, (const T*)v, stride, (const T*)knorm, eps, G, d, dv, block_size, slots, pos,
                          rot_freq, rot_dims, q_row, (T*)k_cache, (T*)v_cache, pool, finish, block_tables, bt_stride, tseq, (T*)pool_k,
                          (T*)pool_v));
  return nvs_check_launch("nvs_qk_rows");
}

extern "C" int nvs_pool_blocks(const void* k_cache, const void* v_cache, int dtype, int G, int d, int dv, int block_size, int pool,
                               const int32_t* slots, const int64_t* pos, const int32_t* block_tables, int64_t bt_stride, const int32_t* tseq,
                               int64_t n, void* pool_k, void* pool_v, void* stream) {
  NVS_REQUIRE(k_cache && v_cache && slots && pos && block_tables && tseq && pool_k && pool_v && n >= 0, "nvs_pool_blocks: null argument");
  NVS_REQUIRE(G > 0 && d > 0 && dv > 0 && block_size > 0 && pool > 0, "nvs_pool_blocks: G %d d %d dv %d block %d pool %d", G, d, dv, block_size, pool);
  if (n == 0) return NVS_OK;
  const int64_t runs = (n + pool - 1) / pool;
  NVS_REQUIRE(runs * pool < (1ll << 31), "nvs_pool_blocks: step too large");
  NVS_DISPATCH(dtype, pool_blocks_kernel<T><<<dim3((unsigned)(runs * pool), 2), dim3(256), 0, (hipStream_t)stream>>>(
                          (const T*)k_cache, (const T*)v_cache, G, d, dv, block_size, pool, n, (unsigned)runs, slots, pos, block_tables, bt_stride, tseq,
                          (T*)pool_k, (T*)pool_v));
  return nvs_check_launch("nvs_pool_blocks");
}
