// What stands between an attention layer's fused projection and its attention call, in one launch: rotation of the query and key
// heads (either pairing, cos and sin times a factor), a norm per head AFTER the rotation, the query's scale, the paged store of keys
// and values, and optionally values blended with those of an earlier layer. The queries are rewritten in place, so the attention
// call takes them as they are.
//
// A workgroup covers `tile` consecutive token rows (32 in long steps, 1 in decoding) and either a share of their query / key heads or
// 128 value columns (grid.y: parts_qk shares, then the value columns). The angles' cos and sin are taken once per token, pair and
// workgroup into LDS. Values are stored transposed inside a page, so they pass through LDS: a wavefront's lanes run along the
// tile's tokens, which are neighbours in memory.
#include "seq_common.h"

namespace {

typedef __attribute__((ext_vector_type(4))) unsigned int u32x4_t;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;

constexpr int MAX_HEAD = 1024, VCOLS = 128;

struct QkvStoreArgs {
  void* q;
  const void *k, *v, *v0;
  int64_t stride, v0_stride, n;
  const float *freq, *mix;
  const int64_t* pos;
  const int32_t* slots;
  void *k_cache, *v_cache;
  int H, G, d, dv, block_size, rot_dims, halves, unit, tile, parts_qk;
  float mag, eps, q_scale;
};

// 128 value columns (starting at col0 of the G * dv) of the tile's tokens; vt: [VCOLS][tile + 2] elements of LDS
template <typename T, bool ROWS8>
__device__ __forceinline__ void store_values(const QkvStoreArgs& A, int64_t t0, int nt, int col0, T* vt) {
  const int cols = A.G * A.dv, tile = A.tile, ldt = tile + 2, tid = threadIdx.x;
  const T* v = (const T*)A.v;
  const T* v0 = (const T*)A.v0;
  const float lam = v0 ? *A.mix : 0.f;
  for (int u = tid; u < nt * (VCOLS / 8); u += 256) {
    const int tt = u / (VCOLS / 8), lc = (u % (VCOLS / 8)) * 8, c = col0 + lc;
    const T* vp = v + (t0 + tt) * A.stride + c;
    const T* op = v0 ? v0 + (t0 + tt) * A.v0_stride + c : nullptr;
    if constexpr (ROWS8) {                          // (bf16, cols % 8 == 0, 16-byte rows)
      if (c >= cols) continue;
      const bf16x8_t a = *(const bf16x8_t*)vp;
      if (!op) {
#pragma unroll
        for (int e = 0; e < 8; ++e) vt[(lc + e) * ldt + tt] = a[e];
      } else {
        const bf16x8_t b = *(const bf16x8_t*)op;
#pragma unroll
        for (int e = 0; e < 8; ++e) stf(&vt[(lc + e) * ldt + tt], (1.f - lam) * (float)a[e] + lam * (float)b[e]);
      }
    } else {
      for (int e = 0; e < 8 && c + e < cols; ++e) {
        float x = ldf(vp + e);
        if (op) x = (1.f - lam) * x + lam * ldf(op + e);
        stf(&vt[(lc + e) * ldt + tt], x);
      }
    }
  }
  __syncthreads();
  for (int u = tid; u < tile * VCOLS; u += 256) {   // (tile is a power of two)
    const int tt = u & (tile - 1), lc = u / tile, c = col0 + lc;
    if (tt >= nt || c >= cols) continue;
    const int slot = A.slots[t0 + tt];
    if (slot < 0) continue;
    const int page = slot / A.block_size, off = slot - page * A.block_size, g = c / A.dv;
    ((T*)A.v_cache)[(((int64_t)page * A.G + g) * A.dv + (c - g * A.dv)) * A.block_size + off] = vt[lc * ldt + tt];
  }
}

// cos and sin (times mag) of the tile's tokens: cs[tt * half + i], sn behind them
__device__ __forceinline__ void angle_table(const QkvStoreArgs& A, int64_t t0, int nt, float* cs, float* sn) {
  const int half = A.rot_dims >> 1;
  for (int u = threadIdx.x; u < nt * half; u += 256) {
    const int tt = u / half;
    float s, c;
    sincosf((float)A.pos[t0 + tt] * A.freq[u - tt * half], &s, &c);
    cs[u] = c * A.mag;
    sn[u] = s * A.mag;
  }
}

// any type and size: one wavefront per (token, head), columns lane, lane + 64, ...
template <typename T, int CH>
__global__ __launch_bounds__(256) void qkv_store_kernel(const QkvStoreArgs A) {
  extern __shared__ __attribute__((aligned(16))) float qkv_lds[];
  const int64_t t0 = (int64_t)blockIdx.x * A.tile;
  const int nt = (int)(A.n - t0 < A.tile ? A.n - t0 : A.tile);
  if ((int)blockIdx.y >= A.parts_qk) {
    store_values<T, false>(A, t0, nt, ((int)blockIdx.y - A.parts_qk) * VCOLS, (T*)qkv_lds);
    return;
  }
  const int half = A.rot_dims >> 1, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float *cs = qkv_lds, *sn = cs + A.tile * half, *row = sn + A.tile * half + wave * A.d;
  angle_table(A, t0, nt, cs, sn);
  const int heads = A.H + A.G, items = nt * heads;
  for (int base = (int)blockIdx.y * 4; base < items; base += A.parts_qk * 4) {      // (the same number of rounds for all four wavefronts)
    const int it = base + wave;
    const bool live = it < items;
    const int tt = live ? it / heads : 0, hd = live ? it - tt * heads : 0;
    const int64_t t = t0 + tt;
    T* src = hd < A.H ? (T*)A.q + t * A.stride + (int64_t)hd * A.d : (T*)A.k + t * A.stride + (int64_t)(hd - A.H) * A.d;
    __syncthreads();                                // the angles are there; the previous round's rows have been read
    for (int c = lane; live && c < A.d; c += 64) row[c] = ldf(src + c);
    __syncthreads();
    if (!live) continue;
    float val[CH], ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = lane + 64 * i;
      val[i] = 0.f;
      if (c >= A.d) continue;
      val[i] = row[c];
      if (c < A.rot_dims) {
        const bool second = A.halves ? c >= half : c & 1;
        const int pair = A.halves ? (second ? c - half : c) : c >> 1;
        const float other = row[A.halves ? (second ? c - half : c + half) : c ^ 1];
        const float cv = cs[tt * half + pair], sv = sn[tt * half + pair];
        val[i] = second ? val[i] * cv + other * sv : val[i] * cv - other * sv;
      }
      ss += val[i] * val[i];
    }
    float r = hd < A.H ? A.q_scale : 1.f;
    if (A.unit) r *= 1.f / sqrtf(wave_sum(ss) / (float)A.d + A.eps);
    T* dst = src;
    if (hd >= A.H) {
      const int64_t slot = A.slots[t];
      if (slot < 0) continue;
      dst = (T*)A.k_cache + (slot * A.G + (hd - A.H)) * A.d;
    }
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = lane + 64 * i;
      if (c < A.d) stf(dst + c, val[i] * r);
    }
  }
}

// bf16 with d % 8 == 0 (d <= 512) and whole pairs of 8-entry units: L lanes (a power of two) per (token, head), eight entries each in
// one 16-byte access; the partner of a unit in the (i, i + rot_dims / 2) pairing is another lane's unit
__global__ __launch_bounds__(256) void qkv_store_rows8_kernel(const QkvStoreArgs A, int L) {
  extern __shared__ __attribute__((aligned(16))) float qkv_lds[];
  const int64_t t0 = (int64_t)blockIdx.x * A.tile;
  const int nt = (int)(A.n - t0 < A.tile ? A.n - t0 : A.tile);
  if ((int)blockIdx.y >= A.parts_qk) {
    store_values<bf16_t, true>(A, t0, nt, ((int)blockIdx.y - A.parts_qk) * VCOLS, (bf16_t*)qkv_lds);
    return;
  }
  const int half = A.rot_dims >> 1, l = threadIdx.x & (L - 1), groups = 256 / L;
  float *cs = qkv_lds, *sn = cs + A.tile * half;
  angle_table(A, t0, nt, cs, sn);
  __syncthreads();
  const int heads = A.H + A.G, items = nt * heads, c0 = l * 8;
  const bool active = c0 < A.d, turns = c0 < A.rot_dims, second = A.halves && c0 >= half;
  const int partner = A.halves && turns ? (second ? l - (half >> 3) : l + (half >> 3)) : l;
  const int pair0 = A.halves ? (second ? c0 - half : c0) : c0 >> 1;
  for (int it = (int)blockIdx.y * groups + threadIdx.x / L; it < items; it += A.parts_qk * groups) {      // (all lanes of a head together)
    const int tt = it / heads, hd = it - tt * heads;
    const int64_t t = t0 + tt;
    bf16_t* src = hd < A.H ? (bf16_t*)A.q + t * A.stride + (int64_t)hd * A.d : (bf16_t*)A.k + t * A.stride + (int64_t)(hd - A.H) * A.d;
    u32x4_t raw = u32x4_t{0u, 0u, 0u, 0u}, oth = raw;
    if (active) raw = *(const u32x4_t*)(src + c0);
    if (A.halves) {
#pragma unroll
      for (int i = 0; i < 4; ++i) oth[i] = __shfl(raw[i], partner, L);
    }
    const bf16x8_t a8 = __builtin_bit_cast(bf16x8_t, raw), b8 = __builtin_bit_cast(bf16x8_t, oth);
    float val[8], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) val[e] = (float)a8[e];
    if (turns) {
      const float *cp = cs + tt * half + pair0, *sp = sn + tt * half + pair0;
      if (A.halves) {
        float cv[8], sv[8];
        ldp<4>(cp, *(float(*)[4])cv), ldp<4>(cp + 4, *(float(*)[4])(cv + 4));
        ldp<4>(sp, *(float(*)[4])sv), ldp<4>(sp + 4, *(float(*)[4])(sv + 4));
#pragma unroll
        for (int e = 0; e < 8; ++e) val[e] = val[e] * cv[e] + (second ? (float)b8[e] : -(float)b8[e]) * sv[e];
      } else {
        float cv[4], sv[4];
        ldp<4>(cp, cv), ldp<4>(sp, sv);
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          const float u = val[e], w = val[e + 1];
          val[e] = u * cv[e >> 1] - w * sv[e >> 1];
          val[e + 1] = w * cv[e >> 1] + u * sv[e >> 1];
        }
      }
    }
    float r = hd < A.H ? A.q_scale : 1.f;
    if (A.unit) {
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += val[e] * val[e];
      for (int o = L >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      r *= 1.f / sqrtf(ss / (float)A.d + A.eps);
    }
    bf16_t* dst = src;
    bool write = active;
    if (hd >= A.H) {
      const int64_t slot = A.slots[t];
      write = write && slot >= 0;
      dst = (bf16_t*)A.k_cache + (slot * A.G + (hd - A.H)) * A.d;
    }
    if (write) {
      bf16x8_t o8;
#pragma unroll
      for (int e = 0; e < 8; ++e) o8[e] = (bf16_t)(val[e] * r);
      *(bf16x8_t*)(dst + c0) = o8;
    }
  }
}

int ceil_div(int64_t a, int64_t b) { return (int)((a + b - 1) / b); }

}  // namespace

extern "C" int nvs_qkv_store(void* q, const void* k, const void* v, int64_t stride, int dtype, int H, int G, int d, int dv, const int64_t* pos,
                             const float* rot_freq, int rot_dims, int rot_halves, float rot_mag, int unit, float eps, float q_scale,
                             const void* v0, int64_t v0_stride, const float* mix, int block_size, const int32_t* slots, int64_t n,
                             void* k_cache, void* v_cache, void* stream) {
  NVS_REQUIRE(q && k && v && slots && k_cache && v_cache && n >= 0, "nvs_qkv_store: null argument");
  NVS_REQUIRE(H > 0 && G > 0 && d > 0 && d <= MAX_HEAD && dv > 0 && dv <= MAX_HEAD && block_size > 0 && (int64_t)G * dv <= (1 << 22),
              "nvs_qkv_store: H %d G %d d %d dv %d", H, G, d, dv);
  NVS_REQUIRE(stride >= (int64_t)H * d && stride >= (int64_t)G * d && stride >= (int64_t)G * dv, "nvs_qkv_store: rows of %lld", (long long)stride);
  NVS_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= d && (rot_dims == 0 || (pos && rot_freq)), "nvs_qkv_store: rotation of %d of %d dimensions",
              rot_dims, d);
  NVS_REQUIRE(!v0 || (mix && v0_stride >= (int64_t)G * dv), "nvs_qkv_store: values to blend with, but no factor (or rows of %lld)", (long long)v0_stride);
  if (n == 0) return NVS_OK;
  QkvStoreArgs a = {};
  a.q = q, a.k = k, a.v = v, a.v0 = v0, a.stride = stride, a.v0_stride = v0_stride, a.n = n, a.freq = rot_freq, a.mix = mix, a.pos = pos, a.slots = slots;
  a.k_cache = k_cache, a.v_cache = v_cache, a.H = H, a.G = G, a.d = d, a.dv = dv, a.block_size = block_size, a.rot_dims = rot_dims;
  a.halves = rot_halves, a.unit = unit, a.mag = rot_mag, a.eps = eps, a.q_scale = q_scale;
  const int64_t vparts = ceil_div((int64_t)G * dv, VCOLS);
  const uintptr_t al = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)v0 | (uintptr_t)k_cache;
  const bool rows8 = dtype == NVS_BF16 && d % 8 == 0 && d <= 512 && (G * dv) % 8 == 0 && stride % 8 == 0 && v0_stride % 8 == 0 && al % 16 == 0 &&
                     rot_dims % (rot_halves ? 16 : 8) == 0;
  a.tile = d > 256 ? 1 : (n >= 2048 ? 32 : (n >= 512 ? 8 : 1));
  const int tiles = ceil_div(n, a.tile);
  int L = 1;
  while (L * 8 < d) L *= 2;
  const int per_round = rows8 ? 256 / L : 4, rounds = ceil_div((int64_t)a.tile * (H + G), per_round);
  a.parts_qk = ceil_div(rounds, a.tile == 1 ? 1 : 16);
  NVS_REQUIRE(a.parts_qk + vparts <= 65535, "nvs_qkv_store: %d + %d heads of %d", H, G, d);
  const size_t esize = dtype == NVS_BF16 ? 2 : 4, angles = (size_t)a.tile * rot_dims * 4, values = (size_t)VCOLS * (a.tile + 2) * esize;
  const size_t rows = rows8 ? 0 : (size_t)4 * d * 4, lds = angles + rows > values ? angles + rows : values;      // (at most 36 KB)
  const dim3 grid((unsigned)tiles, (unsigned)(a.parts_qk + vparts));
  if (rows8) qkv_store_rows8_kernel<<<grid, dim3(256), lds, (hipStream_t)stream>>>(a, L);
  else if (d <= 256) NVS_DISPATCH(dtype, qkv_store_kernel<T, 4><<<grid, dim3(256), lds, (hipStream_t)stream>>>(a));
  else NVS_DISPATCH(dtype, qkv_store_kernel<T, 16><<<grid, dim3(256), lds, (hipStream_t)stream>>>(a));
  return nvs_check_launch("nvs_qkv_store");
}
