// Residual-stream kernels: embedding + sinusoid, output-side scalar RMS norms with the residual add, the final norm on
// selected rows, xIELU. The residual stream is 32-bit; a copy in the activation type feeds the next matrix product.
#include "seq_common.h"
#include <string.h>

namespace {
thread_local char g_err[512] = "";
}
void nvs_set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_err, sizeof(g_err), fmt, ap);
  va_end(ap);
}
int nvs_check_launch(const char* what) {
  hipError_t e = hipGetLastError();
  if (e != hipSuccess) {
    nvs_set_error("%s: HIP launch failed: %s", what, hipGetErrorString(e));
    return NVS_ELAUNCH;
  }
  return NVS_OK;
}
extern "C" int nvs_abi_version(void) { return 7; }   // 7: rotated and normed queries / keys with blended values in one store, norms on a sublayer's output with a layer scale
extern "C" const char* nvs_last_error(void) { return g_err; }

namespace {

template <typename T>
__global__ void embed_sinusoid_kernel(const T* __restrict__ table, const int64_t* __restrict__ ids, const int64_t* __restrict__ pos,
                                      int width, float scale, float log2_base, float* __restrict__ x, T* __restrict__ xh) {
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const float p = (float)pos[t];
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const int i = c >> 1;
    // base^(-2i/width) in 32-bit; the angle is the product of two 32-bit numbers
    const float inv = exp2f(-(2.f * (float)i / (float)width) * log2_base);
    const float ang = p * inv;
    const float pe = log2_base > 0.f ? ((c & 1) ? cosf(ang) : sinf(ang)) : 0.f;      // (no base: no sinusoid)
    const float v = ldf(table + id * width + c) * scale + pe;
    x[t * width + c] = v;
    if (xh) stf(xh + t * width + c, v);
  }
}

// without a sinusoid: table rows times scale, four columns per access
template <typename T>
__global__ void embed_rows_kernel(const T* __restrict__ table, const int64_t* __restrict__ ids, int width, float scale, float* __restrict__ x,
                                  T* __restrict__ xh) {
  const int64_t t = blockIdx.x;
  const T* row = table + ids[t] * width;
  for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
    float v[4];
    ldv<4>(row + c, v);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= scale;
    stv<4>(x + t * width + c, v);
    if (xh) stv<4>(xh + t * width + c, v);
  }
}

// one workgroup per token row
template <typename T>
__global__ void norm_residual_kernel(const T* __restrict__ m, const T* __restrict__ m2, const T* __restrict__ w1,
                                     const T* __restrict__ w2, const T* __restrict__ g, int width, float eps,
                                     float* __restrict__ x, T* __restrict__ xh) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const float gv = ldf(g);
  float ss = 0.f;
  if (m2 == nullptr) {
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      const float v = ldf(m + t * width + c);
      ss += v * v;
    }
    const float r = rsqrtf(block_sum(ss, red) / (float)width + eps);
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      const float v = x[t * width + c] + gv * (ldf(m + t * width + c) * r);
      x[t * width + c] = v;
      if (xh) stf(xh + t * width + c, v);
    }
    return;
  }
  float s2 = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float a = ldf(m + t * width + c), b = ldf(m2 + t * width + c);
    ss += a * a;
    s2 += b * b;
  }
  const float r1 = rsqrtf(block_sum(ss, red) / (float)width + eps);
  const float r2 = rsqrtf(block_sum(s2, red) / (float)width + eps);
  float s3 = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = 0.5f * (ldf(m + t * width + c) * r1 * ldf(w1 + c) + ldf(m2 + t * width + c) * r2 * ldf(w2 + c));
    s3 += v * v;
  }
  const float r3 = rsqrtf(block_sum(s3, red) / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float mm = 0.5f * (ldf(m + t * width + c) * r1 * ldf(w1 + c) + ldf(m2 + t * width + c) * r2 * ldf(w2 + c));
    const float v = x[t * width + c] + gv * (mm * r3);
    x[t * width + c] = v;
    if (xh) stf(xh + t * width + c, v);
  }
}

template <typename T>
__global__ void scalar_norm_rows_kernel(const float* __restrict__ x, const int32_t* __restrict__ rows, int width,
                                        const T* __restrict__ g, float eps, T* __restrict__ out) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t src = rows ? (int64_t)rows[r] : r;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = x[src * width + c];
    ss += v * v;
  }
  const float k = rsqrtf(block_sum(ss, red) / (float)width + eps) * ldf(g);
  for (int c = threadIdx.x; c < width; c += blockDim.x) stf(out + r * width + c, x[src * width + c] * k);
}

template <typename T>
__global__ void xielu_kernel(const T* __restrict__ in, const T* __restrict__ pq, float beta, int64_t numel, T* __restrict__ out) {
  const float ap = softplusf_(ldf(pq)), aq = beta + softplusf_(ldf(pq + 1));
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < numel; i += (int64_t)gridDim.x * blockDim.x) {
    const float z = ldf(in + i);
    const float v = z > 0.f ? ap * z * z + beta * z : aq * (expm1f(z) - z) + beta * z;
    stf(out + i, v);
  }
}

// Input-side ("pre") norm on the 32-bit residual: x[t] += a_mult * a[t] + b[t] first (either may be absent), then every one of
// `groups` equal parts of the row is divided by its own root mean square — or, with `center`, its mean is taken off first and
// it is divided by its standard deviation (a layer norm without bias) — and the row is multiplied by w. One workgroup per
// row; a group is served by one wavefront (several groups per wavefront, in turn, when there are more groups than wavefronts)
// or by `blockDim / 64 / groups` wavefronts together when there are fewer. With `rows` the kernel only reads:
// out[r] = norm(x[rows[r]]).
template <typename T>
__global__ void add_group_norm_kernel(float* __restrict__ x, const T* __restrict__ a, float a_mult, const float* __restrict__ b,
                                      const int32_t* __restrict__ rows, const T* __restrict__ w, int width, int groups, float eps,
                                      int center, T* __restrict__ out) {
  __shared__ float red[2][16];
  const int64_t r = blockIdx.x;
  const int64_t t = rows ? (int64_t)rows[r] : r;
  const int gsz = width / groups, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  float* xr = x + t * width;
  const int wpg = nw > groups ? nw / groups : 1;    // wavefronts per group (the host makes nw a multiple of groups then)
  const int first = wave / wpg, step = nw / wpg, idx = (wave % wpg) * 64 + lane, stride = wpg * 64;
  for (int g = first; g < groups; g += step) {
    const int c0 = g * gsz;
    float ss = 0.f, sm = 0.f;
    for (int c = idx; c < gsz; c += stride) {
      float v = xr[c0 + c];
      if (a) v += a_mult * ldf(a + t * width + c0 + c);
      if (b) v += b[t * width + c0 + c];
      if (a || b) xr[c0 + c] = v;
      ss += v * v;
      sm += v;
    }
    if (!out) continue;                             // (uniform over the workgroup)
    float mean = 0.f;
    if (center) {                                   // the mean first, then the squared deviations (this thread wrote xr[c0 + c])
      sm = wave_sum(sm);
      if (wpg > 1) {
        if (lane == 0) red[1][wave] = sm;
        __syncthreads();
        sm = 0.f;
        for (int i = 0; i < wpg; ++i) sm += red[1][first * wpg + i];
      }
      mean = sm / (float)gsz;
      ss = 0.f;
      for (int c = idx; c < gsz; c += stride) {
        const float dv = xr[c0 + c] - mean;
        ss += dv * dv;
      }
    }
    ss = wave_sum(ss);
    if (wpg > 1) {                                  // (then every wavefront runs this loop exactly once)
      if (lane == 0) red[0][wave] = ss;
      __syncthreads();
      ss = 0.f;
      for (int i = 0; i < wpg; ++i) ss += red[0][first * wpg + i];
    }
    const float k = w ? 1.f / sqrtf(ss / (float)gsz + eps) : 1.f;      // (no weights: the sum itself)
    for (int c = idx; c < gsz; c += stride) stf(out + r * width + c0 + c, (xr[c0 + c] - mean) * k * (w ? ldf(w + c0 + c) : 1.f));
  }
}

// The same for ONE group without centering, four columns per access: the row stays in registers between the two passes
// (PER accesses per thread).
template <typename T, int PER>
__global__ __launch_bounds__(256) void add_norm_row_kernel(float* __restrict__ x, const T* __restrict__ a, float a_mult, const float* __restrict__ b,
                                                           const int32_t* __restrict__ rows, const T* __restrict__ w, int width, float eps,
                                                           T* __restrict__ out) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t t = rows ? (int64_t)rows[r] : r;
  float* xr = x + t * width;
  float v[PER][4];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    ldv<4>(xr + c, v[i]);
    float u[4];
    if (a) {
      ldv<4>(a + t * width + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] += a_mult * u[e];
    }
    if (b) {
      ldv<4>(b + t * width + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] += u[e];
    }
    if (a || b) stv<4>(xr + c, v[i]);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += v[i][e] * v[i][e];
  }
  if (!out) return;
  const float k = w ? 1.f / sqrtf(block_sum(ss, red) / (float)width + eps) : 1.f;      // (no weights: the sum itself)
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    if (w) {
      float u[4];
      ldv<4>(w + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] *= k * u[e];
    }
    stv<4>(out + r * width + c, v[i]);
  }
}

// Norms on BOTH sides of a sublayer, on the 32-bit residual: the sublayer's output y[t] = a_mult * a[t] + a2_mult * a2[t] (a2 may be
// absent) is RMS-normed with the weight (w_off + wa) and added, x[t] += rms(y[t]) * (w_off + wa); then the NEXT sublayer's input
// out[t] = rms(x[t]) * (w_off + w). Either half may be absent (a NULL / out NULL). w_off = 1 serves weights stored as their distance
// from one. With `rows` the kernel only reads: out[r] = norm(x[rows[r]]), or with a as well out[r] = norm(x[rows[r]] + its branch), the
// sum going to `sum`[r] instead of x. One workgroup per row; all sums in 32-bit.
template <typename T>
__global__ void sandwich_norm_kernel(float* __restrict__ x, const T* __restrict__ a, float a_mult, const T* __restrict__ a2, float a2_mult,
                                     const T* __restrict__ wa, const int32_t* __restrict__ rows, const T* __restrict__ w, float w_off,
                                     int width, float eps, float* __restrict__ sum, T* __restrict__ out) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t t = rows ? (int64_t)rows[r] : r;
  const float* xi = x + t * width;
  float* xr = rows && a ? sum + r * width : x + t * width;
  if (a) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      float y = a_mult * ldf(a + t * width + c);
      if (a2) y += a2_mult * ldf(a2 + t * width + c);
      ss += y * y;
    }
    const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      float y = a_mult * ldf(a + t * width + c);
      if (a2) y += a2_mult * ldf(a2 + t * width + c);
      xr[c] = xi[c] + y * k * (w_off + ldf(wa + c));
    }
  }
  if (!out) return;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {     // (every thread reads back what it wrote itself)
    const float v = xr[c];
    ss += v * v;
  }
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) stf(out + r * width + c, xr[c] * k * (w_off + ldf(w + c)));
}

// The same with the rows in registers, four columns per access (PER accesses per thread).
template <typename T, int PER>
__global__ __launch_bounds__(256) void sandwich_row_kernel(float* __restrict__ x, const T* __restrict__ a, float a_mult, const T* __restrict__ a2,
                                                           float a2_mult, const T* __restrict__ wa, const int32_t* __restrict__ rows,
                                                           const T* __restrict__ w, float w_off, int width, float eps, T* __restrict__ out) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t t = rows ? (int64_t)rows[r] : r;
  float v[PER][4];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c < width) ldv<4>(x + t * width + c, v[i]);
  }
  if (a) {
    float y[PER][4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = (i * blockDim.x + threadIdx.x) * 4;
      if (c >= width) continue;
      ldv<4>(a + t * width + c, y[i]);
      float u[4] = {0.f, 0.f, 0.f, 0.f};
      if (a2) ldv<4>(a2 + t * width + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        y[i][e] = a_mult * y[i][e] + a2_mult * u[e];
        ss += y[i][e] * y[i][e];
      }
    }
    const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = (i * blockDim.x + threadIdx.x) * 4;
      if (c >= width) continue;
      float u[4];
      ldv<4>(wa + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] += y[i][e] * k * (w_off + u[e]);
      if (!rows) stv<4>(x + t * width + c, v[i]);   // (selected rows are only read)
    }
  }
  if (!out) return;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    if ((int)(i * blockDim.x + threadIdx.x) * 4 >= width) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += v[i][e] * v[i][e];
  }
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    float u[4];
    ldv<4>(w + c, u);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] *= k * (w_off + u[e]);
    stv<4>(out + r * width + c, v[i]);
  }
}

// A sublayer whose OUTPUT is normed, with a layer scale: y[t] = a[t] + sum_k wts[t, k] rows[pair_row[t, k]] (either part may be absent: the
// output of a product, or a token's chosen experts beside a shared one), x[t] += rms(y[t]) * w * ls, and the new row once more in the
// activation type for the next sublayer's products. One workgroup per row, y and x in registers (PER accesses of four columns per thread).
template <typename T, int PER>
__global__ __launch_bounds__(256) void branch_norm_row_kernel(float* __restrict__ x, const T* __restrict__ a, const T* __restrict__ rows, int64_t ldr,
                                                              const int32_t* __restrict__ pair_row, const float* __restrict__ wts, int top,
                                                              const T* __restrict__ w, const T* __restrict__ ls, int width, float eps,
                                                              T* __restrict__ out) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  float v[PER][4], y[PER][4];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) y[i][e] = 0.f;
    if (c >= width) continue;
    ldv<4>(x + t * width + c, v[i]);
    if (a) ldv<4>(a + t * width + c, y[i]);
  }
  for (int k = 0; k < top; ++k) {
    const int r = pair_row[t * top + k];
    if (r < 0) continue;                            // (uniform over the workgroup)
    const float p = wts[t * top + k];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = (i * blockDim.x + threadIdx.x) * 4;
      if (c >= width) continue;
      float u[4];
      ldv<4>(rows + (int64_t)r * ldr + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[i][e] += p * u[e];
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += y[i][e] * y[i][e];
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    float g[4], s[4] = {1.f, 1.f, 1.f, 1.f};
    ldv<4>(w + c, g);
    if (ls) ldv<4>(ls + c, s);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] += y[i][e] * k * g[e] * s[e];
    stv<4>(x + t * width + c, v[i]);
    if (out) stv<4>(out + t * width + c, v[i]);
  }
}

// the same for any width: y in LDS (every thread only touches its own columns)
template <typename T>
__global__ __launch_bounds__(256) void branch_norm_kernel(float* __restrict__ x, const T* __restrict__ a, const T* __restrict__ rows, int64_t ldr,
                                                          const int32_t* __restrict__ pair_row, const float* __restrict__ wts, int top,
                                                          const T* __restrict__ w, const T* __restrict__ ls, int width, float eps,
                                                          T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float branch_lds[];
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float y = a ? ldf(a + t * width + c) : 0.f;
    for (int k = 0; k < top; ++k) {
      const int r = pair_row[t * top + k];
      if (r >= 0) y += wts[t * top + k] * ldf(rows + (int64_t)r * ldr + c);
    }
    branch_lds[c] = y;
    ss += y * y;
  }
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = x[t * width + c] + branch_lds[c] * k * ldf(w + c) * (ls ? ldf(ls + c) : 1.f);
    x[t * width + c] = v;
    if (out) stf(out + t * width + c, v);
  }
}

// x[t] = rms(table[ids[t]]) * w: one workgroup per token, the row in registers (PER accesses of four columns per thread)
template <typename T, int PER>
__global__ __launch_bounds__(256) void embed_norm_row_kernel(const T* __restrict__ table, const int64_t* __restrict__ ids, int width,
                                                             const T* __restrict__ w, float eps, float* __restrict__ x) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const T* row = table + ids[t] * width;
  float v[PER][4], ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    ldv<4>(row + c, v[i]);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += v[i][e] * v[i][e];
  }
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * 4;
    if (c >= width) continue;
    float u[4];
    ldv<4>(w + c, u);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] *= k * u[e];
    stv<4>(x + t * width + c, v[i]);
  }
}

// the same for any width
template <typename T>
__global__ void embed_norm_kernel(const T* __restrict__ table, const int64_t* __restrict__ ids, int width, const T* __restrict__ w, float eps,
                                  float* __restrict__ x) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const T* row = table + ids[t] * width;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = ldf(row + c);
    ss += v * v;
  }
  const float k = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) x[t * width + c] = ldf(row + c) * k * ldf(w + c);
}

// The add, the norm and the blend with the previous token's normed row, in one pass. A workgroup takes `rows` consecutive token
// rows and keeps the last normed row in LDS; ahead of its first row it norms the row before it once more (x is not updated in
// place, so that row can still be read). The workgroup that holds a portion's FIRST row also norms its LAST one: it alone
// reads and replaces the sequence's state. VEC columns per thread and access (4 where width allows).
template <typename T, int VEC>
__global__ __launch_bounds__(256) void shift_norm_kernel(const float* __restrict__ x, const T* __restrict__ a, const T* __restrict__ wa,
                                                         const T* __restrict__ w, const T* __restrict__ mu, const int32_t* __restrict__ cu_q,
                                                         const int32_t* __restrict__ ctx0, const int32_t* __restrict__ slot,
                                                         const int32_t* __restrict__ tseq, int64_t n, int width, float eps, int rows,
                                                         float* __restrict__ state, float* __restrict__ x_out, T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float shift_lds[];      // yrow | hrow: every thread only touches its own columns
  __shared__ float red[16];
  float *yrow = shift_lds, *hrow = shift_lds + width;
  const int tid = threadIdx.x, step = blockDim.x * VEC;
  // y of row t into yrow (and x_out); returns 1 / rms(y)
  auto load = [&](int64_t t, bool store) {
    float ka = 1.f;
    if (a && wa) {
      float ss = 0.f;
      for (int c = tid * VEC; c < width; c += step) {
        float v[VEC];
        ldv<VEC>(a + t * width + c, v);
#pragma unroll
        for (int i = 0; i < VEC; ++i) ss += v[i] * v[i];
      }
      ka = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
    }
    float ss = 0.f;
    for (int c = tid * VEC; c < width; c += step) {
      float y[VEC];
      ldv<VEC>(x + t * width + c, y);
      if (a) {
        float v[VEC], g[VEC];
        ldv<VEC>(a + t * width + c, v);
        if (wa) ldv<VEC>(wa + c, g);
#pragma unroll
        for (int i = 0; i < VEC; ++i) y[i] += wa ? v[i] * ka * g[i] : v[i];
        if (store) stv<VEC>(x_out + t * width + c, y);
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) ss += y[i] * y[i], yrow[c + i] = y[i];
    }
    return 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  };
  const int64_t t0 = (int64_t)blockIdx.x * rows, t1 = t0 + rows < n ? t0 + rows : n;
  for (int64_t t = t0; t < t1; ++t) {
    const int s = tseq[t];
    const int64_t q0 = cu_q[s], q1 = cu_q[s + 1];
    float* st = state + (int64_t)slot[s] * width;
    const bool head = t == q0, fresh = ctx0[s] == 0;
    if (!head && t == t0) {                         // the row before the workgroup's first one
      const float k = load(t - 1, false);
      for (int c = tid * VEC; c < width; c += step) {
        float g[VEC];
        ldv<VEC>(w + c, g);
#pragma unroll
        for (int i = 0; i < VEC; ++i) hrow[c + i] = yrow[c + i] * k * g[i];
      }
    }
    const float k = load(t, true);
    for (int c = tid * VEC; c < width; c += step) {
      float g[VEC], m[VEC], o[VEC];
      ldv<VEC>(w + c, g);
      ldv<VEC>(mu + c, m);
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        const float h = yrow[c + i] * k * g[i];
        const float before = head ? (fresh ? 0.f : st[c + i]) : hrow[c + i];
        o[i] = h + (before - h) * m[i];
        hrow[c + i] = h;
        if (head && q1 - q0 == 1) st[c + i] = h;
      }
      stv<VEC>(out + t * width + c, o);
    }
    if (head && q1 - q0 > 1) {                      // (hrow stays: the next row of this workgroup blends with it)
      const float kl = load(q1 - 1, false);
      for (int c = tid * VEC; c < width; c += step) {
        float g[VEC];
        ldv<VEC>(w + c, g);
#pragma unroll
        for (int i = 0; i < VEC; ++i) st[c + i] = yrow[c + i] * kl * g[i];
      }
    }
  }
}

template <typename T>
__global__ void gated_lookup_kernel(const T* __restrict__ z, int64_t z_stride, const T* __restrict__ table, int64_t table_stride, int64_t col0,
                                    const int64_t* __restrict__ ids, int dim, int64_t total, T* __restrict__ out) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / dim;
    const int c = (int)(i - t * dim);
    stf(out + i, gelu_tanhf_(ldf(z + t * z_stride + c)) * ldf(table + ids[t] * table_stride + col0 + c));
  }
}

// logits <- cap * tanh(logits * scale / cap) (cap <= 0: logits * scale), 32-bit out
template <typename T>
__global__ void scale_softcap_kernel(const T* __restrict__ in, float scale, float cap, int64_t numel, float* __restrict__ out) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < numel; i += (int64_t)gridDim.x * blockDim.x) {
    const float z = ldf(in + i) * scale;
    out[i] = cap > 0.f ? cap * tanhf(z / cap) : z;
  }
}

// row kernels: threads and accesses of four columns per thread (1, 2, 4 or 8; 0: the row does not fit or is not aligned for them)
int row_plan(int width, uintptr_t al, int* threads) {
  if (width % 4 || width > 8192 || al % 16) return 0;
  *threads = width >= 1024 ? 256 : ((width + 255) / 256) * 64;
  const int per = (width + 1023) / 1024;
  return per <= 1 ? 1 : (per <= 2 ? 2 : (per <= 4 ? 4 : 8));
}
#define NVS_ROW_CASES(per, NAME) \
  switch (per) {                 \
    case 1: NAME(1); break;      \
    case 2: NAME(2); break;      \
    case 4: NAME(4); break;      \
    default: NAME(8);            \
  }

int threads_for(int width) { return width >= 1024 ? 256 : (width >= 256 ? 128 : 64); }

}  // namespace

extern "C" int nvs_embed_sinusoid(const void* table, int dtype, const int64_t* ids, const int64_t* pos, int64_t n, int width,
                                  float scale, float base, float* x, void* xh, void* stream) {
  NVS_REQUIRE(table && ids && pos && x && n >= 0 && width > 0 && (base > 1.f || base == 0.f), "nvs_embed_sinusoid: bad argument");
  if (n == 0) return NVS_OK;
  if (base == 0.f && width % 4 == 0 && ((uintptr_t)table | (uintptr_t)x | (uintptr_t)xh) % 16 == 0) {
    NVS_DISPATCH(dtype, embed_rows_kernel<T><<<dim3((unsigned)n), dim3(width >= 1024 ? 256 : ((width + 255) / 256) * 64), 0, (hipStream_t)stream>>>(
                            (const T*)table, ids, width, scale, x, (T*)xh));
    return nvs_check_launch("nvs_embed_sinusoid (rows)");
  }
  NVS_DISPATCH(dtype, embed_sinusoid_kernel<T><<<dim3((unsigned)n), dim3(threads_for(width)), 0, (hipStream_t)stream>>>(
                          (const T*)table, ids, pos, width, scale, base > 1.f ? log2f(base) : 0.f, x, (T*)xh));
  return nvs_check_launch("nvs_embed_sinusoid");
}

extern "C" int nvs_norm_residual(const void* m, const void* m2, const void* w1, const void* w2, const void* g, int dtype,
                                 int64_t n, int width, float eps, float* x, void* xh, void* stream) {
  NVS_REQUIRE(m && g && x && n >= 0 && width > 0, "nvs_norm_residual: bad argument");
  NVS_REQUIRE(!m2 || (w1 && w2), "nvs_norm_residual: two branches need both channel weights");
  if (n == 0) return NVS_OK;
  NVS_DISPATCH(dtype, norm_residual_kernel<T><<<dim3((unsigned)n), dim3(threads_for(width)), 0, (hipStream_t)stream>>>(
                          (const T*)m, (const T*)m2, (const T*)w1, (const T*)w2, (const T*)g, width, eps, x, (T*)xh));
  return nvs_check_launch("nvs_norm_residual");
}

extern "C" int nvs_scalar_norm_rows(const float* x, const int32_t* rows, int64_t nrows, int width, const void* g, int dtype,
                                    float eps, void* out, void* stream) {
  NVS_REQUIRE(x && g && out && nrows >= 0 && width > 0, "nvs_scalar_norm_rows: bad argument");
  if (nrows == 0) return NVS_OK;
  NVS_DISPATCH(dtype, scalar_norm_rows_kernel<T><<<dim3((unsigned)nrows), dim3(threads_for(width)), 0, (hipStream_t)stream>>>(
                          x, rows, width, (const T*)g, eps, (T*)out));
  return nvs_check_launch("nvs_scalar_norm_rows");
}

extern "C" int nvs_xielu(const void* in, const void* pq, float beta, int dtype, int64_t numel, void* out, void* stream) {
  NVS_REQUIRE(in && pq && out && numel >= 0, "nvs_xielu: bad argument");
  if (numel == 0) return NVS_OK;
  const int64_t blocks = (numel + 255) / 256;
  NVS_DISPATCH(dtype, xielu_kernel<T><<<dim3((unsigned)(blocks > 65536 ? 65536 : blocks)), dim3(256), 0, (hipStream_t)stream>>>(
                          (const T*)in, (const T*)pq, beta, numel, (T*)out));
  return nvs_check_launch("nvs_xielu");
}

extern "C" int nvs_add_group_norm(float* x, const void* a, float a_mult, const float* b, const int32_t* rows, int64_t nrows, const void* w,
                                  int dtype, int width, int groups, float eps, int center, void* out, void* stream) {
  NVS_REQUIRE(x && nrows >= 0 && width > 0 && groups > 0 && width % groups == 0 && (!out || w || !center), "nvs_add_group_norm: width %d groups %d",
              width, groups);
  NVS_REQUIRE(!rows || (!a && !b), "nvs_add_group_norm: selected rows are only read");
  if (nrows == 0) return NVS_OK;
  const uintptr_t al = (uintptr_t)x | (uintptr_t)a | (uintptr_t)b | (uintptr_t)w | (uintptr_t)out;
  int row_threads = 0;
  const int per = groups == 1 && !center ? row_plan(width, al, &row_threads) : 0;
  if (per) {
#define NVS_ROW(PER)                                                                                                           \
  NVS_DISPATCH(dtype, add_norm_row_kernel<T, PER><<<dim3((unsigned)nrows), dim3(row_threads), 0, (hipStream_t)stream>>>(         \
                          x, (const T*)a, a_mult, b, rows, (const T*)w, width, eps, (T*)out))
    NVS_ROW_CASES(per, NVS_ROW)
#undef NVS_ROW
    return nvs_check_launch("nvs_add_group_norm (one group)");
  }
  // a wavefront per group, four groups at a time; wide groups that are fewer than four are shared by 4 / groups wavefronts
  int threads = 64 * (groups < 4 ? groups : 4);
  if (groups < 4 && 4 % groups == 0 && width / groups >= 512) threads = 256;
  NVS_DISPATCH(dtype, add_group_norm_kernel<T><<<dim3((unsigned)nrows), dim3(threads), 0, (hipStream_t)stream>>>(
                          x, (const T*)a, a_mult, b, rows, (const T*)w, width, groups, eps, center, (T*)out));
  return nvs_check_launch("nvs_add_group_norm");
}

extern "C" int nvs_sandwich_norm(float* x, const void* a, float a_mult, const void* a2, float a2_mult, const void* wa, const int32_t* rows,
                                 int64_t nrows, const void* w, float w_off, int dtype, int width, float eps, float* sum, void* out,
                                 void* stream) {
  NVS_REQUIRE(x && nrows >= 0 && width > 0 && (a || out) && (!a || wa) && (!a2 || a) && (!out || w), "nvs_sandwich_norm: bad argument (width %d)", width);
  NVS_REQUIRE(!(rows && a) || sum, "nvs_sandwich_norm: selected rows are only read, their sums need a place of their own");
  if (nrows == 0) return NVS_OK;
  int row_threads = 0;
  const int per = row_plan(width, (uintptr_t)x | (uintptr_t)a | (uintptr_t)a2 | (uintptr_t)wa | (uintptr_t)w | (uintptr_t)out, &row_threads);
  if (per) {
#define NVS_ROW(PER)                                                                                                           \
  NVS_DISPATCH(dtype, sandwich_row_kernel<T, PER><<<dim3((unsigned)nrows), dim3(row_threads), 0, (hipStream_t)stream>>>(         \
                          x, (const T*)a, a_mult, (const T*)a2, a2_mult, (const T*)wa, rows, (const T*)w, w_off, width, eps, (T*)out))
    NVS_ROW_CASES(per, NVS_ROW)
#undef NVS_ROW
    return nvs_check_launch("nvs_sandwich_norm (rows in registers)");
  }
  NVS_DISPATCH(dtype, sandwich_norm_kernel<T><<<dim3((unsigned)nrows), dim3(threads_for(width)), 0, (hipStream_t)stream>>>(
                          x, (const T*)a, a_mult, (const T*)a2, a2_mult, (const T*)wa, rows, (const T*)w, w_off, width, eps, sum, (T*)out));
  return nvs_check_launch("nvs_sandwich_norm");
}

extern "C" int nvs_branch_norm(float* x, const void* a, const void* rows, int64_t ldr, const int32_t* pair_row, const float* wts, int top, int dtype,
                               int64_t n, const void* w, const void* ls, int width, float eps, void* out, void* stream) {
  NVS_REQUIRE(x && w && n >= 0 && width > 0 && width <= 16384 && top >= 0 && (a || top > 0), "nvs_branch_norm: bad argument (width %d, %d choices)", width, top);
  NVS_REQUIRE(top == 0 || (rows && pair_row && wts && ldr >= width), "nvs_branch_norm: %d choices without their rows", top);
  if (n == 0) return NVS_OK;
  int row_threads = 0;
  const uintptr_t al = (uintptr_t)x | (uintptr_t)a | (uintptr_t)(top ? rows : nullptr) | (uintptr_t)w | (uintptr_t)ls | (uintptr_t)out;
  const int per = top == 0 || ldr % 4 == 0 ? row_plan(width, al, &row_threads) : 0;
  if (per) {
#define NVS_ROW(PER)                                                                                                             \
  NVS_DISPATCH(dtype, branch_norm_row_kernel<T, PER><<<dim3((unsigned)n), dim3(row_threads), 0, (hipStream_t)stream>>>(            \
                          x, (const T*)a, (const T*)rows, ldr, pair_row, wts, top, (const T*)w, (const T*)ls, width, eps, (T*)out))
    NVS_ROW_CASES(per, NVS_ROW)
#undef NVS_ROW
    return nvs_check_launch("nvs_branch_norm (rows in registers)");
  }
  const size_t lds = (size_t)width * sizeof(float);      // (at most 64 KB)
  NVS_DISPATCH(dtype, {
    if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)branch_norm_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    branch_norm_kernel<T><<<dim3((unsigned)n), dim3(threads_for(width)), lds, (hipStream_t)stream>>>(
        x, (const T*)a, (const T*)rows, ldr, pair_row, wts, top, (const T*)w, (const T*)ls, width, eps, (T*)out);
  });
  return nvs_check_launch("nvs_branch_norm");
}

extern "C" int nvs_scale_softcap(const void* in, int dtype, float scale, float cap, int64_t numel, float* out, void* stream) {
  NVS_REQUIRE(in && out && numel >= 0, "nvs_scale_softcap: bad argument");
  if (numel == 0) return NVS_OK;
  const int64_t blocks = (numel + 255) / 256;
  NVS_DISPATCH(dtype, scale_softcap_kernel<T><<<dim3((unsigned)(blocks > 65536 ? 65536 : blocks)), dim3(256), 0, (hipStream_t)stream>>>(
                          (const T*)in, scale, cap, numel, out));
  return nvs_check_launch("nvs_scale_softcap");
}

extern "C" int nvs_embed_norm(const void* table, int dtype, const int64_t* ids, int64_t n, int width, const void* w, float eps, float* x,
                              void* stream) {
  NVS_REQUIRE(table && ids && w && x && n >= 0 && width > 0, "nvs_embed_norm: bad argument (width %d)", width);
  if (n == 0) return NVS_OK;
  int row_threads = 0;
  const int per = row_plan(width, (uintptr_t)table | (uintptr_t)w | (uintptr_t)x, &row_threads);
  if (per) {
#define NVS_ROW(PER)                                                                                                        \
  NVS_DISPATCH(dtype, embed_norm_row_kernel<T, PER><<<dim3((unsigned)n), dim3(row_threads), 0, (hipStream_t)stream>>>(        \
                          (const T*)table, ids, width, (const T*)w, eps, x))
    NVS_ROW_CASES(per, NVS_ROW)
#undef NVS_ROW
    return nvs_check_launch("nvs_embed_norm (rows in registers)");
  }
  NVS_DISPATCH(dtype, embed_norm_kernel<T><<<dim3((unsigned)n), dim3(threads_for(width)), 0, (hipStream_t)stream>>>(
                          (const T*)table, ids, width, (const T*)w, eps, x));
  return nvs_check_launch("nvs_embed_norm");
}

extern "C" int nvs_shift_norm(const float* x, const void* a, const void* wa, const void* w, const void* mu, int dtype, const int32_t* cu_q,
                              const int32_t* ctx0, const int32_t* slot, const int32_t* tseq, int nseq, int64_t n, int width, float eps,
                              float* state, float* x_out, void* out, void* stream) {
  NVS_REQUIRE(x && w && mu && cu_q && ctx0 && slot && tseq && state && out && n >= 0 && nseq >= 0, "nvs_shift_norm: null argument");
  NVS_REQUIRE(width > 0 && width <= 16384, "nvs_shift_norm: width %d (up to 16384)", width);
  NVS_REQUIRE(!wa || a, "nvs_shift_norm: a norm weight without a branch");
  NVS_REQUIRE(!a || (x_out && x_out != x), "nvs_shift_norm: the sum needs a tensor of its own (rows of x are read twice)");
  if (n == 0 || nseq == 0) return NVS_OK;
  const int rows = n >= 8192 ? 8 : (n >= 2048 ? 4 : 1);       // (a workgroup reads one row more than it writes)
  const size_t lds = 2 * (size_t)width * sizeof(float);
  const dim3 grid((unsigned)((n + rows - 1) / rows)), block(width >= 1024 ? 256 : (width >= 256 ? 128 : 64));
#define NVS_SHIFT(VEC)                                                                                                                  \
  NVS_DISPATCH(dtype, {                                                                                                                 \
    if (lds > 48 * 1024)                                                                                                                \
      (void)hipFuncSetAttribute((const void*)shift_norm_kernel<T, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);           \
    shift_norm_kernel<T, VEC><<<grid, block, lds, (hipStream_t)stream>>>(x, (const T*)a, (const T*)wa, (const T*)w, (const T*)mu, cu_q, ctx0, \
                                                                         slot, tseq, n, width, eps, rows, state, x_out, (T*)out);        \
  })
  if (width % 4 == 0) {
    NVS_SHIFT(4);
  } else {
    NVS_SHIFT(1);
  }
#undef NVS_SHIFT
  return nvs_check_launch("nvs_shift_norm");
}

extern "C" int nvs_gated_lookup(const void* z, int64_t z_stride, const void* table, int64_t table_stride, int64_t col0, int dtype,
                                const int64_t* ids, int dim, int64_t n, void* out, void* stream) {
  NVS_REQUIRE(z && table && ids && out && dim > 0 && n >= 0 && z_stride >= dim && col0 >= 0 && table_stride >= col0 + dim,
              "nvs_gated_lookup: %d columns from %lld on of rows of %lld", dim, (long long)col0, (long long)table_stride);
  if (n == 0) return NVS_OK;
  int64_t blocks = (n * dim + 255) / 256;
  if (blocks > 65535) blocks = 65535;
  NVS_DISPATCH(dtype, gated_lookup_kernel<T><<<dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream>>>(
                          (const T*)z, z_stride, (const T*)table, table_stride, col0, ids, dim, n * dim, (T*)out));
  return nvs_check_launch("nvs_gated_lookup");
}
