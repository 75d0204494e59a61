// RMS normalisation. The residual stream is fp32 in both precisions; the fused
// kernel adds the pending branch output to it and normalises the sum in one
// pass over the row:
//   r = resid + delta          (fp32, stored back as the new residual)
//   y = r * (1/sqrt(mean(r^2) + eps)) * w
// Reference formulas: kernels/normalization.cu:36-63 (norm) and
// kernels/fused_add_rmsnorm.cu:47-81 (add + norm, two outputs).
#include "common.h"
#include "hector_kernels.h"

template <typename TD, typename TO>
__global__ void add_rmsnorm_kernel(float* __restrict__ resid, const TD* __restrict__ delta,
                                   const void* __restrict__ w, int w_dtype, TO* __restrict__ out,
                                   int D, float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  float* r = resid + row * (int64_t)D;
  float ss = 0.f;
  if (delta != nullptr) {
    const TD* d = delta + row * (int64_t)D;
    for (int i = threadIdx.x; i < D; i += blockDim.x) {
      const float v = r[i] + to_float(d[i]);
      r[i] = v;
      ss += v * v;
    }
  } else {
    for (int i = threadIdx.x; i < D; i += blockDim.x) {
      const float v = r[i];
      ss += v * v;
    }
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)D + eps);
  if (out == nullptr) return;
  TO* o = out + row * (int64_t)D;
  // each thread re-reads exactly the elements it wrote above
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    o[i] = from_float<TO>(r[i] * inv * load_param(w, i, w_dtype));
  }
}

// The same with a row of at most NORM_EPT * blockDim.x elements kept in registers:
// every load of the row is issued before the reduction, nothing is read twice.
#define NORM_EPT 8
template <typename TD, typename TO>
__global__ void add_rmsnorm_reg_kernel(float* __restrict__ resid, const TD* __restrict__ delta,
                                       const void* __restrict__ w, int w_dtype,
                                       TO* __restrict__ out, int D, float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  float* r = resid + row * (int64_t)D;
  const TD* d = delta ? delta + row * (int64_t)D : nullptr;
  float v[NORM_EPT], g[NORM_EPT];
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < NORM_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    v[e] = 0.f;
    g[e] = 0.f;
    if (i < D) {
      v[e] = r[i];
      if (d) v[e] += to_float(d[i]);
      if (out) g[e] = load_param(w, i, w_dtype);
    }
  }
#pragma unroll
  for (int e = 0; e < NORM_EPT; ++e) ss += v[e] * v[e];
  if (d) {
#pragma unroll
    for (int e = 0; e < NORM_EPT; ++e) {
      const int i = threadIdx.x + e * blockDim.x;
      if (i < D) r[i] = v[e];
    }
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)D + eps);
  if (out == nullptr) return;
  TO* o = out + row * (int64_t)D;
#pragma unroll
  for (int e = 0; e < NORM_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    if (i < D) o[i] = from_float<TO>(v[e] * inv * g[e]);
  }
}

// The same with four neighbouring elements a thread and access (16 bytes of the fp32
// residual, 8 of a bf16 tensor): a row of at most 4 * NORM_VEC * blockDim.x elements, D a
// multiple of 4. Tall inputs (prompt steps) are bound by memory traffic; with one element an
// access the kernel reached 3.4 TB/s.
#define NORM_VEC 4
__device__ __forceinline__ void load4(const float* p, float* v) {
  const float4 x = *reinterpret_cast<const float4*>(p);
  v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
}
__device__ __forceinline__ void load4(const bf16_t* p, float* v) {
  const uint2 x = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
  v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
}
__device__ __forceinline__ void store4(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void store4(bf16_t* p, const float* v) {
  uint2 x;
  x.x = (uint32_t)float_to_bf16_bits(v[0]) | ((uint32_t)float_to_bf16_bits(v[1]) << 16);
  x.y = (uint32_t)float_to_bf16_bits(v[2]) | ((uint32_t)float_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = x;
}

template <typename TD, typename TO, typename TW>
__global__ void add_rmsnorm_vec_kernel(float* __restrict__ resid, const TD* __restrict__ delta,
                                       const TW* __restrict__ w, TO* __restrict__ out, int D,
                                       float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  float* r = resid + row * (int64_t)D;
  const TD* d = delta ? delta + row * (int64_t)D : nullptr;
  float v[NORM_VEC][4], g[NORM_VEC][4], a[NORM_VEC][4];
  float ss = 0.f;
  // the loads stand in no per-thread branch (a group beyond the row reads the row's last four
  // elements and counts as zeros), so they all go out before the first is waited for
#pragma unroll
  for (int e = 0; e < NORM_VEC; ++e) load4(r + min(4 * (int)(threadIdx.x + e * blockDim.x), D - 4), v[e]);
  if (d) {
#pragma unroll
    for (int e = 0; e < NORM_VEC; ++e) load4(d + min(4 * (int)(threadIdx.x + e * blockDim.x), D - 4), a[e]);
  }
  if (out) {
#pragma unroll
    for (int e = 0; e < NORM_VEC; ++e) load4(w + min(4 * (int)(threadIdx.x + e * blockDim.x), D - 4), g[e]);
  }
#pragma unroll
  for (int e = 0; e < NORM_VEC; ++e) {
    const bool in = 4 * (int)(threadIdx.x + e * blockDim.x) < D;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[e][j] = in ? v[e][j] + (d ? a[e][j] : 0.f) : 0.f;
      g[e][j] = (in && out) ? g[e][j] : 0.f;
    }
  }
#pragma unroll
  for (int e = 0; e < NORM_VEC; ++e)
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += v[e][j] * v[e][j];
  if (d) {
#pragma unroll
    for (int e = 0; e < NORM_VEC; ++e) {
      const int i = 4 * (threadIdx.x + e * blockDim.x);
      if (i < D) store4(r + i, v[e]);
    }
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)D + eps);
  if (out == nullptr) return;
  TO* o = out + row * (int64_t)D;
#pragma unroll
  for (int e = 0; e < NORM_VEC; ++e) {
    const int i = 4 * (threadIdx.x + e * blockDim.x);
    if (i < D) {
      float y[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = v[e][j] * inv * g[e][j];
      store4(o + i, y);
    }
  }
}

template <typename TD, typename TO>
static void launch_add_rmsnorm_vec(float* resid, const void* delta, const void* w, int w_dtype,
                                   void* out, int rows, int D, float eps, hipStream_t s) {
  int threads = 64;
  while (threads < 512 && 4 * NORM_VEC * threads < D) threads <<= 1;
  while (threads > 64 && 4 * (threads >> 1) >= D) threads >>= 1;
  if (w_dtype == HE_BF16)
    add_rmsnorm_vec_kernel<TD, TO, bf16_t><<<rows, threads, 0, s>>>(
        resid, (const TD*)delta, (const bf16_t*)w, (TO*)out, D, eps);
  else
    add_rmsnorm_vec_kernel<TD, TO, float><<<rows, threads, 0, s>>>(
        resid, (const TD*)delta, (const float*)w, (TO*)out, D, eps);
}

static int norm_threads(int D) { return D >= 2048 ? 512 : (D >= 512 ? 256 : (D >= 128 ? 128 : 64)); }

extern "C" int he_add_rmsnorm(void* resid_f32, const void* delta, const void* weight, void* out,
                              int rows, int D, float eps, int act_dtype, int w_dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0, "he_add_rmsnorm: bad sizes rows=%d D=%d", rows, D);
  HE_REQUIRE(w_dtype == HE_F32 || w_dtype == HE_BF16, "he_add_rmsnorm: bad weight dtype");
  HE_REQUIRE(act_dtype == HE_F32 || act_dtype == HE_BF16, "he_add_rmsnorm: unknown dtype %d",
             act_dtype);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int threads = norm_threads(D);
  if ((D & 3) == 0 && D <= 4 * NORM_VEC * 512 &&
             ((((uintptr_t)resid_f32) | ((uintptr_t)delta) | ((uintptr_t)weight) | ((uintptr_t)out)) & 15) == 0) {
    if (act_dtype == HE_BF16)
      launch_add_rmsnorm_vec<bf16_t, bf16_t>((float*)resid_f32, delta, weight, w_dtype, out, rows, D, eps, s);
    else
      launch_add_rmsnorm_vec<float, float>((float*)resid_f32, delta, weight, w_dtype, out, rows, D, eps, s);
  } else if (D <= NORM_EPT * threads) {
    if (act_dtype == HE_BF16)
      add_rmsnorm_reg_kernel<bf16_t, bf16_t><<<rows, threads, 0, s>>>(
          (float*)resid_f32, (const bf16_t*)delta, weight, w_dtype, (bf16_t*)out, D, eps);
    else
      add_rmsnorm_reg_kernel<float, float><<<rows, threads, 0, s>>>(
          (float*)resid_f32, (const float*)delta, weight, w_dtype, (float*)out, D, eps);
  } else if (act_dtype == HE_BF16) {
    add_rmsnorm_kernel<bf16_t, bf16_t><<<rows, threads, 0, s>>>(
        (float*)resid_f32, (const bf16_t*)delta, weight, w_dtype, (bf16_t*)out, D, eps);
  } else {
    add_rmsnorm_kernel<float, float><<<rows, threads, 0, s>>>(
        (float*)resid_f32, (const float*)delta, weight, w_dtype, (float*)out, D, eps);
  }
  return he_check_launch("he_add_rmsnorm");
}

// Plain row-wise RMS norm of an activation tensor with a row stride (for
// normalising slices such as per-head vectors): x viewed as [rows, D].
template <typename T>
__global__ void rmsnorm_rows_kernel(T* __restrict__ out, const T* __restrict__ x,
                                    const void* __restrict__ w, int w_dtype, int D,
                                    int64_t x_stride, int64_t out_stride, float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const T* xi = x + row * x_stride;
  float ss = 0.f;
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    const float v = to_float(xi[i]);
    ss += v * v;
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)D + eps);
  T* o = out + row * out_stride;
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    const float g = w ? load_param(w, i, w_dtype) : 1.f;
    o[i] = from_float<T>(to_float(xi[i]) * inv * g);
  }
}

extern "C" int he_rmsnorm_rows(void* out, const void* x, const void* weight, int rows, int D,
                               int64_t x_stride, int64_t out_stride, float eps, int dtype,
                               int w_dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0 && x_stride >= D && out_stride >= D,
             "he_rmsnorm_rows: bad sizes rows=%d D=%d", rows, D);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int threads = norm_threads(D);
  if (dtype == HE_BF16)
    rmsnorm_rows_kernel<bf16_t><<<rows, threads, 0, s>>>((bf16_t*)out, (const bf16_t*)x, weight,
                                                         w_dtype, D, x_stride, out_stride, eps);
  else if (dtype == HE_F32)
    rmsnorm_rows_kernel<float><<<rows, threads, 0, s>>>((float*)out, (const float*)x, weight,
                                                        w_dtype, D, x_stride, out_stride, eps);
  else
    HE_REQUIRE(false, "he_rmsnorm_rows: unknown dtype %d", dtype);
  return he_check_launch("he_rmsnorm_rows");
}

// Two stretches of the same rows, each by a root mean square and a gain of its own, in place and in one launch:
// columns [0, D1) with w1 and columns [col2, col2 + D2) with w2 (q and k as they lie behind one product).
template <typename T>
__global__ void rmsnorm_row_pair_kernel(T* __restrict__ x, const void* __restrict__ w1, int D1,
                                        const void* __restrict__ w2, int D2, int col2, int w_dtype,
                                        int64_t stride, float eps) {
  __shared__ float scratch[16];
  const bool second = blockIdx.y == 1;
  const int D = second ? D2 : D1;
  const void* w = second ? w2 : w1;
  T* xi = x + blockIdx.x * stride + (second ? col2 : 0);
  float ss = 0.f;
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    const float v = to_float(xi[i]);
    ss += v * v;
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)D + eps);
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    const float g = w ? load_param(w, i, w_dtype) : 1.f;
    xi[i] = from_float<T>(to_float(xi[i]) * inv * g);
  }
}

extern "C" int he_rmsnorm_row_pair(void* x, const void* w1, int D1, const void* w2, int D2, int col2, int rows,
                                   int64_t stride, float eps, int dtype, int w_dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && D1 > 0 && D2 > 0 && col2 >= D1 && stride >= (int64_t)col2 + D2,
             "he_rmsnorm_row_pair: bad sizes rows=%d D1=%d D2=%d col2=%d", rows, D1, D2, col2);
  HE_REQUIRE(dtype == HE_BF16 || dtype == HE_F32, "he_rmsnorm_row_pair: unknown dtype %d", dtype);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int threads = norm_threads(D1 > D2 ? D1 : D2);
  if (dtype == HE_BF16)
    rmsnorm_row_pair_kernel<bf16_t><<<dim3(rows, 2), threads, 0, s>>>((bf16_t*)x, w1, D1, w2, D2, col2, w_dtype, stride, eps);
  else
    rmsnorm_row_pair_kernel<float><<<dim3(rows, 2), threads, 0, s>>>((float*)x, w1, D1, w2, D2, col2, w_dtype, stride, eps);
  return he_check_launch("he_rmsnorm_row_pair");
}

// Rows x = r * gain whose scale is still owed: out = x / sqrt(sum(partials of the row) / D + eps).
// The partial sums of squares (one per workgroup of the product that made the rows) are
// added as that product's consumers add them: lanes over strided partials, then the wavefront.
// x_pieces: x lies piece-major, 16-byte pieces [D / 8][rows][8]; out is row-major either way.
__global__ void scale_rows_kernel(uint16_t* __restrict__ out, const uint16_t* __restrict__ x,
                                  const float* __restrict__ partials, int count, int D, float eps,
                                  int x_pieces) {
  __shared__ float inv_s;
  const int64_t row = blockIdx.x;
  if (threadIdx.x < 64) {
    float part = 0.f;
    for (int i = threadIdx.x; i < count; i += 64) part += partials[row * count + i];
    const float total = wave_sum(part);
    if (threadIdx.x == 0) inv_s = 1.0f / sqrtf(total / (float)D + eps);
  }
  __syncthreads();
  const float inv = inv_s;
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    const int64_t at = x_pieces ? ((int64_t)(i >> 3) * gridDim.x + row) * 8 + (i & 7) : row * D + i;
    out[row * D + i] = float_to_bf16_bits(bf16_bits_to_float(x[at]) * inv);
  }
}

extern "C" int he_scale_rows_bf16(void* out, const void* x, const void* partials, int count,
                                  int rows, int D, float eps, int x_pieces, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0 && count > 0, "he_scale_rows_bf16: bad sizes rows=%d D=%d count=%d",
             rows, D, count);
  HE_REQUIRE(!x_pieces || D % 8 == 0, "he_scale_rows_bf16: piece-major rows of width %d, not a multiple of 8", D);
  if (rows == 0) return 0;
  scale_rows_kernel<<<rows, norm_threads(D), 0, (hipStream_t)stream>>>(
      (uint16_t*)out, (const uint16_t*)x, (const float*)partials, count, D, eps, x_pieces);
  return he_check_launch("he_scale_rows_bf16");
}

// Dynamic Tanh in place of a norm: y = tanh(alpha * r) * w + b with a scalar alpha and vectors w, b;
// it reduces nothing over the row, so it is one pass over the elements. As the fused add + RMS norm
// above, it first adds the pending branch output: r = resid + delta_scale * delta (fp32, stored
// back as the new residual). alpha is read from device memory (a stored tensor of one element).
template <typename TD, typename TO, typename TW, int VEC>
__global__ void add_dyt_kernel(float* __restrict__ resid, const TD* __restrict__ delta, const TD* __restrict__ delta2,
                               float delta_scale,
                               const TW* __restrict__ w, const TW* __restrict__ b,
                               const TW* __restrict__ alpha_p, TO* __restrict__ out, int64_t n, int D) {
  const float alpha = to_float(alpha_p[0]);
  int64_t i = (blockIdx.x * (int64_t)blockDim.x + threadIdx.x) * VEC;
  const int64_t stride = (int64_t)gridDim.x * blockDim.x * VEC;
  for (; i < n; i += stride) {
    const int c = (int)(i % D);
    float v[VEC], a[VEC], a2[VEC], g[VEC], s[VEC];
    if constexpr (VEC == 4) {
      load4(resid + i, v);
      if (delta) load4(delta + i, a);
      if (delta2) load4(delta2 + i, a2);
      if (out) {
        load4(w + c, g);
        load4(b + c, s);
      }
    } else {
      v[0] = resid[i];
      if (delta) a[0] = to_float(delta[i]);
      if (delta2) a2[0] = to_float(delta2[i]);
      if (out) g[0] = to_float(w[c]), s[0] = to_float(b[c]);
    }
    if (delta) {
      if (delta2) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) a[j] += a2[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = fmaf(delta_scale, a[j], v[j]);
      if constexpr (VEC == 4) store4(resid + i, v);
      else resid[i] = v[0];
    }
    if (out) {
      float y[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) y[j] = fmaf(tanhf(alpha * v[j]), g[j], s[j]);
      if constexpr (VEC == 4) store4(out + i, y);
      else out[i] = from_float<TO>(y[0]);
    }
  }
}

template <typename TD, typename TO, typename TW>
static void launch_add_dyt(float* resid, const void* delta, const void* delta2, float delta_scale, const void* w, const void* b,
                           const void* alpha, void* out, int rows, int D, hipStream_t s) {
  const int64_t n = (int64_t)rows * D;
  const bool vec = (D & 3) == 0 && ((((uintptr_t)resid) | ((uintptr_t)delta) | ((uintptr_t)delta2) | ((uintptr_t)w) | ((uintptr_t)b) |
                                     ((uintptr_t)out)) & 15) == 0;
  const int64_t items = vec ? n / 4 : n;
  int64_t blocks = (items + 255) / 256;
  if (blocks > 65535 * 16) blocks = 65535 * 16;
  if (vec)
    add_dyt_kernel<TD, TO, TW, 4><<<(unsigned)blocks, 256, 0, s>>>(resid, (const TD*)delta, (const TD*)delta2, delta_scale, (const TW*)w,
                                                                   (const TW*)b, (const TW*)alpha, (TO*)out, n, D);
  else
    add_dyt_kernel<TD, TO, TW, 1><<<(unsigned)blocks, 256, 0, s>>>(resid, (const TD*)delta, (const TD*)delta2, delta_scale, (const TW*)w,
                                                                   (const TW*)b, (const TW*)alpha, (TO*)out, n, D);
}

extern "C" int he_add_dyt(void* resid_f32, const void* delta, const void* delta2, float delta_scale, const void* weight,
                          const void* bias, const void* alpha, void* out, int rows, int D, int act_dtype,
                          int w_dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0, "he_add_dyt: bad sizes rows=%d D=%d", rows, D);
  HE_REQUIRE(w_dtype == HE_F32 || w_dtype == HE_BF16, "he_add_dyt: bad parameter dtype");
  HE_REQUIRE(act_dtype == HE_F32 || act_dtype == HE_BF16, "he_add_dyt: unknown dtype %d", act_dtype);
  HE_REQUIRE(out == nullptr || (weight && bias && alpha), "he_add_dyt: weight, bias and alpha are needed");
  HE_REQUIRE(delta2 == nullptr || delta != nullptr, "he_add_dyt: delta2 goes with delta");
  if (rows == 0 || (delta == nullptr && out == nullptr)) return 0;
  hipStream_t s = (hipStream_t)stream;
  float* r = (float*)resid_f32;
#define DYT(TD, TO, TW) launch_add_dyt<TD, TO, TW>(r, delta, delta2, delta_scale, weight, bias, alpha, out, rows, D, s)
  if (act_dtype == HE_BF16) {
    if (w_dtype == HE_BF16) DYT(bf16_t, bf16_t, bf16_t);
    else DYT(bf16_t, bf16_t, float);
  } else {
    if (w_dtype == HE_BF16) DYT(float, float, bf16_t);
    else DYT(float, float, float);
  }
#undef DYT
  return he_check_launch("he_add_dyt");
}

// ---- a branch output that is normed before it joins the stream ("sandwich" norms) ----------------
// resid[r, :] += post_w ? delta[r, :] / sqrt(mean(delta[r, :]^2) + post_eps) * post_w : delta[r, :]
// and then, when out is given,
// out[r, :] = next_w ? resid[r, :] / sqrt(mean(resid[r, :]^2) + next_eps) * next_w : resid[r, :]
// (the rows the next reader wants: normed, or the stream itself in the activation dtype). One workgroup a
// row; the row's new residual values stay in registers between the two sums (D up to PN_EPT * threads).
#define PN_EPT 16
template <typename TD, typename TO>
__global__ void add_normed_kernel(float* __restrict__ resid, const TD* __restrict__ delta, const void* __restrict__ post_w,
                                  float post_eps, const void* __restrict__ next_w, float next_eps, int w_dtype,
                                  TO* __restrict__ out, int D) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  float* r = resid + row * D;
  const TD* d = delta ? delta + row * D : nullptr;
  float x[PN_EPT];
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    x[e] = (d && i < D) ? to_float(d[i]) : 0.f;
    ss = fmaf(x[e], x[e], ss);
  }
  float inv = 1.f;
  if (d && post_w) inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)D + post_eps);
  ss = 0.f;
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    if (i < D) {
      const float g = (d && post_w) ? load_param(post_w, i, w_dtype) : 1.f;
      x[e] = d ? r[i] + x[e] * inv * g : r[i];
      if (d) r[i] = x[e];
    } else {
      x[e] = 0.f;
    }
    ss = fmaf(x[e], x[e], ss);
  }
  if (out == nullptr) return;
  float inv2 = 1.f;
  if (next_w) inv2 = 1.0f / sqrtf(block_sum(ss, scratch) / (float)D + next_eps);
  TO* o = out + row * D;
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    if (i < D) o[i] = from_float<TO>(next_w ? x[e] * inv2 * load_param(next_w, i, w_dtype) : x[e]);
  }
}

// Four neighbouring elements at once (16 bytes of fp32, 8 of bf16)
__device__ __forceinline__ void pn_load4(float* dst, const float* p) {
  const float4 v = *reinterpret_cast<const float4*>(p);
  dst[0] = v.x; dst[1] = v.y; dst[2] = v.z; dst[3] = v.w;
}
__device__ __forceinline__ void pn_load4(float* dst, const bf16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  dst[0] = __uint_as_float(v.x << 16); dst[1] = __uint_as_float(v.x & 0xffff0000u);
  dst[2] = __uint_as_float(v.y << 16); dst[3] = __uint_as_float(v.y & 0xffff0000u);
}
__device__ __forceinline__ void pn_store4(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void pn_store4(bf16_t* p, const float* v) {
  uint2 o;
  o.x = (uint32_t)float_to_bf16_bits(v[0]) | ((uint32_t)float_to_bf16_bits(v[1]) << 16);
  o.y = (uint32_t)float_to_bf16_bits(v[2]) | ((uint32_t)float_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = o;
}

// Four gains at once, whichever dtype they are stored in
__device__ __forceinline__ void pn_param4(float* dst, const void* p, int64_t i, int dtype) {
  if (dtype == HE_BF16) pn_load4(dst, (const bf16_t*)p + i);
  else pn_load4(dst, (const float*)p + i);
}

// Two sums over a block at once (`scratch`: 32 floats), as block_sum forms one
__device__ __forceinline__ void pn_block_sum2(float& a, float& b, float* scratch) {
  const int lane = threadIdx.x & (HE_WAVE - 1), wave = threadIdx.x >> 6, waves = (blockDim.x + HE_WAVE - 1) >> 6;
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if (lane == 0) {
    scratch[wave] = a;
    scratch[16 + wave] = b;
  }
  __syncthreads();
  a = b = 0.f;
  for (int w = 0; w < waves; ++w) {
    a += scratch[w];
    b += scratch[16 + w];
  }
}

// A branch output (a), or with PAIR two of them side by side, each normed over the row with a gain of its own,
//   x = scale * (a / rms(a) * w_a + b / rms(b) * w_b),   rms(z) = sqrt(mean(z^2) + pair_eps),
// on the way above: normed by post_w, added to resid, and out = what the next reader wants of it; without resid
// (PAIR), out = x. Everything in fp32 registers between the loads and out; a thread holds EPT elements in runs of four
// neighbours, and every load of the row, the gains' too, is under way before the first sum is formed. Widths are
// multiples of 4, everything begins on 16 bytes (gains in bf16: 8).
template <typename TD, typename TO, int EPT, bool PAIR>
__global__ __launch_bounds__(1024) void normed_sum_kernel(
    float* __restrict__ resid, const TD* __restrict__ a, const TD* __restrict__ b, const void* __restrict__ w_a,
    const void* __restrict__ w_b, int pair_dtype, float pair_eps, float scale, const void* __restrict__ post_w, float post_eps,
    const void* __restrict__ next_w, float next_eps, int w_dtype, TO* __restrict__ out, int D) {
  __shared__ float scratch[32], scratch_b[16];
  const int64_t row = blockIdx.x;
  float x[EPT], z[PAIR ? EPT : 4], ga[PAIR ? EPT : 4], gb[PAIR ? EPT : 4], r[EPT], gp[EPT], gn[EPT];
#pragma unroll
  for (int e = 0; e < EPT; e += 4) {
    const int i = (threadIdx.x + (e / 4) * blockDim.x) * 4;
    const int at = i < D ? i : 0;        // (lanes past the row read its start and drop it)
    pn_load4(x + e, a + row * D + at);
    if constexpr (PAIR) {
      pn_load4(z + e, b + row * D + at);
      pn_param4(ga + e, w_a, at, pair_dtype);
      pn_param4(gb + e, w_b, at, pair_dtype);
    }
    if (resid) pn_load4(r + e, resid + row * D + at);
    if (post_w) pn_param4(gp + e, post_w, at, w_dtype);
    if (next_w) pn_param4(gn + e, next_w, at, w_dtype);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      x[e + u] = i < D ? x[e + u] : 0.f;
      if constexpr (PAIR) z[e + u] = i < D ? z[e + u] : 0.f;
    }
  }
  float ss = 0.f;
  if constexpr (PAIR) {
    float sb = 0.f;
#pragma unroll
    for (int e = 0; e < EPT; ++e) {
      ss = fmaf(x[e], x[e], ss);
      sb = fmaf(z[e], z[e], sb);
    }
    pn_block_sum2(ss, sb, scratch);
    const float ia = scale / sqrtf(ss / (float)D + pair_eps), ib = scale / sqrtf(sb / (float)D + pair_eps);
#pragma unroll
    for (int e = 0; e < EPT; ++e) x[e] = x[e] * ia * ga[e] + z[e] * ib * gb[e];
  }
  if (resid) {
    float inv = 1.f;
    if (post_w) {
      ss = 0.f;
#pragma unroll
      for (int e = 0; e < EPT; ++e) ss = fmaf(x[e], x[e], ss);
      inv = 1.f / sqrtf(block_sum(ss, scratch_b) / (float)D + post_eps);
    }
    ss = 0.f;
#pragma unroll
    for (int e = 0; e < EPT; e += 4) {
      const int i = (threadIdx.x + (e / 4) * blockDim.x) * 4;
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        x[e + u] = i < D ? r[e + u] + x[e + u] * inv * (post_w ? gp[e + u] : 1.f) : 0.f;
        ss = fmaf(x[e + u], x[e + u], ss);
      }
      if (i < D) pn_store4(resid + row * D + i, x + e);
    }
    if (out == nullptr) return;
    if (next_w) {
      const float inv2 = 1.f / sqrtf(block_sum(ss, scratch_b) / (float)D + next_eps);
#pragma unroll
      for (int e = 0; e < EPT; ++e) x[e] *= inv2 * gn[e];
    }
  }
#pragma unroll
  for (int e = 0; e < EPT; e += 4) {
    const int i = (threadIdx.x + (e / 4) * blockDim.x) * 4;
    if (i < D) pn_store4(out + row * D + i, x + e);
  }
}

static bool pn_vec_gain(const void* w, int dtype) { return ((uintptr_t)w & (dtype == HE_BF16 ? 7 : 15)) == 0; }

// Elements a thread of normed_sum_kernel holds at this width and block
static int pn_ept(int D, int threads) { return D <= 4 * threads ? 4 : D <= 8 * threads ? 8 : 16; }

#define NORMED_SUM(TD, TO, PAIR)                                                                                        \
  do {                                                                                                                  \
    const int ept = pn_ept(D, threads);                                                                                 \
    if (ept == 4) NORMED_SUM_EPT(TD, TO, 4, PAIR);                                                                      \
    else if (ept == 8) NORMED_SUM_EPT(TD, TO, 8, PAIR);                                                                 \
    else NORMED_SUM_EPT(TD, TO, 16, PAIR);                                                                              \
  } while (0)

// The same sum of two branches for any width and address, element by element
template <typename TD, typename TO>
__global__ void add_normed_pair_kernel(float* __restrict__ resid, const TD* __restrict__ a, const TD* __restrict__ b,
                                       const void* __restrict__ w_a, const void* __restrict__ w_b, int pair_dtype,
                                       float pair_eps, float scale, const void* __restrict__ post_w, float post_eps,
                                       const void* __restrict__ next_w, float next_eps, int w_dtype,
                                       TO* __restrict__ out, int D) {
  __shared__ float scratch[32];
  const int64_t row = blockIdx.x;
  float x[PN_EPT], z[PN_EPT];
  float ss = 0.f, sb = 0.f;
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    x[e] = i < D ? to_float(a[row * D + i]) : 0.f;
    z[e] = i < D ? to_float(b[row * D + i]) : 0.f;
    ss = fmaf(x[e], x[e], ss);
    sb = fmaf(z[e], z[e], sb);
  }
  pn_block_sum2(ss, sb, scratch);
  const float ia = scale / sqrtf(ss / (float)D + pair_eps), ib = scale / sqrtf(sb / (float)D + pair_eps);
  ss = 0.f;
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    if (i < D) x[e] = x[e] * ia * load_param(w_a, i, pair_dtype) + z[e] * ib * load_param(w_b, i, pair_dtype);
    ss = fmaf(x[e], x[e], ss);
  }
  float inv2 = 1.f;
  if (resid) {
    const float inv = post_w ? 1.f / sqrtf(block_sum(ss, scratch) / (float)D + post_eps) : 1.f;
    ss = 0.f;
#pragma unroll
    for (int e = 0; e < PN_EPT; ++e) {
      const int i = threadIdx.x + e * blockDim.x;
      if (i < D) {
        x[e] = resid[row * D + i] + x[e] * inv * (post_w ? load_param(post_w, i, w_dtype) : 1.f);
        resid[row * D + i] = x[e];
      }
      ss = fmaf(x[e], x[e], ss);
    }
    if (out == nullptr) return;
    if (next_w) inv2 = 1.f / sqrtf(block_sum(ss, scratch) / (float)D + next_eps);
  }
#pragma unroll
  for (int e = 0; e < PN_EPT; ++e) {
    const int i = threadIdx.x + e * blockDim.x;
    if (i < D) out[row * D + i] = from_float<TO>(resid && next_w ? x[e] * inv2 * load_param(next_w, i, w_dtype) : x[e]);
  }
}

extern "C" int he_add_normed_pair(void* resid_f32, const void* a, const void* b, int delta_dtype, const void* w_a,
                                  const void* w_b, int pair_dtype, float pair_eps, float scale, const void* post_weight,
                                  float post_eps, const void* next_weight, float next_eps, int w_dtype, void* out,
                                  int out_dtype, int rows, int D, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0, "he_add_normed_pair: bad sizes rows=%d D=%d", rows, D);
  HE_REQUIRE(D <= PN_EPT * 1024, "he_add_normed_pair: width %d above %d", D, PN_EPT * 1024);
  HE_REQUIRE(a && b && w_a && w_b && (resid_f32 || out), "he_add_normed_pair: a branch, a gain or the result is missing");
  HE_REQUIRE((w_dtype == HE_F32 || w_dtype == HE_BF16) && (pair_dtype == HE_F32 || pair_dtype == HE_BF16),
             "he_add_normed_pair: bad weight dtype");
  HE_REQUIRE((delta_dtype == HE_F32 || delta_dtype == HE_BF16) && (out_dtype == HE_F32 || out_dtype == HE_BF16),
             "he_add_normed_pair: unknown dtype");
  if (rows == 0) return 0;
  int threads = 64;
  while (threads < 1024 && PN_EPT * threads < D) threads <<= 1;
  while (threads < 256 && 4 * threads < D) threads <<= 1;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = D % 4 == 0 && (((uintptr_t)resid_f32 | (uintptr_t)a | (uintptr_t)b | (uintptr_t)out) & 15) == 0 &&
                   pn_vec_gain(w_a, pair_dtype) && pn_vec_gain(w_b, pair_dtype) && pn_vec_gain(post_weight, w_dtype) &&
                   pn_vec_gain(next_weight, w_dtype);
#define NORMED_SUM_EPT(TD, TO, EPT, PAIR)                                                                               \
  normed_sum_kernel<TD, TO, EPT, PAIR><<<rows, threads, 0, s>>>((float*)resid_f32, (const TD*)a, (const TD*)b, w_a, w_b,  \
                                                                pair_dtype, pair_eps, scale, post_weight, post_eps,      \
                                                                next_weight, next_eps, w_dtype, (TO*)out, D)
#define PN_PAIR(TD, TO)                                                                                                 \
  do {                                                                                                                  \
    if (vec) NORMED_SUM(TD, TO, true);                                                                                  \
    else add_normed_pair_kernel<TD, TO><<<rows, threads, 0, s>>>((float*)resid_f32, (const TD*)a, (const TD*)b, w_a, w_b, \
                                                                 pair_dtype, pair_eps, scale, post_weight, post_eps,     \
                                                                 next_weight, next_eps, w_dtype, (TO*)out, D);           \
  } while (0)
  const bool db = delta_dtype == HE_BF16, ob = out_dtype == HE_BF16;
  if (db && ob) PN_PAIR(bf16_t, bf16_t);
  else if (db) PN_PAIR(bf16_t, float);
  else if (ob) PN_PAIR(float, bf16_t);
  else PN_PAIR(float, float);
#undef PN_PAIR
#undef NORMED_SUM_EPT
  return he_check_launch("he_add_normed_pair");
}

extern "C" int he_add_normed(void* resid_f32, const void* delta, int delta_dtype, const void* post_weight, float post_eps,
                             const void* next_weight, float next_eps, int w_dtype, void* out, int out_dtype, int rows,
                             int D, void* stream) {
  HE_REQUIRE(rows >= 0 && D > 0, "he_add_normed: bad sizes rows=%d D=%d", rows, D);
  HE_REQUIRE(D <= PN_EPT * 1024, "he_add_normed: width %d above %d", D, PN_EPT * 1024);
  HE_REQUIRE(w_dtype == HE_F32 || w_dtype == HE_BF16, "he_add_normed: bad weight dtype");
  HE_REQUIRE((delta == nullptr || delta_dtype == HE_F32 || delta_dtype == HE_BF16) &&
                 (out == nullptr || out_dtype == HE_F32 || out_dtype == HE_BF16),
             "he_add_normed: unknown dtype");
  if (rows == 0) return 0;
  int threads = 64;
  while (threads < 1024 && PN_EPT * threads < D) threads <<= 1;
  while (threads < 256 && 4 * threads < D) threads <<= 1;
  hipStream_t s = (hipStream_t)stream;
#define PN_LAUNCH(TD, TO)                                                                                        \
  add_normed_kernel<TD, TO><<<rows, threads, 0, s>>>((float*)resid_f32, (const TD*)delta, post_weight, post_eps, \
                                                     next_weight, next_eps, w_dtype, (TO*)out, D)
  const bool db = delta != nullptr && delta_dtype == HE_BF16, ob = out != nullptr && out_dtype == HE_BF16;
  if (D % 4 == 0 && (((uintptr_t)resid_f32 | (uintptr_t)delta | (uintptr_t)out) & 15) == 0 && delta != nullptr &&
      pn_vec_gain(post_weight, w_dtype) && pn_vec_gain(next_weight, w_dtype)) {
#define NORMED_SUM_EPT(TD, TO, EPT, PAIR)                                                                            \
  normed_sum_kernel<TD, TO, EPT, PAIR><<<rows, threads, 0, s>>>((float*)resid_f32, (const TD*)delta, (const TD*)nullptr, \
                                                                nullptr, nullptr, HE_F32, 0.f, 1.f, post_weight,      \
                                                                post_eps, next_weight, next_eps, w_dtype, (TO*)out, D)
    if (db && ob) NORMED_SUM(bf16_t, bf16_t, false);
    else if (db) NORMED_SUM(bf16_t, float, false);
    else if (ob) NORMED_SUM(float, bf16_t, false);
    else NORMED_SUM(float, float, false);
#undef NORMED_SUM_EPT
    return he_check_launch("he_add_normed");
  }
  if (db && ob) PN_LAUNCH(bf16_t, bf16_t);
  else if (db) PN_LAUNCH(bf16_t, float);
  else if (ob) PN_LAUNCH(float, bf16_t);
  else PN_LAUNCH(float, float);
#undef PN_LAUNCH
  return he_check_launch("he_add_normed");
}
