// One pass over the projected q/k/v rows of a step: add the projection bias,
// rotate q and k by each row's own position, write q out densely and scatter
// k and v into the paged cache at (slot, position). It replaces the reference's
// add_bias, rope and kv_cache_update launches (kernels/elementwise.cu:307-323,
// kernels/attention.cu:516-558, kernels/attention.cu:1067-1097).
//
// Rotation (half-split pairing): for i < r/2, a = pos * inv_freq[i],
//   y[i]       = x[i] * cos a - x[i + r/2] * sin a
//   y[i + r/2] = x[i] * sin a + x[i + r/2] * cos a
// and dims >= r pass through. All of it in fp32.
//
// Two options of the same pass: every head of q and of k divided by its own root mean square (no gain; a rotation does
// not change it, so it is formed from the rows as they come), and values mixed with an earlier layer's values of the
// same row, v <- (1 - lambda) v + lambda v_first.
#include "cache_layout.h"
#include "hector_kernels.h"

#define ROPE_MAX_HALF 256

// A query's temperature: q at position p is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1), so
// that queries far into a sequence are sharper (every <= 0: none). In fp32.
__device__ __forceinline__ float he_query_temperature(int pos, float coef, int every) {
  return every > 0 ? fmaf(coef, logf((float)((pos + 1) / every + 1)), 1.f) : 1.f;
}

// unit: heads of q and k are divided by sqrt(mean(x^2) + eps). v_first: rows of another layer's values as they were
// projected (KVH * vd_in of them, no bias, `stride` elements apart) that join the own ones with the factor lambda.
struct RopeExtras {
  int unit;
  float eps;
  const void* v_first;
  int64_t v_stride;
  float v_lambda;
};

// hd: the head size of q_out and of the cache pages; hd_in <= hd, vd_in <= hd: the head sizes of the
// projected q/k and v rows (a mixer whose keys and values differ in width keeps both in pages of
// the wider one: q_out's dims from hd_in on are written as zeros, those of the pages are never
// written and stay the zeros the pools were made with). interleaved: the pair of frequency i is
// (2i, 2i + 1) instead of (i, i + r/2). mscale multiplies cos and sin (1: a pure rotation).
template <typename T, typename TI>
__global__ void qkv_rope_cache_kernel(
    T* __restrict__ q_out, T* __restrict__ kpool, T* __restrict__ vpool,
    const TI* __restrict__ q_in, const TI* __restrict__ k_in, const TI* __restrict__ v_in,
    int64_t in_stride, const void* __restrict__ q_bias, const void* __restrict__ k_bias,
    const void* __restrict__ v_bias, int bias_dtype, const int32_t* __restrict__ positions,
    const int32_t* __restrict__ row_seq, const int32_t* __restrict__ seq_slot,
    const int32_t* __restrict__ page_table, int max_blocks, int num_pages,
    const float* __restrict__ inv_freq, int rotary_dim, int H, int KVH, int hd, int hd_in, int vd_in,
    int interleaved, float mscale, float q_coef, int q_every, RopeExtras ex) {
  __shared__ float cs[2][ROPE_MAX_HALF];
  extern __shared__ float inv_rms[];     // ex.unit: one number a head of q, then of k
  const int64_t row = blockIdx.x;
  const int seq = row_seq[row];
  if (seq < 0) return;  // padding row
  const int pos = positions[row];
  const float q_mul = he_query_temperature(pos, q_coef, q_every);
  const int half = rotary_dim >> 1;
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    const float a = (float)pos * inv_freq[i];
    float sn, c;
    sincos_angle(a, &sn, &c);
    cs[0][i] = c * mscale;
    cs[1][i] = sn * mscale;
  }
  if (ex.unit) {
    const int lane = threadIdx.x & 63, heads = H + (k_in ? KVH : 0);
    for (int h = threadIdx.x >> 6; h < heads; h += blockDim.x >> 6) {
      const bool of_q = h < H;
      const int base = (of_q ? h : h - H) * hd_in;
      const TI* in = (of_q ? q_in : k_in) + row * in_stride + base;
      const void* bias = of_q ? q_bias : k_bias;
      float ss = 0.f;
      for (int d = lane; d < hd_in; d += 64) {
        float x = to_float(in[d]);
        if (bias) x += load_param(bias, base + d, bias_dtype);
        ss = fmaf(x, x, ss);
      }
      ss = wave_sum(ss);
      if (lane == 0) inv_rms[h] = 1.f / sqrtf(ss / (float)hd_in + ex.eps);
    }
  }
  __syncthreads();
  // the two dims of pair j
  const int pair_step = interleaved ? 1 : half;
  const int pair_mul = interleaved ? 2 : 1;

  // ---- q: rotate and store densely
  {
    const TI* in = q_in + row * in_stride;
    T* out = q_out + row * (int64_t)H * hd;
    const int per_head = half + (hd - rotary_dim);
    for (int it = threadIdx.x; it < H * per_head; it += blockDim.x) {
      const int h = it / per_head;
      const int j = it - h * per_head;
      const int base = h * hd_in, obase = h * hd;
      const float mul = ex.unit ? q_mul * inv_rms[h] : q_mul;
      if (j < half) {
        const int d0 = pair_mul * j, d1 = d0 + pair_step;
        float x0 = to_float((in + base + d0)[0]);
        float x1 = to_float((in + base + d1)[0]);
        if (q_bias) {
          x0 += load_param(q_bias, base + d0, bias_dtype);
          x1 += load_param(q_bias, base + d1, bias_dtype);
        }
        const float c = cs[0][j], sn = cs[1][j];
        out[obase + d0] = from_float<T>((x0 * c - x1 * sn) * mul);
        out[obase + d1] = from_float<T>((x0 * sn + x1 * c) * mul);
      } else {
        const int d = rotary_dim + (j - half);
        float x = 0.f;
        if (d < hd_in) {
          x = to_float((in + base + d)[0]);
          if (q_bias) x += load_param(q_bias, base + d, bias_dtype);
        }
        out[obase + d] = from_float<T>(x * mul);
      }
    }
  }
  if (k_in == nullptr) return;  // this layer reads another layer's cache

  const int slot = seq_slot[seq];
  const int page = page_table[(int64_t)slot * max_blocks + (pos >> HE_PAGE_SHIFT)];
  if (page < 0 || page >= num_pages) return;  // never for a batch the host has admitted
  const int off = pos & (HE_PAGE_TOKENS - 1);
  // ---- k: rotate and scatter
  {
    const TI* in = k_in + row * in_stride;
    const int per_head = half + (hd_in - rotary_dim);
    for (int it = threadIdx.x; it < KVH * per_head; it += blockDim.x) {
      const int h = it / per_head;
      const int j = it - h * per_head;
      const int base = h * hd_in;
      T* out = kpool + ((int64_t)page * KVH + h) * he_k_page_elems(hd);   // the page, in operand order
      const int KS = he_k_steps(hd);
      const float mul = ex.unit ? inv_rms[H + h] : 1.f;
      if (j < half) {
        const int d0 = pair_mul * j, d1 = d0 + pair_step;
        float x0 = to_float((in + base + d0)[0]);
        float x1 = to_float((in + base + d1)[0]);
        if (k_bias) {
          x0 += load_param(k_bias, base + d0, bias_dtype);
          x1 += load_param(k_bias, base + d1, bias_dtype);
        }
        const float c = cs[0][j], sn = cs[1][j];
        out[he_k_index(off, d0, KS)] = from_float<T>((x0 * c - x1 * sn) * mul);
        out[he_k_index(off, d1, KS)] = from_float<T>((x0 * sn + x1 * c) * mul);
      } else {
        const int d = rotary_dim + (j - half);
        float x = to_float((in + base + d)[0]);
        if (k_bias) x += load_param(k_bias, base + d, bias_dtype);
        out[he_k_index(off, d, KS)] = from_float<T>(x * mul);
      }
    }
  }
  // ---- v: bias and scatter
  {
    const TI* in = v_in + row * in_stride;
    for (int it = threadIdx.x; it < KVH * vd_in; it += blockDim.x) {
      const int h = it / vd_in;
      const int d = it - h * vd_in;
      float x = to_float((in + it)[0]);
      if (v_bias) x += load_param(v_bias, it, bias_dtype);
      if (ex.v_first)
        x = (1.f - ex.v_lambda) * x + ex.v_lambda * to_float(((const TI*)ex.v_first)[row * ex.v_stride + it]);
      vpool[((int64_t)page * KVH + h) * he_v_page_elems(hd) + he_v_index(off, d, he_v_tiles(hd))] =
          from_float<T>(x);
    }
  }
}

// bf16 rows, eight elements per access: one thread rotates the pairs (j..j+7, j+half..)
// of one head (interleaved: the four pairs inside eight neighbouring dims), or copies eight v
// elements. Needs rotary_dim/2 (interleaved: rotary_dim), the head sizes, head_dim - rotary_dim and
// the row stride in multiples of 8. hd_in, vd_in, interleaved, mscale: as the kernel above takes them.
__device__ __forceinline__ void unpack8(const uint4& v, float* f) {
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f[2 * i] = __uint_as_float(w[i] << 16);
    f[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}
__device__ __forceinline__ uint4 pack8(const float* f) {
  uint32_t w[4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
    w[i] = (uint32_t)float_to_bf16_bits(f[2 * i]) | ((uint32_t)float_to_bf16_bits(f[2 * i + 1]) << 16);
  return make_uint4(w[0], w[1], w[2], w[3]);
}

// grid: one workgroup per 8 rows (per row in a step of up to 128 rows) for v, then one per row for q and k.
// V lies transposed in a page (8 keys of one dim are 16 contiguous bytes), so the v values of
// a run of tokens that share such a group are gathered dim by dim and stored together: 16
// bytes a store when the run is a whole group (a prompt), 2 bytes a token otherwise.
__global__ __launch_bounds__(1024) void qkv_rope_cache_vec_kernel(
    uint16_t* __restrict__ q_out, uint16_t* __restrict__ kpool, uint16_t* __restrict__ vpool,
    const uint16_t* __restrict__ q_in, const uint16_t* __restrict__ k_in,
    const uint16_t* __restrict__ v_in, int64_t in_stride, const uint16_t* __restrict__ q_bias,
    const uint16_t* __restrict__ k_bias, const uint16_t* __restrict__ v_bias,
    const int32_t* __restrict__ positions, const int32_t* __restrict__ row_seq,
    const int32_t* __restrict__ seq_slot, const int32_t* __restrict__ page_table, int max_blocks,
    int num_pages, const float* __restrict__ inv_freq, int rotary_dim, int rows, int H, int KVH,
    int hd, int hd_in, int vd_in, int interleaved, float mscale, int v_span, float q_coef, int q_every,
    RopeExtras ex) {
  __shared__ float cs[2][ROPE_MAX_HALF];
  extern __shared__ float squares[];     // ex.unit: an item's share of its head's sum of squares
  const int v_blocks = (int)gridDim.x - rows;   // they come first: theirs is the longest chain of dependent loads
  if ((int)blockIdx.x < v_blocks) {
    // ---- v: the runs of tokens that begin in rows [r0, r0 + v_span). In a step of few rows (one token a
    // sequence) every row has a workgroup of its own: a workgroup takes its rows one after the other, and
    // each is a chain of dependent loads (sequence, slot, page) that eight rows in a row made 14 us long.
    const int r0 = v_span * (int)blockIdx.x;
    const int NT = he_v_tiles(hd);
    for (int r = r0; r < min(r0 + v_span, rows); ++r) {
      const int seq = row_seq[r];
      if (seq < 0) continue;
      const int pos = positions[r];
      const bool begins = (pos & 7) == 0 || r == 0 || row_seq[r - 1] != seq || positions[r - 1] != pos - 1;
      if (!begins) continue;
      int n = 1;   // tokens of the run: the same sequence, consecutive positions, one group of 8 keys
      while (n < 8 - (pos & 7) && r + n < rows && row_seq[r + n] == seq && positions[r + n] == pos + n) ++n;
      const int page = page_table[(int64_t)seq_slot[seq] * max_blocks + (pos >> HE_PAGE_SHIFT)];
      if (page < 0 || page >= num_pages) continue;
      const int off = pos & (HE_PAGE_TOKENS - 1);
      for (int e = threadIdx.x; e < KVH * vd_in; e += blockDim.x) {
        const int h = e / vd_in, d = e - h * vd_in;
        const float b = v_bias ? bf16_bits_to_float(v_bias[e]) : 0.f;
        uint16_t vals[8];
        // eight loads with no branch around them (a token beyond the run reads the run's last
        // row and is dropped): they go out together
#pragma unroll
        for (int i = 0; i < 8; ++i) vals[i] = v_in[(int64_t)(r + min(i, n - 1)) * in_stride + e];
        if (ex.v_first) {
          uint16_t firsts[8];
#pragma unroll
          for (int i = 0; i < 8; ++i)
            firsts[i] = ((const uint16_t*)ex.v_first)[(int64_t)(r + min(i, n - 1)) * ex.v_stride + e];
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            vals[i] = float_to_bf16_bits((1.f - ex.v_lambda) * (bf16_bits_to_float(vals[i]) + b) +
                                         ex.v_lambda * bf16_bits_to_float(firsts[i]));
          }
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if (v_bias && !ex.v_first) vals[i] = float_to_bf16_bits(bf16_bits_to_float(vals[i]) + b);
          if (i >= n) vals[i] = 0;
        }
        uint16_t* out = vpool + ((int64_t)page * KVH + h) * he_v_page_elems(hd) + he_v_index(off, d, NT);
        if (n == 8) {
          *reinterpret_cast<uint4*>(out) =
              make_uint4(vals[0] | ((uint32_t)vals[1] << 16), vals[2] | ((uint32_t)vals[3] << 16),
                         vals[4] | ((uint32_t)vals[5] << 16), vals[6] | ((uint32_t)vals[7] << 16));
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i)
            if (i < n) out[i] = vals[i];
        }
      }
    }
    return;
  }
  // ---- q and k of one row
  const int64_t row = (int)blockIdx.x - v_blocks;
  const int seq = row_seq[row];
  if (seq < 0) return;  // padding row
  const int half = rotary_dim >> 1;
  const int rot8 = (interleaved ? rotary_dim : half) >> 3;   // rotated groups per head: 8 pairs, or, interleaved, 8 dims
  // groups of 8 pass-through dims per head: q_out has hd dims a head (those from hd_in on are zeros), a key hd_in
  const int per_head_q = rot8 + ((hd - rotary_dim) >> 3), per_head_k = rot8 + ((hd_in - rotary_dim) >> 3);
  const int q_items = H * per_head_q;
  const int items = q_items + (k_in ? KVH * per_head_k : 0);
  // an item: eight pairs (j.., j + half..) of one head (interleaved: the dims j..j+7, four pairs), or eight
  // pass-through dims from j on
  struct Item {
    const uint16_t* in;
    const uint16_t* bias;
    int h, j;
    bool is_q, rotated, pad;
  };
  auto item = [&](int it) {
    Item im;
    im.is_q = it < q_items;
    const int idx = im.is_q ? it : it - q_items;
    const int per_head = im.is_q ? per_head_q : per_head_k;
    im.h = idx / per_head;
    const int g = idx - im.h * per_head;
    im.rotated = g < rot8;
    im.j = im.rotated ? 8 * g : rotary_dim + 8 * (g - rot8);
    im.pad = !im.rotated && im.j >= hd_in;       // dims of q_out beyond the rows' head size
    im.in = (im.is_q ? q_in : k_in) + row * in_stride + im.h * hd_in;
    const uint16_t* bias = im.is_q ? q_bias : k_bias;
    im.bias = bias ? bias + im.h * hd_in : nullptr;
    return im;
  };
  const uint4 zero = make_uint4(0, 0, 0, 0);
  // four loads with no branch around them, so that they go out together: an item without a
  // partner, or a row without a bias, reads its own eight elements again and drops them
  auto load = [&](const Item& im, uint4 (&raw)[4]) {
    const int j = im.pad ? 0 : im.j;             // (padding reads the head's first dims and drops them)
    const int partner = im.rotated && !interleaved ? j + half : j;
    const uint16_t* b = im.bias ? im.bias : im.in;
    const uint4 x0 = *reinterpret_cast<const uint4*>(im.in + j);
    const uint4 x1 = *reinterpret_cast<const uint4*>(im.in + partner);
    const uint4 b0 = *reinterpret_cast<const uint4*>(b + j);
    const uint4 b1 = *reinterpret_cast<const uint4*>(b + partner);
    raw[0] = im.pad ? zero : x0;
    raw[1] = im.rotated ? x1 : zero;
    raw[2] = im.bias && !im.pad ? b0 : zero;
    raw[3] = im.bias && im.rotated ? b1 : zero;
  };
  // the loads of a thread's first item are on their way while the angles are computed
  Item first;
  uint4 first_raw[4];
  const bool has_first = (int)threadIdx.x < items;
  if (has_first) {
    first = item(threadIdx.x);
    load(first, first_raw);
  }
  const int pos = positions[row];
  int page = -1;
  if (k_in != nullptr) page = page_table[(int64_t)seq_slot[seq] * max_blocks + (pos >> HE_PAGE_SHIFT)];
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    float sn, c;
    sincos_angle((float)pos * inv_freq[i], &sn, &c);
    cs[0][i] = c * mscale;
    cs[1][i] = sn * mscale;
  }
  if (ex.unit) {
    auto square = [&](int it, const Item& im, const uint4 (&raw)[4]) {
      float ss = 0.f;
#pragma unroll
      for (int half_of = 0; half_of < 2; ++half_of) {       // the item's own elements, then its partners'
        if (half_of == 1 && (!im.rotated || interleaved)) break;
        float x[8], b[8];
        unpack8(raw[half_of], x);
        unpack8(raw[2 + half_of], b);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss = fmaf(x[i] + b[i], x[i] + b[i], ss);
      }
      squares[it] = ss;
    };
    if (has_first) square(threadIdx.x, first, first_raw);
    for (int it = threadIdx.x + blockDim.x; it < items; it += blockDim.x) {
      const Item im = item(it);
      uint4 raw[4];
      load(im, raw);
      square(it, im, raw);
    }
  }
  __syncthreads();
  // what a head is multiplied by: the shares of its items, added in their order
  auto unit_mul = [&](const Item& im) {
    if (!ex.unit) return 1.f;
    const int per_head = im.is_q ? per_head_q : per_head_k;
    const float* p = squares + (im.is_q ? 0 : q_items) + im.h * per_head;
    float ss = 0.f;
    for (int i = 0; i < per_head; ++i) ss += p[i];
    return 1.f / sqrtf(ss / (float)hd_in + ex.eps);
  };
  const bool cache_ok = page >= 0 && page < num_pages;
  const int off = pos & (HE_PAGE_TOKENS - 1);
  const int KS = he_k_steps(hd);
  const float q_mul = he_query_temperature(pos, q_coef, q_every);
  const bool tempered = q_mul != 1.f;
  const bool scaled = tempered || ex.unit;
  auto finish = [&](const Item& im, const uint4 (&raw)[4]) {
    // where the eight elements from dim d on go: the q row, or the cache page in operand order
    uint16_t* out;
    if (im.is_q) {
      out = q_out + row * (int64_t)H * hd + im.h * hd;
    } else {
      if (!cache_ok) return;
      out = kpool + ((int64_t)page * KVH + im.h) * he_k_page_elems(hd);
    }
    auto at = [&](int d) { return out + (im.is_q ? d : he_k_index(off, d, KS)); };
    const float mul = (im.is_q ? q_mul : 1.f) * unit_mul(im);
    float x0[8], x1[8], b0[8], b1[8];
    unpack8(raw[0], x0);
    unpack8(raw[2], b0);
    if (im.rotated && interleaved) {
      float y[8];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float a0 = x0[2 * i] + b0[2 * i], a1 = x0[2 * i + 1] + b0[2 * i + 1];
        const float c = cs[0][(im.j >> 1) + i], sn = cs[1][(im.j >> 1) + i];
        y[2 * i] = a0 * c - a1 * sn;
        y[2 * i + 1] = a0 * sn + a1 * c;
      }
      if (scaled) {
#pragma unroll
        for (int i = 0; i < 8; ++i) y[i] *= mul;
      }
      *reinterpret_cast<uint4*>(at(im.j)) = pack8(y);
    } else if (im.rotated) {
      unpack8(raw[1], x1);
      unpack8(raw[3], b1);
      float y0[8], y1[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float a0 = x0[i] + b0[i], a1 = x1[i] + b1[i];
        const float c = cs[0][im.j + i], sn = cs[1][im.j + i];
        y0[i] = a0 * c - a1 * sn;
        y1[i] = a0 * sn + a1 * c;
      }
      if (scaled) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          y0[i] *= mul;
          y1[i] *= mul;
        }
      }
      *reinterpret_cast<uint4*>(at(im.j)) = pack8(y0);
      *reinterpret_cast<uint4*>(at(im.j + half)) = pack8(y1);
    } else {
      if (im.bias || scaled) {
#pragma unroll
        for (int i = 0; i < 8; ++i) x0[i] = (x0[i] + b0[i]) * mul;
        *reinterpret_cast<uint4*>(at(im.j)) = pack8(x0);
      } else {
        *reinterpret_cast<uint4*>(at(im.j)) = raw[0];
      }
    }
  };
  if (has_first) finish(first, first_raw);
  for (int it = threadIdx.x + blockDim.x; it < items; it += blockDim.x) {
    const Item im = item(it);
    uint4 raw[4];
    load(im, raw);
    finish(im, raw);
  }
}

extern "C" int he_qkv_rope_cache(void* q_out, void* kpool, void* vpool, const void* q_in,
                                 const void* k_in, const void* v_in, int64_t in_stride,
                                 const void* q_bias, const void* k_bias, const void* v_bias,
                                 int bias_dtype, const void* positions, const void* row_seq,
                                 const void* seq_slot, const void* page_table, int max_blocks,
                                 int num_pages, const void* inv_freq, int rotary_dim, int rows,
                                 int H, int KVH, int hd, int hd_in, int vd_in, int interleaved,
                                 float mscale, float q_coef, int q_every, int unit, float unit_eps,
                                 const void* v_first, int64_t v_stride, float v_lambda, int dtype,
                                 void* stream) {
  HE_REQUIRE(rows >= 0 && H > 0 && KVH >= 0 && hd > 0, "he_qkv_rope_cache: bad sizes");
  if (hd_in <= 0) hd_in = hd;
  if (vd_in <= 0) vd_in = hd;
  HE_REQUIRE(hd_in <= hd && vd_in <= hd,
             "he_qkv_rope_cache: the rows' head sizes %d and %d exceed the pages' %d", hd_in, vd_in, hd);
  HE_REQUIRE(rotary_dim >= 0 && rotary_dim <= hd_in && (rotary_dim & 1) == 0,
             "he_qkv_rope_cache: rotary_dim %d must be even and at most head_dim %d", rotary_dim,
             hd_in);
  HE_REQUIRE(rotary_dim / 2 <= ROPE_MAX_HALF, "he_qkv_rope_cache: rotary_dim %d above %d",
             rotary_dim, 2 * ROPE_MAX_HALF);
  HE_REQUIRE(rotary_dim == 0 || inv_freq != nullptr, "he_qkv_rope_cache: missing inv_freq");
  HE_REQUIRE((k_in == nullptr) == (v_in == nullptr), "he_qkv_rope_cache: k and v go together");
  HE_REQUIRE(k_in == nullptr || (kpool && vpool && page_table && max_blocks > 0 && KVH > 0),
             "he_qkv_rope_cache: cache arguments missing");
  HE_REQUIRE(dtype == HE_BF16 || dtype == HE_F32, "he_qkv_rope_cache: unknown dtype %d", dtype);
  HE_REQUIRE(v_first == nullptr || (k_in != nullptr && v_stride >= (int64_t)KVH * vd_in),
             "he_qkv_rope_cache: rows of other values are %lld wide, not %d", (long long)v_stride, KVH * vd_in);
  HE_REQUIRE(H + KVH <= 8192, "he_qkv_rope_cache: %d heads", H + KVH);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int threads = 256;
  RopeExtras ex;
  ex.unit = unit;
  ex.eps = unit_eps;
  ex.v_first = v_first;
  ex.v_stride = v_stride;
  ex.v_lambda = v_lambda;
  const size_t head_floats = unit ? sizeof(float) * (H + KVH) : 0;
#define ROPE_LAUNCH(T, TI)                                                                      \
  qkv_rope_cache_kernel<T, TI><<<rows, threads, head_floats, s>>>(                                      \
      (T*)q_out, (T*)kpool, (T*)vpool, (const TI*)q_in, (const TI*)k_in, (const TI*)v_in,       \
      in_stride, q_bias, k_bias, v_bias, bias_dtype,                                            \
      (const int32_t*)positions, (const int32_t*)row_seq, (const int32_t*)seq_slot,             \
      (const int32_t*)page_table, max_blocks, num_pages, (const float*)inv_freq, rotary_dim, H, \
      KVH, hd, hd_in, vd_in, interleaved, mscale, q_coef, q_every, ex)
  const bool vec_ok = dtype == HE_BF16 &&
                      (q_bias == nullptr || bias_dtype == HE_BF16) &&
                      ((interleaved ? rotary_dim : rotary_dim >> 1) & 7) == 0 && ((hd - rotary_dim) & 7) == 0 &&
                      (in_stride & 7) == 0 && (hd & 7) == 0 && (hd_in & 7) == 0 &&
                      ((((uintptr_t)q_in) | ((uintptr_t)k_in) | ((uintptr_t)v_in) |
                        ((uintptr_t)q_bias) | ((uintptr_t)k_bias) | ((uintptr_t)v_bias) |
                        ((uintptr_t)q_out) | ((uintptr_t)kpool)) & 15) == 0;
  if (vec_ok) {
    const int rot8 = (interleaved ? rotary_dim : rotary_dim >> 1) >> 3;
    const int items = H * (rot8 + ((hd - rotary_dim) >> 3)) + (k_in ? KVH * (rot8 + ((hd_in - rotary_dim) >> 3)) : 0);
    HE_REQUIRE(!unit || items <= 12288, "he_qkv_rope_cache: %d heads are too many to norm", H + KVH);
    const int vec_threads = min(1024, max(64, (items + 63) / 64 * 64));
    const int v_span = rows <= 128 ? 1 : 8;
    const int v_blocks = k_in ? (rows + v_span - 1) / v_span : 0;
    qkv_rope_cache_vec_kernel<<<rows + v_blocks, vec_threads, unit ? sizeof(float) * items : 0, s>>>(
        (uint16_t*)q_out, (uint16_t*)kpool, (uint16_t*)vpool, (const uint16_t*)q_in,
        (const uint16_t*)k_in, (const uint16_t*)v_in, in_stride, (const uint16_t*)q_bias,
        (const uint16_t*)k_bias, (const uint16_t*)v_bias, (const int32_t*)positions,
        (const int32_t*)row_seq, (const int32_t*)seq_slot, (const int32_t*)page_table, max_blocks,
        num_pages, (const float*)inv_freq, rotary_dim, rows, H, KVH, hd, hd_in, vd_in, interleaved, mscale, v_span, q_coef,
        q_every, ex);
  } else if (dtype == HE_BF16) {
    ROPE_LAUNCH(bf16_t, bf16_t);
  } else {
    ROPE_LAUNCH(float, float);
  }
#undef ROPE_LAUNCH
  return he_check_launch("he_qkv_rope_cache");
}
