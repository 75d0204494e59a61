// What a latent attention needs around the shared attention kernels. Its keys and values are one latent
// vector c a token (plus one rotated key part shared by all heads); a head's own key part is W_uk,h c and
// its value W_uv,h c. Because q . (W_uk,h c) = (W_uk,h^T q) . c, the cache keeps [rotated part | c] as the
// one key of a token and c as its value, the queries are taken through W_uk,h^T, and a head's attention
// result over the latents goes through W_uv,h afterwards: two products per head.
//   he_head_product(_mfma)   out[r, h, :] = x[r, h, :] W_h for a matrix a head, optionally times a gate's sigmoid
//   he_latent_cache          the latent's norm, both rotations and the cache write, one launch
#include "cache_layout.h"
#include "hector_kernels.h"

#define HP_ROWS 8
#define HP_KCHUNK 256
// out[r, h, n] = sum_k x[r, h, k] * w[h, k, n] in fp32: k in chunks of HP_KCHUNK; inside a chunk each of the
// workgroup's four wavefronts takes a quarter of the k (a chain of multiply-adds in ascending k, eight weight loads
// in flight), the four sums meet in wavefront order, and the chunks' sums are added in chunk order: one order a
// row whatever else the step holds. x at x_row / x_head element strides, out likewise; w [H][K][N]. A workgroup
// takes HP_ROWS rows of one head and 64 neighbouring n; the rows' x values are staged in LDS a chunk at a time.
// gate (or null): the result is multiplied by sigmoid(gate[r * gate_row + h * N + n]).
template <typename T, typename TW>
__global__ __launch_bounds__(256) void head_product_kernel(T* __restrict__ out, int64_t o_row, int64_t o_head,
                                                           const T* __restrict__ x, int64_t x_row, int64_t x_head,
                                                           const TW* __restrict__ w, int rows, int K, int N,
                                                           const T* __restrict__ gate, int64_t gate_row) {
  __shared__ float xs[HP_ROWS][HP_KCHUNK];
  __shared__ float part[4][HP_ROWS][64];
  const int h = blockIdx.y;
  const int64_t r0 = (int64_t)blockIdx.z * HP_ROWS;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int n = blockIdx.x * 64 + lane;
  const int nc = min(n, N - 1);            // a lane beyond N reads the last column and stores nothing
  const TW* wh = w + (int64_t)h * K * N;
  float total[HP_ROWS];
#pragma unroll
  for (int r = 0; r < HP_ROWS; ++r) total[r] = 0.f;
  for (int k0 = 0; k0 < K; k0 += HP_KCHUNK) {
    const int kc = min(HP_KCHUNK, K - k0);
    __syncthreads();
    for (int i = threadIdx.x; i < HP_ROWS * kc; i += blockDim.x) {
      const int r = i / kc, k = i % kc;
      xs[r][k] = r0 + r < rows ? to_float(x[(r0 + r) * x_row + h * x_head + k0 + k]) : 0.f;
    }
    __syncthreads();
    const int per = (kc + 3) / 4;
    const int ka = wave * per, kb = min(kc, ka + per);
    float acc[HP_ROWS];
#pragma unroll
    for (int r = 0; r < HP_ROWS; ++r) acc[r] = 0.f;
    for (int k = ka; k < kb; k += 8) {
      float wv[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) wv[u] = to_float(wh[(int64_t)(k0 + min(k + u, kb - 1)) * N + nc]);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (k + u < kb) {
#pragma unroll
          for (int r = 0; r < HP_ROWS; ++r) acc[r] = fmaf(xs[r][k + u], wv[u], acc[r]);
        }
    }
#pragma unroll
    for (int r = 0; r < HP_ROWS; ++r) part[wave][r][lane] = acc[r];
    __syncthreads();
    if (wave == 0) {
#pragma unroll
      for (int r = 0; r < HP_ROWS; ++r)
        total[r] += ((part[0][r][lane] + part[1][r][lane]) + part[2][r][lane]) + part[3][r][lane];
    }
  }
  if (wave != 0 || n >= N) return;
#pragma unroll
  for (int r = 0; r < HP_ROWS; ++r)
    if (r0 + r < rows) {
      float v = total[r];
      if (gate != nullptr) v = v / (1.f + expf(-to_float(gate[(r0 + r) * gate_row + (int64_t)h * N + n])));
      out[(r0 + r) * o_row + h * o_head + n] = from_float<T>(v);
    }
}

extern "C" int he_head_product(void* out, int64_t o_row, int64_t o_head, const void* x, int64_t x_row, int64_t x_head,
                               const void* w, int w_dtype, int rows, int H, int K, int N, const void* gate,
                               int64_t gate_row, int dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && H > 0 && K > 0 && N > 0 && H <= 65535, "he_head_product: bad sizes H=%d K=%d N=%d", H, K, N);
  HE_REQUIRE((dtype == HE_BF16 || dtype == HE_F32) && (w_dtype == HE_BF16 || w_dtype == HE_F32), "he_head_product: unknown dtype");
  if (rows == 0) return 0;
  const int threads = 256;
  const dim3 grid((N + 63) / 64, H, (rows + HP_ROWS - 1) / HP_ROWS);
  HE_REQUIRE(grid.z <= 65535, "he_head_product: %d rows are too many for one launch", rows);
  hipStream_t s = (hipStream_t)stream;
#define HP_LAUNCH(T, TW)                                                                                    \
  head_product_kernel<T, TW><<<grid, threads, 0, s>>>((T*)out, o_row, o_head, (const T*)x, x_row, x_head, \
                                                      (const TW*)w, rows, K, N, (const T*)gate, gate_row)
  if (dtype == HE_BF16 && w_dtype == HE_BF16) {
    HP_LAUNCH(bf16_t, bf16_t);
  } else if (dtype == HE_BF16) {
    HP_LAUNCH(bf16_t, float);
  } else if (w_dtype == HE_BF16) {
    HP_LAUNCH(float, bf16_t);
  } else {
    HP_LAUNCH(float, float);
  }
#undef HP_LAUNCH
  return he_check_launch("he_head_product");
}

// The same products on the matrix cores (v_mfma_f32_16x16x32_bf16): w [H][N][K], so that a weight row's eight
// consecutive k are one 16-byte load, as an x row's are. Weight rows are the rows of a tile and step rows its columns:
// a lane then holds four neighbouring n of one row and stores them together. A wavefront takes NTL tiles of 16 n and MT
// tiles of 16 rows; the workgroup's four wavefronts are WN along n times 4 / WN along the rows. k runs in ascending steps
// of 32 whatever the tile shape: a row's sums do not depend on the rest of the step. K is a multiple of 8 (a step past the
// end multiplies zeros); n and rows beyond the ends read the last ones and store nothing.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 hp_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float hp_floatx4;

template <int MT, int NTL, int WN>
__global__ __launch_bounds__(256) void head_product_mfma_kernel(
    uint16_t* __restrict__ out, int64_t o_row, int64_t o_head, const uint16_t* __restrict__ x, int64_t x_row,
    int64_t x_head, const uint16_t* __restrict__ w, int rows, int K, int N, const uint16_t* __restrict__ gate,
    int64_t gate_row, int out_vec, int gate_vec) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.y;
  const int n0 = 16 * NTL * ((int)blockIdx.x * WN + wave % WN);
  const int64_t r0 = 16 * MT * ((int64_t)blockIdx.z * (4 / WN) + wave / WN);
  if (n0 >= N || r0 >= rows) return;
  const uint16_t* wp[NTL];
  const uint16_t* xp[MT];
#pragma unroll
  for (int u = 0; u < NTL; ++u) wp[u] = w + ((int64_t)h * N + min(n0 + 16 * u + lr, N - 1)) * K;
#pragma unroll
  for (int t = 0; t < MT; ++t) xp[t] = x + min(r0 + 16 * t + lr, (int64_t)rows - 1) * x_row + h * x_head;
  hp_floatx4 acc[NTL][MT];
#pragma unroll
  for (int u = 0; u < NTL; ++u)
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[u][t] = hp_floatx4{0.f, 0.f, 0.f, 0.f};
  constexpr int UNROLL = MT * NTL >= 8 ? 2 : 4;
#pragma unroll UNROLL
  for (int k0 = 0; k0 < K; k0 += 32) {
    const int k = k0 + 8 * lg;
    const bool in = k < K;
    const int kc = in ? k : 0;
    const uint4 zero = make_uint4(0, 0, 0, 0);
    hp_bf16x8 a[NTL], b[MT];
#pragma unroll
    for (int u = 0; u < NTL; ++u) {
      const uint4 v = *reinterpret_cast<const uint4*>(wp[u] + kc);
      a[u] = __builtin_bit_cast(hp_bf16x8, in ? v : zero);
    }
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      const uint4 v = *reinterpret_cast<const uint4*>(xp[t] + kc);
      b[t] = __builtin_bit_cast(hp_bf16x8, in ? v : zero);
    }
#pragma unroll
    for (int u = 0; u < NTL; ++u)
#pragma unroll
      for (int t = 0; t < MT; ++t) acc[u][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u], b[t], acc[u][t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int64_t m = r0 + 16 * t + lr;
    if (m >= rows) continue;
#pragma unroll
    for (int u = 0; u < NTL; ++u) {
      const int n = n0 + 16 * u + 4 * lg;
      if (n >= N) continue;
      float v[4] = {acc[u][t][0], acc[u][t][1], acc[u][t][2], acc[u][t][3]};
      const bool whole = n + 4 <= N;
      if (gate != nullptr) {
        const uint16_t* gp = gate + m * gate_row + (int64_t)h * N + n;
        float g[4];
        if (gate_vec && whole) {
          const uint2 raw = *reinterpret_cast<const uint2*>(gp);
          g[0] = __uint_as_float(raw.x << 16), g[1] = __uint_as_float(raw.x & 0xffff0000u);
          g[2] = __uint_as_float(raw.y << 16), g[3] = __uint_as_float(raw.y & 0xffff0000u);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) g[i] = bf16_bits_to_float(gp[min(i, N - 1 - n)]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = v[i] / (1.f + expf(-g[i]));
      }
      uint16_t* o = out + m * o_row + h * o_head + n;
      if (out_vec && whole) {
        *reinterpret_cast<uint2*>(o) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < N) o[i] = float_to_bf16_bits(v[i]);
      }
    }
  }
}

extern "C" int he_head_product_mfma(void* out, int64_t o_row, int64_t o_head, const void* x, int64_t x_row, int64_t x_head,
                                    const void* w, int rows, int H, int K, int N, const void* gate, int64_t gate_row,
                                    void* stream) {
  HE_REQUIRE(rows >= 0 && H > 0 && K > 0 && N > 0 && H <= 65535, "he_head_product_mfma: bad sizes H=%d K=%d N=%d", H, K, N);
  HE_REQUIRE((K & 7) == 0 && (x_row & 7) == 0 && (x_head & 7) == 0 && ((((uintptr_t)x) | ((uintptr_t)w)) & 15) == 0,
             "he_head_product_mfma: K=%d, the strides of x and its address must be multiples of 8 elements", K);
  if (rows == 0) return 0;
  const int out_vec = ((o_row | o_head) & 3) == 0 && (((uintptr_t)out) & 7) == 0;
  const int gate_vec = gate != nullptr && (gate_row & 3) == 0 && (N & 3) == 0 && (((uintptr_t)gate) & 7) == 0;
  hipStream_t s = (hipStream_t)stream;
  // few rows: the weights are what is read, so the n are spread over as many wavefronts as there are tiles; many rows: tiles
  // of 64 x 64, the four wavefronts of a workgroup over the same weights
#define HPM_LAUNCH(MT, NTL, WN)                                                                                          \
  do {                                                                                                                   \
    const dim3 grid((N + 16 * NTL * WN - 1) / (16 * NTL * WN), H, (rows + 16 * MT * (4 / WN) - 1) / (16 * MT * (4 / WN))); \
    HE_REQUIRE(grid.z <= 65535, "he_head_product_mfma: %d rows are too many for one launch", rows);                      \
    head_product_mfma_kernel<MT, NTL, WN><<<grid, 256, 0, s>>>((uint16_t*)out, o_row, o_head, (const uint16_t*)x, x_row, \
                                                               x_head, (const uint16_t*)w, rows, K, N,                  \
                                                               (const uint16_t*)gate, gate_row, out_vec, gate_vec);     \
  } while (0)
  if (rows <= 16) HPM_LAUNCH(1, 1, 4);
  else if (rows <= 128) HPM_LAUNCH(2, 1, 4);
  else HPM_LAUNCH(4, 4, 1);
#undef HPM_LAUNCH
  return he_check_launch("he_head_product_mfma");
}

// One pass over the projected rows of a latent attention's step. q [row][H][d + r] (rows q_row elements apart): a head's
// last r dims, rotated at the row's position, go to the first r dims of its pd dims of q_out (rows q_out_row apart), and
// what lies behind the r + rank dims in use becomes zeros; the rank dims in between are a head product's to write.
// down [row][rank + r] (rows down_row apart; null: the latents are another layer's): c = rms(first rank dims) * gain, in
// fp32, rounded once; the key [rotated last r dims | c] and the value c go into the row's cache page (one kv head of pd dims).
// Rotation: frequency i turns the dims (i, i + r/2), or, interleaved, (2i, 2i + 1); cos and sin times mscale.
//
// grid: the key/value workgroups first (span rows each: one in a step of few rows, else eight, two a wavefront), then a
// workgroup a row for q. A page holds V transposed (eight tokens of a dim are neighbours), so the workgroup keeps its rows'
// c in LDS and stores a whole group of eight tokens at once where it has one.
template <typename T>
__global__ __launch_bounds__(256) void latent_cache_kernel(
    T* __restrict__ q_out, int64_t q_out_row, T* __restrict__ kpool, T* __restrict__ vpool, const T* __restrict__ q,
    int64_t q_row, const T* __restrict__ down, int64_t down_row, const void* __restrict__ gain, int gain_dtype, float eps,
    const int32_t* __restrict__ positions, const int32_t* __restrict__ row_seq, const int32_t* __restrict__ seq_slot,
    const int32_t* __restrict__ page_table, int max_blocks, int num_pages, const float* __restrict__ inv_freq,
    int interleaved, float mscale, int rows, int H, int d, int r, int rank, int pd, int kv_blocks, int span) {
  extern __shared__ char lds[];
  const int half = r >> 1;
  const int pair_step = interleaved ? 1 : half, pair_mul = interleaved ? 2 : 1;
  if ((int)blockIdx.x >= kv_blocks) {
    // ---- the queries of one row
    const int64_t row = (int)blockIdx.x - kv_blocks;
    if (row_seq[row] < 0) return;   // padding row
    float* cs = reinterpret_cast<float*>(lds);
    const int pos = positions[row];
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
      float sn, c;
      sincos_angle((float)pos * inv_freq[i], &sn, &c);
      cs[2 * i] = c * mscale;
      cs[2 * i + 1] = sn * mscale;
    }
    __syncthreads();
    const int pad = pd - r - rank;
    const T* in = q + row * q_row;
    T* o = q_out + row * q_out_row;
    for (int it = threadIdx.x; it < H * half; it += blockDim.x) {
      const int h = it / half, j = it - h * half;
      const int d0 = pair_mul * j, d1 = d0 + pair_step;
      const T* qh = in + (int64_t)h * (d + r) + d;
      const float x0 = to_float(qh[d0]), x1 = to_float(qh[d1]);
      const float c = cs[2 * j], sn = cs[2 * j + 1];
      o[(int64_t)h * pd + d0] = from_float<T>(x0 * c - x1 * sn);
      o[(int64_t)h * pd + d1] = from_float<T>(x0 * sn + x1 * c);
    }
    for (int it = threadIdx.x; it < H * pad; it += blockDim.x)
      o[(int64_t)(it / pad) * pd + r + rank + it % pad] = from_float<T>(0.f);
    return;
  }
  // ---- keys and values of span rows
  T* c_sh = reinterpret_cast<T*>(lds);       // [span][rank]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r0 = span * (int)blockIdx.x;
  const int KS = he_k_steps(pd), NT = he_v_tiles(pd);
  for (int i = wave; i < span && r0 + i < rows; i += 4) {
    const int64_t row = r0 + i;
    const int seq = row_seq[row];
    if (seq < 0) continue;
    const T* dn = down + row * down_row;
    float sq = 0.f;
    for (int k = lane; k < rank; k += 64) {
      const float v = to_float(dn[k]);
      sq = fmaf(v, v, sq);
    }
    const float inv = 1.f / sqrtf(wave_sum(sq) / (float)rank + eps);
    const int pos = positions[row];
    const int page = page_table[(int64_t)seq_slot[seq] * max_blocks + (pos >> HE_PAGE_SHIFT)];
    const bool ok = page >= 0 && page < num_pages;      // always, for a batch the host has admitted
    const int off = pos & (HE_PAGE_TOKENS - 1);
    T* kp = kpool + (int64_t)(ok ? page : 0) * he_k_page_elems(pd);
    for (int k = lane; k < rank; k += 64) {
      const T c = from_float<T>(to_float(dn[k]) * inv * load_param(gain, k, gain_dtype));
      c_sh[i * rank + k] = c;
      if (ok) kp[he_k_index(off, r + k, KS)] = c;
    }
    for (int j = lane; j < half; j += 64) {
      float sn, c;
      sincos_angle((float)pos * inv_freq[j], &sn, &c);
      c *= mscale;
      sn *= mscale;
      const int d0 = pair_mul * j, d1 = d0 + pair_step;
      const float x0 = to_float(dn[rank + d0]), x1 = to_float(dn[rank + d1]);
      if (ok) {
        kp[he_k_index(off, d0, KS)] = from_float<T>(x0 * c - x1 * sn);
        kp[he_k_index(off, d1, KS)] = from_float<T>(x0 * sn + x1 * c);
      }
    }
  }
  __syncthreads();
  for (int i = 0; i < span && r0 + i < rows;) {
    const int row = r0 + i;
    const int seq = row_seq[row];
    if (seq < 0) {
      ++i;
      continue;
    }
    const int pos = positions[row];
    int n = 1;   // tokens of the run: this workgroup's, of one sequence, consecutive, inside one group of eight
    while (n < 8 - (pos & 7) && i + n < span && row + n < rows && row_seq[row + n] == seq && positions[row + n] == pos + n) ++n;
    const int page = page_table[(int64_t)seq_slot[seq] * max_blocks + (pos >> HE_PAGE_SHIFT)];
    if (page >= 0 && page < num_pages) {
      T* vp = vpool + (int64_t)page * he_v_page_elems(pd);
      const int off = pos & (HE_PAGE_TOKENS - 1);
      for (int e = threadIdx.x; e < rank; e += blockDim.x) {
        T* o = vp + he_v_index(off, e, NT);
        if (sizeof(T) == 2 && n == 8) {
          const uint16_t* c = reinterpret_cast<const uint16_t*>(c_sh) + i * rank + e;
          uint32_t pair[4];
#pragma unroll
          for (int u = 0; u < 4; ++u) pair[u] = c[2 * u * rank] | ((uint32_t)c[(2 * u + 1) * rank] << 16);
          *reinterpret_cast<uint4*>(o) = make_uint4(pair[0], pair[1], pair[2], pair[3]);
        } else {
          for (int u = 0; u < n; ++u) o[u] = c_sh[(i + u) * rank + e];
        }
      }
    }
    i += n;
  }
}

extern "C" int he_latent_cache(void* q_out, int64_t q_out_row, void* kpool, void* vpool, const void* q, int64_t q_row,
                               const void* down, int64_t down_row, const void* gain, int gain_dtype, float eps,
                               const void* positions, const void* row_seq, const void* seq_slot, const void* page_table,
                               int max_blocks, int num_pages, const void* inv_freq, int interleaved, float mscale, int rows,
                               int H, int d, int r, int rank, int pd, int dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && H > 0 && d >= 0 && r >= 0 && (r & 1) == 0 && rank > 0 && pd >= r + rank,
             "he_latent_cache: bad sizes H=%d d=%d r=%d rank=%d pd=%d", H, d, r, rank, pd);
  HE_REQUIRE(dtype == HE_BF16 || dtype == HE_F32, "he_latent_cache: unknown dtype %d", dtype);
  HE_REQUIRE(r == 0 || inv_freq != nullptr, "he_latent_cache: missing inv_freq");
  HE_REQUIRE(q_row >= (int64_t)H * (d + r) && q_out_row >= (int64_t)H * pd && (down == nullptr || down_row >= rank + r),
             "he_latent_cache: rows narrower than their contents");
  HE_REQUIRE(down == nullptr || (kpool && vpool && page_table && gain && max_blocks > 0), "he_latent_cache: cache arguments missing");
  if (rows == 0) return 0;
  const int span = rows <= 128 ? 1 : 8;
  const int kv_blocks = down != nullptr ? (rows + span - 1) / span : 0;
  const size_t es = dtype == HE_BF16 ? 2 : 4;
  size_t bytes = (size_t)r * sizeof(float);
  if (kv_blocks > 0 && bytes < span * (size_t)rank * es) bytes = span * (size_t)rank * es;
  HE_REQUIRE(bytes <= 64 * 1024, "he_latent_cache: a latent of %d dims is too wide", rank);
  hipStream_t s = (hipStream_t)stream;
#define LATENT_LAUNCH(T)                                                                                             \
  latent_cache_kernel<T><<<rows + kv_blocks, 256, bytes, s>>>(                                                       \
      (T*)q_out, q_out_row, (T*)kpool, (T*)vpool, (const T*)q, q_row, (const T*)down, down_row, gain, gain_dtype, eps, \
      (const int32_t*)positions, (const int32_t*)row_seq, (const int32_t*)seq_slot, (const int32_t*)page_table,       \
      max_blocks, num_pages, (const float*)inv_freq, interleaved, mscale, rows, H, d, r, rank, pd, kv_blocks, span)
  if (dtype == HE_BF16) LATENT_LAUNCH(bf16_t);
  else LATENT_LAUNCH(float);
#undef LATENT_LAUNCH
  return he_check_launch("he_latent_cache");
}
