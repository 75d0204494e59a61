// A memory per head that fades by a constant factor a token (linear attention with a fixed decay):
//   S_t = decay S_(t-1) + k_t v_t^T        (dk x dv)
//   y_t = S_t^T q_t
// q, k and v may first pass SiLU (element by element), q and k a rotation at the row's position (the first 2 * half
// dims of a head, pair (i, i + half)), and k a factor; all of that, and everything behind it, is fp32 arithmetic:
// only the projected rows themselves are read in the activation dtype. S starts at zero and lives in 32-bit floats in
// the sequence's row of the cache's state area.
//
// Steps of a few tokens a sequence walk them one by one (dm_step_kernel). Longer ones go by chunks of DM_C rows, whose
// sums are matrix products on the fp32 MFMA units: with n rows in a chunk, row i of it (from 0) and S the memory
// before the chunk,
//   y_i = decay^(i+1) S^T q_i + sum over j <= i of decay^(i-j) (q_i . k_j) v_j
//   S'  = decay^n S + sum over j of decay^(n-1-j) k_j v_j^T
// in four launches: the rows made ready (rotated, scaled, as 32-bit numbers), every chunk's own share of S' (all chunks
// at once), the memory before every chunk (one walk over the chunks of a sequence, element by element), and every chunk's
// rows (all at once). A chunk begins at the first row
// a step brings, every power of the decay is at most the decay's own, and no exponent is ever positive: how the rows
// were cut shows in rounding only. The powers come from a table [H][DM_C + 1] formed in double precision on the host.
#include "common.h"
#include "hector_kernels.h"

#define DM_C 64       // rows of a chunk
#define DM_B 64       // dims of a block of keys or of values
#define DM_LD 68      // floats between rows in LDS (a multiple of 4, and four banks on from row to row)
#define DM_WALK 8     // steps of at most so many rows a sequence are walked
#define DM_STEP_TILE 32            // value dims of a workgroup of the walk
#define DM_MAX_KEY 512             // key dims the walk holds
#define DM_WINDOW_FLOATS (64 << 20)   // memories held between the launches at once (256 MiB)

typedef float dm_acc __attribute__((ext_vector_type(16)));

static inline int dm_fours(int n) { return (n + 3) / 4 * 4; }

extern "C" int64_t he_decay_state_floats(int H, int dk, int dv) {
  if (H <= 0 || dk <= 0 || dv <= 0) return 0;
  return (int64_t)H * dk * dm_fours(dv);       // [H][dk][dv padded to 4]
}

static int64_t dm_window(int rows, int num_seqs, int64_t memory) {
  const int64_t chunks = (int64_t)rows / DM_C + num_seqs;      // no fewer than the sequences' chunks
  int64_t most = DM_WINDOW_FLOATS / memory;
  if (most > 32768) most = 32768;
  return chunks < most ? chunks : (most < 1 ? 1 : most);
}

extern "C" int64_t he_decay_workspace_floats(int rows, int num_seqs, int max_q_len, int H, int dk, int dv) {
  if (rows <= 0 || num_seqs <= 0 || max_q_len <= DM_WALK) return 0;
  const int64_t ready = (int64_t)rows * H * (2 * dm_fours(dk) + dm_fours(dv));
  return ready + dm_window(rows, num_seqs, he_decay_state_floats(H, dk, dv)) * he_decay_state_floats(H, dk, dv);
}

__device__ __forceinline__ float dm_silu(float z) { return z / (1.f + expf(-z)); }

__device__ __forceinline__ void dm_vec4(float* x, const float* p) {
  const float4 v = *reinterpret_cast<const float4*>(p);
  x[0] = v.x; x[1] = v.y; x[2] = v.z; x[3] = v.w;
}
__device__ __forceinline__ void dm_vec4(float* x, const bf16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  x[0] = __uint_as_float(v.x << 16); x[1] = __uint_as_float(v.x & 0xffff0000u);
  x[2] = __uint_as_float(v.y << 16); x[3] = __uint_as_float(v.y & 0xffff0000u);
}

// ---- which chunk is whose ------------------------------------------------------------------------------
__device__ __forceinline__ int dm_chunks(const int32_t* cu, int s) { return (cu[s + 1] - cu[s] + DM_C - 1) / DM_C; }

// Chunk t of the step, counted through its sequences: the sequence and the chunk inside it. Every wavefront finds it
// for itself (64 sequences a turn). False: the step has no chunk t.
__device__ __forceinline__ bool dm_find(int t, const int32_t* __restrict__ cu, int num_seqs, int& seq, int& chunk) {
  const int lane = threadIdx.x & 63;
  int base = 0;
  for (int s0 = 0; s0 < num_seqs; s0 += 64) {
    const int s = s0 + lane;
    const int n = s < num_seqs ? dm_chunks(cu, s) : 0;
    int upto = n;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int u = __shfl_up(upto, o);
      if (lane >= o) upto += u;
    }
    const unsigned long long hit = __ballot(t < base + upto);
    if (hit != 0) {
      const int f = __ffsll((long long)hit) - 1;
      seq = s0 + f;
      chunk = t - base - __shfl(upto - n, f);
      return true;
    }
    base += __shfl(upto, 63);
  }
  return false;
}

// what every kernel of a scan reads
template <typename T>
struct DmArgs {
  const T* q;                // the projected rows
  const T* k;
  const T* v;
  int64_t stride;            // elements between rows
  const float* powers;       // [H][DM_C + 1]: decay^0 .. decay^DM_C
  const float* inv_freq;     // [half]
  int half;
  int act;                   // q, k and v pass SiLU
  float k_scale;
  const int32_t* positions;
  const int32_t* cu;
  const int32_t* slot;
  int rows;                  // of the step; those from cu[num_seqs] on belong to no sequence
  int num_seqs, H, dk, dv;
  int dkp, dvp;              // dk and dv in fours
  uint8_t* state;
  int64_t state_stride, state_offset;
  // where chunks are used: the rows ready for the products, [rows][H][dkp] and [rows][H][dvp], and the window's
  // memories, [chunk of the window][H][dk][dvp]
  float* qf;
  float* kf;
  float* vf;
  float* ws;
};

// ---- the rows made ready for the chunks' products --------------------------------------------------------
// One workgroup a row: q, k and v as 32-bit numbers in heads of whole fours (zeros behind a head's own), through SiLU,
// q and k rotated by the row's position, k times its factor. VEC: widths and strides in fours, so that four neighbours
// (and their four partners in the rotation) are one load.
#define DM_MAX_HALF (DM_MAX_KEY / 2)
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void dm_ready_kernel(DmArgs<T> a) {
  __shared__ float cs[DM_MAX_HALF], sn[DM_MAX_HALF];
  const int64_t row = blockIdx.x;
  if (row >= a.cu[a.num_seqs]) return;
  for (int i = threadIdx.x; i < a.half; i += 256) sincos_angle((float)a.positions[row] * a.inv_freq[i], sn + i, cs + i);
  __syncthreads();
  const int qn = a.H * a.dkp / 4, vn = a.H * a.dvp / 4;
  for (int it = threadIdx.x; it < 2 * qn + vn; it += 256) {
    const int part = it < qn ? 0 : it < 2 * qn ? 1 : 2;          // q, k, v
    const int idx = it - part * qn, width = part == 2 ? a.dv : a.dk, wp = part == 2 ? a.dvp : a.dkp;
    const int h = 4 * idx / wp, d = 4 * idx - h * wp;
    const T* p = (part == 0 ? a.q : part == 1 ? a.k : a.v) + row * a.stride + (int64_t)h * width;
    float* out = (part == 0 ? a.qf : part == 1 ? a.kf : a.vf) + (row * a.H + h) * wp + d;
    float x[4], y[4] = {0.f, 0.f, 0.f, 0.f};
    const bool turns = part < 2 && d < 2 * a.half;
    if (VEC) {
      dm_vec4(x, p + d);
      if (turns) dm_vec4(y, p + (d < a.half ? d + a.half : d - a.half));
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        x[e] = d + e < width ? to_float(p[d + e]) : 0.f;
        if (turns && d + e < 2 * a.half) y[e] = to_float(p[d + e < a.half ? d + e + a.half : d + e - a.half]);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (a.act) x[e] = dm_silu(x[e]);
      if (turns && d + e < 2 * a.half) {
        if (a.act) y[e] = dm_silu(y[e]);
        const bool low = d + e < a.half;
        const int i = low ? d + e : d + e - a.half;
        x[e] = low ? x[e] * cs[i] - y[e] * sn[i] : x[e] * cs[i] + y[e] * sn[i];
      }
      if (part == 1) x[e] *= a.k_scale;
    }
    *reinterpret_cast<float4*>(out) = make_float4(x[0], x[1], x[2], x[3]);
  }
}

// Four numbers at dim d of a row of a chunk (n rows from `first` on, `stride` floats apart), zeros beyond the chunk or
// the head; the load itself stands behind no condition, so that a tile's loads go out together.
__device__ __forceinline__ float4 dm_tile4(const float* first, int64_t stride, int row, int n, int d, int width) {
  const float4 v = *reinterpret_cast<const float4*>(first + min(row, n - 1) * stride + (d < width ? d : 0));
  return row < n && d < width ? v : make_float4(0.f, 0.f, 0.f, 0.f);
}

// ---- every chunk's own share of the memory behind it -----------------------------------------------------
// One workgroup of four wavefronts a (64 key dims x 64 value dims, head, chunk); a wavefront 32 x 32 of it, two rows
// of the chunk an instruction (v_mfma_f32_32x32x2_f32: A lane l holds A[l % 32][l / 32], B likewise, D register r
// of lane l is D[8 (r / 4) + 4 (l / 32) + r % 4][l % 32]).
template <typename T>
__global__ __launch_bounds__(256) void dm_share_kernel(DmArgs<T> a, int t0) {
  __shared__ __attribute__((aligned(16))) float ks[DM_C * DM_LD], vs[DM_C * DM_LD];
  const int h = blockIdx.y;
  int seq, chunk;
  if (!dm_find(t0 + (int)blockIdx.z, a.cu, a.num_seqs, seq, chunk)) return;
  if (a.slot[seq] < 0) return;
  const int vb = (a.dvp + DM_B - 1) / DM_B;
  const int d0 = ((int)blockIdx.x / vb) * DM_B, c0 = ((int)blockIdx.x % vb) * DM_B;
  const int64_t r0 = a.cu[seq] + (int64_t)chunk * DM_C;
  const int n = min(DM_C, (int)(a.cu[seq + 1] - r0));
  const float* pw = a.powers + h * (DM_C + 1);
  const int t = threadIdx.x, d = 4 * (t & 15);
  const float* kr = a.kf + (r0 * a.H + h) * a.dkp;
  const float* vr = a.vf + (r0 * a.H + h) * a.dvp;
  float4 kx[4], vx[4];
  float fade[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (t >> 4) + 16 * i;
    kx[i] = dm_tile4(kr, (int64_t)a.H * a.dkp, row, n, d0 + d, a.dkp);
    vx[i] = dm_tile4(vr, (int64_t)a.H * a.dvp, row, n, c0 + d, a.dvp);
    fade[i] = pw[max(n - 1 - row, 0)];
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (t >> 4) + 16 * i;
    *reinterpret_cast<float4*>(ks + row * DM_LD + d) =
        make_float4(kx[i].x * fade[i], kx[i].y * fade[i], kx[i].z * fade[i], kx[i].w * fade[i]);
    *reinterpret_cast<float4*>(vs + row * DM_LD + d) = vx[i];
  }
  __syncthreads();
  const int wave = t >> 6, l32 = t & 31, hl = (t >> 5) & 1;
  const int i0 = (wave >> 1) * 32, j0 = (wave & 1) * 32;
  dm_acc acc = {0.f};
  for (int g = 0; g < n; g += 8) {
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int row = g + 4 * hl + m;
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ks[row * DM_LD + i0 + l32], vs[row * DM_LD + j0 + l32], acc, 0, 0, 0);
    }
  }
  float* out = a.ws + ((int64_t)blockIdx.z * a.H + h) * a.dk * a.dvp;
  const int col = c0 + j0 + l32;
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int od = d0 + i0 + 8 * (r >> 2) + 4 * hl + (r & 3);
    if (od < a.dk && col < a.dvp) out[(int64_t)od * a.dvp + col] = acc[r];
  }
}

// ---- the memory before every chunk ---------------------------------------------------------------------
// A thread holds four neighbouring elements of a sequence's S and walks its chunks in the window [t0, t0 + nt): the
// chunk's share is taken out, the memory before the chunk put in its place.
template <typename T>
__global__ __launch_bounds__(256) void dm_carry_kernel(DmArgs<T> a, int t0, int nt) {
  const int seq = blockIdx.z, h = blockIdx.y;
  const int slot = a.slot[seq];
  const int len = a.cu[seq + 1] - a.cu[seq];
  if (slot < 0 || len <= 0) return;
  int before = 0;
  for (int s0 = 0; s0 < seq; s0 += 64) {
    const int s = s0 + (int)(threadIdx.x & 63);
    int n = s < seq ? dm_chunks(a.cu, s) : 0;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o);
    before += n;
  }
  const int chunks = dm_chunks(a.cu, seq);
  const int first = max(0, t0 - before), end = min(chunks, t0 + nt - before);
  if (first >= end) return;
  const int64_t memory = (int64_t)a.dk * a.dvp;
  const int64_t at = 4 * (blockIdx.x * 256ll + threadIdx.x);
  if (at >= memory) return;
  float* st = reinterpret_cast<float*>(a.state + (int64_t)slot * a.state_stride + a.state_offset) + h * memory + at;
  const float full = a.powers[h * (DM_C + 1) + DM_C];
  const float tail = a.powers[h * (DM_C + 1) + len - (chunks - 1) * DM_C];      // of the sequence's last chunk
  float* w = a.ws + ((int64_t)(before + first - t0) * a.H + h) * memory + at;
  const int64_t step = (int64_t)a.H * memory;
  float4 S = *reinterpret_cast<const float4*>(st);
  constexpr int AHEAD = 8;
  for (int c = first; c < end; c += AHEAD) {
    float4 own[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
      own[u] = *reinterpret_cast<const float4*>(w + min(u, end - 1 - c) * step);
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      if (c + u < end) {
        const float f = c + u == chunks - 1 ? tail : full;
        *reinterpret_cast<float4*>(w + u * step) = S;
        S.x = fmaf(f, S.x, own[u].x);
        S.y = fmaf(f, S.y, own[u].y);
        S.z = fmaf(f, S.z, own[u].z);
        S.w = fmaf(f, S.w, own[u].w);
      }
    }
    w += AHEAD * step;
  }
  *reinterpret_cast<float4*>(st) = S;
}

// ---- every chunk's rows --------------------------------------------------------------------------------
// One workgroup of four wavefronts a (64 value dims, head, chunk), a wavefront 32 rows x 32 columns: the rows'
// products with the keys of the chunk (a square of which the part behind the diagonal is left out) and with the
// memory before it, block by block of 32 key dims; then the square, faded, on the values. One chunk more than the
// window's (`tail`): the step's rows that belong to no sequence get zeros.
#define DM_KB 32      // key dims of a block here
#define DM_KLD 36     // floats between its rows in LDS
template <typename T>
__global__ __launch_bounds__(256, 4) void dm_rows_kernel(float* __restrict__ y, DmArgs<T> a, int t0, int tail) {
  // rows of q, rows of k, key dims of the memory; later the square and the values
  __shared__ __attribute__((aligned(16))) float lds[2 * DM_C * DM_LD];
  static_assert(2 * DM_C * DM_KLD + DM_KB * DM_LD <= 2 * DM_C * DM_LD, "the blocks fit where the square and the values will be");
  float* qs = lds;
  float* ks = qs + DM_C * DM_KLD;
  float* ss = ks + DM_C * DM_KLD;
  float* square_s = lds;
  float* vs = lds + DM_C * DM_LD;
  __shared__ float pw[DM_C + 1];
  const int h = blockIdx.y;
  const int c0 = (int)blockIdx.x * DM_B;
  const int t = threadIdx.x, wave = t >> 6, l32 = t & 31, hl = (t >> 5) & 1;
  if (tail && blockIdx.z + 1 == gridDim.z) {
    const int col = c0 + (t & 63);
    if (col < a.dv)
      for (int64_t r = a.cu[a.num_seqs] + wave; r < a.rows; r += 4) y[r * a.H * a.dv + (int64_t)h * a.dv + col] = 0.f;
    return;
  }
  int seq, chunk;
  if (!dm_find(t0 + (int)blockIdx.z, a.cu, a.num_seqs, seq, chunk)) return;
  if (a.slot[seq] < 0) return;
  const int64_t r0 = a.cu[seq] + (int64_t)chunk * DM_C;
  const int n = min(DM_C, (int)(a.cu[seq + 1] - r0));
  const int i0 = (wave >> 1) * 32, j0 = (wave & 1) * 32;
  if (t <= DM_C) pw[t] = a.powers[h * (DM_C + 1) + t];
  const float* S = a.ws + ((int64_t)blockIdx.z * a.H + h) * a.dk * a.dvp;
  const float* qr = a.qf + (r0 * a.H + h) * a.dkp;
  const float* kr = a.kf + (r0 * a.H + h) * a.dkp;
  dm_acc square = {0.f}, out = {0.f};
  for (int d0 = 0; d0 < a.dk; d0 += DM_KB) {
    // thread t: rows t / 8 + 32 i and dims 4 (t % 8) of q and k; dims t / 16 + 16 i and columns 4 (t % 16) of the memory
    const int d = 4 * (t & 7), sc = 4 * (t & 15);
    float4 sx[2], qx[2], kx[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int sd = d0 + (t >> 4) + 16 * i;
      const bool there = sd < a.dk && c0 + sc < a.dvp;
      const float4 v = *reinterpret_cast<const float4*>(S + (there ? (int64_t)sd * a.dvp + c0 + sc : 0));
      sx[i] = there ? v : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      qx[i] = dm_tile4(qr, (int64_t)a.H * a.dkp, (t >> 3) + 32 * i, n, d0 + d, a.dkp);
      kx[i] = dm_tile4(kr, (int64_t)a.H * a.dkp, (t >> 3) + 32 * i, n, d0 + d, a.dkp);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      *reinterpret_cast<float4*>(qs + ((t >> 3) + 32 * i) * DM_KLD + d) = qx[i];
      *reinterpret_cast<float4*>(ks + ((t >> 3) + 32 * i) * DM_KLD + d) = kx[i];
      *reinterpret_cast<float4*>(ss + ((t >> 4) + 16 * i) * DM_LD + sc) = sx[i];
    }
    __syncthreads();
    const int dims = min(DM_KB, a.dk - d0);
    for (int g = 0; g < dims; g += 8) {
      float qa[4], ka[4];
      dm_vec4(qa, qs + (i0 + l32) * DM_KLD + g + 4 * hl);
      dm_vec4(ka, ks + (j0 + l32) * DM_KLD + g + 4 * hl);
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        if (j0 <= i0) square = __builtin_amdgcn_mfma_f32_32x32x2f32(qa[m], ka[m], square, 0, 0, 0);
        out = __builtin_amdgcn_mfma_f32_32x32x2f32(qa[m], ss[(g + 4 * hl + m) * DM_LD + j0 + l32], out, 0, 0, 0);
      }
    }
  }
  float4 vx[4];
  {
    const int d = 4 * (t & 15);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      vx[i] = dm_tile4(a.vf + (r0 * a.H + h) * a.dvp, (int64_t)a.H * a.dvp, (t >> 4) + 16 * i, n, c0 + d, a.dvp);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<float4*>(vs + ((t >> 4) + 16 * i) * DM_LD + d) = vx[i];
  }
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int i = i0 + 8 * (r >> 2) + 4 * hl + (r & 3), j = j0 + l32;
    square_s[i * DM_LD + j] = i >= j ? square[r] * pw[i - j] : 0.f;
    out[r] *= pw[i + 1];
  }
  __syncthreads();
  for (int g = 0; g < i0 + 32; g += 8) {      // rows up to the wavefront's last one
    float pa[4];
    dm_vec4(pa, square_s + (i0 + l32) * DM_LD + g + 4 * hl);
#pragma unroll
    for (int m = 0; m < 4; ++m)
      out = __builtin_amdgcn_mfma_f32_32x32x2f32(pa[m], vs[(g + 4 * hl + m) * DM_LD + j0 + l32], out, 0, 0, 0);
  }
  const int col = c0 + j0 + l32;
  if (col < a.dv) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = i0 + 8 * (r >> 2) + 4 * hl + (r & 3);
      if (i < n) y[(r0 + i) * a.H * a.dv + (int64_t)h * a.dv + col] = out[r];
    }
  }
}

// ---- a few rows a sequence -----------------------------------------------------------------------------
// One workgroup a (tile of 32 value dims, head, sequence). Thread t holds the value dims 4 (t % 8) .. + 3 of the
// tile and the key dims t / 8 + 32 e, e < E: its share of S is E runs of 16 bytes.
template <typename T, int E>
__global__ __launch_bounds__(256) void dm_step_kernel(float* __restrict__ y, DmArgs<T> a) {
  __shared__ float qs[32 * E], ks[32 * E], vs[DM_STEP_TILE], part[4][DM_STEP_TILE];
  const int seq = blockIdx.z, h = blockIdx.y;
  if (seq == a.num_seqs) {       // the step's rows that belong to no sequence get zeros
    const int col = (int)blockIdx.x * DM_STEP_TILE + (threadIdx.x & 31);
    if (col < a.dv)
      for (int64_t r = a.cu[seq] + (threadIdx.x >> 5); r < a.rows; r += 8) y[r * a.H * a.dv + (int64_t)h * a.dv + col] = 0.f;
    return;
  }
  const int slot = a.slot[seq];
  const int r0 = a.cu[seq], r1 = a.cu[seq + 1];
  if (slot < 0 || r0 >= r1) return;
  const int t = threadIdx.x, quad = t & 7, g = t >> 3, c0 = (int)blockIdx.x * DM_STEP_TILE;
  const bool active = c0 + 4 * quad < a.dvp;
  const int64_t memory = (int64_t)a.dk * a.dvp;
  float* st = reinterpret_cast<float*>(a.state + (int64_t)slot * a.state_stride + a.state_offset) + h * memory + c0 + 4 * quad;
  float S[E][4];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int d = g + 32 * e;
    if (active && d < a.dk) dm_vec4(S[e], st + (int64_t)d * a.dvp);
    else S[e][0] = S[e][1] = S[e][2] = S[e][3] = 0.f;
  }
  const float decay = a.powers[h * (DM_C + 1) + 1];
  for (int r = r0; r < r1; ++r) {
    const int64_t at = (int64_t)r * a.stride;
    const T* q = a.q + at + (int64_t)h * a.dk;
    const T* k = a.k + at + (int64_t)h * a.dk;
    for (int d = t; d < 32 * E; d += 256) {
      float qx = 0.f, kx = 0.f;
      if (d < a.dk) {
        qx = to_float(q[d]);
        kx = to_float(k[d]);
        if (a.act) { qx = dm_silu(qx); kx = dm_silu(kx); }
        if (d < 2 * a.half) {
          const bool lo = d < a.half;
          const int i = lo ? d : d - a.half, o = lo ? d + a.half : i;
          float qy = to_float(q[o]), ky = to_float(k[o]);
          if (a.act) { qy = dm_silu(qy); ky = dm_silu(ky); }
          float sn, cs;
          sincos_angle((float)a.positions[r] * a.inv_freq[i], &sn, &cs);
          if (lo) sn = -sn;
          qx = fmaf(qx, cs, qy * sn);
          kx = fmaf(kx, cs, ky * sn);
        }
        kx *= a.k_scale;
      }
      qs[d] = qx;
      ks[d] = kx;
    }
    if (t < DM_STEP_TILE) {
      float v = c0 + t < a.dv ? to_float(a.v[at + (int64_t)h * a.dv + c0 + t]) : 0.f;
      if (a.act) v = dm_silu(v);
      vs[t] = v;
    }
    __syncthreads();
    float p[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const float kd = ks[g + 32 * e], qd = qs[g + 32 * e];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        S[e][u] = fmaf(decay, S[e][u], kd * vs[4 * quad + u]);
        p[u] = fmaf(qd, S[e][u], p[u]);
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      p[u] = xor32_sum(p[u]);
      p[u] = xor16_sum(p[u]);
      p[u] += lane_xor8(p[u]);
    }
    if ((t & 63) < 8) {
#pragma unroll
      for (int u = 0; u < 4; ++u) part[t >> 6][4 * quad + u] = p[u];
    }
    __syncthreads();
    if (t < DM_STEP_TILE && c0 + t < a.dv)
      y[(int64_t)r * a.H * a.dv + (int64_t)h * a.dv + c0 + t] = (part[0][t] + part[1][t]) + (part[2][t] + part[3][t]);
  }
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int d = g + 32 * e;
    if (active && d < a.dk) *reinterpret_cast<float4*>(st + (int64_t)d * a.dvp) = make_float4(S[e][0], S[e][1], S[e][2], S[e][3]);
  }
}

template <typename T>
static int dm_run(float* y, DmArgs<T> a, int rows, int max_q_len, float* workspace, hipStream_t s) {
  if (max_q_len <= DM_WALK) {
    const dim3 grid((a.dv + DM_STEP_TILE - 1) / DM_STEP_TILE, a.H, a.num_seqs + 1);
    const int e = (a.dk + 31) / 32;
    if (e <= 1) dm_step_kernel<T, 1><<<grid, 256, 0, s>>>(y, a);
    else if (e <= 2) dm_step_kernel<T, 2><<<grid, 256, 0, s>>>(y, a);
    else if (e <= 4) dm_step_kernel<T, 4><<<grid, 256, 0, s>>>(y, a);
    else if (e <= 8) dm_step_kernel<T, 8><<<grid, 256, 0, s>>>(y, a);
    else dm_step_kernel<T, 16><<<grid, 256, 0, s>>>(y, a);
    return he_check_launch("he_decay_scan");
  }
  a.qf = workspace;
  a.kf = a.qf + (int64_t)rows * a.H * a.dkp;
  a.vf = a.kf + (int64_t)rows * a.H * a.dkp;
  a.ws = a.vf + (int64_t)rows * a.H * a.dvp;
  const int64_t memory = (int64_t)a.H * a.dk * a.dvp;
  const int window = (int)dm_window(rows, a.num_seqs, memory);
  const int chunks = rows / DM_C + a.num_seqs;
  const bool vec = a.dk % 4 == 0 && a.dv % 4 == 0 && a.half % 4 == 0 && a.stride % 4 == 0 &&
                   (((uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.v) & (4 * sizeof(T) - 1)) == 0;
  if (vec) dm_ready_kernel<T, true><<<rows, 256, 0, s>>>(a);
  else dm_ready_kernel<T, false><<<rows, 256, 0, s>>>(a);
  const int kb = (a.dk + DM_B - 1) / DM_B, vb = (a.dvp + DM_B - 1) / DM_B;
  for (int t0 = 0; t0 < chunks; t0 += window) {
    const int nt = chunks - t0 < window ? chunks - t0 : window;
    const dim3 share(kb * vb, a.H, nt), carry((unsigned)(((int64_t)a.dk * a.dvp / 4 + 255) / 256), a.H, a.num_seqs);
    const int tail = t0 + nt >= chunks;
    const dim3 out(vb, a.H, nt + tail);
    dm_share_kernel<T><<<share, 256, 0, s>>>(a, t0);
    dm_carry_kernel<T><<<carry, 256, 0, s>>>(a, t0, nt);
    dm_rows_kernel<T><<<out, 256, 0, s>>>(y, a, t0, tail);
  }
  return he_check_launch("he_decay_scan");
}

extern "C" int he_decay_scan(void* y_f32, const void* q, const void* k, const void* v, int64_t in_stride,
                             const void* powers_f32, int act, float k_scale, const void* inv_freq_f32, int half,
                             const void* positions, void* state, int64_t state_stride, int64_t state_offset,
                             const void* cu_seqlens, const void* seq_slot, int rows, int num_seqs, int max_q_len, int H,
                             int dk, int dv, void* workspace_f32, int64_t workspace_floats, int dtype, void* stream) {
  HE_REQUIRE(rows >= 0 && num_seqs >= 0 && H > 0 && dk > 0 && dv > 0, "he_decay_scan: bad sizes H=%d dk=%d dv=%d", H, dk, dv);
  HE_REQUIRE(H <= 65535 && num_seqs < 65535, "he_decay_scan: more than 65535 heads or sequences");
  HE_REQUIRE(dk <= DM_MAX_KEY, "he_decay_scan: key size %d above %d", dk, DM_MAX_KEY);
  HE_REQUIRE(dtype == HE_BF16 || dtype == HE_F32, "he_decay_scan: unknown dtype %d", dtype);
  HE_REQUIRE(half >= 0 && 2 * half <= dk && (half == 0 || (inv_freq_f32 != nullptr && positions != nullptr)),
             "he_decay_scan: %d rotated dims of %d", 2 * half, dk);
  HE_REQUIRE(state != nullptr && state_offset % 16 == 0 && state_stride % 16 == 0 && ((uintptr_t)state & 15) == 0 &&
                 state_stride >= state_offset + 4 * he_decay_state_floats(H, dk, dv),
             "he_decay_scan: the state row is too short or not aligned");
  const int64_t need = he_decay_workspace_floats(rows, num_seqs, max_q_len, H, dk, dv);
  HE_REQUIRE(need == 0 || (workspace_f32 != nullptr && workspace_floats >= need && ((uintptr_t)workspace_f32 & 15) == 0),
             "he_decay_scan: the workspace has %lld floats of %lld, or is not aligned", (long long)workspace_floats, (long long)need);
  if (rows == 0 || num_seqs == 0) return 0;
#define DM_FILL(T)                                                                                                     \
  DmArgs<T> a;                                                                                                         \
  a.q = (const T*)q; a.k = (const T*)k; a.v = (const T*)v; a.stride = in_stride; a.powers = (const float*)powers_f32;   \
  a.inv_freq = (const float*)inv_freq_f32; a.half = half; a.act = act; a.k_scale = k_scale;     \
  a.positions = (const int32_t*)positions; a.cu = (const int32_t*)cu_seqlens; a.slot = (const int32_t*)seq_slot;       \
  a.rows = rows; a.num_seqs = num_seqs; a.H = H; a.dk = dk; a.dv = dv; a.dkp = dm_fours(dk); a.dvp = dm_fours(dv); a.state = (uint8_t*)state;                 \
  a.state_stride = state_stride; a.state_offset = state_offset; a.qf = a.kf = a.vf = a.ws = nullptr;                   \
  return dm_run<T>((float*)y_f32, a, rows, max_q_len, (float*)workspace_f32, (hipStream_t)stream)
  if (dtype == HE_BF16) {
    DM_FILL(bf16_t);
  }
  DM_FILL(float);
#undef DM_FILL
}
