// Linear attention with one decay per head and token (decay_scan.hip says what it computes) for
// prompt portions: chunks of 128 rows on the matrix cores, all chunks of a step side by side.
//
// With b_t the running sum of the decays' logarithms inside a chunk (b_t <= 0) and S the state
// before it, the recurrence written out is
//
//   o_t = e^(r_t + m) S^T q_t + sum_{j <= t} P[t][j] v_j,   P[t][j] = (q_t . k_j) e^(r_t + c_j) w_j
//   S'  = e^(r_last + m) S + sum_j e^(r_last + c_j) w_j k_j v_j^T
//
// with, in the form kScanStep, r = b, c = -b, w = dt and m = 0; in the form kScanExp, c = i - b,
// w = 1, m the running maximum before the chunk and r_t = -max(m, max_{j <= t} c_j), so that the
// running maximum after row t is b_t - r_t. Every exponent is <= 0. The sum of the keys n and its
// product with the query are the same with v = 1. The running sums are formed in 64-bit and kept
// as two 32-bit numbers each: under strong decays they are large, and the exponents are their small
// differences.
//
//   scan_chunk_gates     b, c and w (or the running maximum of c) of every row: a wave per (chunk,
//                        head), two rows a lane, prefix sums and maxima by lane exchanges
//   scan_chunk_maxima    kScanExp: m before every chunk
//   scan_chunk_states    the sum in S' of every chunk by itself
//   scan_chunk_carry     the states before the chunks, in place: S <- E S + sum, a piece per thread
//   scan_chunk_outputs   the outputs
//
// Queries, keys and values are bfloat16 and enter v_mfma_f32_16x16x32_bf16 as they are. What is
// 32-bit (the state, P, the weighted values) enters as three bfloat16 numbers whose sum is the
// 32-bit one to its last bit or two, and the products of the three parts are added up in the
// 32-bit accumulators: three instructions where one would round, a fifth of what the 32-bit matrix
// instruction takes. Operands that have to be read along the rows (keys and values in the sums over
// rows, the state) come from LDS through the transposing read; a sum's terms may come in any order,
// so P goes from the accumulators of one product into the operand of the next without moving.
#include "decay_scan.h"

namespace ninfer {

constexpr int kScRows = 128;         // rows of a chunk
constexpr int kScMaxDim = 256;
constexpr int kScCt = 4;             // tiles of 16 value columns of a block
constexpr int kScCols = 16 * kScCt;
constexpr int kScVRow = kScCols + 8; // row length of values in LDS
constexpr float kScLog2e = 1.44269504088896f;

typedef __bf16 sc_bf16x8 __attribute__((ext_vector_type(8)));
typedef float sc_f32x4 __attribute__((ext_vector_type(4)));
typedef short sc_short4 __attribute__((ext_vector_type(4)));
typedef short sc_short8 __attribute__((ext_vector_type(8)));
typedef unsigned int sc_u32x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) sc_short4 sc_lds_short4;

struct ScanChunkArgs {
  ScanArgs s;
  float2* b;      // [H, T]       (pairs: a number and what its rounding left)
  float2* c;      // [H, T]
  float2* w;      // [H, T] (w, 0), or (kScanExp) the running maximum of c
  float2* b_last; // [chunks, H]
  float2* c_max;  // [chunks, H]
  float* m_in;    // [chunks, H]
  float* sums;    // [chunks, H, dim, vdim]: a chunk's sum, then the state before it
  float* keys;    // [chunks, H, dim]: the same of n
};

// Chunk `at` of the step (chunks of the requests from first_seq on, counted request after request).
__device__ __forceinline__ bool scan_find_chunk(const ScanArgs& a, int at, int* row0, int* rows) {
  for (int s = a.first_seq; s < a.S; ++s) {
    const int r = a.seq_row_start[s], n = a.seq_row_start[s + 1] - r;
    const int chunks = (n + kScRows - 1) / kScRows;
    if (at < chunks) {
      *row0 = r + at * kScRows;
      *rows = min(kScRows, n - at * kScRows);
      return true;
    }
    at -= chunks;
  }
  return false;
}

__device__ __forceinline__ float2 sc_pair(double x) {
  const float hi = (float)x;
  return make_float2(hi, (float)(x - (double)hi));
}
__device__ __forceinline__ double sc_double(float2 p) { return (double)p.x + (double)p.y; }
// -max(m, p) as a pair
__device__ __forceinline__ float2 sc_minus_max(float m, float2 p) {
  return (double)m > sc_double(p) ? make_float2(-m, 0.f) : make_float2(-p.x, -p.y);
}

__device__ __forceinline__ float sc_exp(float x) { return __builtin_amdgcn_exp2f(x * kScLog2e); }

__global__ __launch_bounds__(256) void scan_chunk_gates_kernel(ScanChunkArgs a) {
  int row0, L;
  if (!scan_find_chunk(a.s, blockIdx.x, &row0, &L)) return;
  const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6), H = a.s.H;
  if (h >= H) return;   // (no barrier below: a wave works alone)
  const bool exp_form = a.s.form == kScanExp;
  float g[2], in[2];   // the decay's logarithm; dt, or the write gate's logarithm
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int i = 2 * lane + e;
    g[e] = 0.f;
    in[e] = exp_form ? -1e30f : 0.f;
    if (i < L) {
      if (exp_form) {
        scan_exp_gates(a.s, row0 + i, h, &in[e], &g[e]);
      } else {
        in[e] = scan_softplus(a.s.z[(int64_t)(row0 + i) * H + h] + a.s.z_bias[h]);
        g[e] = -a.s.rate[h] * in[e];
      }
    }
  }
  double sum = (double)g[0] + (double)g[1];
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double up = __shfl_up(sum, off, 64);
    if (lane >= off) sum += up;
  }
  double before = __shfl_up(sum, 1, 64);
  if (lane == 0) before = 0.0;
  double b[2], c[2], w[2];
  b[0] = before + (double)g[0];
  b[1] = b[0] + (double)g[1];
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    c[e] = exp_form ? (double)in[e] - b[e] : -b[e];
    w[e] = in[e];
  }
  if (exp_form) {
    double mx = fmax(c[0], c[1]);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const double up = __shfl_up(mx, off, 64);
      if (lane >= off) mx = fmax(mx, up);
    }
    double mb = __shfl_up(mx, 1, 64);
    if (lane == 0) mb = -1e30;
    w[0] = fmax(mb, c[0]);
    w[1] = fmax(w[0], c[1]);
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int i = 2 * lane + e;
    if (i < L) {
      const int64_t at = (int64_t)h * a.s.T + row0 + i;
      a.b[at] = sc_pair(b[e]);
      a.c[at] = sc_pair(c[e]);
      a.w[at] = sc_pair(w[e]);
    }
  }
  if (lane == 63) {   // (rows beyond the last change neither)
    a.b_last[(int64_t)blockIdx.x * H + h] = sc_pair(b[1]);
    a.c_max[(int64_t)blockIdx.x * H + h] = sc_pair(w[1]);
  }
}

__global__ __launch_bounds__(64) void scan_chunk_maxima_kernel(ScanChunkArgs a) {
  const int s = a.s.first_seq + blockIdx.x, h = blockIdx.y * 64 + threadIdx.x, H = a.s.H;
  if (h >= H) return;
  int first = 0;
  for (int i = a.s.first_seq; i < s; ++i)
    first += (a.s.seq_row_start[i + 1] - a.s.seq_row_start[i] + kScRows - 1) / kScRows;
  const int count = (a.s.seq_row_start[s + 1] - a.s.seq_row_start[s] + kScRows - 1) / kScRows;
  float* m_at = a.s.state + (int64_t)a.s.seq_slots[s] * a.s.state_stride + (int64_t)H * a.s.dim * (a.s.vdim + 1) + h;
  float m = *m_at;
#pragma unroll 8
  for (int i = 0; i < count; ++i) {
    const int64_t at = (int64_t)(first + i) * H + h;
    const double bl = sc_double(a.b_last[at]), cm = sc_double(a.c_max[at]);
    a.m_in[at] = m;
    m = (float)(bl + fmax((double)m, cm));
  }
  *m_at = m;
}

// e^(r_last + m) of a chunk
__device__ __forceinline__ float scan_chunk_keep(const ScanChunkArgs& a, int64_t chunk_head) {
  if (a.s.form == kScanStep) return sc_exp(a.b_last[chunk_head].x);
  const float m = a.m_in[chunk_head];
  const float2 r = sc_minus_max(m, a.c_max[chunk_head]);
  return sc_exp((m + r.x) + r.y);
}

// x as three bfloat16 numbers
__device__ __forceinline__ void split3(float x, __bf16& p0, __bf16& p1, __bf16& p2) {
  p0 = (__bf16)x;
  const float r = x - (float)p0;
  p1 = (__bf16)r;
  p2 = (__bf16)(r - (float)p1);
}

// What a lane needs of an operand that lies in LDS row by row when the sum runs over the rows: rows
// `r` .. + 3 and `r + gap` .. + 3 (of this lane's group of 16 lanes) of its column. `p` points at
// the lane's place in row `r`: row + lane % 16 / 4, column + 4 (lane % 4).
__device__ __forceinline__ sc_bf16x8 tr_read(const unsigned short* p, int gap_elements) {
  const sc_short4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((sc_lds_short4*)p);
  const sc_short4 up = __builtin_amdgcn_ds_read_tr16_b64_v4i16((sc_lds_short4*)(p + gap_elements));
  sc_short8 both;
  both.s0 = lo.x; both.s1 = lo.y; both.s2 = lo.z; both.s3 = lo.w;
  both.s4 = up.x; both.s5 = up.y; both.s6 = up.z; both.s7 = up.w;
  return __builtin_bit_cast(sc_bf16x8, both);
}

// A block: the sum of one (chunk, head) in 64 value columns. Wave w owns the key channels' tiles
// of 16 w, w + 4, .. (at most 64 NPW channels). Every load is unconditional and under way before the
// first result is used: rows, channels and columns beyond the last are fetched from the last.
template <int NPW>
__global__ __launch_bounds__(256) void scan_chunk_states_kernel(ScanChunkArgs a) {
  constexpr int DP = 64 * NPW, KROW = DP + 8, KPC = DP / 8, KP = kScRows * KPC / 256;
  constexpr int VP = kScRows * 2 * kScCt / 256;
  extern __shared__ __attribute__((aligned(16))) unsigned short lds[];
  int row0, L;
  if (!scan_find_chunk(a.s, blockIdx.x, &row0, &L)) return;
  const int h = blockIdx.y, col0 = blockIdx.z * kScCols, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int dim = a.s.dim, vdim = a.s.vdim, H = a.s.H, g_head = h / (H / a.s.G);
  const int64_t chunk_head = (int64_t)blockIdx.x * H + h;
  unsigned short* k_s = lds;                        // [128][KROW]
  unsigned short* v_s = k_s + kScRows * KROW;       // [3][128][kScVRow]
  float* e_s = (float*)(v_s + 3 * kScRows * kScVRow);   // [128]
  const unsigned short* rows = (const unsigned short*)a.s.rows + (int64_t)row0 * a.s.stride;
  const sc_u32x4 zero4 = {0u, 0u, 0u, 0u};
  sc_u32x4 kreg[KP], vreg[VP];
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int p = i * 256 + tid, r = p / (2 * kScCt), d = 8 * (p % (2 * kScCt));
    vreg[i] = *(const sc_u32x4*)(rows + (int64_t)min(r, L - 1) * a.s.stride + a.s.v_off + h * vdim + min(col0 + d, vdim - 8));
  }
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int p = i * 256 + tid, r = p / KPC, d = 8 * (p % KPC);
    kreg[i] = *(const sc_u32x4*)(rows + (int64_t)min(r, L - 1) * a.s.stride + a.s.k_off + g_head * dim + min(d, dim - 8));
  }
  if (tid < kScRows) {
    const int64_t at = (int64_t)h * a.s.T + row0 + min(tid, L - 1);
    const bool step = a.s.form == kScanStep;
    const float2 r = step ? a.b_last[chunk_head] : sc_minus_max(a.m_in[chunk_head], a.c_max[chunk_head]);
    const float2 cj = a.c[at];
    const float e = sc_exp((r.x + cj.x) + (r.y + cj.y)) * (step ? a.w[at].x : 1.f);
    e_s[tid] = tid < L ? e : 0.f;
  }
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int p = i * 256 + tid, r = p / KPC, d = 8 * (p % KPC);
    *(sc_u32x4*)(k_s + r * KROW + d) = r < L && d < dim ? kreg[i] : zero4;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int p = i * 256 + tid, r = p / (2 * kScCt), d = 8 * (p % (2 * kScCt));
    union { __bf16 b[8]; sc_u32x4 v; } o[3];
    const float e = col0 + d < vdim ? e_s[r] : 0.f;   // (0 for rows beyond the last)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      split3(__uint_as_float(vreg[i][x] << 16) * e, o[0].b[2 * x], o[1].b[2 * x], o[2].b[2 * x]);
      split3(__uint_as_float(vreg[i][x] & 0xffff0000u) * e, o[0].b[2 * x + 1], o[1].b[2 * x + 1], o[2].b[2 * x + 1]);
    }
#pragma unroll
    for (int sp = 0; sp < 3; ++sp) *(sc_u32x4*)(v_s + (sp * kScRows + r) * kScVRow + d) = o[sp].v;
  }
  if (a.s.form == kScanExp && blockIdx.z == 0 && tid < dim) {   // (dim <= 256)
    float n[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int j = 0; j < kScRows; j += 4)
#pragma unroll
      for (int x = 0; x < 4; ++x)
        n[x] = fmaf(e_s[j + x], __uint_as_float((unsigned)k_s[(j + x) * KROW + tid] << 16), n[x]);
    a.keys[chunk_head * dim + tid] = (n[0] + n[1]) + (n[2] + n[3]);
  }
  __syncthreads();
  const int c = lane & 15, g = lane >> 4, n_tiles = (dim + 15) / 16, rows32 = (L + 31) / 32 * 32;
  sc_f32x4 acc[NPW][kScCt];
#pragma unroll
  for (int i = 0; i < NPW; ++i)
#pragma unroll
    for (int ct = 0; ct < kScCt; ++ct) acc[i][ct] = sc_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int j0 = 0; j0 < rows32; j0 += 32) {
    const int r = j0 + 8 * g + (c >> 2);
    sc_bf16x8 va[kScCt][3], kb[NPW];
#pragma unroll
    for (int i = 0; i < NPW; ++i) kb[i] = tr_read(k_s + r * KROW + 16 * (wave + 4 * i) + 4 * (c & 3), 4 * KROW);
#pragma unroll
    for (int ct = 0; ct < kScCt; ++ct)
#pragma unroll
      for (int sp = 0; sp < 3; ++sp)
        va[ct][sp] = tr_read(v_s + (sp * kScRows + r) * kScVRow + 16 * ct + 4 * (c & 3), 4 * kScVRow);
#pragma unroll
    for (int i = 0; i < NPW; ++i) {
      if (wave + 4 * i < n_tiles) {
#pragma unroll
        for (int sp = 2; sp >= 0; --sp)
#pragma unroll
          for (int ct = 0; ct < kScCt; ++ct)
            acc[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va[ct][sp], kb[i], acc[i][ct], 0, 0, 0);
      }
    }
  }
  // lane (c, g) holds channel 16 nt + c, value columns 16 ct + 4 g ..
#pragma unroll
  for (int i = 0; i < NPW; ++i) {
    const int d = 16 * (wave + 4 * i) + c;
    if (d >= dim) continue;
#pragma unroll
    for (int ct = 0; ct < kScCt; ++ct) {
      const int col = col0 + 16 * ct + 4 * g;
      if (col < vdim) *(sc_f32x4*)(a.sums + (chunk_head * dim + d) * vdim + col) = acc[i][ct];
    }
  }
}

__global__ __launch_bounds__(256) void scan_chunk_carry_kernel(ScanChunkArgs a) {
  const int s = a.s.first_seq + blockIdx.y, H = a.s.H, dim = a.s.dim, vdim = a.s.vdim;
  const int64_t n_state = (int64_t)H * dim * vdim;
  int64_t e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  const int64_t total = n_state + (a.s.form == kScanExp ? (int64_t)H * dim : 0);
  if (e >= total) return;
  int first = 0;
  for (int i = a.s.first_seq; i < s; ++i)
    first += (a.s.seq_row_start[i + 1] - a.s.seq_row_start[i] + kScRows - 1) / kScRows;
  const int count = (a.s.seq_row_start[s + 1] - a.s.seq_row_start[s] + kScRows - 1) / kScRows;
  sc_f32x4* slot = (sc_f32x4*)(a.s.state + (int64_t)a.s.seq_slots[s] * a.s.state_stride + e);
  const bool is_n = e >= n_state;
  if (is_n) e -= n_state;
  const int h = (int)(e / (is_n ? dim : (int64_t)dim * vdim));
  float* base = (is_n ? a.keys : a.sums) + e;
  const int64_t step = is_n ? (int64_t)H * dim : n_state;
  sc_f32x4 S = *slot;
#pragma unroll 4
  for (int i = 0; i < count; ++i) {
    sc_f32x4* at = (sc_f32x4*)(base + (first + i) * step);
    const sc_f32x4 sum = *at;
    const float keep = scan_chunk_keep(a, (int64_t)(first + i) * H + h);
    *at = S;
    S = S * keep + sum;
  }
  *slot = S;
}

// A block: the outputs of one (chunk, head) in 64 value columns; wave w owns rows 32 w .. + 31, in
// two tiles of 16. In the accumulators lane (c, g) holds row c of a tile and value columns 4 g ..
template <int KS, int FORM>
__global__ __launch_bounds__(256, KS <= 4 ? 3 : 1) void scan_chunk_outputs_kernel(ScanChunkArgs a) {
  constexpr int DP = 32 * KS, KROW = DP + 8;
  extern __shared__ __attribute__((aligned(16))) unsigned short lds[];
  __shared__ __attribute__((aligned(16))) float c_s[kScRows], cl_s[kScRows], w_s[kScRows];
  __shared__ float n_s[FORM == kScanExp ? DP : 1];
  int row0, L;
  if (!scan_find_chunk(a.s, blockIdx.x, &row0, &L)) return;
  const int h = blockIdx.y, col0 = blockIdx.z * kScCols, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int dim = a.s.dim, vdim = a.s.vdim, H = a.s.H, g_head = h / (H / a.s.G);
  const int c = lane & 15, g = lane >> 4;
  const int64_t chunk_head = (int64_t)blockIdx.x * H + h, gates0 = (int64_t)h * a.s.T + row0;
  const unsigned short* rows = (const unsigned short*)a.s.rows + (int64_t)row0 * a.s.stride;
  const sc_u32x4 zero4 = {0u, 0u, 0u, 0u};
  // All loads set out here, every one unconditional: rows, channels and columns beyond the last are
  // fetched from the last. First the state, then queries and gates, then keys and values, which
  // are not wanted before the state's part is done.
  constexpr int SP = DP * 4 * kScCt / 256, KPC = DP / 8, KP = kScRows * KPC / 256, VP = kScRows * 2 * kScCt / 256;
  sc_f32x4 sreg[SP];
  sc_u32x4 kreg[KP], vreg[VP];
  const float* S = a.sums + chunk_head * dim * vdim;
#pragma unroll
  for (int i = 0; i < SP; ++i) {
    const int p = i * 256 + tid, d = p / (4 * kScCt), col = 4 * (p % (4 * kScCt));
    sreg[i] = *(const sc_f32x4*)(S + (int64_t)min(d, dim - 1) * vdim + min(col0 + col, vdim - 4));
  }
  // this lane's queries (operand of both products)
  sc_bf16x8 qf[2][KS];
  float2 r_t[2];
  float scale_in[2];
  const float m_in = FORM == kScanExp ? a.m_in[chunk_head] : 0.f;
#pragma unroll
  for (int tt = 0; tt < 2; ++tt) {
    const int t = min(32 * wave + 16 * tt + c, L - 1);
    const unsigned short* qr = rows + (int64_t)t * a.s.stride + a.s.q_off + g_head * dim;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      qf[tt][ks] = __builtin_bit_cast(sc_bf16x8, *(const sc_u32x4*)(qr + min(32 * ks + 8 * g, dim - 8)));
    r_t[tt] = FORM == kScanExp ? a.w[gates0 + t] : a.b[gates0 + t];
  }
  const float2 c_t = a.c[gates0 + min(tid & (kScRows - 1), L - 1)], w_t = a.w[gates0 + min(tid & (kScRows - 1), L - 1)];
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int p = i * 256 + tid, r = p / KPC, d = 8 * (p % KPC);
    kreg[i] = *(const sc_u32x4*)(rows + (int64_t)min(r, L - 1) * a.s.stride + a.s.k_off + g_head * dim + min(d, dim - 8));
  }
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int p = i * 256 + tid, r = p / (2 * kScCt), d = 8 * (p % (2 * kScCt));
    vreg[i] = *(const sc_u32x4*)(rows + (int64_t)min(r, L - 1) * a.s.stride + a.s.v_off + h * vdim + min(col0 + d, vdim - 8));
  }
#pragma unroll
  for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      if (32 * ks + 8 * g >= dim) qf[tt][ks] = __builtin_bit_cast(sc_bf16x8, zero4);
    if (FORM == kScanExp) r_t[tt] = sc_minus_max(m_in, r_t[tt]);
    scale_in[tt] = sc_exp((m_in + r_t[tt].x) + r_t[tt].y);
  }
  if (tid < kScRows) {
    c_s[tid] = tid < L ? c_t.x : 0.f;
    cl_s[tid] = tid < L ? c_t.y : 0.f;
    w_s[tid] = FORM == kScanExp ? 1.f : tid < L ? w_t.x : 0.f;
  }
  // 1. the state before the chunk, in three parts: [3][DP][kScVRow]
#pragma unroll
  for (int i = 0; i < SP; ++i) {
    const int p = i * 256 + tid, d = p / (4 * kScCt), col = 4 * (p % (4 * kScCt));
    const bool in = d < dim && col0 + col < vdim;
    union { __bf16 b[4]; uint2 u; } o[3];
#pragma unroll
    for (int x = 0; x < 4; ++x) split3(in ? sreg[i][x] : 0.f, o[0].b[x], o[1].b[x], o[2].b[x]);
#pragma unroll
    for (int sp = 0; sp < 3; ++sp) *(uint2*)(lds + (sp * DP + d) * kScVRow + col) = o[sp].u;
  }
  if constexpr (FORM == kScanExp) {
    if (tid < DP) n_s[tid] = tid < dim ? a.keys[chunk_head * dim + tid] : 0.f;
  }
  __syncthreads();
  sc_f32x4 acc[kScCt][2];
#pragma unroll
  for (int ct = 0; ct < kScCt; ++ct)
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) acc[ct][tt] = sc_f32x4{0.f, 0.f, 0.f, 0.f};
  float dn[2] = {0.f, 0.f};
  const bool live = 32 * wave < L;
  if (live) {
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int r = 32 * ks + 8 * g + (c >> 2);
#pragma unroll
      for (int ct = 0; ct < kScCt; ++ct)
#pragma unroll
        for (int sp = 2; sp >= 0; --sp) {
          const sc_bf16x8 sa = tr_read(lds + (sp * DP + r) * kScVRow + 16 * ct + 4 * (c & 3), 4 * kScVRow);
#pragma unroll
          for (int tt = 0; tt < 2; ++tt)
            acc[ct][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sa, qf[tt][ks], acc[ct][tt], 0, 0, 0);
        }
      if constexpr (FORM == kScanExp) {
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
#pragma unroll
          for (int e = 0; e < 8; ++e) dn[tt] = fmaf((float)qf[tt][ks][e], n_s[32 * ks + 8 * g + e], dn[tt]);
      }
    }
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
      for (int ct = 0; ct < kScCt; ++ct) acc[ct][tt] *= scale_in[tt];
      dn[tt] *= scale_in[tt];
    }
  }
  __syncthreads();   // everyone has read the state: keys and values take its place
  // 2. keys [128][KROW] and values [128][kScVRow]
  unsigned short* k_s = lds;
  unsigned short* v_s = lds + kScRows * KROW;
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int p = i * 256 + tid, r = p / KPC, d = 8 * (p % KPC);
    *(sc_u32x4*)(k_s + r * KROW + d) = r < L && d < dim ? kreg[i] : zero4;
  }
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int p = i * 256 + tid, r = p / (2 * kScCt), d = 8 * (p % (2 * kScCt));
    *(sc_u32x4*)(v_s + r * kScVRow + d) = r < L && col0 + d < vdim ? vreg[i] : zero4;
  }
  __syncthreads();
  if (!live) return;
  for (int j0 = 0; j0 <= 32 * wave; j0 += 32) {
    // P^T: keys j0 + 16 jt + 4 g + x of row c
    sc_f32x4 s[2][2];
#pragma unroll
    for (int jt = 0; jt < 2; ++jt) {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) s[jt][tt] = sc_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const sc_bf16x8 ka = *(const sc_bf16x8*)(k_s + (j0 + 16 * jt + c) * KROW + 32 * ks + 8 * g);
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
          s[jt][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, qf[tt][ks], s[jt][tt], 0, 0, 0);
      }
    }
    sc_bf16x8 pb[3][2];
#pragma unroll
    for (int jt = 0; jt < 2; ++jt) {
      const int j = j0 + 16 * jt + 4 * g;
      const sc_f32x4 cj = *(const sc_f32x4*)(c_s + j), cl = *(const sc_f32x4*)(cl_s + j);
      const sc_f32x4 wj = *(const sc_f32x4*)(w_s + j);
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        const int t = 32 * wave + 16 * tt + c;
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          const float ex = (r_t[tt].x + cj[x]) + (r_t[tt].y + cl[x]);
          float p = s[jt][tt][x] * (sc_exp(fminf(ex, 0.f)) * wj[x]);
          if (j + x > t || j + x >= L) p = 0.f;
          dn[tt] += p;
          __bf16 p0, p1, p2;
          split3(p, p0, p1, p2);
          pb[0][tt][4 * jt + x] = p0;
          pb[1][tt][4 * jt + x] = p1;
          pb[2][tt][4 * jt + x] = p2;
        }
      }
    }
#pragma unroll
    for (int ct = 0; ct < kScCt; ++ct) {
      const sc_bf16x8 va = tr_read(v_s + (j0 + 4 * g + (c >> 2)) * kScVRow + 16 * ct + 4 * (c & 3), 16 * kScVRow);
#pragma unroll
      for (int sp = 2; sp >= 0; --sp)
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
          acc[ct][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pb[sp][tt], acc[ct][tt], 0, 0, 0);
    }
  }
  const float skip = FORM == kScanStep ? a.s.skip[h] : 0.f;
#pragma unroll
  for (int tt = 0; tt < 2; ++tt) {
    const int t = 32 * wave + 16 * tt + c;
    if constexpr (FORM == kScanExp) {
      dn[tt] += __shfl_xor(dn[tt], 16, 64);
      dn[tt] += __shfl_xor(dn[tt], 32, 64);
      if (t < L && g == 0 && blockIdx.z == 0) {
        const float2 b = a.b[gates0 + t];
        a.s.den[(int64_t)(row0 + t) * H + h] =
            fmaxf(fabsf(dn[tt] * a.s.q_scale), sc_exp((r_t[tt].x - b.x) + (r_t[tt].y - b.y))) + 1e-6f;
      }
    }
    if (t >= L) continue;
    float* o = a.s.out + ((int64_t)(row0 + t) * H + h) * vdim + col0;
#pragma unroll
    for (int ct = 0; ct < kScCt; ++ct) {
      const int col = 16 * ct + 4 * g;
      if (col0 + col >= vdim) continue;
      sc_f32x4 y = acc[ct][tt] * a.s.q_scale;
      if constexpr (FORM == kScanStep) {
        const uint2 v = *(const uint2*)(v_s + t * kScVRow + col);
        y[0] = fmaf(skip, __uint_as_float(v.x << 16), y[0]);
        y[1] = fmaf(skip, __uint_as_float(v.x & 0xffff0000u), y[1]);
        y[2] = fmaf(skip, __uint_as_float(v.y << 16), y[2]);
        y[3] = fmaf(skip, __uint_as_float(v.y & 0xffff0000u), y[3]);
      }
      *(sc_f32x4*)(o + col) = y;
    }
  }
}

static int64_t most_chunks(const ScanArgs& a) { return a.T / kScRows + a.S - a.first_seq; }   // no step has more

bool scan_chunks_take(const ScanArgs& a) {
  return a.dtype == kBF16 && a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= kScMaxDim && a.stride % 8 == 0 &&
         a.q_off % 8 == 0 && a.k_off % 8 == 0 && a.v_off % 8 == 0 && (uintptr_t)a.rows % 16 == 0 &&
         a.state_stride % 4 == 0 && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.out % 16 == 0;
}

int64_t scan_chunks_work_floats(const ScanArgs& a) {
  const int64_t n = most_chunks(a), gates = ((int64_t)6 * a.H * a.T + 5 * n * a.H + 3) / 4 * 4;
  return gates + n * a.H * a.dim * (a.vdim + (a.form == kScanExp ? 1 : 0));
}

template <typename K>
static int scan_lds(K kern, size_t lds, bool* raised) {
  if (lds > 64 * 1024 && !*raised) {
    hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024);
    if (e != hipSuccess) return set_error(-2, "decay_scan: %zu bytes of LDS refused: %s", lds, hipGetErrorString(e));
    *raised = true;
  }
  return 0;
}

template <int NPW>
static int launch_states(const ScanChunkArgs& a, dim3 grid, hipStream_t stream) {
  const size_t lds = ((size_t)kScRows * (64 * NPW + 8) + 3 * kScRows * kScVRow) * 2 + kScRows * sizeof(float);
  static bool raised = false;
  if (int rc = scan_lds(scan_chunk_states_kernel<NPW>, lds, &raised)) return rc;
  scan_chunk_states_kernel<NPW><<<grid, 256, lds, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return 0;
}

template <int KS, int FORM>
static int launch_outputs(const ScanChunkArgs& a, dim3 grid, hipStream_t stream) {
  constexpr size_t state = (size_t)3 * 32 * KS * kScVRow * 2, rows = (size_t)kScRows * (32 * KS + 8 + kScVRow) * 2;
  constexpr size_t lds = state > rows ? state : rows;
  static bool raised = false;
  if (int rc = scan_lds(scan_chunk_outputs_kernel<KS, FORM>, lds, &raised)) return rc;
  scan_chunk_outputs_kernel<KS, FORM><<<grid, 256, lds, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return 0;
}

int scan_chunks(const ScanArgs& s, hipStream_t stream) {
  ScanChunkArgs a;
  a.s = s;
  const int64_t n = most_chunks(s), ht = (int64_t)s.H * s.T;
  a.b = (float2*)s.work;
  a.c = a.b + ht;
  a.w = a.c + ht;
  a.b_last = a.w + ht;
  a.c_max = a.b_last + n * s.H;
  a.m_in = (float*)(a.c_max + n * s.H);
  a.sums = s.work + (6 * ht + 5 * n * s.H + 3) / 4 * 4;
  a.keys = a.sums + n * s.H * s.dim * s.vdim;
  scan_chunk_gates_kernel<<<dim3(n, (s.H + 3) / 4), 256, 0, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  const int seqs = s.S - s.first_seq;
  if (s.form == kScanExp) {
    scan_chunk_maxima_kernel<<<dim3(seqs, (s.H + 63) / 64), 64, 0, stream>>>(a);
    NINFER_LAUNCH_CHECK();
  }
  const dim3 grid(n, s.H, (s.vdim + kScCols - 1) / kScCols);
  const int tiles = (s.dim + 15) / 16;
  int rc = tiles <= 4 ? launch_states<1>(a, grid, stream) : tiles <= 8 ? launch_states<2>(a, grid, stream)
                                                                       : launch_states<4>(a, grid, stream);
  if (rc) return rc;
  const int64_t pieces = ((int64_t)s.H * s.dim * (s.vdim + (s.form == kScanExp ? 1 : 0)) / 4 + 255) / 256;
  scan_chunk_carry_kernel<<<dim3(pieces, seqs), 256, 0, stream>>>(a);
  NINFER_LAUNCH_CHECK();
#define NINFER_SCAN_OUT(FORM)                                                    \
  return s.dim <= 64 ? launch_outputs<2, FORM>(a, grid, stream)                  \
                     : s.dim <= 128 ? launch_outputs<4, FORM>(a, grid, stream)   \
                                    : launch_outputs<8, FORM>(a, grid, stream)
  if (s.form == kScanExp) NINFER_SCAN_OUT(kScanExp);
  NINFER_SCAN_OUT(kScanStep);
#undef NINFER_SCAN_OUT
}

}  // namespace ninfer

using namespace ninfer;

// Floats of workspace with which requests first_seq .. of this step run in chunks; 0 when the
// sizes do not fit (the row-by-row kernels take them).
extern "C" long long ninfer_decay_scan_chunk_floats(const ScanArgs* a) {
  return scan_chunks_take(*a) ? scan_chunks_work_floats(*a) : 0;
}

extern "C" int ninfer_decay_scan_chunks(const ScanArgs* args, hipStream_t stream) {
  const ScanArgs& a = *args;
  if (int rc = scan_check(a)) return rc;
  NINFER_REQUIRE(scan_chunks_take(a), "decay_scan: these sizes do not run in chunks");
  NINFER_REQUIRE(a.work && (uintptr_t)a.work % 16 == 0 && a.out && (a.form == kScanStep || a.den),
                 "decay_scan: no room for gates or outputs");
  return scan_chunks(a, stream);
}
