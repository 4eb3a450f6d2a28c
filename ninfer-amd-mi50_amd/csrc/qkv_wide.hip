// What lies between the q/k/v product and attention when queries and keys are normed over their
// whole projections, in one kernel (a block per row):
//
//   q' = q rsqrt(mean(q^2) + eps) gain   over all Hq * dim numbers of the row (k alike over its
//        Hkv * dim; gains null: no norm), before the numbers are split into heads;
//   the first rot_dim numbers of every head turn by pos * inv_freq[i], cosine and sine times
//        `magnitude`: pair i is (i, i + rot_dim / 2), or the neighbours (2i, 2i + 1) when
//        `interleaved`; a query head is multiplied by head_scale[h] where that is given (a
//        factor on the head's scores);
//   with `unit_heads` every query and key head is divided by its root mean square instead (over
//        its dim numbers, eps inside the root, no gain): before or after it turns is the same, a
//        rotation keeps the sum of the squares (`magnitude` is 1 then);
//   queries go to q_out [T, Hq * dim]; keys and values to the request's pages. Values are columns
//        of the projected row from v_col on: columns of their own, or the keys' own columns
//        (values that are the keys as projected, before norm and rotation).
//
// With `block` > 0 the cache also holds one key and one value for every whole block of `block`
// tokens: the means of what the pages hold for them (rounded as they are there), formed in
// 32-bit in the order of the positions. In steps in which every request brings one row the
// row's own block of threads forms the means of the block its token completes; otherwise a
// second kernel does so for all blocks that the step completes, with the same sums.
// All sums are 32-bit; their order depends on the sizes alone.
#include "common.h"

namespace ninfer {

struct QkvWideArgs {
  const void* u;            // [T, stride] projected rows
  void* q_out;              // [T, Hq * dim]
  void* kpool;              // [pages, Hkv, page_size, dim]
  void* vpool;              // [pages, Hkv, page_size, vdim]
  const int* block_table;   // [S, bt_stride]
  void* kblk;               // [pages, Hkv, blk_page_size, dim], or null
  void* vblk;               // [pages, Hkv, blk_page_size, vdim]
  const int* blk_table;     // [S, blk_bt_stride]
  const int* positions;     // [T]
  const int* row_seq;       // [T]
  const int* seq_row_start; // [S + 1]
  const int* seq_pos0;      // [S]
  const float* q_gain;      // [Hq * dim] or null
  const float* k_gain;      // [Hkv * dim] or null
  const float* inv_freq;    // [rot_dim / 2] or null
  const float* head_scale;  // [Hq] or null
  int stride;
  int q_col;
  int k_col;
  int v_col;
  int bt_stride;
  int blk_bt_stride;
  int T;
  int S;
  int Hq;
  int Hkv;
  int dim;
  int vdim;
  int rot_dim;
  int interleaved;
  int page_size;
  int blk_page_size;
  int block;                // tokens of a block (0: no means are kept)
  int dtype;
  float eps;
  float magnitude;
  int all_single;           // every request of the step brings one row
  int force_plain;          // tests: 1 the kernel of single numbers, 2 the kernel of whole pieces
  int unit_heads;           // every query and key head divided by its root mean square
};

constexpr int kWideThreads = 256;
constexpr int kWideMaxLds = 150 * 1024;
typedef unsigned int wide_u32x4 __attribute__((ext_vector_type(4)));

// VEC consecutive numbers as 32-bit ones and back
template <typename T, int VEC>
__device__ __forceinline__ void wide_load(const T* p, float* f) {
  if constexpr (VEC == 8) {
    const wide_u32x4 v = *(const wide_u32x4*)p;
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
    f[4] = __uint_as_float(v.z << 16); f[5] = __uint_as_float(v.z & 0xffff0000u);
    f[6] = __uint_as_float(v.w << 16); f[7] = __uint_as_float(v.w & 0xffff0000u);
  } else {
    f[0] = to_f32(p[0]);
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void wide_store(T* p, const float* f) {
  if constexpr (VEC == 8) {
    union { __bf16 b[8]; wide_u32x4 v; } o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o.b[e] = (__bf16)f[e];
    *(wide_u32x4*)p = o.v;
  } else {
    p[0] = from_f32<T>(f[0]);
  }
}

// The mean of VEC numbers (from number e0 of the keys, or of the values when `is_v`) over the
// block's positions first .. first + block - 1; the last position's numbers come from `last`
// when that is given (they are on their way to the page).
template <typename T, int VEC>
__device__ __forceinline__ void wide_block_mean(const QkvWideArgs& a, const int* bt, bool is_v, int e0,
                                                int first, const float* last, float* out) {
  const int n = is_v ? a.vdim : a.dim;
  const T* pool = (const T*)(is_v ? a.vpool : a.kpool);
  const int g = e0 / n, d = e0 - g * n;
  float sum[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) sum[e] = 0.f;
  const int upto = a.block - (last ? 1 : 0);
#pragma unroll 8
  for (int j = 0; j < upto; ++j) {
    const int p = first + j;
    float v[VEC];
    wide_load<T, VEC>(pool + (((int64_t)bt[p / a.page_size] * a.Hkv + g) * a.page_size + p % a.page_size) * n + d, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) sum[e] += v[e];
  }
  if (last) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) sum[e] += last[e];
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) out[e] = sum[e] / (float)a.block;
}

template <typename T, int VEC>
__device__ __forceinline__ void wide_store_mean(const QkvWideArgs& a, int seq, bool is_v, int e0, int b, const float* m) {
  const int n = is_v ? a.vdim : a.dim;
  T* pool = (T*)(is_v ? a.vblk : a.kblk);
  const int g = e0 / n, d = e0 - g * n;
  const int64_t page = a.blk_table[(int64_t)seq * a.blk_bt_stride + b / a.blk_page_size];
  wide_store<T, VEC>(pool + ((page * a.Hkv + g) * a.blk_page_size + b % a.blk_page_size) * n + d, m);
}

// A thread moves pieces of VEC consecutive numbers; the row's queries and keys lie in LDS in
// 32-bit between the two phases (sums of squares; norm, rotation, stores). VEC 8 wants heads
// of whole pieces, and whole pieces in each half of the turning numbers unless the pairs are
// neighbours.
template <typename T, int VEC>
__global__ __launch_bounds__(kWideThreads) void qkv_wide_kernel(QkvWideArgs a) {
  extern __shared__ float smem[];
  __shared__ float red[2][kWideThreads / 64];
  const int nq = a.Hq * a.dim, nk = a.Hkv * a.dim, nv = a.Hkv * a.vdim;
  float* row_s = smem;                 // [nq + nk]
  float* trig = row_s + nq + nk;       // [rot_dim]: cos, then sin
  float* inv_s = trig + a.rot_dim;     // [Hq + Hkv] 1 / root mean square of each head, with unit_heads
  const int t = blockIdx.x, tid = threadIdx.x;
  const int s = a.row_seq[t], pos = a.positions[t];
  const int half = a.rot_dim / 2;
  const T* u = (const T*)a.u + (int64_t)t * a.stride;
  const int* bt = a.block_table + (int64_t)s * a.bt_stride;
  for (int i = tid; i < half; i += kWideThreads) {
    float sn, cs;
    sincosf((float)pos * a.inv_freq[i], &sn, &cs);
    trig[i] = cs * a.magnitude;
    trig[half + i] = sn * a.magnitude;
  }
  float sq = 0.f, sk = 0.f;
  for (int i = VEC * tid; i < nq + nk; i += VEC * kWideThreads) {
    float x[VEC];
    wide_load<T, VEC>(i < nq ? u + a.q_col + i : u + a.k_col + (i - nq), x);
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      ss = fmaf(x[e], x[e], ss);
      row_s[i + e] = x[e];
    }
    if (i < nq) sq += ss;
    else sk += ss;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) red[0][tid >> 6] = sq, red[1][tid >> 6] = sk;
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < kWideThreads / 64; ++i) sq += red[0][i], sk += red[1][i];
  const float inv_q = a.q_gain ? 1.f / sqrtf(sq / (float)nq + a.eps) : 1.f;
  const float inv_k = a.k_gain ? 1.f / sqrtf(sk / (float)nk + a.eps) : 1.f;
  if (a.unit_heads) {   // a wave per head
    for (int hd = tid >> 6; hd < a.Hq + a.Hkv; hd += kWideThreads / 64) {
      float ss = 0.f;
      for (int d = tid & 63; d < a.dim; d += 64) ss = fmaf(row_s[hd * a.dim + d], row_s[hd * a.dim + d], ss);
      ss = wave_sum(ss);
      if ((tid & 63) == 0) inv_s[hd] = 1.f / sqrtf(ss / (float)a.dim + a.eps);
    }
    __syncthreads();
  }
  const int64_t page = bt[pos / a.page_size];
  const int slot = pos % a.page_size;
  // the block that this row's token completes, when the row itself forms its means
  const bool means = a.block > 0 && a.all_single && (pos + 1) % a.block == 0;
  const int b = means ? pos / a.block : 0;

  for (int i = VEC * tid; i < nq + nk; i += VEC * kWideThreads) {
    const bool is_q = i < nq;
    const int j0 = is_q ? i : i - nq;            // in the projection
    const int hd = j0 / a.dim, d0 = j0 - hd * a.dim;
    const float* head = row_s + i - d0;
    const float* gain = is_q ? a.q_gain : a.k_gain;
    const float* hg = gain ? gain + j0 - d0 : nullptr;
    const float inv = a.unit_heads ? inv_s[is_q ? hd : a.Hq + hd] : is_q ? inv_q : inv_k;
    const float plain = a.unit_heads ? inv : 1.f;   // the factor where there are no gains
    float x[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] = head[d0 + e] * (hg ? inv * hg[d0 + e] : plain);
    if constexpr (VEC == 8) {
      if (a.interleaved) {
#pragma unroll
        for (int e = 0; e < VEC; e += 2) {
          if (d0 + e < a.rot_dim) {
            const int p = (d0 + e) >> 1;
            const float cs = trig[p], sn = trig[half + p], x0 = x[e], x1 = x[e + 1];
            x[e] = x0 * cs - x1 * sn;
            x[e + 1] = x1 * cs + x0 * sn;
          }
        }
      } else if (d0 < a.rot_dim) {   // (a piece lies wholly in one half, and so does its partner)
        const bool first = d0 < half;
        const int o0 = first ? d0 + half : d0 - half, p0 = first ? d0 : d0 - half;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          const float y = head[o0 + e] * (hg ? inv * hg[o0 + e] : plain);
          const float cs = trig[p0 + e], sn = trig[half + p0 + e];
          x[e] = first ? x[e] * cs - y * sn : x[e] * cs + y * sn;
        }
      }
    } else if (d0 < a.rot_dim) {
      const bool first = a.interleaved ? !(d0 & 1) : d0 < half;
      const int o = a.interleaved ? d0 ^ 1 : first ? d0 + half : d0 - half;
      const int p = a.interleaved ? d0 >> 1 : first ? d0 : d0 - half;
      const float y = head[o] * (hg ? inv * hg[o] : plain);
      x[0] = first ? x[0] * trig[p] - y * trig[half + p] : x[0] * trig[p] + y * trig[half + p];
    }
    if (is_q) {
      if (a.head_scale) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[e] *= a.head_scale[hd];
      }
      wide_store<T, VEC>((T*)a.q_out + (int64_t)t * nq + i, x);
    } else {
      wide_store<T, VEC>((T*)a.kpool + ((page * a.Hkv + hd) * a.page_size + slot) * a.dim + d0, x);
      if (means) {
        float own[VEC], m[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) own[e] = to_f32(from_f32<T>(x[e]));   // as the page holds it
        wide_block_mean<T, VEC>(a, bt, false, j0, b * a.block, own, m);
        wide_store_mean<T, VEC>(a, s, false, j0, b, m);
      }
    }
  }
  for (int i = VEC * tid; i < nv; i += VEC * kWideThreads) {
    float x[VEC];
    wide_load<T, VEC>(u + a.v_col + i, x);
    const int g = i / a.vdim, d0 = i - g * a.vdim;
    wide_store<T, VEC>((T*)a.vpool + ((page * a.Hkv + g) * a.page_size + slot) * a.vdim + d0, x);
    if (means) {
      float m[VEC];
      wide_block_mean<T, VEC>(a, bt, true, i, b * a.block, x, m);
      wide_store_mean<T, VEC>(a, s, true, i, b, m);
    }
  }
}

// The same for bfloat16 rows of whole pieces, ROWS rows to a block of as many threads as a row
// has pieces of queries and keys: a thread keeps its piece's gains and its piece of every row
// in registers, so that gains are fetched once for ROWS rows and the rows' loads are under way
// together; only pieces whose partners lie in another thread's (half-split pairs) go through
// LDS. One barrier.
constexpr int kWideRowsMaxThreads = 1024;
template <int ROWS>
__global__ __launch_bounds__(kWideRowsMaxThreads) void qkv_wide_rows_kernel(QkvWideArgs a) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  __shared__ float red[ROWS][kWideRowsMaxThreads / 64][2];
  const int nq = a.Hq * a.dim, nk = a.Hkv * a.dim, nv = a.Hkv * a.vdim;
  const int tid = threadIdx.x, nt = blockDim.x, wave = tid >> 6;
  const int half = a.rot_dim / 2, t0 = blockIdx.x * ROWS;
  float* trig = smem;                          // [ROWS][rot_dim]: cos, then sin
  float* x_s = smem + ROWS * a.rot_dim;        // [ROWS][nq + nk], for half-split pairs
  // [ROWS][pieces] the squares' sums of the pieces, with unit_heads
  float* piece_s = x_s + (a.interleaved ? 0 : ROWS * (nq + nk));
  const int i = 8 * tid;
  const bool live = i < nq + nk, is_q = i < nq;
  const int j0 = is_q ? i : i - nq;
  const int hd = j0 / a.dim, d0 = j0 - hd * a.dim;
  const bool split = !a.interleaved && d0 < a.rot_dim;   // the partners are another piece
  const float* gain = is_q ? a.q_gain : a.k_gain;
  wide_u32x4 raw[ROWS];
  int pos[ROWS], seq[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int t = min(t0 + r, a.T - 1);
    pos[r] = a.positions[t];
    seq[r] = a.row_seq[t];
    const unsigned short* u = (const unsigned short*)a.u + (int64_t)t * a.stride;
    raw[r] = live ? *(const wide_u32x4*)(u + (is_q ? a.q_col : a.k_col) + j0) : wide_u32x4{0u, 0u, 0u, 0u};
  }
  float g[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) g[e] = 1.f;
  if (gain && live) {
    const float4 g0 = *(const float4*)(gain + j0), g1 = *(const float4*)(gain + j0 + 4);
    g[0] = g0.x; g[1] = g0.y; g[2] = g0.z; g[3] = g0.w; g[4] = g1.x; g[5] = g1.y; g[6] = g1.z; g[7] = g1.w;
  }
  for (int idx = tid; idx < ROWS * half; idx += nt) {
    const int r = idx / half, p = idx - r * half;
    float sn, cs;
    sincosf((float)a.positions[min(t0 + r, a.T - 1)] * a.inv_freq[p], &sn, &cs);
    trig[r * a.rot_dim + p] = cs * a.magnitude;
    trig[r * a.rot_dim + half + p] = sn * a.magnitude;
  }
  const bool has_q = wave * 512 < nq, has_k = wave * 512 + 511 >= nq;
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    float f[8], ss = 0.f;
    wide_load<bf16, 8>((const bf16*)&raw[r], f);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(f[e], f[e], ss);
    if (live && split) {
      float* dst = x_s + r * (nq + nk) + i;
      *(float4*)dst = make_float4(f[0] * g[0], f[1] * g[1], f[2] * g[2], f[3] * g[3]);
      *(float4*)(dst + 4) = make_float4(f[4] * g[4], f[5] * g[5], f[6] * g[6], f[7] * g[7]);
    }
    if (a.unit_heads) {
      if (live) piece_s[r * ((nq + nk) / 8) + tid] = ss;
      continue;
    }
    const float sq = has_q ? wave_sum(is_q ? ss : 0.f) : 0.f;
    const float sk = has_k ? wave_sum(is_q ? 0.f : ss) : 0.f;
    if ((tid & 63) == 0) red[r][wave][0] = sq, red[r][wave][1] = sk;
  }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int t = t0 + r;
    if (t >= a.T) break;
    float sum = 0.f, over = (float)(is_q ? nq : nk);
    if (a.unit_heads) {   // (heads of whole pieces: the piece's head begins d0 / 8 pieces before it)
      const float* p = piece_s + r * ((nq + nk) / 8) + (live ? tid - d0 / 8 : 0);
      for (int i = 0; i < a.dim / 8; ++i) sum += p[i];
      over = (float)a.dim;
    } else {
      for (int w = 0; w < nt / 64; ++w) sum += red[r][w][is_q ? 0 : 1];
    }
    const float inv = gain || a.unit_heads ? 1.f / sqrtf(sum / over + a.eps) : 1.f;
    const int* bt = a.block_table + (int64_t)seq[r] * a.bt_stride;
    const int64_t page = bt[pos[r] / a.page_size];
    const int slot = pos[r] % a.page_size;
    const bool means = ROWS == 1 && a.block > 0 && a.all_single && (pos[r] + 1) % a.block == 0;
    const int b = means ? pos[r] / a.block : 0;
    const float* tr = trig + r * a.rot_dim;
    if (live) {
      float x[8];
      wide_load<bf16, 8>((const bf16*)&raw[r], x);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= inv * g[e];
      if (split) {
        const bool first = d0 < half;
        const float* other = x_s + r * (nq + nk) + i + (first ? half : -half);
        const int p0 = first ? d0 : d0 - half;
        const float4 y0 = *(const float4*)other, y1 = *(const float4*)(other + 4);
        const float y[8] = {y0.x, y0.y, y0.z, y0.w, y1.x, y1.y, y1.z, y1.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float cs = tr[p0 + e], sn = tr[half + p0 + e], z = y[e] * inv * sn;
          x[e] = first ? x[e] * cs - z : x[e] * cs + z;
        }
      } else if (d0 < a.rot_dim) {
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          if (d0 + e < a.rot_dim) {
            const int p = (d0 + e) >> 1;
            const float cs = tr[p], sn = tr[half + p], x0 = x[e], x1 = x[e + 1];
            x[e] = x0 * cs - x1 * sn;
            x[e + 1] = x1 * cs + x0 * sn;
          }
        }
      }
      if (is_q) {
        if (a.head_scale) {
          const float hs = a.head_scale[hd];
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] *= hs;
        }
        wide_store<bf16, 8>((bf16*)a.q_out + (int64_t)t * nq + i, x);
      } else {
        const int64_t at = ((page * a.Hkv + hd) * a.page_size + slot) * a.dim + d0;
        wide_store<bf16, 8>((bf16*)a.kpool + at, x);
        if (means) {
          float own[8], m[8];
#pragma unroll
          for (int e = 0; e < 8; ++e) own[e] = to_f32(from_f32<bf16>(x[e]));   // as the page holds it
          wide_block_mean<bf16, 8>(a, bt, false, j0, b * a.block, own, m);
          wide_store_mean<bf16, 8>(a, seq[r], false, j0, b, m);
        }
      }
    }
    for (int v = 8 * tid; v < nv; v += 8 * nt) {
      const wide_u32x4 val = *(const wide_u32x4*)((const unsigned short*)a.u + (int64_t)t * a.stride + a.v_col + v);
      const int gv = v / a.vdim, dv = v - gv * a.vdim;
      *(wide_u32x4*)((unsigned short*)a.vpool + ((page * a.Hkv + gv) * a.page_size + slot) * a.vdim + dv) = val;
      if (means) {
        float own[8], m[8];
        wide_load<bf16, 8>((const bf16*)&val, own);
        wide_block_mean<bf16, 8>(a, bt, true, v, b * a.block, own, m);
        wide_store_mean<bf16, 8>(a, seq[r], true, v, b, m);
      }
    }
  }
}

// The means of all blocks that the step's rows complete: a block of threads per token block,
// counted request after request.
template <typename T, int VEC>
__global__ __launch_bounds__(kWideThreads) void block_means_kernel(QkvWideArgs a) {
  int seq = -1, b = blockIdx.x;
  for (int s = 0; s < a.S; ++s) {
    const int p0 = a.seq_pos0[s], n = a.seq_row_start[s + 1] - a.seq_row_start[s];
    const int from = p0 / a.block, count = (p0 + n) / a.block - from;
    if (b < count) {
      seq = s;
      b += from;
      break;
    }
    b -= count;
  }
  if (seq < 0) return;
  const int* bt = a.block_table + (int64_t)seq * a.bt_stride;
  const int nk = a.Hkv * a.dim, nv = a.Hkv * a.vdim;
  for (int i = VEC * threadIdx.x; i < nk + nv; i += VEC * kWideThreads) {
    const bool is_v = i >= nk;
    const int e0 = is_v ? i - nk : i;
    float m[VEC];
    wide_block_mean<T, VEC>(a, bt, is_v, e0, b * a.block, nullptr, m);
    wide_store_mean<T, VEC>(a, seq, is_v, e0, b, m);
  }
}

template <typename K>
static int wide_lds(K kern, size_t lds, bool* raised) {
  if (lds > 64 * 1024 && !*raised) {
    hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, kWideMaxLds);
    if (e != hipSuccess) return set_error(-2, "qkv_wide: %zu bytes of LDS refused: %s", lds, hipGetErrorString(e));
    *raised = true;
  }
  return 0;
}

template <typename T, int VEC>
static int launch_means(const QkvWideArgs& a, hipStream_t stream) {
  if (a.block > 0 && !a.all_single) {
    // no step completes more: every request adds at most one block begun before
    const int most = a.T / a.block + a.S;
    block_means_kernel<T, VEC><<<most, kWideThreads, 0, stream>>>(a);
    NINFER_LAUNCH_CHECK();
  }
  return 0;
}

// Rows of bfloat16 whole pieces: several rows to a block where there are many.
template <int ROWS>
static int launch_wide_rows(const QkvWideArgs& a, hipStream_t stream) {
  const int n = (a.Hq + a.Hkv) * a.dim;
  const size_t lds = (size_t)ROWS * (a.rot_dim + (a.interleaved ? 0 : n) + (a.unit_heads ? n / 8 : 0)) * sizeof(float);
  static bool raised = false;
  if (int rc = wide_lds(qkv_wide_rows_kernel<ROWS>, lds, &raised)) return rc;
  qkv_wide_rows_kernel<ROWS><<<(a.T + ROWS - 1) / ROWS, (n / 8 + 63) / 64 * 64, lds, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return launch_means<bf16, 8>(a, stream);
}

template <typename T, int VEC>
static int launch_wide(const QkvWideArgs& a, hipStream_t stream) {
  const size_t lds = (size_t)((a.Hq + a.Hkv) * (a.dim + (a.unit_heads ? 1 : 0)) + a.rot_dim) * sizeof(float);
  NINFER_REQUIRE(lds <= (size_t)kWideMaxLds, "qkv_wide: rows of %d queries' and keys' numbers exceed LDS",
                 (a.Hq + a.Hkv) * a.dim);
  static bool raised = false;
  if (int rc = wide_lds(qkv_wide_kernel<T, VEC>, lds, &raised)) return rc;
  qkv_wide_kernel<T, VEC><<<a.T, kWideThreads, lds, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return launch_means<T, VEC>(a, stream);
}

}  // namespace ninfer

using namespace ninfer;

extern "C" int ninfer_qkv_wide(const QkvWideArgs* args, hipStream_t stream) {
  const QkvWideArgs& a = *args;
  NINFER_REQUIRE(a.T > 0 && a.S > 0 && a.Hq > 0 && a.Hkv > 0 && a.dim > 0 && a.vdim > 0,
                 "qkv_wide: T=%d S=%d heads=%d/%d dim=%d vdim=%d must be positive", a.T, a.S, a.Hq,
                 a.Hkv, a.dim, a.vdim);
  const int nq = a.Hq * a.dim, nk = a.Hkv * a.dim, nv = a.Hkv * a.vdim;
  NINFER_REQUIRE(a.q_col >= 0 && a.k_col >= 0 && a.v_col >= 0 && a.q_col + nq <= a.stride &&
                 a.k_col + nk <= a.stride && a.v_col + nv <= a.stride,
                 "qkv_wide: columns outside rows of %d", a.stride);
  NINFER_REQUIRE(a.rot_dim >= 0 && a.rot_dim % 2 == 0 && a.rot_dim <= a.dim && (a.rot_dim == 0 || a.inv_freq),
                 "qkv_wide: %d turning numbers of %d", a.rot_dim, a.dim);
  NINFER_REQUIRE(!a.unit_heads || (!a.q_gain && !a.k_gain && a.magnitude == 1.f),
                 "qkv_wide: heads of unit size beside gains or a scaled rotation");
  NINFER_REQUIRE(a.kpool && a.vpool && a.block_table && a.page_size > 0 && a.bt_stride > 0,
                 "qkv_wide: keys and values without pages");
  NINFER_REQUIRE(a.block >= 0 && (a.block == 0 || (a.kblk && a.vblk && a.blk_table && a.blk_page_size > 0 &&
                                                   a.blk_bt_stride > 0 && a.seq_pos0 && a.seq_row_start)),
                 "qkv_wide: blocks of %d tokens without pages", a.block);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "qkv_wide: unknown dtype %d", a.dtype);
  if (a.dtype == kF32) return launch_wide<float, 1>(a, stream);
  // whole pieces of 8: heads, columns and rows, and the turning part's halves unless neighbours pair
  const bool pieces = a.dim % 8 == 0 && a.vdim % 8 == 0 && (a.interleaved || a.rot_dim % 16 == 0) &&
                      a.stride % 8 == 0 && a.q_col % 8 == 0 && a.k_col % 8 == 0 && a.v_col % 8 == 0 &&
                      (uintptr_t)a.u % 16 == 0;
  if (pieces && a.force_plain != 1) {
    const int n = (a.Hq + a.Hkv) * a.dim;
    const bool aligned = (uintptr_t)a.q_gain % 16 == 0 && (uintptr_t)a.k_gain % 16 == 0;
    auto fits = [&](int rows) {
      return aligned && n <= 8 * kWideRowsMaxThreads &&
             (size_t)rows * (a.rot_dim + (a.interleaved ? 0 : n) + (a.unit_heads ? n / 8 : 0)) * sizeof(float) <=
                 (size_t)kWideMaxLds;
    };
    if (!a.all_single && a.T >= 512 && fits(2)) return launch_wide_rows<2>(a, stream);
    if (fits(1)) return launch_wide_rows<1>(a, stream);
    return launch_wide<bf16, 8>(a, stream);
  }
  return launch_wide<bf16, 1>(a, stream);
}
