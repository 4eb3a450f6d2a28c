// Gated linear attention: linear attention whose state decays per key channel by a factor
// that every token brings, token by token:
//
//   alpha_t = sigmoid(z_t)^(1 / tau)                     (per head and key channel, in (0, 1))
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T              (S: [dim, vdim] per head, 32-bit)
//   o_t = S_t^T (q_t q_scale)
//
// z comes in 32-bit (the decay's logits after their bias); the decay is formed here as
// exp(log_sigmoid(z) / tau).
//
// A second form of the same recurrence has a forget gate that also says how much is written, and
// no keys of its own (`lower` given): from the gate's projected columns w and its bias b,
//
//   f_t = l + (1 - l) sigmoid(w_t + b),  S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,
//   o_t = S_t^T (silu(q_t) q_scale)
//
// with a lower bound l in [0, 1] per head and channel; 1 - f is formed as (1 - l) sigmoid(-w - b).
//
// The state comes from and returns to the request's slot, so a
// request may be cut into steps anywhere and every row sees exactly the sums it would see in
// one piece.
//
// A block of four waves owns 64 value columns of one (request, head) and walks the request's
// rows of the step in order; a wave owns 16 of the columns. Lane (part, col) keeps S[d][col]
// for the DPL key channels d = part DPL .. in registers, updates them and forms its part of
// o_t[col]; the four parts are added by two lane exchanges. q, k and the decay of a row are
// staged in LDS by the block's threads, a channel each (two buffers, one barrier a row); the
// rows come from global memory eight at a time, one batch ahead of the one being computed, so
// that the loads' latency is paid once per batch. The order of every sum depends on dim alone.
#include "common.h"

namespace ninfer {

constexpr int kGlaCols = 16;    // value columns per wave
constexpr int kGlaParts = 4;    // parts of the key channels, one per 16 lanes
constexpr int kGlaWaves = 4;    // waves per block
constexpr int kGlaBatch = 8;    // rows fetched at a time

__device__ __forceinline__ float log_sigmoid(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

struct GlaArgs {
  const void* qkv;        // [T, stride] rows: q at q_off, k at k_off (H x dim), v at v_off (H x vdim)
  const float* z;         // [T, H * dim] the decay's logits
  float* state;           // + slot * state_stride: [H, dim, vdim]
  float* out;             // [T, H * vdim]
  const int* seq_row_start;
  const int* seq_slots;
  int64_t state_stride;
  int stride, q_off, k_off, v_off;
  int H, dim, vdim;
  float inv_tau, q_scale;
  // the form with a forget gate: its columns' first one, bias and lower bounds [H * dim] (z, k_off
  // and inv_tau are not used then)
  int f_off;
  const float* f_bias;
  const float* lower;
};

// What a token brings to a key channel: how much of the state stays, what is written, and the
// logarithm of the former.
struct GlaGate {
  float keep, write, log_keep;
};
// the forget gate's form from its logit (with bias) and lower bound
__device__ __forceinline__ GlaGate forget_gate(float z, float lower) {
  const float e = expf(-fabsf(z)), r = 1.f / (1.f + e);
  const float up = z >= 0.f ? r : e * r, down = z >= 0.f ? e * r : r;   // sigmoid(z), sigmoid(-z)
  GlaGate g;
  g.keep = fmaf(1.f - lower, up, lower);
  g.write = (1.f - lower) * down;
  g.log_keep = fmaxf(log1pf(-g.write), -80.f);   // (exp(-80) is as good as nothing, and finite)
  return g;
}
__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }

template <typename T, int DPL, bool FORGET>
__global__ __launch_bounds__(64 * kGlaWaves) void gla_seq_kernel(GlaArgs a) {
  constexpr int DIM = DPL * kGlaParts;            // channels held (>= dim; the rest stay 0)
  static_assert(DIM <= 64 * kGlaWaves, "a thread stages one channel");
  __shared__ __attribute__((aligned(16))) float q_s[2][DIM], k_s[2][DIM], a_s[2][DIM];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = (blockIdx.z * kGlaWaves + wave) * kGlaCols + (lane & (kGlaCols - 1));
  const int part = lane / kGlaCols;
  const bool has_col = col < a.vdim;
  const int r0 = a.seq_row_start[s], n = a.seq_row_start[s + 1] - r0;
  const int dim = a.dim, vdim = a.vdim;
  float* st = a.state + (int64_t)a.seq_slots[s] * a.state_stride + (int64_t)h * dim * vdim;

  float S[DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = part * DPL + i;
    S[i] = has_col && d < dim ? st[(int64_t)d * vdim + col] : 0.f;
  }
  // the batch of rows a thread fetches ahead: q, k and the decay's logit of its channel (thread
  // tid looks after channel tid), and v of its column
  const bool stages = tid < DIM, in_dim = tid < dim;
  float fq[kGlaBatch], fk[kGlaBatch], fz[kGlaBatch], fv[kGlaBatch];
  const float f_bias = FORGET && in_dim ? a.f_bias[h * dim + tid] : 0.f;
  const float lower = FORGET && in_dim ? a.lower[h * dim + tid] : 0.f;
  auto fetch = [&](int first) {
#pragma unroll
    for (int j = 0; j < kGlaBatch; ++j) {
      const int row = r0 + min(first + j, n - 1);   // (rows beyond the last are fetched again, not used)
      const T* r = (const T*)a.qkv + (int64_t)row * a.stride;
      fq[j] = in_dim ? to_f32(r[a.q_off + h * dim + tid]) : 0.f;
      if constexpr (FORGET) {
        fz[j] = in_dim ? to_f32(r[a.f_off + h * dim + tid]) : 0.f;
      } else {
        fk[j] = in_dim ? to_f32(r[a.k_off + h * dim + tid]) : 0.f;
        fz[j] = in_dim ? a.z[((int64_t)row * a.H + h) * dim + tid] : 0.f;
      }
      fv[j] = has_col ? to_f32(r[a.v_off + h * vdim + col]) : 0.f;
    }
  };
  if (n > 0) fetch(0);
  for (int base = 0; base < n; base += kGlaBatch) {
    float cq[kGlaBatch], ck[kGlaBatch], ca[kGlaBatch], cv[kGlaBatch];
#pragma unroll
    for (int j = 0; j < kGlaBatch; ++j) {
      if constexpr (FORGET) {
        const GlaGate g = forget_gate(fz[j] + f_bias, lower);
        cq[j] = silu_f(fq[j]) * a.q_scale;
        ck[j] = in_dim ? g.write : 0.f;
        ca[j] = in_dim ? g.keep : 1.f;
      } else {
        cq[j] = fq[j] * a.q_scale;
        ck[j] = fk[j];
        ca[j] = in_dim ? expf(log_sigmoid(fz[j]) * a.inv_tau) : 1.f;
      }
      cv[j] = fv[j];
    }
    if (base + kGlaBatch < n) fetch(base + kGlaBatch);
#pragma unroll
    for (int j = 0; j < kGlaBatch; ++j) {
      if (base + j >= n) break;
      const int b = j & 1;
      if (stages) {
        q_s[b][tid] = cq[j];
        k_s[b][tid] = ck[j];
        a_s[b][tid] = ca[j];
      }
      // (a barrier that waits for LDS traffic only: the batch on its way and the outputs' stores
      // stay in flight)
      lds_barrier();   // the row is in LDS; the other buffer's readers are done
      const float v_t = cv[j];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = part * DPL + i;
        const float sn = fmaf(a_s[b][d], S[i], k_s[b][d] * v_t);
        S[i] = sn;
        o = fmaf(sn, q_s[b][d], o);
      }
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
      if (part == 0 && has_col) a.out[((int64_t)(r0 + base + j) * a.H + h) * vdim + col] = o;
    }
  }
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = part * DPL + i;
    if (has_col && d < dim) st[(int64_t)d * vdim + col] = S[i];
  }
}

}  // namespace ninfer

using namespace ninfer;

// qkv: [T, stride] rows of the activation dtype with the heads' q at column q_off, k at k_off
// (heads x dim each) and v at v_off (heads x vdim); z: [T, heads * dim] 32-bit; out:
// [T, heads * vdim] 32-bit. With `lower` [heads * dim] the form with a forget gate: its columns
// (heads x dim) at f_off, its bias f_bias [heads * dim]; z, k_off and tau are not read.
extern "C" int ninfer_gated_linear_attention(const void* qkv, int stride, int q_off, int k_off,
                                             int v_off, const float* z, float tau, float q_scale,
                                             float* state, long long state_stride, float* out,
                                             const int* seq_row_start, const int* seq_slots,
                                             int T, int S, int H, int dim, int vdim, int dtype,
                                             int f_off, const float* f_bias, const float* lower,
                                             hipStream_t stream) {
  NINFER_REQUIRE(T > 0 && S > 0 && H > 0 && dim > 0 && vdim > 0,
                 "gated_linear_attention: T=%d S=%d heads=%d dim=%d vdim=%d must be positive", T,
                 S, H, dim, vdim);
  NINFER_REQUIRE(dim <= 256, "gated_linear_attention: %d key channels exceed 256", dim);
  NINFER_REQUIRE(tau > 0.f, "gated_linear_attention: tau (%g) must be positive", tau);
  NINFER_REQUIRE(state_stride >= (long long)H * dim * vdim,
                 "gated_linear_attention: a request's state of %lld floats holds no %d x %d x %d",
                 state_stride, H, dim, vdim);
  NINFER_REQUIRE(dtype == kF32 || dtype == kBF16, "gated_linear_attention: unknown dtype %d", dtype);
  GlaArgs a;
  a.qkv = qkv, a.z = z, a.state = state, a.out = out;
  a.seq_row_start = seq_row_start, a.seq_slots = seq_slots, a.state_stride = state_stride;
  a.stride = stride, a.q_off = q_off, a.k_off = k_off, a.v_off = v_off;
  a.H = H, a.dim = dim, a.vdim = vdim, a.inv_tau = 1.f / tau, a.q_scale = q_scale;
  a.f_off = f_off, a.f_bias = f_bias, a.lower = lower;
  NINFER_REQUIRE(!lower == !f_bias && (lower || z), "gated_linear_attention: a forget gate without its bias, or no gate");
  const int cols = kGlaCols * kGlaWaves;
  const dim3 grid(S, H, (vdim + cols - 1) / cols);
#define NINFER_GLA(DPL)                                                                               \
  do {                                                                                                \
    if (lower) {                                                                                      \
      if (dtype == kF32) gla_seq_kernel<float, DPL, true><<<grid, 64 * kGlaWaves, 0, stream>>>(a);    \
      else gla_seq_kernel<bf16, DPL, true><<<grid, 64 * kGlaWaves, 0, stream>>>(a);                   \
    } else {                                                                                          \
      if (dtype == kF32) gla_seq_kernel<float, DPL, false><<<grid, 64 * kGlaWaves, 0, stream>>>(a);   \
      else gla_seq_kernel<bf16, DPL, false><<<grid, 64 * kGlaWaves, 0, stream>>>(a);                  \
    }                                                                                                 \
  } while (0)
  if (dim <= 16) NINFER_GLA(4);
  else if (dim <= 32) NINFER_GLA(8);
  else if (dim <= 64) NINFER_GLA(16);
  else if (dim <= 128) NINFER_GLA(32);
  else NINFER_GLA(64);
#undef NINFER_GLA
  NINFER_LAUNCH_CHECK();
  return 0;
}

// ---- prompt portions in chunks of 16 rows, on the 32-bit matrix instruction ---------------------
//
// With b_i = sum of ln alpha over the rows 0 .. i of a chunk (per key channel, <= 0) and the
// state S before the chunk, the recurrence written out is
//
//   o_i = (q_i * e^(b_i))^T S  +  sum_{j <= i} A[i][j] v_j,   A[i][j] = sum_d q_i[d] k_j[d] e^(b_i[d] - b_j[d])
//   S' = diag(e^(b_(L-1))) S + sum_j (k_j * e^(b_(L-1) - b_j)) v_j^T
//
// Every exponent is <= 0, so nothing grows, however strong the decay. A first kernel, one block
// per (chunk, head) and so as wide as the step, forms q e^b, k e^(b_last - b), e^b and A in
// 32-bit: A not from exponentials but as the recurrence does, by multiplying k_j with the decays
// of the rows that follow it, one after the other. A second kernel walks a request's chunks
// in order: a wave keeps 16 value columns of the state in the accumulators of
// v_mfma_f32_16x16x4_f32 (they are that instruction's second operand as they are: the order of
// a sum's terms is free), and a chunk costs it dim / 4 + 4 products for the outputs and
// dim / 4 for the state, with the operands of the next chunk on their way meanwhile. Nothing
// is rounded to a shorter type.
//
// A request's chunks in order are a long chain on few blocks when the step has few requests.
// Then they are cut into segments of kGlaSegment chunks: every segment's state from a zero start
// and its decays' products (all segments side by side), the states in front of the segments from
// those (one pass over the segments, S <- E S + S_segment, a number of the state per thread),
// and the outputs of all segments side by side, each from the state in front of it.
namespace ninfer {

typedef float gla_f32x4 __attribute__((ext_vector_type(4)));
constexpr int kGlaChunk = 16;
constexpr int kGlaChunkMaxDim = 128;
constexpr int kGlaSegment = 8;                              // chunks of a segment
constexpr int kGlaSegmentRows = kGlaSegment * kGlaChunk;

struct GlaChunkArgs {
  GlaArgs g;
  float* qe;     // [H, T, dim]  q q_scale e^b  (a chunk of a head is one piece of memory)
  float* ke;     // [H, T, dim]  k e^(b_last - b)
  float* eb;     // [H, T, dim]  e^b
  float* A;      // [H, T, 16]
  float* seg;    // [segments, H, dim, vdim]: a segment's state from zero, then the state in front of it
  float* seg_e;  // [segments, H, dim]: the products of a segment's decays
  int T, S;
};

// The request and the first row of chunk `c` of the step (chunks of `rows` rows are counted
// request after request); false if the step has fewer chunks.
__device__ __forceinline__ bool gla_find_chunk(const int* seq_row_start, int S, int c, int* r0,
                                               int* i0, int* n, int* seq = nullptr, int rows = kGlaChunk) {
  for (int s = 0; s < S; ++s) {
    const int a = seq_row_start[s], len = seq_row_start[s + 1] - a;
    const int chunks = (len + rows - 1) / rows;
    if (c < chunks) {
      *r0 = a, *i0 = c * rows, *n = len;
      if (seq) *seq = s;
      return true;
    }
    c -= chunks;
  }
  return false;
}

template <typename T, bool FORGET>
__global__ __launch_bounds__(256) void gla_chunk_prepare_kernel(GlaChunkArgs a) {
  __shared__ float q_s[kGlaChunk][kGlaChunkMaxDim], k_s[kGlaChunk][kGlaChunkMaxDim];
  __shared__ float al_s[kGlaChunk][kGlaChunkMaxDim], b_s[kGlaChunk][kGlaChunkMaxDim];
  int r0, i0, n;
  if (!gla_find_chunk(a.g.seq_row_start, a.S, blockIdx.x, &r0, &i0, &n)) return;
  const int h = blockIdx.y, tid = threadIdx.x;
  const int dim = a.g.dim, H = a.g.H;
  const int L = min(kGlaChunk, n - i0), base = r0 + i0;
  // 1. the rows' q, k and decays; rows beyond the chunk's last count as absent (k = 0, alpha = 1)
  for (int e = tid; e < kGlaChunk * dim; e += 256) {
    const int t = e / dim, d = e % dim;
    float qv = 0.f, kv = 0.f, g = 0.f, al = 1.f;
    if (t < L) {
      const T* r = (const T*)a.g.qkv + (int64_t)(base + t) * a.g.stride;
      qv = to_f32(r[a.g.q_off + h * dim + d]) * a.g.q_scale;
      if constexpr (FORGET) {
        const GlaGate f = forget_gate(to_f32(r[a.g.f_off + h * dim + d]) + a.g.f_bias[h * dim + d],
                                      a.g.lower[h * dim + d]);
        qv = silu_f(to_f32(r[a.g.q_off + h * dim + d])) * a.g.q_scale;
        kv = f.write, g = f.log_keep, al = f.keep;
      } else {
        kv = to_f32(r[a.g.k_off + h * dim + d]);
        g = log_sigmoid(a.g.z[((int64_t)(base + t) * H + h) * dim + d]) * a.g.inv_tau;
        al = expf(g);
      }
    }
    q_s[t][d] = qv, k_s[t][d] = kv, al_s[t][d] = al, b_s[t][d] = g;
  }
  __syncthreads();
  // 2. b: the running sum of the logarithms, a channel per thread
  if (tid < dim) {
    float b = 0.f;
#pragma unroll
    for (int t = 0; t < kGlaChunk; ++t) {
      b += b_s[t][tid];
      b_s[t][tid] = b;
    }
  }
  __syncthreads();
  // 3. the scaled rows
  for (int e = tid; e < L * dim; e += 256) {
    const int t = e / dim, d = e % dim;
    const float eb = expf(b_s[t][d]);
    const int64_t at = ((int64_t)h * a.T + base + t) * dim + d;
    a.qe[at] = q_s[t][d] * eb;
    a.ke[at] = k_s[t][d] * expf(b_s[L - 1][d] - b_s[t][d]);
    a.eb[at] = eb;
  }
  // 4. A: thread (j, part) carries k_j times the decays since row j for the channels part,
  // part + 16, ..; the sixteen parts of a (row, j) are added by lane exchanges
  {
    const int j = tid >> 4, part = tid & 15;
    constexpr int PER = kGlaChunkMaxDim / 16;
    float kp[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int d = part + 16 * i;
      kp[i] = d < dim ? k_s[j][d] : 0.f;
    }
    for (int t = 0; t < L; ++t) {
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int d = part + 16 * i;
        if (d < dim) {
          if (t > j) kp[i] *= al_s[t][d];
          acc = fmaf(q_s[t][d], kp[i], acc);
        }
      }
      acc += __shfl_xor(acc, 1, 64);
      acc += __shfl_xor(acc, 2, 64);
      acc += __shfl_xor(acc, 4, 64);
      acc += __shfl_xor(acc, 8, 64);
      if (part == 0) a.A[((int64_t)h * a.T + base + t) * kGlaChunk + j] = j <= t ? acc : 0.f;
    }
  }
}

// A chunk's operands as the lanes of a wave hold them. Lane (c, g) = (lane % 16, lane / 16).
template <int DT>
struct GlaChunkRegs {
  gla_f32x4 q[DT];    // qe[row c][16 dt + 4 g ..]
  gla_f32x4 e[DT];    // eb[last row][16 dt + 4 g ..]
  float k[4][DT];     // ke[row 4 g + x][16 dt + c]
  gla_f32x4 A;        // A[row c][4 g ..]
  float v[4];         // v[row 4 g + x][column c of the wave]
};

// What a block of the scan walks: a request's rows of the step; a segment of them from a zero
// state, for the state it leaves only; a segment from the state in front of it, for its outputs.
enum GlaScan : int { kGlaWhole, kGlaSegmentState, kGlaSegmentOut };

template <typename T, int DT, int MODE>
__global__ __launch_bounds__(64 * kGlaWaves) void gla_chunk_scan_kernel(GlaChunkArgs a) {
  int s = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const int col = (blockIdx.z * kGlaWaves + wave) * kGlaCols + c;
  const int dim = a.g.dim, vdim = a.g.vdim, H = a.g.H;
  const bool has_col = col < vdim;
  int r0, n;
  bool ends = true;   // the last piece of its request: the state after it goes to the request's slot
  if constexpr (MODE == kGlaWhole) {
    r0 = a.g.seq_row_start[s], n = a.g.seq_row_start[s + 1] - r0;
  } else {
    int i0;
    if (!gla_find_chunk(a.g.seq_row_start, a.S, blockIdx.x, &r0, &i0, &n, &s, kGlaSegmentRows)) return;
    ends = i0 + kGlaSegmentRows >= n;
    r0 += i0, n = min(kGlaSegmentRows, n - i0);
    if (MODE == kGlaSegmentState && ends) return;   // nobody starts from its state
  }
  float* slot = a.g.state + (int64_t)a.g.seq_slots[s] * a.g.state_stride + (int64_t)h * dim * vdim;
  float* st = MODE == kGlaWhole ? slot : a.seg + ((int64_t)blockIdx.x * H + h) * dim * vdim;
  const int64_t head_row0 = (int64_t)h * a.T;   // the head's first row in the workspace
  // the state: S[16 dt + 4 g + x][col] in Sreg[dt][x]
  gla_f32x4 Sreg[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int d = 16 * dt + 4 * g + x;
      Sreg[dt][x] = MODE != kGlaSegmentState && has_col && d < dim ? st[(int64_t)d * vdim + col] : 0.f;
    }
  gla_f32x4 Ereg[DT];   // the products of the decays so far
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) Ereg[dt] = gla_f32x4{1.f, 1.f, 1.f, 1.f};
  const gla_f32x4 zero4 = {0.f, 0.f, 0.f, 0.f};
  // The loads of a chunk's operands, every one of them unconditional (a load inside a branch is
  // waited for where the branch ends): rows, channels and columns beyond the last are fetched
  // from the last, a chunk beyond the last from the last, and `chunk` puts zeros where they count.
  const int last_chunk = n > 0 ? (n - 1) / kGlaChunk * kGlaChunk : 0;
  const int col_c = min(col, vdim - 1);
  auto fetch = [&](GlaChunkRegs<DT>& R, int i0) {
    i0 = min(i0, last_chunk);
    const int L = min(kGlaChunk, n - i0), base = r0 + i0;
    const float* qrow = a.qe + (head_row0 + base + min(c, L - 1)) * dim;
    const float* erow = a.eb + (head_row0 + base + L - 1) * dim;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int d = min(16 * dt + 4 * g, dim - 4);   // (dim is a multiple of 4)
      if constexpr (MODE != kGlaSegmentState) R.q[dt] = *(const gla_f32x4*)(qrow + d);
      R.e[dt] = *(const gla_f32x4*)(erow + d);
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int64_t row = base + min(4 * g + x, L - 1);
      const float* krow = a.ke + (head_row0 + row) * dim;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) R.k[x][dt] = krow[min(16 * dt + c, dim - 1)];
      R.v[x] = to_f32(((const T*)a.g.qkv)[row * a.g.stride + a.g.v_off + h * vdim + col_c]);
    }
    if constexpr (MODE != kGlaSegmentState)
      R.A = *(const gla_f32x4*)(a.A + (head_row0 + base + min(c, L - 1)) * kGlaChunk + 4 * g);
  };
  // a chunk: its outputs from the state before it, then the state after it; the operands of the
  // chunk after the next one set out first (three sets of registers take turns)
  auto chunk = [&](GlaChunkRegs<DT>& cur, int i0, GlaChunkRegs<DT>& ahead) {
    const int L = min(kGlaChunk, n - i0);
    fetch(ahead, i0 + 2 * kGlaChunk);
    // zeros where a sum runs over rows or channels that are not there
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      if (16 * dt + 4 * g >= dim) {
        if constexpr (MODE != kGlaSegmentState) cur.q[dt] = zero4;
        cur.e[dt] = zero4;
      }
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (4 * g + x >= L || 16 * dt + c >= dim) cur.k[x][dt] = 0.f;
    }
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (4 * g + x >= L) cur.v[x] = 0.f;
    // the outputs: rows 4 g + x of column c in o[x] + o2[x]
    if constexpr (MODE != kGlaSegmentState) {
    gla_f32x4 o = zero4, o2 = zero4;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.q[dt][0], Sreg[dt][0], o, 0, 0, 0);
      o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.q[dt][1], Sreg[dt][1], o2, 0, 0, 0);
      o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.q[dt][2], Sreg[dt][2], o, 0, 0, 0);
      o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.q[dt][3], Sreg[dt][3], o2, 0, 0, 0);
    }
    o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.A[0], cur.v[0], o, 0, 0, 0);
    o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.A[1], cur.v[1], o2, 0, 0, 0);
    o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.A[2], cur.v[2], o, 0, 0, 0);
    o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.A[3], cur.v[3], o2, 0, 0, 0);
    if (has_col) {
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int t = 4 * g + x;
        if (t < L) a.g.out[((int64_t)(r0 + i0 + t) * H + h) * vdim + col] = o[x] + o2[x];
      }
    }
    }
    // the state after the chunk
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        Sreg[dt][x] *= cur.e[dt][x];
        if constexpr (MODE == kGlaSegmentState) Ereg[dt][x] *= cur.e[dt][x];
      }
#pragma unroll
      for (int x = 0; x < 4; ++x)
        Sreg[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.k[x][dt], cur.v[x], Sreg[dt], 0, 0, 0);
    }
  };
  GlaChunkRegs<DT> R0, R1, R2;
  if (n <= 0) return;
  fetch(R0, 0);
  fetch(R1, kGlaChunk);
  for (int i0 = 0; i0 < n; i0 += 3 * kGlaChunk) {
    chunk(R0, i0, R2);
    if (i0 + kGlaChunk >= n) break;
    chunk(R1, i0 + kGlaChunk, R0);
    if (i0 + 2 * kGlaChunk >= n) break;
    chunk(R2, i0 + 2 * kGlaChunk, R1);
  }
  if (MODE == kGlaSegmentOut && !ends) return;
  float* to = MODE == kGlaSegmentState ? st : slot;
  if (has_col) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int d = 16 * dt + 4 * g + x;
        if (d < dim) to[(int64_t)d * vdim + col] = Sreg[dt][x];
      }
  }
  if (MODE == kGlaSegmentState && blockIdx.z == 0 && wave == 0 && c == 0) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int d = 16 * dt + 4 * g + x;
        if (d < dim) a.seg_e[((int64_t)blockIdx.x * H + h) * dim + d] = Ereg[dt][x];
      }
  }
}

// The states in front of a request's segments, in place of the states the segments leave from
// zero: a number of the state per thread.
__global__ __launch_bounds__(256) void gla_segment_states_kernel(GlaChunkArgs a) {
  const int s = blockIdx.y, dim = a.g.dim, vdim = a.g.vdim, H = a.g.H;
  const int n = H * dim * vdim, e = blockIdx.x * 256 + threadIdx.x;
  if (e >= n) return;
  int first = 0;
  for (int i = 0; i < s; ++i)
    first += (a.g.seq_row_start[i + 1] - a.g.seq_row_start[i] + kGlaSegmentRows - 1) / kGlaSegmentRows;
  const int count = (a.g.seq_row_start[s + 1] - a.g.seq_row_start[s] + kGlaSegmentRows - 1) / kGlaSegmentRows;
  float S = a.g.state[(int64_t)a.g.seq_slots[s] * a.g.state_stride + e];
  const int hd = e / vdim;
#pragma unroll 8
  for (int i = 0; i < count; ++i) {
    float* at = a.seg + (int64_t)(first + i) * n + e;
    // (the last segment has left neither a state nor decays: nothing comes after it)
    const bool more = i + 1 < count;
    const float left = more ? *at : 0.f, keep = more ? a.seg_e[(int64_t)(first + i) * H * dim + hd] : 0.f;
    *at = S;
    S = fmaf(keep, S, left);
  }
}

}  // namespace ninfer

// The same as ninfer_gated_linear_attention for bfloat16 rows, in chunks of 16 rows on the
// matrix cores: for steps that bring prompt portions. `work` holds T * (3 heads dim + 16 heads)
// floats. `segments` (or null): as many floats as ninfer_gla_segment_floats asks for, and the
// step runs in segments. Returns 1 (nothing launched) when the sizes do not fit.
extern "C" int ninfer_gated_linear_attention_chunks(const void* qkv, int stride, int q_off, int k_off,
                                                    int v_off, const float* z, float tau,
                                                    float q_scale, float* state,
                                                    long long state_stride, float* out,
                                                    const int* seq_row_start, const int* seq_slots,
                                                    float* work, int T, int S, int H, int dim,
                                                    int vdim, int dtype, int f_off, const float* f_bias,
                                                    const float* lower, float* segments,
                                                    hipStream_t stream) {
  NINFER_REQUIRE(T > 0 && S > 0 && H > 0 && dim > 0 && vdim > 0,
                 "gated_linear_attention: T=%d S=%d heads=%d dim=%d vdim=%d must be positive", T,
                 S, H, dim, vdim);
  NINFER_REQUIRE(tau > 0.f, "gated_linear_attention: tau (%g) must be positive", tau);
  NINFER_REQUIRE(state_stride >= (long long)H * dim * vdim,
                 "gated_linear_attention: a request's state of %lld floats holds no %d x %d x %d",
                 state_stride, H, dim, vdim);
  NINFER_REQUIRE(!lower == !f_bias && (lower || z), "gated_linear_attention: a forget gate without its bias, or no gate");
  NINFER_REQUIRE(work != nullptr, "gated_linear_attention: the chunks need their workspace");
  if (dtype != kBF16 || dim > kGlaChunkMaxDim || dim % 4 != 0 || (uintptr_t)work % 16 != 0) return 1;
  GlaChunkArgs a;
  a.g.qkv = qkv, a.g.z = z, a.g.state = state, a.g.out = out;
  a.g.seq_row_start = seq_row_start, a.g.seq_slots = seq_slots, a.g.state_stride = state_stride;
  a.g.stride = stride, a.g.q_off = q_off, a.g.k_off = k_off, a.g.v_off = v_off;
  a.g.H = H, a.g.dim = dim, a.g.vdim = vdim, a.g.inv_tau = 1.f / tau, a.g.q_scale = q_scale;
  const int64_t thd = (int64_t)T * H * dim;
  a.qe = work, a.ke = work + thd, a.eb = work + 2 * thd, a.A = work + 3 * thd;
  a.T = T, a.S = S;
  a.g.f_off = f_off, a.g.f_bias = f_bias, a.g.lower = lower;
  const int chunks = T / kGlaChunk + S;   // no step has more: each request adds at most one short chunk
  if (lower) gla_chunk_prepare_kernel<bf16, true><<<dim3(chunks, H), 256, 0, stream>>>(a);
  else gla_chunk_prepare_kernel<bf16, false><<<dim3(chunks, H), 256, 0, stream>>>(a);
  const int cols = kGlaCols * kGlaWaves;
  dim3 grid(S, H, (vdim + cols - 1) / cols);
#define NINFER_GLA_SCAN(MODE)                                                                              \
  do {                                                                                                     \
    if (dim <= 16) gla_chunk_scan_kernel<bf16, 1, MODE><<<grid, 64 * kGlaWaves, 0, stream>>>(a);           \
    else if (dim <= 32) gla_chunk_scan_kernel<bf16, 2, MODE><<<grid, 64 * kGlaWaves, 0, stream>>>(a);      \
    else if (dim <= 64) gla_chunk_scan_kernel<bf16, 4, MODE><<<grid, 64 * kGlaWaves, 0, stream>>>(a);      \
    else gla_chunk_scan_kernel<bf16, 8, MODE><<<grid, 64 * kGlaWaves, 0, stream>>>(a);                     \
  } while (0)
  if (segments) {
    const int n_seg = T / kGlaSegmentRows + S;   // no step has more
    a.seg = segments, a.seg_e = segments + (int64_t)n_seg * H * dim * vdim;
    grid.x = n_seg;
    NINFER_GLA_SCAN(kGlaSegmentState);
    gla_segment_states_kernel<<<dim3((H * dim * vdim + 255) / 256, S), 256, 0, stream>>>(a);
    NINFER_GLA_SCAN(kGlaSegmentOut);
  } else {
    NINFER_GLA_SCAN(kGlaWhole);
  }
#undef NINFER_GLA_SCAN
  NINFER_LAUNCH_CHECK();
  return 0;
}

// Floats of workspace with which a step of this shape runs in segments; 0 when it does not pay:
// few rows, or requests enough to fill the device with one block per request, head and columns.
extern "C" long long ninfer_gla_segment_floats(int T, int S, int H, int dim, int vdim) {
  const int cols = kGlaCols * kGlaWaves;
  if (T < 2 * kGlaSegmentRows * S || (long long)S * H * ((vdim + cols - 1) / cols) >= 2LL * device_cu_count()) return 0;
  return (long long)(T / kGlaSegmentRows + S) * H * dim * (vdim + 1);
}
