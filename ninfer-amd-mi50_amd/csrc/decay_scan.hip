// Linear attention with one decay per head and token, row by row:
//
//   S_t = keep_t S_(t-1) + write_t k_t v_t^T        (S: [dim, vdim] per head, 32-bit)
//   o_t = S_t^T q_t q_scale
//
// with keys and queries that the heads of a group share, in two forms:
//
//   kScanStep   dt = softplus(z + b), keep = exp(-rate dt), write = dt, and o_t += skip v_t
//   kScanExp    i = c(z_i + b_i), f = log_sigmoid(c(z_f + b_f)), c(x) = cap tanh(x / cap);
//               m_t = max(f + m_(t-1), i), keep = exp(f + m_(t-1) - m_t), write = exp(i - m_t);
//               n_t = keep n_(t-1) + write k_t beside S, and the output is to be divided by
//               max(|n_t . q_t q_scale|, exp(-m_t)) + 1e-6
//
// Gates, decays, the running maximum and the sums are 32-bit. The state comes from and returns to
// the request's slot, so a request may be cut into steps anywhere.
//
// Three kernels. scan_gates_kernel: keep, write (and m) of every row, a thread per (request, head)
// walking its rows. scan_seq_kernel: the recurrence of any number of rows; a block of four waves
// owns 64 value columns of one (request, head), a wave 16 of them, lane (part, col) keeps S[d][col]
// of a quarter of the key channels in registers; q and k of a row are staged in LDS (two buffers,
// one barrier a row) and fetched eight rows ahead. n is treated as one more value column whose
// values are 1: the wave that owns it writes the divisors. The order of every sum depends on dim
// alone. scan_step_kernel: requests that bring one row (decoding), gates, state, output and, in the
// form kScanExp, divisor, head norm and output gate in one pass over the state.
#include "decay_scan.h"

namespace ninfer {

constexpr int kSeqCols = 16, kSeqParts = 4, kSeqWaves = 4, kSeqBatch = 8;

int scan_check(const ScanArgs& a) {
  NINFER_REQUIRE(a.T > 0 && a.S > 0 && a.H > 0 && a.G > 0 && a.dim > 0 && a.vdim > 0 && a.H % a.G == 0,
                 "decay_scan: T=%d S=%d heads=%d groups=%d dim=%d vdim=%d do not fit", a.T, a.S, a.H, a.G, a.dim, a.vdim);
  NINFER_REQUIRE(a.dim <= 512, "decay_scan: %d key channels exceed 512", a.dim);
  NINFER_REQUIRE(a.form == kScanStep || a.form == kScanExp, "decay_scan: unknown form %d", a.form);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "decay_scan: unknown dtype %d", a.dtype);
  NINFER_REQUIRE(a.rows && a.z && a.z_bias && a.state && a.seq_row_start && a.seq_slots, "decay_scan: rows, gates or state are missing");
  NINFER_REQUIRE(a.form == kScanExp ? a.cap > 0.f : (a.rate && a.skip), "decay_scan: the gates' constants are missing");
  const long long floats = (long long)a.H * a.dim * a.vdim + (a.form == kScanExp ? (long long)a.H * (a.dim + 1) : 0);
  NINFER_REQUIRE(a.state_stride >= floats, "decay_scan: a request's state of %lld floats holds no %lld",
                 (long long)a.state_stride, floats);
  NINFER_REQUIRE(a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.q_off + a.G * a.dim <= a.stride &&
                 a.k_off + a.G * a.dim <= a.stride && a.v_off + a.H * a.vdim <= a.stride,
                 "decay_scan: columns outside rows of %d", a.stride);
  NINFER_REQUIRE(a.first_seq >= 0 && a.first_seq < a.S, "decay_scan: no request is left after %d", a.first_seq);
  return 0;
}

// work: [T, H, 2] keep and write, then (kScanExp) [T, H] m
__global__ __launch_bounds__(64) void scan_gates_kernel(ScanArgs a) {
  const int s = a.first_seq + blockIdx.x, h = blockIdx.y * 64 + threadIdx.x;
  if (h >= a.H) return;
  const int r0 = a.seq_row_start[s], r1 = a.seq_row_start[s + 1];
  float2* kw = (float2*)a.work;
  if (a.form == kScanStep) {
    const float rate = a.rate[h], b = a.z_bias[h];
    for (int r = r0; r < r1; ++r) {
      const float dt = scan_softplus(a.z[(int64_t)r * a.H + h] + b);
      kw[(int64_t)r * a.H + h] = make_float2(expf(-rate * dt), dt);
    }
    return;
  }
  float* m_at = a.state + (int64_t)a.seq_slots[s] * a.state_stride + (int64_t)a.H * a.dim * (a.vdim + 1) + h;
  float* m_rows = a.work + 2 * (int64_t)a.T * a.H;
  float m = *m_at;
  for (int r = r0; r < r1; ++r) {
    float i, f;
    scan_exp_gates(a, r, h, &i, &f);
    const float up = f + m, m_new = fmaxf(up, i);
    kw[(int64_t)r * a.H + h] = make_float2(expf(up - m_new), expf(i - m_new));
    m_rows[(int64_t)r * a.H + h] = m_new;
    m = m_new;
  }
  *m_at = m;
}

template <typename T, int DPL, int FORM>
__global__ __launch_bounds__(64 * kSeqWaves) void scan_seq_kernel(ScanArgs a) {
  constexpr int DIM = DPL * kSeqParts, NT = 64 * kSeqWaves;
  constexpr int CPT = (DIM + NT - 1) / NT;     // channels that a thread stages
  __shared__ __attribute__((aligned(16))) float q_s[2][DIM], k_s[2][DIM];
  const int s = a.first_seq + blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = (blockIdx.z * kSeqWaves + wave) * kSeqCols + (lane & (kSeqCols - 1)), part = lane / kSeqCols;
  const int dim = a.dim, vdim = a.vdim, H = a.H, g = h / (H / a.G);
  const bool has_v = col < vdim, ones = FORM == kScanExp && col == vdim, live = has_v || ones;
  const int r0 = a.seq_row_start[s], n = a.seq_row_start[s + 1] - r0;
  if (n <= 0) return;
  float* slot = a.state + (int64_t)a.seq_slots[s] * a.state_stride;
  // a column of the state: of S, or n
  float* st = ones ? slot + (int64_t)H * dim * vdim + (int64_t)h * dim : slot + (int64_t)h * dim * vdim + col;
  const int step = ones ? 1 : vdim;
  float S[DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = part * DPL + i;
    S[i] = live && d < dim ? st[(int64_t)d * step] : 0.f;
  }
  const float2* kw = (const float2*)a.work;
  const float* m_rows = a.work + 2 * (int64_t)a.T * H;
  const float skip = FORM == kScanStep ? a.skip[h] : 0.f;
  float fq[kSeqBatch][CPT], fk[kSeqBatch][CPT], fv[kSeqBatch];
  float2 fg[kSeqBatch];
  auto fetch = [&](int first) {
#pragma unroll
    for (int j = 0; j < kSeqBatch; ++j) {
      const int64_t row = r0 + min(first + j, n - 1);   // (rows beyond the last are fetched again, not used)
      const T* r = (const T*)a.rows + row * a.stride;
#pragma unroll
      for (int x = 0; x < CPT; ++x) {
        const int d = tid + x * NT;
        fq[j][x] = d < dim ? to_f32(r[a.q_off + g * dim + d]) : 0.f;
        fk[j][x] = d < dim ? to_f32(r[a.k_off + g * dim + d]) : 0.f;
      }
      fv[j] = has_v ? to_f32(r[a.v_off + h * vdim + col]) : ones ? 1.f : 0.f;
      fg[j] = kw[row * H + h];
    }
  };
  fetch(0);
  for (int base = 0; base < n; base += kSeqBatch) {
    float cq[kSeqBatch][CPT], ck[kSeqBatch][CPT], cv[kSeqBatch];
    float2 cg[kSeqBatch];
#pragma unroll
    for (int j = 0; j < kSeqBatch; ++j) {
#pragma unroll
      for (int x = 0; x < CPT; ++x) cq[j][x] = fq[j][x] * a.q_scale, ck[j][x] = fk[j][x];
      cv[j] = fv[j];
      cg[j] = fg[j];
    }
    if (base + kSeqBatch < n) fetch(base + kSeqBatch);
#pragma unroll
    for (int j = 0; j < kSeqBatch; ++j) {
      if (base + j >= n) break;
      const int b = j & 1;
#pragma unroll
      for (int x = 0; x < CPT; ++x) {
        const int d = tid + x * NT;
        if (d < DIM) q_s[b][d] = cq[j][x], k_s[b][d] = ck[j][x];
      }
      lds_barrier();   // the row is in LDS; the other buffer's readers are done
      const float keep = cg[j].x, w = cg[j].y * cv[j];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = part * DPL + i;
        const float sn = fmaf(keep, S[i], k_s[b][d] * w);
        S[i] = sn;
        o = fmaf(sn, q_s[b][d], o);
      }
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
      if (part == 0) {
        const int64_t at = (int64_t)(r0 + base + j) * H + h;
        if (has_v) a.out[at * vdim + col] = FORM == kScanStep ? fmaf(skip, cv[j], o) : o;
        else if (ones) a.den[at] = fmaxf(fabsf(o), expf(-m_rows[at])) + 1e-6f;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = part * DPL + i;
    if (live && d < dim) st[(int64_t)d * step] = S[i];
  }
}

// ---- requests that bring one row each -------------------------------------------------------------
//
// A block of NT threads owns one (request, head) and, in the form kScanStep, TX * VEC value columns
// of it. Thread (row, col) moves VEC neighbouring columns of every (NT / TX)th key channel; all
// loads of a group of TX * VEC columns are under way together, before anything else is asked for.
constexpr int kStepMaxDim = 512, kStepMaxV = 1024;

template <int VEC>
__device__ __forceinline__ void step_load(const float* p, float* f) {
  if constexpr (VEC == 4) {
    const float4 v = *(const float4*)p;
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  } else {
    f[0] = p[0];
  }
}
template <int VEC>
__device__ __forceinline__ void step_store(float* p, const float* f) {
  if constexpr (VEC == 4) *(float4*)p = make_float4(f[0], f[1], f[2], f[3]);
  else p[0] = f[0];
}

template <typename T, int NT, int VEC, int TX, int PASSES, int FORM>
__global__ __launch_bounds__(NT) void scan_step_kernel(ScanArgs a) {
  constexpr int COLS = TX * VEC, ROWS = NT / TX, WAVES = NT / 64;
  static_assert(COLS <= NT, "a thread adds up one column");
  __shared__ float q_s[kStepMaxDim], k_s[kStepMaxDim];
  __shared__ __attribute__((aligned(16))) float part_s[WAVES][COLS];
  __shared__ float o_s[FORM == kScanExp ? kStepMaxV : 1];
  __shared__ float red[16];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int dim = a.dim, vdim = a.vdim, H = a.H, g = h / (H / a.G);
  const int64_t row = a.seq_row_start[s];
  const T* r = (const T*)a.rows + row * a.stride;
  float* slot = a.state + (int64_t)a.seq_slots[s] * a.state_stride;
  float* st = slot + (int64_t)h * dim * vdim;
  const int ty = tid / TX, tx = tid % TX;
  const int c_begin = FORM == kScanExp ? 0 : blockIdx.z * COLS;
  const int c_end = FORM == kScanExp ? vdim : min(vdim, c_begin + COLS);
  float S[PASSES][VEC];
  // (channels and columns beyond the last are fetched from the last: loads inside branches would
  // be waited for one by one)
  auto fetch = [&](int c0) {
    const int col = min(c0 + tx * VEC, vdim - VEC);
#pragma unroll
    for (int p = 0; p < PASSES; ++p) step_load<VEC>(st + (int64_t)min(p * ROWS + ty, dim - 1) * vdim + col, S[p]);
  };
  fetch(c_begin);
  for (int d = tid; d < dim; d += NT) {
    q_s[d] = to_f32(r[a.q_off + g * dim + d]) * a.q_scale;
    k_s[d] = to_f32(r[a.k_off + g * dim + d]);
  }
  float keep, write, m_new = 0.f;
  if constexpr (FORM == kScanStep) {
    const float dt = scan_softplus(a.z[row * H + h] + a.z_bias[h]);
    keep = expf(-a.rate[h] * dt);
    write = dt;
  } else {
    const float m = slot[(int64_t)H * dim * (vdim + 1) + h];
    float i, f;
    scan_exp_gates(a, row, h, &i, &f);
    m_new = fmaxf(f + m, i);
    keep = expf(f + m - m_new);
    write = expf(i - m_new);
  }
  __syncthreads();   // q and k are there; everyone has read m
  float inv_den = 1.f;
  if constexpr (FORM == kScanExp) {
    float* n = slot + (int64_t)H * dim * vdim + (int64_t)h * dim;
    float nq = 0.f;
    for (int d = tid; d < dim; d += NT) {
      const float nn = fmaf(keep, n[d], write * k_s[d]);
      n[d] = nn;
      nq = fmaf(nn, q_s[d], nq);
    }
    nq = block_sum(nq, red);
    inv_den = 1.f / (fmaxf(fabsf(nq), expf(-m_new)) + 1e-6f);
    if (tid == 0) slot[(int64_t)H * dim * (vdim + 1) + h] = m_new;
  }
  for (int c0 = c_begin; c0 < c_end; c0 += COLS) {
    if (c0 > c_begin) fetch(c0);
    const int col = c0 + tx * VEC;
    float v[VEC], acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      v[e] = col + e < vdim ? to_f32(r[a.v_off + h * vdim + col + e]) * write : 0.f;
      acc[e] = 0.f;
    }
#pragma unroll
    for (int p = 0; p < PASSES; ++p) {
      const int d = p * ROWS + ty;
      if (d < dim && col < vdim) {
        const float k = k_s[d], q = q_s[d];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          S[p][e] = fmaf(keep, S[p][e], k * v[e]);
          acc[e] = fmaf(S[p][e], q, acc[e]);
        }
        step_store<VEC>(st + (int64_t)d * vdim + col, S[p]);
      }
    }
    // the rows of a wave, then the waves
#pragma unroll
    for (int off = TX; off < 64; off <<= 1)
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] += __shfl_xor(acc[e], off, 64);
    if (lane < TX) step_store<VEC>(&part_s[wave][tx * VEC], acc);
    __syncthreads();
    if (tid < COLS && c0 + tid < vdim) {
      float o = 0.f;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) o += part_s[w][tid];
      if constexpr (FORM == kScanStep)
        a.out[(row * H + h) * vdim + c0 + tid] =
            fmaf(a.skip[h], to_f32(r[a.v_off + h * vdim + c0 + tid]), o);
      else
        o_s[c0 + tid] = o * inv_den;
    }
    __syncthreads();
  }
  if constexpr (FORM == kScanExp) {   // the head's norm and gate
    float ss = 0.f;
    for (int c = tid; c < vdim; c += NT) ss = fmaf(o_s[c], o_s[c], ss);
    ss = block_sum(ss, red);
    const float inv = 1.f / sqrtf(ss / (float)vdim + a.eps);
    for (int c = tid; c < vdim; c += NT) {
      const float zg = to_f32(((const T*)a.gate)[row * a.gate_stride + h * vdim + c]);
      ((T*)a.normed)[(row * H + h) * vdim + c] =
          from_f32<T>(o_s[c] * inv * a.norm_w[h * vdim + c] / (1.f + expf(-zg)));
    }
  }
}

template <typename T, int NT, int VEC, int TX, int FORM>
static int launch_step_tx(const ScanArgs& a, int n, hipStream_t stream) {
  const dim3 grid(n, a.H, FORM == kScanExp ? 1 : (a.vdim + TX * VEC - 1) / (TX * VEC));
  const int passes = (a.dim + NT / TX - 1) / (NT / TX);
  if (passes <= 1) scan_step_kernel<T, NT, VEC, TX, 1, FORM><<<grid, NT, 0, stream>>>(a);
  else if (passes <= 2) scan_step_kernel<T, NT, VEC, TX, 2, FORM><<<grid, NT, 0, stream>>>(a);
  else if (passes <= 4) scan_step_kernel<T, NT, VEC, TX, 4, FORM><<<grid, NT, 0, stream>>>(a);
  else if (passes <= 8) scan_step_kernel<T, NT, VEC, TX, 8, FORM><<<grid, NT, 0, stream>>>(a);
  else if constexpr (NT == 512) scan_step_kernel<T, NT, VEC, TX, 16, FORM><<<grid, NT, 0, stream>>>(a);
  else return set_error(-1, "decay_scan: %d key channels in more passes than there are kernels for", a.dim);
  NINFER_LAUNCH_CHECK();
  return 0;
}

template <typename T, int VEC, int FORM>
static int launch_step(const ScanArgs& a, int n, hipStream_t stream) {
  if constexpr (FORM == kScanStep) {
    return launch_step_tx<T, 512, VEC, 16, FORM>(a, n, stream);
  } else {
    // as many columns at a time as a head has, while a thread's share of the channels is at most 8
    if constexpr (VEC == 4) {
      if (a.vdim > 128 && a.dim <= 128) return launch_step_tx<T, 1024, VEC, 64, FORM>(a, n, stream);
      if (a.vdim > 64 && a.dim <= 256) return launch_step_tx<T, 1024, VEC, 32, FORM>(a, n, stream);
    }
    return launch_step_tx<T, 1024, VEC, 16, FORM>(a, n, stream);
  }
}

template <typename T, int FORM>
static int launch_seq(const ScanArgs& a, hipStream_t stream) {
  const int n = a.S - a.first_seq;
  scan_gates_kernel<<<dim3(n, (a.H + 63) / 64), 64, 0, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  const int cols = a.vdim + (FORM == kScanExp ? 1 : 0), per = kSeqCols * kSeqWaves;
  const dim3 grid(n, a.H, (cols + per - 1) / per);
  if (a.dim <= 32) scan_seq_kernel<T, 8, FORM><<<grid, 64 * kSeqWaves, 0, stream>>>(a);
  else if (a.dim <= 64) scan_seq_kernel<T, 16, FORM><<<grid, 64 * kSeqWaves, 0, stream>>>(a);
  else if (a.dim <= 128) scan_seq_kernel<T, 32, FORM><<<grid, 64 * kSeqWaves, 0, stream>>>(a);
  else if (a.dim <= 256) scan_seq_kernel<T, 64, FORM><<<grid, 64 * kSeqWaves, 0, stream>>>(a);
  else scan_seq_kernel<T, 128, FORM><<<grid, 64 * kSeqWaves, 0, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return 0;
}

}  // namespace ninfer

using namespace ninfer;

// Requests first_seq .. of the step, row by row. work: T * H * (2, or 3 in the form kScanExp)
// floats. Outputs to `out` (and `den`).
extern "C" int ninfer_decay_scan(const ScanArgs* args, hipStream_t stream) {
  const ScanArgs& a = *args;
  if (int rc = scan_check(a)) return rc;
  NINFER_REQUIRE(a.work && a.out && (a.form == kScanStep || a.den), "decay_scan: no room for gates or outputs");
  if (a.form == kScanStep)
    return a.dtype == kF32 ? launch_seq<float, kScanStep>(a, stream) : launch_seq<bf16, kScanStep>(a, stream);
  return a.dtype == kF32 ? launch_seq<float, kScanExp>(a, stream) : launch_seq<bf16, kScanExp>(a, stream);
}

// The step's first n requests, which bring one row each. kScanStep: outputs to `out`; kScanExp:
// divided, normed and gated, to `normed`. Returns 1 (nothing launched) when the sizes do not fit.
extern "C" int ninfer_decay_scan_single(const ScanArgs* args, int n, hipStream_t stream) {
  const ScanArgs& a = *args;
  if (int rc = scan_check(a)) return rc;
  NINFER_REQUIRE(n > 0 && n <= a.S, "decay_scan: %d single rows of %d requests", n, a.S);
  NINFER_REQUIRE(a.form == kScanStep ? a.out != nullptr : (a.gate && a.norm_w && a.normed && a.gate_stride >= a.H * a.vdim),
                 "decay_scan: no room for the outputs");
  if (a.form == kScanExp && a.vdim > kStepMaxV) return 1;
  const bool vec = a.vdim % 4 == 0 && a.state_stride % 4 == 0 && (uintptr_t)a.state % 16 == 0;
#define NINFER_SCAN_STEP(TYPE)                                                                        \
  do {                                                                                                \
    if (a.form == kScanStep)                                                                          \
      return vec ? launch_step<TYPE, 4, kScanStep>(a, n, stream) : launch_step<TYPE, 1, kScanStep>(a, n, stream); \
    return vec ? launch_step<TYPE, 4, kScanExp>(a, n, stream) : launch_step<TYPE, 1, kScanExp>(a, n, stream);     \
  } while (0)
  if (a.dtype == kF32) NINFER_SCAN_STEP(float);
  NINFER_SCAN_STEP(bf16);
#undef NINFER_SCAN_STEP
}
