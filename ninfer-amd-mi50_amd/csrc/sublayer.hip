// Row-wise kernels around a sublayer whose norm sits on its output:
//
//   short_conv     h_t + sum_j w[:, j] h_(t - taps + 1 + j): a causal convolution over the
//                  rows of each request, channel by channel, added to its input. The last
//                  taps - 1 inputs of a request are per-request state (32-bit), so a request
//                  may be cut into steps anywhere; before a request's start they are zero.
//   norm_add       x += y rsqrt(mean(y^2) + eps) g, g one number or one per channel; optionally
//                  with the row's mean taken off first (a layer norm), and with y a weighted
//                  sum of rows.
//   gated_rmsnorm  out = o rsqrt(mean(o^2) + eps) w sigmoid(g) (or w g sigmoid(g)), the norm
//                  over the whole row or over every group of columns (a head's) by itself;
//                  without a gate the last factor is 1. Or with the gate in front of the norm,
//                  o <- o act(g) first; with a divisor per group, o <- o / den first.
//   post_norm      x <- z rsqrt(mean(z^2) + eps) g with z = alpha x + y, written in 32-bit and
//                  once more in the activation dtype for whoever reads x next; y a row, a
//                  weighted sum of rows, or half-and-half of two normed rows.
//
// All sums are 32-bit and their order depends on the row alone (taps ascending; the block
// reduction's order depends on the width), never on how a request was cut or on the batch.
#include "common.h"

namespace ninfer {

// out[t, c] for all rows. Inputs before the step's first row of a request come from the
// request's state: state[slot][i * H + c] is the input at the request's position
// pos0 - (taps - 1) + i. With `update` (steps in which every request brings one row) the
// thread also shifts the state; otherwise short_conv_state_kernel does so afterwards.
template <typename T>
__global__ void short_conv_kernel(const float* __restrict__ x, const float* __restrict__ w,
                                  float* __restrict__ state, int64_t state_stride,
                                  T* __restrict__ out, const int* __restrict__ row_seq,
                                  const int* __restrict__ seq_row_start,
                                  const int* __restrict__ seq_slots, int H, int taps, int update) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= H) return;
  const int s = row_seq[t];
  const int r0 = seq_row_start[s];
  const int i = t - r0;
  float* st = state + (int64_t)seq_slots[s] * state_stride;
  const float* wc = w + (int64_t)c * taps;
  const float cur = x[(int64_t)t * H + c];
  float acc = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int src = i - (taps - 1 - j);
    const float v = src >= 0 ? x[(int64_t)(r0 + src) * H + c] : st[(int64_t)(taps - 1 + src) * H + c];
    acc = fmaf(wc[j], v, acc);
  }
  out[(int64_t)t * H + c] = from_f32<T>(cur + acc);
  if (update) {   // this row is the request's only one: the state moves on by one input
    for (int k = 0; k + 2 < taps; ++k) st[(int64_t)k * H + c] = st[(int64_t)(k + 1) * H + c];
    if (taps > 1) st[(int64_t)(taps - 2) * H + c] = cur;
  }
}

// state <- the last taps - 1 inputs of each request after this step's n rows. Entry k is the
// input at index n - (taps - 1) + k of the step's rows; a negative index is the old entry
// k + n, which lies above k, so ascending k never reads what it has written.
__global__ void short_conv_state_kernel(const float* __restrict__ x, float* __restrict__ state,
                                        int64_t state_stride,
                                        const int* __restrict__ seq_row_start,
                                        const int* __restrict__ seq_slots, int H, int taps) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= H) return;
  const int r0 = seq_row_start[s];
  const int n = seq_row_start[s + 1] - r0;
  float* st = state + (int64_t)seq_slots[s] * state_stride;
  for (int k = 0; k < taps - 1; ++k) {
    const int p = n - (taps - 1) + k;
    st[(int64_t)k * H + c] = p >= 0 ? x[(int64_t)(r0 + p) * H + c] : st[(int64_t)(k + n) * H + c];
  }
}

// x += norm(y) g with norm(y) = y rsqrt(mean(y^2) + eps), or with `center` the layer norm
// (y - mean) rsqrt(mean((y - mean)^2) + eps). y is a row of `y`, or with `w` the weighted sum of
// k rows, y_r = sum_j w[r, j] y[r k + j] (a sparse feed-forward's chosen experts), formed in
// 32-bit in the order of j. A thread keeps its (at most 8) numbers of the row in registers, in
// groups of VEC consecutive ones (VEC 4: whole 8- and 16-byte loads and stores).
constexpr int kNormAddPerThread = 8;
template <int VEC>
__device__ __forceinline__ void na_load(const float* p, float* f) {
  if constexpr (VEC == 4) {
    const float4 v = *(const float4*)p;
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  } else {
    f[0] = p[0];
  }
}
template <int VEC>
__device__ __forceinline__ void na_load(const bf16* p, float* f) {
  if constexpr (VEC == 4) {
    const uint2 v = *(const uint2*)p;   // four bf16: the upper halves of four floats
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
  } else {
    f[0] = to_f32(p[0]);
  }
}

template <typename T, int VEC>
__global__ void norm_add_kernel(float* __restrict__ x, const T* __restrict__ y,
                                const float* __restrict__ w, int k,
                                const float* __restrict__ gain, int gain_n, int H, float eps,
                                int center) {
  constexpr int G = kNormAddPerThread / VEC;
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  float vals[G][VEC];
  float sum = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
#pragma unroll
    for (int e = 0; e < VEC; ++e) vals[c][e] = 0.f;
    if (i < H) {
      if (w) {
        for (int j = 0; j < k; ++j) {
          float yv[VEC];
          na_load<VEC>(y + (r * k + j) * H + i, yv);
          const float wj = w[r * k + j];
#pragma unroll
          for (int e = 0; e < VEC; ++e) vals[c][e] = fmaf(wj, yv[e], vals[c][e]);
        }
      } else {
        na_load<VEC>(y + r * H + i, vals[c]);
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) sum += vals[c][e];
  }
  const float mean = center ? block_sum(sum, red) / (float)H : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const bool in = VEC * (threadIdx.x + c * blockDim.x) < H;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float d = in ? vals[c][e] - mean : 0.f;
      ss = fmaf(d, d, ss);
    }
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)H + eps);
  float* xr = x + r * H;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i < H) {
      float xv[VEC], gv[VEC];
      na_load<VEC>(xr + i, xv);
      if (gain_n == 1) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) gv[e] = gain[0];
      } else {
        na_load<VEC>(gain + i, gv);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) xv[e] += (vals[c][e] - mean) * inv * gv[e];
      if constexpr (VEC == 4) *(float4*)(xr + i) = make_float4(xv[0], xv[1], xv[2], xv[3]);
      else xr[i] = xv[0];
    }
  }
}

// x <- norm(alpha x + y), norm(z) = z rsqrt(mean(z^2) + eps) gain; also as T into `out` when that
// is given. y: a row of `y`; with `w` the weighted sum of k rows (as norm_add has it); with `y2`
// factor * (rms(y) gain1 + rms(y2) gain2). The pieces of a row stay in registers throughout.
struct PostNormArgs {
  float* x;            // [T, H]
  const void* y;       // [T, H], or [T k, H] with w
  const void* y2;      // [T, H] or null
  const float* gain1;  // [H] with y2
  const float* gain2;
  const float* w;      // [T, k] or null
  const float* gain;   // [H]
  void* out;           // [T, H] or null
  int T;
  int H;
  int k;
  int dtype;
  float alpha;
  float eps;
  float factor;
};

// Two sums over a block at once; every thread gets both.
__device__ __forceinline__ void block_sum2(float& u, float& v, float (*red)[2]) {
  u = wave_sum(u);
  v = wave_sum(v);
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();
  if (lane == 0) red[wv][0] = u, red[wv][1] = v;
  __syncthreads();
  u = v = 0.f;
  for (int i = 0; i < nw; ++i) u += red[i][0], v += red[i][1];
}

template <typename T, int VEC>
__global__ void post_norm_kernel(PostNormArgs a) {
  constexpr int G = kNormAddPerThread / VEC;
  __shared__ float red[16];
  __shared__ float red2[16][2];
  const int64_t r = blockIdx.x;
  const int H = a.H;
  const T* y = (const T*)a.y;
  float* xr = a.x + r * H;
  float z[G][VEC];
  if (a.y2) {
    const T* y2 = (const T*)a.y2;
    float b[G][VEC];
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int c = 0; c < G; ++c) {
      const int i = VEC * (threadIdx.x + c * blockDim.x);
#pragma unroll
      for (int e = 0; e < VEC; ++e) z[c][e] = b[c][e] = 0.f;
      if (i < H) {
        na_load<VEC>(y + r * H + i, z[c]);
        na_load<VEC>(y2 + r * H + i, b[c]);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) sa = fmaf(z[c][e], z[c][e], sa), sb = fmaf(b[c][e], b[c][e], sb);
    }
    block_sum2(sa, sb, red2);
    const float ia = a.factor / sqrtf(sa / (float)H + a.eps), ib = a.factor / sqrtf(sb / (float)H + a.eps);
#pragma unroll
    for (int c = 0; c < G; ++c) {
      const int i = VEC * (threadIdx.x + c * blockDim.x);
      if (i < H) {
        float ga[VEC], gb[VEC];
        na_load<VEC>(a.gain1 + i, ga);
        na_load<VEC>(a.gain2 + i, gb);
#pragma unroll
        for (int e = 0; e < VEC; ++e) z[c][e] = z[c][e] * ia * ga[e] + b[c][e] * ib * gb[e];
      }
    }
  } else {
#pragma unroll
    for (int c = 0; c < G; ++c) {
      const int i = VEC * (threadIdx.x + c * blockDim.x);
#pragma unroll
      for (int e = 0; e < VEC; ++e) z[c][e] = 0.f;
      if (i < H) {
        if (a.w) {
          for (int j = 0; j < a.k; ++j) {
            float yv[VEC];
            na_load<VEC>(y + (r * a.k + j) * H + i, yv);
            const float wj = a.w[r * a.k + j];
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[c][e] = fmaf(wj, yv[e], z[c][e]);
          }
        } else {
          na_load<VEC>(y + r * H + i, z[c]);
        }
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i < H) {
      float xv[VEC];
      na_load<VEC>(xr + i, xv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        z[c][e] = fmaf(a.alpha, xv[e], z[c][e]);
        ss = fmaf(z[c][e], z[c][e], ss);
      }
    }
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)H + a.eps);
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i < H) {
      float g[VEC];
      na_load<VEC>(a.gain + i, g);
#pragma unroll
      for (int e = 0; e < VEC; ++e) z[c][e] *= inv * g[e];
      if constexpr (VEC == 4) {
        *(float4*)(xr + i) = make_float4(z[c][0], z[c][1], z[c][2], z[c][3]);
      } else {
        xr[i] = z[c][0];
      }
      if (a.out) {
        T* o = (T*)a.out + r * H + i;
        if constexpr (VEC == 4 && sizeof(T) == 2) {
          union { __bf16 b[4]; uint2 u; } p;
#pragma unroll
          for (int e = 0; e < 4; ++e) p.b[e] = (__bf16)z[c][e];
          *(uint2*)o = p.u;
        } else {
#pragma unroll
          for (int e = 0; e < VEC; ++e) o[e] = from_f32<T>(z[c][e]);
        }
      }
    }
  }
}

struct GatedNormArgs {
  const float* o;       // [T, N]
  const void* gate;     // [T, gate_stride] or null
  const float* w;       // [w_n]: a number per column of the row (w_n = N) or of a group
  const float* den;     // [T, N / group] or null: what a group's numbers are divided by first
  void* out;            // [T, N]
  int gate_stride, T, N, group, w_n, silu, gate_first, dtype;
  float eps;
};

// VEC numbers of the row as the norm takes them, and the factors that follow the norm.
template <typename T, int VEC>
__device__ __forceinline__ void gated_norm_in(const GatedNormArgs& a, int64_t r, int i, float inv_den, float* v, float* after) {
  na_load<VEC>(a.o + r * a.N + i, v);
  float z[VEC];
  if (a.gate) na_load<VEC>((const T*)a.gate + r * a.gate_stride + i, z);
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    v[e] *= inv_den;
    after[e] = a.gate ? (a.silu ? z[e] : 1.f) * sigmoid_for<T>(z[e]) : 1.f;
    if (a.gate_first) v[e] *= after[e], after[e] = 1.f;
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void gated_norm_out(const GatedNormArgs& a, int64_t r, int i, const float* w, float inv,
                                               const float* v, const float* after) {
  T* out = (T*)a.out + r * a.N + i;
  float g[VEC], y[VEC];
  na_load<VEC>(w, g);
#pragma unroll
  for (int e = 0; e < VEC; ++e) y[e] = v[e] * inv * g[e] * after[e];
  if constexpr (VEC == 4 && sizeof(T) == 4) {
    *(float4*)out = make_float4(y[0], y[1], y[2], y[3]);
  } else if constexpr (VEC == 4) {
    union { __bf16 b[4]; uint2 u; } p;
#pragma unroll
    for (int e = 0; e < 4; ++e) p.b[e] = (__bf16)y[e];
    *(uint2*)out = p.u;
  } else {
    out[0] = from_f32<T>(y[0]);
  }
}

// A block per (row, group); a thread keeps its (at most 16) numbers in registers, in groups of VEC
// consecutive ones.
constexpr int kGatedPerThread = 16;
template <typename T, int VEC>
__global__ void gated_rmsnorm_kernel(GatedNormArgs a) {
  constexpr int G = kGatedPerThread / VEC;
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int g0 = blockIdx.y * a.group;
  const float inv_den = a.den ? 1.f / a.den[r * gridDim.y + blockIdx.y] : 1.f;
  const float* w = a.w + (a.w_n == a.N ? g0 : 0);
  float v[G][VEC], sg[G][VEC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i < a.group) {
      gated_norm_in<T, VEC>(a, r, g0 + i, inv_den, v[c], sg[c]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(v[c][e], v[c][e], ss);
    }
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)a.group + a.eps);
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i < a.group) gated_norm_out<T, VEC>(a, r, g0 + i, w + i, inv, v[c], sg[c]);
  }
}

// The same for groups of few columns (a head's values): one wave per (row, group), four groups
// to a block.
constexpr int kGatedWaveMax = 512;
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gated_group_rmsnorm_kernel(GatedNormArgs a) {
  constexpr int PER = kGatedWaveMax / 64 / VEC;
  const int64_t r = blockIdx.x;
  const int g = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int g0 = g * a.group;
  if (g0 >= a.N) return;
  const float inv_den = a.den ? 1.f / a.den[r * (a.N / a.group) + g] : 1.f;
  const float* w = a.w + (a.w_n == a.N ? g0 : 0);
  float v[PER][VEC], sg[PER][VEC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < PER; ++c) {
    const int i = VEC * (lane + 64 * c);
    if (i < a.group) {
      gated_norm_in<T, VEC>(a, r, g0 + i, inv_den, v[c], sg[c]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(v[c][e], v[c][e], ss);
    }
  }
  ss = wave_sum(ss);
  const float inv = 1.f / sqrtf(ss / (float)a.group + a.eps);
#pragma unroll
  for (int c = 0; c < PER; ++c) {
    const int i = VEC * (lane + 64 * c);
    if (i < a.group) gated_norm_out<T, VEC>(a, r, g0 + i, w + i, inv, v[c], sg[c]);
  }
}

template <typename T, int VEC>
static void launch_gated_norm(const GatedNormArgs& a, hipStream_t stream) {
  const int groups = a.N / a.group;
  if (a.group <= kGatedWaveMax && groups > 1) {
    gated_group_rmsnorm_kernel<T, VEC><<<dim3(a.T, (groups + 3) / 4), 256, 0, stream>>>(a);
  } else {
    const int want = ((a.group + VEC - 1) / VEC + 63) / 64 * 64;
    gated_rmsnorm_kernel<T, VEC><<<dim3(a.T, groups), want > 1024 ? 1024 : want, 0, stream>>>(a);
  }
}

static int row_block(int H) {
  int b = (H + 63) / 64 * 64;
  return b > 256 ? 256 : b;
}

}  // namespace ninfer

using namespace ninfer;

extern "C" int ninfer_short_conv(const float* x, const float* w, float* state,
                                 long long state_stride, void* out, const int* row_seq,
                                 const int* seq_row_start, const int* seq_slots, int T, int S,
                                 int H, int taps, int all_single, int dtype, hipStream_t stream) {
  NINFER_REQUIRE(T > 0 && S > 0 && H > 0, "short_conv: T=%d S=%d H=%d must be positive", T, S, H);
  NINFER_REQUIRE(taps >= 1, "short_conv: %d taps", taps);
  NINFER_REQUIRE(state_stride >= (long long)(taps - 1) * H,
                 "short_conv: a request's state of %lld floats holds no %d x %d inputs",
                 state_stride, taps - 1, H);
  NINFER_REQUIRE(dtype == kF32 || dtype == kBF16, "short_conv: unknown dtype %d", dtype);
  const int block = row_block(H);
  const dim3 grid(T, (H + block - 1) / block);
  if (dtype == kF32)
    short_conv_kernel<float><<<grid, block, 0, stream>>>(x, w, state, state_stride, (float*)out,
                                                         row_seq, seq_row_start, seq_slots, H,
                                                         taps, all_single);
  else
    short_conv_kernel<bf16><<<grid, block, 0, stream>>>(x, w, state, state_stride, (bf16*)out,
                                                        row_seq, seq_row_start, seq_slots, H, taps,
                                                        all_single);
  NINFER_LAUNCH_CHECK();
  if (!all_single && taps > 1) {
    short_conv_state_kernel<<<dim3(S, (H + block - 1) / block), block, 0, stream>>>(
        x, state, state_stride, seq_row_start, seq_slots, H, taps);
    NINFER_LAUNCH_CHECK();
  }
  return 0;
}

extern "C" int ninfer_norm_add(float* x, const void* y, const float* gain, int gain_n, int T, int H,
                               float eps, int dtype, int center, const float* w, int k,
                               hipStream_t stream) {
  NINFER_REQUIRE(T > 0 && H > 0, "norm_add: T=%d H=%d must be positive", T, H);
  NINFER_REQUIRE(gain_n == 1 || gain_n == H, "norm_add: %d gains for %d channels", gain_n, H);
  NINFER_REQUIRE(dtype == kF32 || dtype == kBF16, "norm_add: unknown dtype %d", dtype);
  NINFER_REQUIRE(H <= 1024 * kNormAddPerThread, "norm_add: width %d exceeds %d", H,
                 1024 * kNormAddPerThread);
  NINFER_REQUIRE(!w || k > 0, "norm_add: a weighted sum of %d rows", k);
  // groups of 4 consecutive numbers when every row stays 16-byte aligned
  auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = H % 4 == 0 && aligned(x) && aligned(y) && (gain_n == 1 || aligned(gain));
  const int per_thread = vec ? 4 : 1;
  int block = ((H + per_thread - 1) / per_thread + 63) / 64 * 64;
  if (block > 1024) block = 1024;
  NINFER_REQUIRE((int64_t)block * kNormAddPerThread >= H, "norm_add: width %d exceeds the kernel's", H);
  if (dtype == kF32) {
    if (vec) norm_add_kernel<float, 4><<<T, block, 0, stream>>>(x, (const float*)y, w, k, gain, gain_n, H, eps, center);
    else norm_add_kernel<float, 1><<<T, block, 0, stream>>>(x, (const float*)y, w, k, gain, gain_n, H, eps, center);
  } else {
    if (vec) norm_add_kernel<bf16, 4><<<T, block, 0, stream>>>(x, (const bf16*)y, w, k, gain, gain_n, H, eps, center);
    else norm_add_kernel<bf16, 1><<<T, block, 0, stream>>>(x, (const bf16*)y, w, k, gain, gain_n, H, eps, center);
  }
  NINFER_LAUNCH_CHECK();
  return 0;
}

extern "C" int ninfer_post_norm(const PostNormArgs* args, hipStream_t stream) {
  const PostNormArgs& a = *args;
  NINFER_REQUIRE(a.T > 0 && a.H > 0 && a.x && a.y && a.gain, "post_norm: T=%d H=%d must be positive", a.T, a.H);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "post_norm: unknown dtype %d", a.dtype);
  NINFER_REQUIRE(!a.w || a.k > 0, "post_norm: a weighted sum of %d rows", a.k);
  NINFER_REQUIRE(!a.y2 || (a.gain1 && a.gain2 && !a.w), "post_norm: two normed rows need their gains and no weights");
  auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = a.H % 4 == 0 && aligned(a.x) && aligned(a.y) && aligned(a.gain) && aligned(a.y2) &&
                   aligned(a.gain1) && aligned(a.gain2) && aligned(a.out);
  const int per_thread = vec ? 4 : 1;
  int block = ((a.H + per_thread - 1) / per_thread + 63) / 64 * 64;
  if (block > 1024) block = 1024;
  NINFER_REQUIRE((int64_t)block * kNormAddPerThread >= a.H, "post_norm: width %d exceeds the kernel's", a.H);
  if (a.dtype == kF32) {
    if (vec) post_norm_kernel<float, 4><<<a.T, block, 0, stream>>>(a);
    else post_norm_kernel<float, 1><<<a.T, block, 0, stream>>>(a);
  } else {
    if (vec) post_norm_kernel<bf16, 4><<<a.T, block, 0, stream>>>(a);
    else post_norm_kernel<bf16, 1><<<a.T, block, 0, stream>>>(a);
  }
  NINFER_LAUNCH_CHECK();
  return 0;
}

// group 0 (or N): the norm over the whole row; else over every group of `group` columns by
// itself, with a weight of `group` numbers that the groups share or of N.
extern "C" int ninfer_gated_rmsnorm(const GatedNormArgs* args, hipStream_t stream) {
  GatedNormArgs a = *args;
  NINFER_REQUIRE(a.T > 0 && a.N > 0 && (!a.gate || a.gate_stride >= a.N), "gated_rmsnorm: T=%d N=%d gate stride %d", a.T,
                 a.N, a.gate_stride);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "gated_rmsnorm: unknown dtype %d", a.dtype);
  if (a.group == 0) a.group = a.N;
  NINFER_REQUIRE(a.group > 0 && a.N % a.group == 0, "gated_rmsnorm: groups of %d columns do not fill rows of %d",
                 a.group, a.N);
  NINFER_REQUIRE(a.w_n == a.N || a.w_n == a.group, "gated_rmsnorm: %d weights for groups of %d columns", a.w_n, a.group);
  NINFER_REQUIRE(a.group <= 1024 * kGatedPerThread, "gated_rmsnorm: %d columns exceed %d", a.group, 1024 * kGatedPerThread);
  NINFER_REQUIRE(!a.gate_first || a.gate, "gated_rmsnorm: no gate to apply first");
  auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = a.group % 4 == 0 && (!a.gate || a.gate_stride % 4 == 0) && aligned(a.o) && aligned(a.gate) &&
                   aligned(a.w) && aligned(a.out);
  if (a.dtype == kF32) {
    if (vec) launch_gated_norm<float, 4>(a, stream);
    else launch_gated_norm<float, 1>(a, stream);
  } else {
    if (vec) launch_gated_norm<bf16, 4>(a, stream);
    else launch_gated_norm<bf16, 1>(a, stream);
  }
  NINFER_LAUNCH_CHECK();
  return 0;
}
