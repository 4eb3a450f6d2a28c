// The 32-bit residual stream between two sublayers, in one kernel (a block per row): what the
// last sublayer left is added to the stream, and the stream is handed on, normed or as it is:
//
//   z = x + add,  add = nothing | f1 y1 + f2 y2 + bias | rms(y1) gain1      (rms(y) =
//                                                          y rsqrt(mean(y^2) + eps1))
//   x <- z (when something was added),  out = z rsqrt(mean(z^2) + eps) gain, or z itself
//
// With `rows` only those rows are read, and x is left as it is. A row's numbers stay in registers
// between the passes; all sums are 32-bit and their order depends on the width alone.
//
// Beside it: g = gelu(z) * table[token, columns], the gate of a per-layer token input.
#include "common.h"

namespace ninfer {

struct StreamNormArgs {
  float* x;             // [*, H]
  const void* y1;       // [*, H] or null
  const void* y2;       // [*, H] or null
  const float* bias;    // [H] or null
  const float* gain1;   // [H] or null: y1 is normed
  const float* gain;    // [H] or null: z is not normed
  void* out;            // [n_rows, H] or null
  const int* rows;      // [n_rows] or null
  int n_rows, H, dtype;
  float f1, f2, eps1, eps;
};

constexpr int kStreamPerThread = 8;

template <int VEC>
__device__ __forceinline__ void sn_load(const float* p, float* f) {
  if constexpr (VEC == 4) {
    const float4 v = *(const float4*)p;
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  } else {
    f[0] = p[0];
  }
}
template <int VEC>
__device__ __forceinline__ void sn_load(const bf16* p, float* f) {
  if constexpr (VEC == 4) {
    const uint2 v = *(const uint2*)p;
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
  } else {
    f[0] = to_f32(p[0]);
  }
}
template <int VEC>
__device__ __forceinline__ void sn_store(float* p, const float* f) {
  if constexpr (VEC == 4) *(float4*)p = make_float4(f[0], f[1], f[2], f[3]);
  else p[0] = f[0];
}
template <int VEC>
__device__ __forceinline__ void sn_store(bf16* p, const float* f) {
  if constexpr (VEC == 4) {
    union { __bf16 b[4]; uint2 u; } w;
#pragma unroll
    for (int e = 0; e < 4; ++e) w.b[e] = (__bf16)f[e];
    *(uint2*)p = w.u;
  } else {
    p[0] = from_f32<bf16>(f[0]);
  }
}

template <typename T, int VEC>
__global__ void stream_norm_kernel(StreamNormArgs a) {
  constexpr int G = kStreamPerThread / VEC;
  __shared__ float red[16];
  const int H = a.H;
  const int64_t r_out = blockIdx.x, r = a.rows ? a.rows[r_out] : r_out;
  float* xr = a.x + r * H;
  const T* y1 = a.y1 ? (const T*)a.y1 + r * H : nullptr;
  const T* y2 = a.y2 ? (const T*)a.y2 + r * H : nullptr;
  float z[G][VEC], y[G][VEC];
  float sy = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
#pragma unroll
    for (int e = 0; e < VEC; ++e) z[c][e] = y[c][e] = 0.f;
    if (i < H) {
      sn_load<VEC>(xr + i, z[c]);
      if (y1) sn_load<VEC>(y1 + i, y[c]);
      if (!a.gain1) {
        float t[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[c][e] *= a.f1;
        if (y2) {
          sn_load<VEC>(y2 + i, t);
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[c][e] = fmaf(a.f2, t[e], y[c][e]);
        }
        if (a.bias) {
          sn_load<VEC>(a.bias + i, t);
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[c][e] += t[e];
        }
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) sy = fmaf(y[c][e], y[c][e], sy);
  }
  if (a.gain1) {
    const float inv = 1.f / sqrtf(block_sum(sy, red) / (float)H + a.eps1);
#pragma unroll
    for (int c = 0; c < G; ++c) {
      const int i = VEC * (threadIdx.x + c * blockDim.x);
      if (i < H) {
        float g[VEC];
        sn_load<VEC>(a.gain1 + i, g);
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[c][e] *= inv * g[e];
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < G; ++c)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      z[c][e] += y[c][e];
      ss = fmaf(z[c][e], z[c][e], ss);
    }
  const float inv = a.gain ? 1.f / sqrtf(block_sum(ss, red) / (float)H + a.eps) : 1.f;
  const bool back = !a.rows && (a.y1 || a.bias);
#pragma unroll
  for (int c = 0; c < G; ++c) {
    const int i = VEC * (threadIdx.x + c * blockDim.x);
    if (i >= H) continue;
    if (back) sn_store<VEC>(xr + i, z[c]);
    if (!a.out) continue;
    if (a.gain) {
      float g[VEC];
      sn_load<VEC>(a.gain + i, g);
#pragma unroll
      for (int e = 0; e < VEC; ++e) z[c][e] *= inv * g[e];
    }
    sn_store<VEC>((T*)a.out + r_out * H + i, z[c]);
  }
}

// out[t, i] = gelu(z[t, i]) table[tokens[t], column0 + i], gelu(z) = z / 2 (1 + tanh(sqrt(2 / pi)
// (z + 0.044715 z^3)))
template <typename T>
__global__ void token_gate_kernel(const T* __restrict__ z, const T* __restrict__ table,
                                  const int* __restrict__ tokens, T* __restrict__ out, int T_rows, int d,
                                  int width, int column0) {
  const int idx = blockIdx.x * blockDim.x + threadIdx.x;
  const int t = idx / d, i = idx - t * d;
  if (t >= T_rows) return;
  const float v = to_f32(z[idx]);
  const float e = to_f32(table[(int64_t)tokens[t] * width + column0 + i]);
  out[idx] = from_f32<T>(0.5f * v * (1.f + tanhf(0.7978845608028654f * (v + 0.044715f * v * v * v))) * e);
}

}  // namespace ninfer

using namespace ninfer;

extern "C" int ninfer_stream_norm(const StreamNormArgs* args, hipStream_t stream) {
  const StreamNormArgs& a = *args;
  NINFER_REQUIRE(a.n_rows > 0 && a.H > 0 && a.x, "stream_norm: rows=%d H=%d must be positive", a.n_rows, a.H);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "stream_norm: unknown dtype %d", a.dtype);
  NINFER_REQUIRE(!a.gain1 || (a.y1 && !a.y2 && !a.bias), "stream_norm: one normed row is added by itself");
  NINFER_REQUIRE(!a.y2 || a.y1, "stream_norm: a second row without a first");
  NINFER_REQUIRE(a.H <= 1024 * kStreamPerThread, "stream_norm: width %d exceeds %d", a.H, 1024 * kStreamPerThread);
  auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = a.H % 4 == 0 && aligned(a.x) && aligned(a.y1) && aligned(a.y2) && aligned(a.bias) &&
                   aligned(a.gain1) && aligned(a.gain) && aligned(a.out);
  const int per_thread = vec ? 4 : 1;
  int block = ((a.H + per_thread - 1) / per_thread + 63) / 64 * 64;
  if (block > 1024) block = 1024;
  if (a.dtype == kF32) {
    if (vec) stream_norm_kernel<float, 4><<<a.n_rows, block, 0, stream>>>(a);
    else stream_norm_kernel<float, 1><<<a.n_rows, block, 0, stream>>>(a);
  } else {
    if (vec) stream_norm_kernel<bf16, 4><<<a.n_rows, block, 0, stream>>>(a);
    else stream_norm_kernel<bf16, 1><<<a.n_rows, block, 0, stream>>>(a);
  }
  NINFER_LAUNCH_CHECK();
  return 0;
}

extern "C" int ninfer_token_gate(const void* z, const void* table, const int* tokens, void* out, int T, int d,
                                 int width, int column0, int dtype, hipStream_t stream) {
  NINFER_REQUIRE(T > 0 && d > 0 && column0 >= 0 && column0 + d <= width,
                 "token_gate: T=%d, columns %d .. + %d of %d", T, column0, d, width);
  NINFER_REQUIRE(dtype == kF32 || dtype == kBF16, "token_gate: unknown dtype %d", dtype);
  NINFER_REQUIRE((int64_t)T * d < (1LL << 31), "token_gate: %d rows of %d are too many", T, d);
  const int blocks = (int)(((int64_t)T * d + 255) / 256);
  if (dtype == kF32)
    token_gate_kernel<float><<<blocks, 256, 0, stream>>>((const float*)z, (const float*)table, tokens, (float*)out, T, d, width, column0);
  else
    token_gate_kernel<bf16><<<blocks, 256, 0, stream>>>((const bf16*)z, (const bf16*)table, tokens, (bf16*)out, T, d, width, column0);
  NINFER_LAUNCH_CHECK();
  return 0;
}
