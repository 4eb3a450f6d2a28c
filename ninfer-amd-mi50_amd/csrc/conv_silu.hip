// A short causal convolution over time per channel with a bias, and silu:
//
//   out[t, c] = silu(b[c] + sum_j w[j, c] u[t - taps + 1 + j, c]),   j = 0 .. taps - 1
//
// over the rows of each request. The inputs before a step's first row come from the request's
// state (32-bit, state[slot][k * C + c] the input at its position pos0 - (taps - 1) + k; zeros at a
// request's start), so a request may be cut into steps anywhere. Sums are 32-bit, taps ascending.
// A thread owns VEC neighbouring channels of one row, or of ROWS rows one after the other, whose
// inputs it then reads once. In steps in which every request brings one row the thread moves the
// state on itself; otherwise a second kernel does so.
#include "common.h"

namespace ninfer {

struct ConvSiluArgs {
  const void* u;            // [T, stride] rows, C columns from u on
  const float* w;           // [taps, C]
  const float* b;           // [C]
  float* state;
  void* out;                // [T, C]
  const int* row_seq;
  const int* seq_row_start;
  const int* seq_slots;
  int64_t state_stride;
  int stride, T, S, C, taps, all_single, dtype;
};

typedef unsigned int cs_u32x4 __attribute__((ext_vector_type(4)));

template <typename T, int VEC>
__device__ __forceinline__ void cs_load(const T* p, float* f) {
  if constexpr (VEC == 8) {
    const cs_u32x4 v = *(const cs_u32x4*)p;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[2 * i] = __uint_as_float(v[i] << 16);
      f[2 * i + 1] = __uint_as_float(v[i] & 0xffff0000u);
    }
  } else {
    f[0] = to_f32(p[0]);
  }
}
template <int VEC>
__device__ __forceinline__ void cs_load32(const float* p, float* f) {
  if constexpr (VEC == 8) {
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
  } else {
    f[0] = p[0];
  }
}
template <int VEC>
__device__ __forceinline__ void cs_store32(float* p, const float* f) {
  if constexpr (VEC == 8) {
    *(float4*)p = make_float4(f[0], f[1], f[2], f[3]);
    *(float4*)(p + 4) = make_float4(f[4], f[5], f[6], f[7]);
  } else {
    p[0] = f[0];
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void cs_store(T* p, const float* f) {
  if constexpr (VEC == 8) {
    union { __bf16 b[8]; cs_u32x4 v; } o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o.b[e] = (__bf16)f[e];
    *(cs_u32x4*)p = o.v;
  } else {
    p[0] = from_f32<T>(f[0]);
  }
}

// the input of row r0 + src of a request whose step begins at row r0 (src < 0: from its state)
template <typename T, int VEC>
__device__ __forceinline__ void cs_input(const ConvSiluArgs& a, const float* st, int r0, int src, int c, float* f) {
  if (src >= 0) cs_load<T, VEC>((const T*)a.u + (int64_t)(r0 + src) * a.stride + c, f);
  else cs_load32<VEC>(st + (int64_t)(a.taps - 1 + src) * a.C + c, f);
}

template <typename T, int VEC>
__global__ void conv_silu_kernel(ConvSiluArgs a) {
  const int pieces = a.C / VEC;
  const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  const int t = (int)(idx / pieces), c = (int)(idx - (int64_t)t * pieces) * VEC;
  if (t >= a.T) return;
  const int s = a.row_seq[t], r0 = a.seq_row_start[s], i = t - r0;
  float* st = a.state ? a.state + (int64_t)a.seq_slots[s] * a.state_stride : nullptr;
  float acc[VEC], v[VEC], w[VEC];
  cs_load32<VEC>(a.b + c, acc);
  for (int j = 0; j < a.taps; ++j) {
    cs_input<T, VEC>(a, st, r0, i - (a.taps - 1 - j), c, v);
    cs_load32<VEC>(a.w + (int64_t)j * a.C + c, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = fmaf(w[e], v[e], acc[e]);
  }
  if (a.all_single && a.taps > 1) {   // this row is the request's only one: the state moves on by one input
    float n[VEC];
    for (int k = 0; k + 2 < a.taps; ++k) {
      cs_load32<VEC>(st + (int64_t)(k + 1) * a.C + c, n);
      cs_store32<VEC>(st + (int64_t)k * a.C + c, n);
    }
    cs_store32<VEC>(st + (int64_t)(a.taps - 2) * a.C + c, v);   // (v: the row's own input, the last tap's)
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) acc[e] *= sigmoid_for<T>(acc[e]);
  cs_store<T, VEC>((T*)a.out + (int64_t)t * a.C + c, acc);
}

// ROWS consecutive rows per thread, TAPS known: every input is read once, all reads of a thread
// under way together (a thread whose rows and their inputs lie in one request; the others take
// their inputs one by one).
template <typename T, int VEC, int TAPS, int ROWS>
__global__ __launch_bounds__(256) void conv_silu_rows_kernel(ConvSiluArgs a) {
  const int pieces = a.C / VEC;
  const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  const int tile = (int)(idx / pieces), c = (int)(idx - (int64_t)tile * pieces) * VEC;
  const int t0 = tile * ROWS;
  if (t0 >= a.T) return;
  const int t1 = min(t0 + ROWS, a.T) - 1;
  const int s0 = a.row_seq[t0], s1 = a.row_seq[t1], r0 = a.seq_row_start[s0];
  float in[ROWS + TAPS - 1][VEC];
#pragma unroll
  for (int k = 0; k < ROWS + TAPS - 1; ++k)
    cs_load<T, VEC>((const T*)a.u + (int64_t)min(max(t0 + k - (TAPS - 1), 0), a.T - 1) * a.stride + c, in[k]);
  float w[TAPS][VEC], bias[VEC];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) cs_load32<VEC>(a.w + (int64_t)j * a.C + c, w[j]);
  cs_load32<VEC>(a.b + c, bias);
  const bool plain = s0 == s1 && t0 - (TAPS - 1) >= r0;
#pragma unroll
  for (int k = 0; k < ROWS; ++k) {
    const int t = t0 + k;
    if (t >= a.T) break;
    float acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = bias[e];
    if (plain) {
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = fmaf(w[j][e], in[k + j][e], acc[e]);
    } else {
      const int s = a.row_seq[t], first = a.seq_row_start[s];
      const float* st = a.state ? a.state + (int64_t)a.seq_slots[s] * a.state_stride : nullptr;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        float v[VEC];
        cs_input<T, VEC>(a, st, first, t - first - (TAPS - 1 - j), c, v);
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = fmaf(w[j][e], v[e], acc[e]);
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] *= sigmoid_for<T>(acc[e]);
    cs_store<T, VEC>((T*)a.out + (int64_t)t * a.C + c, acc);
  }
}

// state <- the last taps - 1 inputs of each request after this step's rows (ascending: an entry
// that is moved lies above the one it goes to)
template <typename T, int VEC>
__global__ void conv_silu_state_kernel(ConvSiluArgs a) {
  const int s = blockIdx.y, c = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (c >= a.C) return;
  const int r0 = a.seq_row_start[s], n = a.seq_row_start[s + 1] - r0;
  float* st = a.state + (int64_t)a.seq_slots[s] * a.state_stride;
  for (int k = 0; k < a.taps - 1; ++k) {
    float v[VEC];
    const int p = n - (a.taps - 1) + k;
    if (p >= 0) cs_load<T, VEC>((const T*)a.u + (int64_t)(r0 + p) * a.stride + c, v);
    else cs_load32<VEC>(st + (int64_t)(k + n) * a.C + c, v);
    cs_store32<VEC>(st + (int64_t)k * a.C + c, v);
  }
}

template <typename T, int VEC>
static int launch_conv_silu(const ConvSiluArgs& a, hipStream_t stream) {
  constexpr int ROWS = 8;
  const int64_t pieces = a.C / VEC;
  if (!a.all_single && a.taps >= 2 && a.taps <= 4 && a.T >= 256) {
    const int64_t n = (a.T + ROWS - 1) / ROWS * pieces;
    const int blocks = (int)((n + 255) / 256);
    if (a.taps == 2) conv_silu_rows_kernel<T, VEC, 2, ROWS><<<blocks, 256, 0, stream>>>(a);
    else if (a.taps == 3) conv_silu_rows_kernel<T, VEC, 3, ROWS><<<blocks, 256, 0, stream>>>(a);
    else conv_silu_rows_kernel<T, VEC, 4, ROWS><<<blocks, 256, 0, stream>>>(a);
  } else {
    const int64_t n = a.T * pieces;
    const int block = n < 65536 ? 64 : 256;
    conv_silu_kernel<T, VEC><<<(int)((n + block - 1) / block), block, 0, stream>>>(a);
  }
  NINFER_LAUNCH_CHECK();
  if (!a.all_single && a.taps > 1) {
    conv_silu_state_kernel<T, VEC><<<dim3((int)((pieces + 63) / 64), a.S), 64, 0, stream>>>(a);
    NINFER_LAUNCH_CHECK();
  }
  return 0;
}

}  // namespace ninfer

using namespace ninfer;

extern "C" int ninfer_conv_silu(const ConvSiluArgs* args, hipStream_t stream) {
  const ConvSiluArgs& a = *args;
  NINFER_REQUIRE(a.T > 0 && a.S > 0 && a.C > 0 && a.taps >= 1, "conv_silu: T=%d S=%d C=%d taps=%d must be positive",
                 a.T, a.S, a.C, a.taps);
  NINFER_REQUIRE(a.stride >= a.C, "conv_silu: rows of %d hold no %d channels", a.stride, a.C);
  NINFER_REQUIRE(a.taps == 1 || (a.state && a.state_stride >= (long long)(a.taps - 1) * a.C),
                 "conv_silu: a request's state holds no %d x %d inputs", a.taps - 1, a.C);
  NINFER_REQUIRE(a.dtype == kF32 || a.dtype == kBF16, "conv_silu: unknown dtype %d", a.dtype);
  if (a.dtype == kF32) return launch_conv_silu<float, 1>(a, stream);
  auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  if (a.C % 8 == 0 && a.stride % 8 == 0 && a.state_stride % 4 == 0 && aligned(a.u) && aligned(a.w) && aligned(a.b) &&
      aligned(a.state) && aligned(a.out))
    return launch_conv_silu<bf16, 8>(a, stream);
  return launch_conv_silu<bf16, 1>(a, stream);
}
