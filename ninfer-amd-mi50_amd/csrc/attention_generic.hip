// Paged attention, plain form: one wave per (row, query head).
//
// A row at position p of its request sees the keys of that request at
// positions lo..p, lo = max(0, p - window + 1) (window 0: all). Keys are
// walked in tiles of 64 aligned to absolute positions, with an online softmax
// (running max m, running sum l, rescale by exp(m_old - m_new): reference
// src/ops/attention.hip:62-75, :228-241; normalised at the end :92, :265), so
// the order of every sum depends only on the row's own position, never on how
// the request was cut into steps or what else is in the batch. Query head h
// reads kv head h / (Hq / Hkv) (reference src/ops/attention.hip:27-28).
// Scores, softmax and the value sum are 32-bit. This is the kernel of the true
// 32-bit path and of head sizes the MFMA kernels refuse. Values may have another size than
// keys (Dv), and the softmax may have a sink: one more term exp(0) in its denominator that
// belongs to no key, so that the weights of a row add up to less than one. Where the cache keeps
// one key and value per block of tokens, the blocks a row sees are walked first, in tiles of 64
// too. The output may be gated, element by element.
#include "attention.h"

namespace ninfer {

constexpr int kMaxDPerLane = 8;  // head sizes up to 512

template <typename T>
__global__ __launch_bounds__(64) void paged_attention_generic_kernel(AttnArgs a) {
  extern __shared__ float smem[];
  const int D = a.D, Dv = a.Dv, Hkv = a.Hkv;
  float* q_s = smem;                 // [D]
  float* p_s = smem + D;             // [64]
  int64_t* off_s = (int64_t*)(p_s + 64);  // [64] page's slot (page * Hkv + g) * page_size + slot of each key

  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int g = h / (a.Hq / Hkv);
  const int pos = a.positions[t];
  const float slope = a.slopes ? a.slopes[h] : 0.f;

  const T* qr = (const T*)a.q + (int64_t)t * a.q_stride + h * D;
  for (int d = lane; d < D; d += 64) q_s[d] = to_f32(qr[d]);
  __syncthreads();

  // (a sink is a key without a value: the running maximum starts at its score, the sum at 1)
  float m = a.sink ? attention_sink(a, h) : -INFINITY, l = a.sink ? 1.f : 0.f;
  float acc[kMaxDPerLane];
#pragma unroll
  for (int i = 0; i < kMaxDPerLane; ++i) acc[i] = 0.f;

  // entries lo .. last of a pair of pools
  auto walk = [&](const T* kpool, const T* vpool, const int* bt, int page_size, int lo, int last) {
    for (int tile = (lo / 64) * 64; tile <= last; tile += 64) {
      int j = tile + lane;
      bool valid = j >= lo && j <= last;
      float s = -INFINITY;
      int64_t off = 0;
      if (valid) {
        int page = bt[j / page_size];
        off = ((int64_t)page * Hkv + g) * page_size + (j % page_size);
        const T* kr = kpool + off * D;
        float dot = 0.f;
        for (int d = 0; d < D; ++d) dot = fmaf(q_s[d], to_f32(kr[d]), dot);
        s = fmaf(slope, (float)(j - pos), dot * a.scale);
      }
      float m_new = fmaxf(m, wave_max(s));
      float p = valid ? expf(s - m_new) : 0.f;
      float alpha = expf(m - m_new);  // 0 on the first tile (m = -inf)
      l = l * alpha + wave_sum(p);
      m = m_new;
      p_s[lane] = p;
      off_s[lane] = off;
      __syncthreads();
      int n_keys = min(64, last - tile + 1);
      int first = max(0, lo - tile);
#pragma unroll
      for (int i = 0; i < kMaxDPerLane; ++i) {
        int d = lane + i * 64;
        if (d < Dv) {
          float x = acc[i] * alpha;
          for (int jj = first; jj < n_keys; ++jj) x = fmaf(p_s[jj], to_f32(vpool[off_s[jj] * Dv + d]), x);
          acc[i] = x;
        }
      }
      __syncthreads();
    }
  };
  const int s = a.row_seq[t];
  if (a.kblk)
    walk((const T*)a.kblk, (const T*)a.vblk, a.blk_table + (int64_t)s * a.blk_bt_stride, a.blk_page_size, 0,
         attention_blocks_seen(pos, a.window, a.block) - 1);
  walk((const T*)a.kpool, (const T*)a.vpool, a.block_table + (int64_t)s * a.bt_stride, a.page_size,
       a.window > 0 ? max(0, pos - a.window + 1) : 0, pos);
  const int64_t orow = ((int64_t)t * a.Hq + h) * Dv;
  const T* gate = a.gate ? (const T*)a.gate + (int64_t)t * a.gate_stride + h * Dv : nullptr;
  float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < kMaxDPerLane; ++i) {
    int d = lane + i * 64;
    if (d < Dv) {
      float x = acc[i] * inv;
      if (gate) x /= 1.f + expf(-to_f32(gate[d]));
      ((T*)a.out)[orow + d] = from_f32<T>(x);
    }
  }
}

int attention_generic(const AttnArgs& args, hipStream_t stream) {
  AttnArgs a = args;
  if (a.Dv <= 0) a.Dv = a.D;
  NINFER_REQUIRE(a.D <= 64 * kMaxDPerLane && a.Dv <= 64 * kMaxDPerLane,
                 "paged_attention: head sizes %d, %d exceed %d", a.D, a.Dv, 64 * kMaxDPerLane);
  dim3 grid(a.T, a.Hq);
  size_t lds = (a.D + 64) * sizeof(float) + 64 * sizeof(int64_t);
  if (a.dtype == kF32) paged_attention_generic_kernel<float><<<grid, 64, lds, stream>>>(a);
  else paged_attention_generic_kernel<bf16><<<grid, 64, lds, stream>>>(a);
  NINFER_LAUNCH_CHECK();
  return 0;
}

}  // namespace ninfer
