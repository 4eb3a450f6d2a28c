// Arguments of paged attention. One struct serves the plain kernel and the
// MFMA kernels; the entry point picks by dtype, head size and batch shape.
#pragma once
#include "common.h"

namespace ninfer {

struct AttnArgs {
  const void* q;            // [T, q_stride] rows; head h of row t at q + t*q_stride + h*D
  const void* kpool;        // [pages, Hkv, page_size, D]
  const void* vpool;
  void* out;                // [T, Hq*D]
  const int* block_table;   // [S, bt_stride] page of each logical page, -1 when given back
  const int* positions;     // [T] absolute position of each row
  const int* row_seq;       // [T] request (index in this step) of each row
  const int* seq_row_start; // [S + 1] first row of each request, then T
  const int* seq_qlen;      // [S]
  const int* seq_pos0;      // [S]
  float* workspace;         // split-KV partial results, or null
  int64_t workspace_floats;
  int q_stride;
  int bt_stride;
  int T;
  int S;
  int Hq;
  int Hkv;
  int D;
  int page_size;
  int window;               // 0: all keys
  float scale;
  int dtype;
  int max_qlen;             // host-side bounds used to size launches
  int max_kv_len;
  int single_rows;          // the first single_rows requests bring one row each: rows
                            // 0 .. single_rows - 1 (0 when the caller does not sort them)
  const float* slopes;      // [Hq] or null: head h's scores get slopes[h] * (key position - row's
                            // position) added before the softmax (a distance-based position bias)
  int Dv;                   // numbers of a value head: vpool is [pages, Hkv, page_size, Dv] and out
                            // [T, Hq*Dv] (0: the same as D)
  int sink;                 // != 0: the softmax's denominator has one more term, exp(0), that
                            // belongs to no key (a sink with score 0 and no value)
                            // (with `sinks`, below, exp(sinks[h]): a sink of a learned score)
  // Beside the keys of its window a row may see one key and value per block of `block` tokens
  // that lies wholly before the window: block b (positions b block .. b block + block - 1) where
  // b block + block - 1 <= position - window. Keys and blocks share one softmax.
  const void* kblk;         // [pages, Hkv, blk_page_size, D], or null: no blocks
  const void* vblk;         // [pages, Hkv, blk_page_size, Dv]
  const int* blk_table;     // [S, blk_bt_stride]
  int blk_bt_stride;
  int blk_page_size;
  int block;
  // a gate on the output: out[t, c] times sigmoid(gate[t * gate_stride + c]), c < Hq * Dv
  const void* gate;         // of the activation dtype, or null
  int gate_stride;
  const float* sinks;       // [Hq] or null (0): the score of head h's sink, not scaled
};

// The score of head h's sink.
__device__ __forceinline__ float attention_sink(const AttnArgs& a, int h) { return a.sinks ? a.sinks[h] : 0.f; }

// How many blocks a row at this position sees (they are the first ones of its request).
__host__ __device__ inline int attention_blocks_seen(int pos, int window, int block) {
  return pos >= window ? (pos - window + 1) / block : 0;
}

int attention_check(const AttnArgs& a);
int attention_generic(const AttnArgs& a, hipStream_t stream);

int64_t attention_decode_workspace_floats(int T, int Hq, int D, int max_kv_len);
bool attention_decode_takes(const AttnArgs& a);
int attention_decode(const AttnArgs& a, hipStream_t stream);
void attention_decode_plan(const AttnArgs& a, bool* heads, int* chunk, int* n_chunks);
bool attention_decode_heads_takes(const AttnArgs& a);
int attention_decode_heads(const AttnArgs& a, int chunk, int n_chunks, hipStream_t stream);
bool attention_prefill_takes(const AttnArgs& a);
int attention_prefill(const AttnArgs& a, hipStream_t stream);
// keys of D and values of Dv numbers (multiples of 8 up to 256), a window or none, a sink or
// none: row tiles on the matrix cores; single rows with the heads of a kv head as the tile's rows
bool attention_tiles_takes(const AttnArgs& a);
int attention_tiles(const AttnArgs& a, int first_seq, hipStream_t stream);
bool attention_tiles_heads_takes(const AttnArgs& a);
int attention_tiles_heads(const AttnArgs& a, hipStream_t stream);

}  // namespace ninfer
