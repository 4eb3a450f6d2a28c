// Entry point of paged attention: checks the arguments and picks a kernel.
#include "attention.h"

using namespace ninfer;

namespace ninfer {
// What every kernel of the family assumes of the arguments.
int attention_check(const AttnArgs& args) {
  const AttnArgs* a = &args;
  NINFER_REQUIRE(a->T > 0 && a->S > 0, "paged_attention: T=%d S=%d must be positive", a->T, a->S);
  NINFER_REQUIRE(a->Hq > 0 && a->Hkv > 0 && a->Hq % a->Hkv == 0,
                 "paged_attention: %d query heads are not a multiple of %d kv heads", a->Hq,
                 a->Hkv);
  NINFER_REQUIRE(a->D > 0 && a->D % 2 == 0, "paged_attention: head size %d must be even", a->D);
  NINFER_REQUIRE(a->page_size > 0 && a->bt_stride > 0, "paged_attention: bad page size %d or "
                 "table width %d", a->page_size, a->bt_stride);
  NINFER_REQUIRE(a->scale > 0.f, "paged_attention: scale %g must be positive", (double)a->scale);
  NINFER_REQUIRE(a->window >= 0, "paged_attention: window %d must be >= 0", a->window);
  NINFER_REQUIRE(a->dtype == kF32 || a->dtype == kBF16, "paged_attention: unknown dtype %d",
                 a->dtype);
  NINFER_REQUIRE(a->q_stride >= a->Hq * a->D, "paged_attention: row stride %d < %d", a->q_stride,
                 a->Hq * a->D);
  NINFER_REQUIRE(a->Dv >= 0, "paged_attention: value size %d is negative", a->Dv);
  NINFER_REQUIRE(a->max_qlen >= 1 && a->max_kv_len >= 1, "paged_attention: bad size hints");
  NINFER_REQUIRE(a->single_rows >= 0 && a->single_rows <= a->S && a->single_rows <= a->T,
                 "paged_attention: %d single rows of %d requests", a->single_rows, a->S);
  NINFER_REQUIRE(!a->kblk || (a->vblk && a->blk_table && a->blk_bt_stride > 0 && a->blk_page_size > 0 &&
                              a->block > 0 && a->window > 0),
                 "paged_attention: blocks of %d tokens before a window of %d", a->block, a->window);
  NINFER_REQUIRE(!a->kblk || !a->slopes, "paged_attention: a position bias beside blocks is not built");
  NINFER_REQUIRE(!a->gate || a->gate_stride >= a->Hq * (a->Dv > 0 ? a->Dv : a->D),
                 "paged_attention: the gate's rows of %d are too short", a->gate_stride);
  NINFER_REQUIRE(!a->sinks || a->sink, "paged_attention: scores of sinks without a sink");
  return 0;
}
}  // namespace ninfer

// force_generic != 0 runs the plain one-wave-per-(row, head) kernel whatever
// the shape (tests compare the fast kernels with it).
extern "C" int ninfer_paged_attention(const AttnArgs* a, int force_generic, hipStream_t stream) {
  if (int rc = attention_check(*a)) return rc;
  if (!force_generic && a->max_qlen == 1 && attention_decode_takes(*a))
    return attention_decode(*a, stream);
  if (!force_generic && a->single_rows > 0 && a->single_rows < a->S &&
      attention_decode_takes(*a) && attention_prefill_takes(*a)) {
    // A step that mixes decoded tokens with prompt portions: the single rows, which come
    // first, walk their contexts split over many blocks; in the prompt kernel each would be
    // one block that walks its whole context alone.
    const int n = a->single_rows;
    AttnArgs d = *a;
    d.T = n;
    d.S = n;
    d.max_qlen = 1;
    if (int rc = attention_decode(d, stream)) return rc;
    AttnArgs p = *a;   // rows and their positions stay where they are: only the requests move
    p.seq_row_start += n;
    p.seq_qlen += n;
    p.seq_pos0 += n;
    p.block_table += (int64_t)n * a->bt_stride;
    p.S = a->S - n;
    p.T = a->T - n;
    return attention_prefill(p, stream);
  }
  // single rows (which come first) of layers with values of another size, a sink, blocks or a
  // gate: the heads of a kv head as a tile's rows
  const int n = a->max_qlen == 1 ? a->S : a->single_rows;
  const bool tiles = !force_generic && attention_tiles_takes(*a);
  const bool apart = tiles && n > 0 && attention_tiles_heads_takes(*a) &&
                     (!attention_prefill_takes(*a) || a->kblk || a->gate || a->sink);
  if (apart) {
    AttnArgs d = *a;
    d.T = n;
    d.S = n;
    d.max_qlen = 1;
    if (int rc = attention_tiles_heads(d, stream)) return rc;
    if (n == a->S) return 0;
  }
  if (!force_generic && attention_prefill_takes(*a)) {
    if (!apart) return attention_prefill(*a, stream);
    AttnArgs p = *a;
    p.seq_row_start += n;
    p.seq_qlen += n;
    p.seq_pos0 += n;
    p.block_table += (int64_t)n * a->bt_stride;
    if (p.kblk) p.blk_table += (int64_t)n * a->blk_bt_stride;
    p.S = a->S - n;
    p.T = a->T - n;
    return attention_prefill(p, stream);
  }
  // ... and prompt portions of any such shape on the matrix cores
  if (tiles) return attention_tiles(*a, apart ? n : 0, stream);
  return attention_generic(*a, stream);
}

// 32-bit floats of workspace the split-KV decode kernel needs for this shape.
extern "C" long long ninfer_attention_workspace_floats(int T, int Hq, int D, int max_kv_len) {
  return attention_decode_workspace_floats(T, Hq, D, max_kv_len);
}

// How a step of single-token rows would run (nothing is launched): kernel 0 = the plain
// kernel, 1 = split contexts on scalar FMAs, 2 = split contexts on the matrix cores (grouped
// heads); the keys per chunk and the number of chunks the merge kernel adds up. Tests name
// the kernel variant they mean to reach with it.
extern "C" int ninfer_attention_decode_plan(const AttnArgs* a, int* kernel, int* chunk, int* n_chunks) {
  *kernel = 0;
  *chunk = *n_chunks = 0;
  if (int rc = attention_check(*a)) return rc;
  if (!attention_decode_takes(*a)) return 0;
  bool heads;
  attention_decode_plan(*a, &heads, chunk, n_chunks);
  *kernel = heads ? 2 : 1;
  return 0;
}
