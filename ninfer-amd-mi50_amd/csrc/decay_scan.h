// Arguments of linear attention with one decay per head and token (decay_scan.hip: row by row;
// decay_scan_chunks.hip: prompt portions in chunks on the matrix cores).
#pragma once
#include "common.h"

namespace ninfer {

enum ScanForm : int {
  kScanStep = 0,    // a step size dt = softplus(z + bias): keep = exp(-rate dt), write = dt; the
                    // output gets skip_h v_t added
  kScanExp = 1,     // two exponential gates with a running maximum, and the sum of the keys beside
                    // the state, whose product with the query the output is divided by
};

struct ScanArgs {
  const void* rows;         // [T, stride]: q at q_off, k at k_off (G x dim each), v at v_off (H x vdim)
  const float* z;           // [T, H] the step sizes' logits; or [T, 2 H] the write gates', then the
                            // forget gates' logits
  const float* z_bias;      // [H] or [2 H]
  const float* rate;        // [H]   (kScanStep)
  const float* skip;        // [H]   (kScanStep)
  float* state;             // + slot * state_stride: S [H, dim, vdim], then (kScanExp) n [H, dim], m [H]
  float* out;               // [T, H * vdim] 32-bit
  float* den;               // [T, H] (kScanExp) what the outputs are to be divided by
  float* work;              // gates of the rows and, for chunks, their states: see scan_chunks_work_floats
  const int* seq_row_start; // [S + 1]
  const int* seq_slots;     // [S]
  int64_t state_stride;
  // kScanExp in the kernel of single rows: the head's norm and gate, which it applies itself
  const void* gate;         // [T, gate_stride] columns (H x vdim)
  const float* norm_w;      // [H * vdim]
  void* normed;             // [T, H * vdim] of the activation dtype
  int gate_stride;
  int stride, q_off, k_off, v_off;
  int H, G, dim, vdim;      // head h reads q and k of group h / (H / G)
  int T, S;                 // all rows and requests of the step
  int first_seq;            // requests first_seq .. are run (the ones before bring one row each)
  int form, dtype;
  float cap, q_scale, eps;
};

__device__ __forceinline__ float scan_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float scan_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// the logarithms of the write gate and of the forget gate of a head in a row
__device__ __forceinline__ void scan_exp_gates(const ScanArgs& a, int64_t row, int h, float* write, float* keep) {
  const float* z = a.z + row * 2 * a.H;
  *write = a.cap * tanhf((z[h] + a.z_bias[h]) / a.cap);
  *keep = scan_log_sigmoid(a.cap * tanhf((z[a.H + h] + a.z_bias[a.H + h]) / a.cap));
}

int scan_check(const ScanArgs& a);
int scan_chunks(const ScanArgs& a, hipStream_t stream);
bool scan_chunks_take(const ScanArgs& a);
int64_t scan_chunks_work_floats(const ScanArgs& a);

}  // namespace ninfer
