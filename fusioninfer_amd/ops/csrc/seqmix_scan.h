// Launchers of the kernels around sublayers with a norm on both sides
// (seqmix_sandwich.hip) and of the selective scan (seqmix_scan.hip).
#pragma once

#include "seqmix.h"

namespace fi {

template <typename A>
void launch_norm_residual_norm(float* resid, const A* y, const float* w_post,
                               const float* w_next, A* out, float eps, int T,
                               int W, hipStream_t st);

// operands of headnorm_rope_cache: column slices of projection outputs and
// the paged caches
template <typename A>
struct HeadRopeArgs {
  A* q_out;                       // [T, H, D]
  const A *q, *k, *v, *v_first;   // v_first null: values as they are
  int64_t qs, ks, vs, fs;         // row strides
  const float* lam;               // one number, read with v_first
  const int* positions;
  const float *q_w, *k_w, *inv_freq;
  float eps;
  A *k_cache, *v_cache;           // [blocks, G, bs, D | V]
  const int* slot_mapping;
  int T, H, G, D, V, bs, n;       // n: rotated pairs
};
template <typename A>
void launch_headnorm_rope_cache(HeadRopeArgs<A> a, hipStream_t st);

template <typename A>
void launch_gelu_tanh(A* out, const A* x, int T, int N, hipStream_t st);

template <typename A>
void launch_causal_conv_silu(A* out, const A* x, int64_t x_stride,
                             const float* conv_w, const float* conv_b,
                             float* conv_state, const int* seq_cu,
                             const int* row_seq, const int* seq_slots,
                             const int* positions, int T, int S, int C,
                             int taps, int hist, int max_rows,
                             hipStream_t st);
// (seqmix_parallel.hip)
template <typename A>
void launch_conv_tail_update(const A* x, int64_t x_stride, float* conv_state,
                             const int* seq_cu, const int* seq_slots,
                             const int* positions, int S, int C, int taps,
                             int hist, hipStream_t st);

// operands of the selective scan; dt, B, C and z may be column slices
template <typename A>
struct ScanArgs {
  A* out;                         // [T, W]
  const A *u, *dt, *B, *C, *z;    // u [T, W] dense
  int64_t dts, bs, cs, zs;        // row strides
  const float *dt_bias, *a_log, *d_skip;   // [W], [W, N], [W]
  float* state;                   // [slots, W, N]
  const int *seq_cu, *seq_slots, *positions;
  int W, N;
  int vec;                        // set by the launcher of the row form
};
int scan_lanes(int N);            // lanes that share a channel
// rows per segment when the leading groups' longest one is cut so that the
// launch fills the chip (0: not cut)
int scan_segment_rows(int groups, int max_rows, int W, int N);
// groups 0 .. groups-1; seg_rows > 0: cut into segments, with scratch
// seg_state [groups, segs, W, 4 lanes] and seg_dt [groups, segs, W]
template <typename A>
void launch_selective_scan_portions(ScanArgs<A> a, int groups, int max_rows,
                                    int seg_rows, float* seg_state,
                                    float* seg_dt, hipStream_t st);
// groups s0 .. S-1, row by row
template <typename A>
void launch_selective_scan_rows(ScanArgs<A> a, int s0, int S, hipStream_t st);

}  // namespace fi
