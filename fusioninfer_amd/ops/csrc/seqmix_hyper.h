// Launchers of the stream-copy, latent-projection and matrix-memory kernels
// (seqmix_hyper.hip, seqmix_memory.hip).
#pragma once

#include "seqmix.h"

namespace fi {

// y = sum_j c_j[t] * y_j[t, :] of one to three sublayer terms; c null: 1;
// sig: c passes a sigmoid first
template <typename A>
struct HyperTerms {
  const A* y[3];
  const float* c[3];
  int64_t c_stride[3];
  int sig[3];
};

template <typename A>
void launch_hyper_start(float* xs, A* h, const int64_t* ids, const A* embed,
                        const float* w_in, const float* norm_w, float eps,
                        int T, int S, int W, hipStream_t st);
template <typename A>
void launch_hyper_update(float* xs, A* h, HyperTerms<A> terms,
                         const float* mix, const float* w_out,
                         const float* w_in, const float* norm_w, float eps,
                         int T, int S, int W, hipStream_t st);
template <typename A>
void launch_latent_norm_cache(A* q_out, const A* dq, int64_t dq_stride, int Q,
                              const A* dkv, int64_t dkv_stride,
                              const int* positions, const float* inv_freq,
                              int rot_pairs, float rot_mult, const float* q_w,
                              const float* c_w, float eps, A* kv_cache,
                              const int* slot_mapping, int T, int C, int R,
                              int half, hipStream_t st);
template <typename A>
void launch_latent_query_rope(A* q_out, const A* q, int64_t q_stride,
                              const int* positions, const float* inv_freq,
                              int rot_pairs, float rot_mult, int T, int H,
                              int D, int R, int C, int half, hipStream_t st);
void launch_paged_rows_gather(void* out, const void* cache, const int* slots,
                              int rows, int64_t row_bytes, hipStream_t st);
template <typename A>
void launch_silu_and_mul(A* out, const A* gu, int T, int F, hipStream_t st);

// operands of the matrix memory: q/k/v [T, H*D | H*D | H*V] and gate inputs
// [T, H], each a column slice of a wider row
template <typename A>
struct MemoryInputs {
  const A *q, *k, *v, *i, *f;
  int64_t qs, ks, vs, is, fs;
  const float *i_bias, *f_bias;
  float cap;
};

constexpr int kMemoryCols = 64;     // value columns per workgroup

// row groups s0 .. S-1 token by token
template <typename A>
void launch_gated_memory_scan(float* out, MemoryInputs<A> in, float* mem,
                              float* aux, const int* seq_cu,
                              const int* seq_slots, const int* positions,
                              int s0, int S, int H, int D, int V,
                              hipStream_t st);

// groups 0 .. groups-1 (the ones the tile table covers) in chunks; scratch:
// chunk_mem [2 tiles, H, ceil(V/64), 64, 16 row_tiles], chunk_n [2 tiles, H,
// 16 row_tiles], meta [2 tiles, H, 3]
bool gated_memory_has_chunks(int D);
int gated_memory_row_tiles(int D);
template <typename A>
void launch_gated_memory_chunks(float* out, float* chunk_mem, float* chunk_n,
                                double* meta, MemoryInputs<A> in, float* mem,
                                float* aux, const int* seq_cu,
                                const int* seq_slots, const int* positions,
                                const int* tile_seq, const int* tile_row0,
                                int tiles, int groups, int H, int D, int V,
                                hipStream_t st);

}  // namespace fi
