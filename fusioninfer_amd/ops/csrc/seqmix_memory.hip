// Matrix memory with exponential gates (gfx950, wave64).
//
// Per head, with log gates i and f = log sigmoid(.) (both behind a tanh
// cap) and a running maximum m that starts at 0:
//
//   m_t = max(f + m_(t-1), i)
//   S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k v^T   (n alike, k)
//   o_t = S_t^T q' / (max(|n_t . q'|, exp(-m_t)) + 1e-6),  q' = D^-1/2 q
//
// All of it is fp32 whatever the activation type. State per slot and head:
// mem [D, V], aux [copies, D + 1] (normalizer and maximum, one equal copy per
// workgroup of a head, so that no workgroup reads what another one writes).
//
//  * gated_memory_scan: token by token. A workgroup owns 64 value columns of
//    one (group, head); its four waves split the state's rows, lanes own
//    columns, so a state slice is read and written once with whole-line
//    accesses and lives in registers in between.

#include <math.h>

#include "seqmix.h"
#include "seqmix_hyper.h"

namespace fi {

namespace {

FI_DEV float capped(float z, float cap) { return cap * tanhf(z / cap); }

// log sigmoid without overflow on either side
FI_DEV float log_sigmoid(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

template <typename A>
FI_DEV void load_gates(const MemoryInputs<A>& in, int64_t t, int head,
                       float& li, float& lf) {
  li = capped(Act<A>::ld(in.i + t * in.is + head) + in.i_bias[head], in.cap);
  lf = log_sigmoid(
      capped(Act<A>::ld(in.f + t * in.fs + head) + in.f_bias[head], in.cap));
}

constexpr int kScanTokens = 8;      // tokens staged through LDS at a time

template <typename A, int RPW>      // state rows per wave, D <= 4 * RPW
__global__ __launch_bounds__(256) void gated_memory_scan_kernel(
    float* __restrict__ out, MemoryInputs<A> in, float* __restrict__ mem,
    float* __restrict__ aux, const int* __restrict__ seq_cu,
    const int* __restrict__ seq_slots, const int* __restrict__ positions,
    int s0, int H, int D, int V) {
  constexpr int DP = 4 * RPW;
  constexpr int NL = (RPW + 63) / 64;          // normalizer rows per lane
  __shared__ __attribute__((aligned(16))) float q_lds[kScanTokens][DP];
  __shared__ __attribute__((aligned(16))) float k_lds[kScanTokens][DP];
  __shared__ float v_lds[kScanTokens][kMemoryCols];
  __shared__ float li_lds[kScanTokens], lf_lds[kScanTokens];
  __shared__ float part[2][4][kMemoryCols];
  __shared__ float part_n[2][4];

  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64;
  const int head = blockIdx.y, s = s0 + blockIdx.z;
  const int row0 = seq_cu[s], row1 = seq_cu[s + 1];
  if (row1 <= row0) return;
  const int slot = seq_slots[s];
  const int col0 = blockIdx.x * kMemoryCols, col = col0 + lane;
  const int d0 = wave * RPW;
  const float q_scale = rsqrtf(static_cast<float>(D));

  float S[RPW], n[NL], m = 0.f;
#pragma unroll
  for (int r = 0; r < RPW; ++r) S[r] = 0.f;
#pragma unroll
  for (int x = 0; x < NL; ++x) n[x] = 0.f;
  float *sp = nullptr, *ap = nullptr;
  if (slot >= 0) {
    const int64_t sh = static_cast<int64_t>(slot) * H + head;
    sp = mem + sh * D * V;
    ap = aux + (sh * gridDim.x + blockIdx.x) * (D + 1);
    if (positions[row0] > 0) {
      if (col < V) {
#pragma unroll
        for (int r = 0; r < RPW; ++r)
          if (d0 + r < D) S[r] = sp[static_cast<int64_t>(d0 + r) * V + col];
      }
#pragma unroll
      for (int x = 0; x < NL; ++x) {
        const int r = lane + 64 * x;
        if (r < RPW && d0 + r < D) n[x] = ap[d0 + r];
      }
      m = ap[D];
    }
  }

  for (int t0 = row0; t0 < row1; t0 += kScanTokens) {
    const int nt = min(kScanTokens, row1 - t0);
    // every reader of the staged tokens has passed the last token's barrier
    for (int i = tid; i < nt * DP; i += 256) {
      const int j = i / DP, d = i % DP;
      const int64_t t = t0 + j;
      float qv = 0.f, kv = 0.f;
      if (d < D) {
        qv = Act<A>::ld(in.q + t * in.qs + head * D + d) * q_scale;
        kv = Act<A>::ld(in.k + t * in.ks + head * D + d);
      }
      q_lds[j][d] = qv;
      k_lds[j][d] = kv;
    }
    for (int i = tid; i < nt * kMemoryCols; i += 256) {
      const int j = i / kMemoryCols, c = i % kMemoryCols;
      const int64_t t = t0 + j;
      v_lds[j][c] = col0 + c < V
          ? Act<A>::ld(in.v + t * in.vs + head * V + col0 + c) : 0.f;
    }
    if (tid < nt) load_gates(in, t0 + tid, head, li_lds[tid], lf_lds[tid]);
    __syncthreads();
    for (int j = 0; j < nt; ++j) {
      const float carried = lf_lds[j] + m;
      m = fmaxf(carried, li_lds[j]);
      const float keep = expf(carried - m), add = expf(li_lds[j] - m);
      const float va = add * v_lds[j][lane];
      const float* kr = k_lds[j] + d0;
      const float* qr = q_lds[j] + d0;
      float o = 0.f, nq = 0.f;
#pragma unroll
      for (int r = 0; r < RPW; ++r) {
        S[r] = keep * S[r] + kr[r] * va;
        o += S[r] * qr[r];
      }
#pragma unroll
      for (int x = 0; x < NL; ++x) {
        const int r = lane + 64 * x;
        if (r < RPW) {
          n[x] = keep * n[x] + add * kr[r];
          nq += n[x] * qr[r];
        }
      }
      nq = wave_reduce_sum(nq);
      part[j & 1][wave][lane] = o;
      if (lane == 0) part_n[j & 1][wave] = nq;
      __syncthreads();
      if (wave == (j & 3) && col < V) {
        const float (*p)[kMemoryCols] = part[j & 1];
        const float* pn = part_n[j & 1];
        const float num = p[0][lane] + p[1][lane] + p[2][lane] + p[3][lane];
        const float nd = pn[0] + pn[1] + pn[2] + pn[3];
        out[static_cast<int64_t>(t0 + j) * H * V + head * V + col] =
            num / (fmaxf(fabsf(nd), expf(-m)) + 1e-6f);
      }
    }
  }
  if (sp == nullptr) return;
  if (col < V) {
#pragma unroll
    for (int r = 0; r < RPW; ++r)
      if (d0 + r < D) sp[static_cast<int64_t>(d0 + r) * V + col] = S[r];
  }
#pragma unroll
  for (int x = 0; x < NL; ++x) {
    const int r = lane + 64 * x;
    if (r < RPW && d0 + r < D) ap[d0 + r] = n[x];
  }
  if (tid == 0) ap[D] = m;
}

}  // namespace

template <typename A>
void launch_gated_memory_scan(float* out, MemoryInputs<A> in, float* mem,
                              float* aux, const int* seq_cu,
                              const int* seq_slots, const int* positions,
                              int s0, int S, int H, int D, int V,
                              hipStream_t st) {
  if (S <= s0) return;
  const dim3 grid(ceil_div(V, kMemoryCols), H, S - s0);
#define FI_SCAN(R_)                                                            \
  hipLaunchKernelGGL((gated_memory_scan_kernel<A, R_>), grid, dim3(256), 0,    \
                     st, out, in, mem, aux, seq_cu, seq_slots, positions, s0,  \
                     H, D, V)
  if (D <= 64) FI_SCAN(16);
  else if (D <= 128) FI_SCAN(32);
  else if (D <= 256) FI_SCAN(64);
  else FI_SCAN(128);
#undef FI_SCAN
}

#define FI_INST(A)                                                             \
  template void launch_gated_memory_scan<A>(                                   \
      float*, MemoryInputs<A>, float*, float*, const int*, const int*,         \
      const int*, int, int, int, int, int, hipStream_t);
FI_INST(float)
FI_INST(u16)
#undef FI_INST

}  // namespace fi
