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
//    accesses and lives in registers in between. Decoded rows use it, and
//    key sizes above 256.
//  * gated_memory chunks: prompt portions, 64 tokens at a time and all chunks
//    side by side. With F_t the sum of f over the chunk's tokens up to t,
//    g_j = i_j - F_j and G_t = max(m_0, max_{j<=t} g_j), the recurrence
//    unrolls to m_t = F_t + G_t and
//
//      o_t ~ e^(m_0 - G_t) S_0^T q_t + sum_{j<=t} e^(g_j - G_t) (q_t.k_j) v_j
//
//    with every exponent <= 0. Three launches:
//      state: each chunk's own contribution sum_j e^(g_j - max g) k_j v_j^T
//      carry: runs over a sequence's chunks, replaces each contribution by
//             the state the chunk starts from, leaves the last one in the slot
//      read:  scores, decayed values, start-state part and denominator
//    F and g are kept in fp64 (one number per token), everything else is
//    fp32: the products run on the fp32 matrix cores (16x16x4), query-key
//    scores of bf16 activations on the bf16 ones (exact products, fp32 sums).
//    Chunk states sit in scratch in accumulator order [64-column tile][wave]
//    [16-row tile][lane][4], so that all three launches move them as whole
//    16-byte lanes.

#include <math.h>

#include <type_traits>

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

typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(4))) float floatx4;

constexpr int kChunk = 64;          // tokens per chunk
constexpr int kTileRows = 128;      // rows per entry of the tile table

// rows [row0, row0 + n) of the step that chunk c covers (n <= 0: none);
// two chunks per tile-table entry
FI_DEV int chunk_rows(int c, const int* tile_seq, const int* tile_row0,
                      const int* seq_cu, int& row0) {
  const int s = tile_seq[c / 2];
  const int base = seq_cu[s] + tile_row0[c / 2];
  row0 = base + (c & 1) * kChunk;
  const int end = min(seq_cu[s + 1], base + kTileRows);
  return min(kChunk, end - row0);
}

// one wave: lane j < n holds token j. Returns g_j, its running maximum and
// F_j (fp64, inclusive); lanes beyond n repeat the last token's F and M and
// have g = -inf.
template <typename A>
FI_DEV void chunk_gates(const MemoryInputs<A>& in, int row0, int n, int head,
                        int lane, double& g, double& gmax, double& F) {
  float li = 0.f, lf = 0.f;
  if (lane < n) load_gates(in, row0 + lane, head, li, lf);
  F = lf;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double o = __shfl_up(F, off, 64);
    if (lane >= off) F += o;
  }
  g = lane < n ? static_cast<double>(li) - F : -INFINITY;
  gmax = g;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double o = __shfl_up(gmax, off, 64);
    if (lane >= off) gmax = fmax(gmax, o);
  }
}

// rows x cols of an activation matrix into an LDS tile of ROWS x COLS
// entries (pitch P), zero beyond
template <typename A, int VW, int ROWS, int COLS, int P>
FI_DEV void load_tile(A* dst, const A* src, int64_t stride, int rows,
                      int cols) {
  constexpr int CV = COLS / VW;
  for (int i = threadIdx.x; i < ROWS * CV; i += 256) {
    const int r = i / CV, c = (i % CV) * VW;
    A v[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) v[e] = A(0);
    if (r < rows && c < cols) {
      // VW > 1 only where cols is a multiple of it
      __builtin_memcpy(v, __builtin_assume_aligned(src + r * stride + c,
                                                   VW * sizeof(A)),
                       sizeof(v));
    }
    __builtin_memcpy(__builtin_assume_aligned(dst + r * P + c,
                                              VW * sizeof(A)),
                     v, sizeof(v));
  }
}

// meta per (chunk, head), fp64: m of the chunk's own contribution, F of its
// last token, m at its start
constexpr int kMeta = 3;

template <typename A, int DT, int VW>
__global__ __launch_bounds__(256) void gated_memory_state_kernel(
    float* __restrict__ chunk_mem,    // [chunks, H, CT, 4, DT, 64, 4]
    float* __restrict__ chunk_n,      // [chunks, H, DT * 16]
    double* __restrict__ meta, MemoryInputs<A> in,
    const int* __restrict__ seq_cu, const int* __restrict__ tile_seq,
    const int* __restrict__ tile_row0, int H, int D, int V) {
  constexpr int KP = DT * 16 + 8;
  constexpr int VP = kMemoryCols + 8;
  __shared__ __attribute__((aligned(16))) A k_lds[kChunk * KP];
  __shared__ __attribute__((aligned(16))) A v_lds[kChunk * VP];
  __shared__ float w_lds[kChunk];
  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64;
  const int g4 = lane / 16, c16 = lane % 16;
  const int head = blockIdx.y, c = blockIdx.z;
  const int col0 = blockIdx.x * kMemoryCols;
  int row0;
  const int n = chunk_rows(c, tile_seq, tile_row0, seq_cu, row0);
  if (n <= 0) return;
  const int64_t ch = static_cast<int64_t>(c) * H + head;

  load_tile<A, VW, kChunk, DT * 16, KP>(k_lds, in.k + row0 * in.ks + head * D,
                                        in.ks, n, D);
  load_tile<A, VW, kChunk, kMemoryCols, VP>(
      v_lds, in.v + row0 * in.vs + head * V + col0, in.vs, n,
      min(kMemoryCols, V - col0));
  if (wave == 0) {
    double g, gmax, F;
    chunk_gates(in, row0, n, head, lane, g, gmax, F);
    const double top = __shfl(gmax, n - 1, 64);
    w_lds[lane] = lane < n ? expf(static_cast<float>(g - top)) : 0.f;
    if (blockIdx.x == 0 && lane == n - 1) {
      meta[ch * kMeta] = F + top;
      meta[ch * kMeta + 1] = F;
    }
  }
  __syncthreads();

  float wv[kChunk / 4];
#pragma unroll
  for (int kk = 0; kk < kChunk / 4; ++kk) {
    const int j = 4 * kk + g4;
    wv[kk] = w_lds[j] * Act<A>::ld(v_lds + j * VP + wave * 16 + c16);
  }
  float* dst = chunk_mem +
      (((ch * gridDim.x + blockIdx.x) * 4 + wave) * DT * 64 + lane) * 4;
#pragma unroll
  for (int t = 0; t < DT; ++t) {
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < kChunk / 4; ++kk)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(
          Act<A>::ld(k_lds + (4 * kk + g4) * KP + 16 * t + c16), wv[kk], acc,
          0, 0, 0);
    *reinterpret_cast<floatx4*>(dst + t * 256) = acc;
  }
  if (blockIdx.x == 0) {
    for (int d = tid; d < DT * 16; d += 256) {
      float sum = 0.f;
      for (int j = 0; j < kChunk; ++j)
        sum += w_lds[j] * Act<A>::ld(k_lds + j * KP + d);
      chunk_n[ch * DT * 16 + d] = sum;
    }
  }
}

// grid x: 256-lane slices of the state, then one workgroup for the
// normalizer and the maximum; z: row group
template <int DT>
__global__ __launch_bounds__(256) void gated_memory_carry_kernel(
    float* __restrict__ chunk_mem, float* __restrict__ chunk_n,
    double* __restrict__ meta, float* __restrict__ mem,
    float* __restrict__ aux, const int* __restrict__ seq_cu,
    const int* __restrict__ seq_slots, const int* __restrict__ positions,
    int H, int D, int V, int CT) {
  __shared__ float scratch[8];
  const int tid = threadIdx.x;
  const int head = blockIdx.y, s = blockIdx.z;
  // first chunk of this group: two per tile entry of the groups before it
  float before = 0.f, dummy = 0.f;
  for (int i = tid; i < s; i += 256)
    before += static_cast<float>(
        (seq_cu[i + 1] - seq_cu[i] + kTileRows - 1) / kTileRows);
  block_reduce_sum2_256(before, dummy, scratch);
  const int row0 = seq_cu[s], rows = seq_cu[s + 1] - row0;
  if (rows <= 0) return;
  const int c0 = 2 * static_cast<int>(before + 0.5f);
  const int nc = (rows + kChunk - 1) / kChunk;
  const int slot = seq_slots[s];
  const bool resume = slot >= 0 && positions[row0] > 0;
  const int64_t sh = static_cast<int64_t>(slot < 0 ? 0 : slot) * H + head;
  double m = resume ? static_cast<double>(aux[sh * CT * (D + 1) + D]) : 0.0;
  const double* mp = meta + (static_cast<int64_t>(c0) * H + head) * kMeta;
  const int64_t ms = static_cast<int64_t>(H) * kMeta;

  if (blockIdx.x == gridDim.x - 1) {
    // every copy of (normalizer, maximum) was equal: read the first
    for (int d = tid; d < DT * 16; d += 256) {
      double mm = m;
      float acc = resume && d < D ? aux[sh * CT * (D + 1) + d] : 0.f;
      for (int c = 0; c < nc; ++c) {
        float* p = chunk_n + ((static_cast<int64_t>(c0 + c)) * H + head) *
                                 (DT * 16) + d;
        const double own = mp[c * ms], F = mp[c * ms + 1];
        const double mn = fmax(mm + F, own);
        const float add = *p;
        *p = acc;
        acc = expf(static_cast<float>(mm + F - mn)) * acc +
              expf(static_cast<float>(own - mn)) * add;
        mm = mn;
      }
      if (slot >= 0 && d < D)
        for (int x = 0; x < CT; ++x) aux[(sh * CT + x) * (D + 1) + d] = acc;
    }
    // the maximum goes out only after every thread has read the old one
    __syncthreads();
    if (tid == 0) {
      double* mw = meta + (static_cast<int64_t>(c0) * H + head) * kMeta;
      for (int c = 0; c < nc; ++c) {
        mw[c * ms + 2] = m;
        m = fmax(m + mw[c * ms + 1], mw[c * ms]);
      }
    }
    return;
  }
  // slice index -> (column tile, wave, row tile, lane)
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 256 + tid;
  if (item >= static_cast<int64_t>(CT) * 4 * DT * 64) return;
  const int lane = item % 64, t = (item / 64) % DT;
  const int wave = (item / (64 * DT)) % 4, ct = item / (256 * DT);
  const int d = 16 * t + 4 * (lane / 16);
  const int col = ct * kMemoryCols + wave * 16 + lane % 16;
  floatx4 S = {0.f, 0.f, 0.f, 0.f};
  float* sp = mem + sh * D * V;
  if (resume && col < V) {
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (d + r < D) S[r] = sp[static_cast<int64_t>(d + r) * V + col];
  }
  float* p = chunk_mem + (static_cast<int64_t>(c0) * H + head) *
                             (static_cast<int64_t>(CT) * DT * 1024) + item * 4;
  const int64_t ps = static_cast<int64_t>(H) * CT * DT * 1024;
  constexpr int AHEAD = 4;            // chunk loads in flight
  for (int cb = 0; cb < nc; cb += AHEAD) {
    floatx4 add[AHEAD];
#pragma unroll
    for (int x = 0; x < AHEAD; ++x)
      if (cb + x < nc)
        add[x] = *reinterpret_cast<const floatx4*>(p + (cb + x) * ps);
#pragma unroll
    for (int x = 0; x < AHEAD; ++x) {
      if (cb + x >= nc) break;
      *reinterpret_cast<floatx4*>(p + (cb + x) * ps) = S;
      const double own = mp[(cb + x) * ms], F = mp[(cb + x) * ms + 1];
      const double mn = fmax(m + F, own);
      const float a = expf(static_cast<float>(m + F - mn));
      const float b = expf(static_cast<float>(own - mn));
#pragma unroll
      for (int r = 0; r < 4; ++r) S[r] = a * S[r] + b * add[x][r];
      m = mn;
    }
  }
  if (slot >= 0 && col < V) {
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (d + r < D) sp[static_cast<int64_t>(d + r) * V + col] = S[r];
  }
}

// the maxima of all copies, after every reader of the carry launch is done
__global__ void gated_memory_max_kernel(
    const double* __restrict__ meta, float* __restrict__ aux,
    const int* __restrict__ seq_cu, const int* __restrict__ seq_slots, int G,
    int H, int D, int CT) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= G * H) return;
  const int s = i / H, head = i % H;
  const int slot = seq_slots[s];
  const int rows = seq_cu[s + 1] - seq_cu[s];
  if (slot < 0 || rows <= 0) return;
  int c0 = 0;
  for (int x = 0; x < s; ++x)
    c0 += 2 * ((seq_cu[x + 1] - seq_cu[x] + kTileRows - 1) / kTileRows);
  const int last = c0 + (rows + kChunk - 1) / kChunk - 1;
  const double* mp = meta + (static_cast<int64_t>(last) * H + head) * kMeta;
  const float m = static_cast<float>(fmax(mp[2] + mp[1], mp[0]));
  for (int x = 0; x < CT; ++x)
    aux[((static_cast<int64_t>(slot) * H + head) * CT + x) * (D + 1) + D] = m;
}

template <typename A, int DT, int VW>
__global__ __launch_bounds__(256) void gated_memory_read_kernel(
    float* __restrict__ out, const float* __restrict__ chunk_mem,
    const float* __restrict__ chunk_n, const double* __restrict__ meta,
    MemoryInputs<A> in, const int* __restrict__ seq_cu,
    const int* __restrict__ tile_seq, const int* __restrict__ tile_row0,
    int H, int D, int V, int CT) {
  constexpr bool BF = std::is_same<A, u16>::value;
  constexpr int DP = DT * 16;
  constexpr int QP = DP + 8;
  constexpr int VP = kMemoryCols + 8;
  constexpr int AP = kChunk + 4;
  constexpr int RT = kChunk / 16;
  // the key tile's space is used again for the scores
  constexpr int KBYTES = kChunk * QP * sizeof(A);
  constexpr int ABYTES = kChunk * AP * sizeof(float);
  __shared__ __attribute__((aligned(16))) A q_lds[kChunk * QP];
  __shared__ __attribute__((aligned(16))) char ka_lds[KBYTES > ABYTES
                                                          ? KBYTES : ABYTES];
  __shared__ __attribute__((aligned(16))) A v_lds[kChunk * VP];
  __shared__ double g_lds[kChunk], top_lds[kChunk];
  __shared__ float start_lds[kChunk], floor_lds[kChunk], inv_lds[kChunk];
  A* k_lds = reinterpret_cast<A*>(ka_lds);
  float* a_lds = reinterpret_cast<float*>(ka_lds);

  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64;
  const int g4 = lane / 16, c16 = lane % 16;
  const int head = blockIdx.x, c = blockIdx.y;
  int row0;
  const int n = chunk_rows(c, tile_seq, tile_row0, seq_cu, row0);
  if (n <= 0) return;
  const int64_t ch = static_cast<int64_t>(c) * H + head;
  const float q_scale = rsqrtf(static_cast<float>(D));

  load_tile<A, VW, kChunk, DP, QP>(q_lds, in.q + row0 * in.qs + head * D,
                                   in.qs, n, D);
  load_tile<A, VW, kChunk, DP, QP>(k_lds, in.k + row0 * in.ks + head * D,
                                   in.ks, n, D);
  if (wave == 0) {
    double g, gmax, F;
    chunk_gates(in, row0, n, head, lane, g, gmax, F);
    const double m0 = meta[ch * kMeta + 2];
    const double top = fmax(m0, gmax);
    g_lds[lane] = g;
    top_lds[lane] = top;
    start_lds[lane] = expf(static_cast<float>(m0 - top));
    floor_lds[lane] = expf(static_cast<float>(-(F + top)));
  }
  __syncthreads();

  // causal 16x16 score tiles, dealt to the waves in turn
  constexpr int NT = RT * (RT + 1) / 2;
  floatx4 sc[(NT + 3) / 4];
#pragma unroll
  for (int x = 0; x < (NT + 3) / 4; ++x) {
    const int tile = wave + 4 * x;
    sc[x] = floatx4{0.f, 0.f, 0.f, 0.f};
    if (tile >= NT) continue;
    int rt = 0;
    while ((rt + 1) * (rt + 2) / 2 <= tile) ++rt;
    const int kt = tile - rt * (rt + 1) / 2;
    const A* qr = q_lds + (16 * rt + c16) * QP;
    const A* kr = k_lds + (16 * kt + c16) * QP;
    if constexpr (BF) {
#pragma unroll
      for (int t = 0; t < DT; ++t)
        sc[x] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(
            *reinterpret_cast<const short4v*>(qr + 16 * t + 4 * g4),
            *reinterpret_cast<const short4v*>(kr + 16 * t + 4 * g4), sc[x], 0,
            0, 0);
    } else {
#pragma unroll
      for (int t = 0; t < 4 * DT; ++t)
        sc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(
            qr[4 * t + g4], kr[4 * t + g4], sc[x], 0, 0, 0);
    }
  }
  __syncthreads();                    // keys are no longer needed
#pragma unroll
  for (int x = 0; x < (NT + 3) / 4; ++x) {
    const int tile = wave + 4 * x;
    if (tile >= NT) continue;
    int rt = 0;
    while ((rt + 1) * (rt + 2) / 2 <= tile) ++rt;
    const int kt = tile - rt * (rt + 1) / 2;
    const int j = 16 * kt + c16;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * rt + 4 * g4 + r;
      a_lds[i * AP + j] =
          j <= i ? sc[x][r] * expf(static_cast<float>(g_lds[j] - top_lds[i]))
                 : 0.f;
    }
  }
  __syncthreads();
  {
    // denominators: four neighbouring threads share a row
    const int i = tid / 4, part = tid % 4;
    const float* np = chunk_n + ch * DP;
    float own = 0.f, start = 0.f;
    for (int j = part; j < 16 * (i / 16 + 1); j += 4) own += a_lds[i * AP + j];
    for (int d = part; d < DP; d += 4)
      start += Act<A>::ld(q_lds + i * QP + d) * np[d];
    float nd = own + start_lds[i] * start;
    nd += __shfl_xor(nd, 1, 64);
    nd += __shfl_xor(nd, 2, 64);
    if (part == 0)
      inv_lds[i] = q_scale / (fmaxf(fabsf(nd * q_scale), floor_lds[i]) + 1e-6f);
  }

  for (int ct = 0; ct < CT; ++ct) {
    const int col0 = ct * kMemoryCols;
    const float* src = chunk_mem +
        (((ch * CT + ct) * 4 + wave) * DT * 64 + lane) * 4;
    floatx4 S[DT];
#pragma unroll
    for (int t = 0; t < DT; ++t)
      S[t] = *reinterpret_cast<const floatx4*>(src + t * 256);
    load_tile<A, VW, kChunk, kMemoryCols, VP>(
        v_lds, in.v + row0 * in.vs + head * V + col0, in.vs, n,
        min(kMemoryCols, V - col0));
    __syncthreads();
    float vr[kChunk / 4];
#pragma unroll
    for (int kk = 0; kk < kChunk / 4; ++kk)
      vr[kk] = Act<A>::ld(v_lds + (4 * kk + g4) * VP + wave * 16 + c16);
    __syncthreads();
    const int col = col0 + wave * 16 + c16;
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      floatx4 own = {0.f, 0.f, 0.f, 0.f}, start = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < 4 * (rt + 1); ++kk)
        own = __builtin_amdgcn_mfma_f32_16x16x4f32(
            a_lds[(16 * rt + c16) * AP + 4 * kk + g4], vr[kk], own, 0, 0, 0);
#pragma unroll
      for (int t = 0; t < DT; ++t) {
        float q4[4];
        ldv<A, 4>(q_lds + (16 * rt + c16) * QP + 16 * t + 4 * g4, q4);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          start = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], S[t][r], start,
                                                       0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * rt + 4 * g4 + r;
        if (i < n && col < V)
          out[static_cast<int64_t>(row0 + i) * H * V + head * V + col] =
              (own[r] + start_lds[i] * start[r]) * inv_lds[i];
      }
    }
  }
}

}  // namespace

bool gated_memory_has_chunks(int D) { return D <= 256; }

int gated_memory_row_tiles(int D) {
  return D <= 32 ? 2 : D <= 64 ? 4 : D <= 128 ? 8 : 16;
}

template <typename A>
void launch_gated_memory_chunks(float* out, float* chunk_mem, float* chunk_n,
                                double* meta, MemoryInputs<A> in, float* mem,
                                float* aux, const int* seq_cu,
                                const int* seq_slots, const int* positions,
                                const int* tile_seq, const int* tile_row0,
                                int tiles, int groups, int H, int D, int V,
                                hipStream_t st) {
  if (tiles == 0 || groups == 0) return;
  const int CT = ceil_div(V, kMemoryCols);
  const int chunks = 2 * tiles;
  auto fits = [](const A* p, int64_t stride, int size) {
    return reinterpret_cast<uintptr_t>(p) % (4 * sizeof(A)) == 0 &&
           stride % 4 == 0 && size % 4 == 0;
  };
  const bool vec = fits(in.q, in.qs, D) && fits(in.k, in.ks, D) &&
                   fits(in.v, in.vs, V);
#define FI_CHUNKS(DT_, VW_)                                                      do {                                                                             hipLaunchKernelGGL((gated_memory_state_kernel<A, DT_, VW_>),                                      dim3(CT, H, chunks), dim3(256), 0, st, chunk_mem,                              chunk_n, meta, in, seq_cu, tile_seq, tile_row0, H, D,                          V);                                                         hipLaunchKernelGGL((gated_memory_carry_kernel<DT_>),                                              dim3(CT * DT_ + 1, H, groups), dim3(256), 0, st,                               chunk_mem, chunk_n, meta, mem, aux, seq_cu, seq_slots,                         positions, H, D, V, CT);                                    hipLaunchKernelGGL(gated_memory_max_kernel,                                                       dim3(ceil_div(groups * H, 64)), dim3(64), 0, st, meta,                         aux, seq_cu, seq_slots, groups, H, D, CT);                  hipLaunchKernelGGL((gated_memory_read_kernel<A, DT_, VW_>),                                       dim3(H, chunks), dim3(256), 0, st, out, chunk_mem,                             chunk_n, meta, in, seq_cu, tile_seq, tile_row0, H, D,                          V, CT);                                                   } while (0)
#define FI_CHUNKS_D(DT_)                                                         case DT_:                                                                        if (vec) FI_CHUNKS(DT_, 4);                                                    else FI_CHUNKS(DT_, 1);                                                        break
  switch (gated_memory_row_tiles(D)) {
    FI_CHUNKS_D(2);
    FI_CHUNKS_D(4);
    FI_CHUNKS_D(8);
    FI_CHUNKS_D(16);
  }
#undef FI_CHUNKS_D
#undef FI_CHUNKS
}

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
      const int*, int, int, int, int, int, hipStream_t);                       \
  template void launch_gated_memory_chunks<A>(                                 \
      float*, float*, float*, double*, MemoryInputs<A>, float*, float*,        \
      const int*, const int*, const int*, const int*, const int*, int, int,    \
      int, int, int, hipStream_t);
FI_INST(float)
FI_INST(u16)
#undef FI_INST

}  // namespace fi
