// Selective state-space recurrence and its short convolution (gfx950,
// wave64). Per channel c and state n, with dt = softplus(dt_lin + bias) and
// A = -exp(a_log):
//
//     S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c u_c B_n
//     out_c = (sum_n S[c, n] C_n + D_c u_c) * silu(z_c)
//
//  * causal_conv_silu: u = silu(causal convolution of x). A thread walks a
//    run of rows with the last taps - 1 inputs in registers, so every input
//    is read once; a step of one-row groups updates the tails in the same
//    launch.
//  * selective_scan_portion: LN adjacent lanes share a channel (four states
//    each), a 256-thread workgroup takes 256 / LN channels of one group (or
//    one segment of it). Blocks of kScanTokens tokens go global ->
//    registers -> LDS with step sizes, inputs and B / C rows converted once;
//    the loads of the next block are in flight while the current one is
//    applied from LDS. The read-outs of a token are summed over the LN lanes
//    by DPP and leave through LDS with the skip term and the gate.
//    Few long groups are cut into segments: end state from a zero start and
//    sum of the step sizes per segment (the decay of a whole segment is
//    exp(A sum dt)), an elementwise pass over the segments, then every
//    segment from its start state.
//  * selective_scan_rows: the same for decoded rows, straight from global
//    memory: bound by reading and writing the state.

#include "seqmix_scan.h"

namespace fi {

namespace {

FI_DEV float silu_f(float z) { return z * sigmoid_hw(z); }

// ------------------------------------------------------------ convolution

// ROWS consecutive rows per thread; their inputs are loaded up front
template <typename A, int VW, int TAPS, int ROWS>
__global__ __launch_bounds__(256) void causal_conv_silu_kernel(
    A* __restrict__ out, const A* __restrict__ x, int64_t x_stride,
    const float* __restrict__ conv_w, const float* __restrict__ conv_b,
    float* __restrict__ conv_state, const int* __restrict__ seq_cu,
    const int* __restrict__ row_seq, const int* __restrict__ seq_slots,
    const int* __restrict__ positions, int T, int C, int hist,
    int keep_tail) {
  constexpr int HW = TAPS > 1 ? TAPS - 1 : 1;
  const int c = (blockIdx.y * 256 + threadIdx.x) * VW;
  if (c >= C) return;
  const int t0 = blockIdx.x * ROWS;
  float w[VW][TAPS], b[VW], win[HW][VW], xs[ROWS][VW];
#pragma unroll
  for (int i = 0; i < ROWS; ++i)
    ldv<A, VW>(x + static_cast<int64_t>(min(t0 + i, T - 1)) * x_stride + c,
               xs[i]);
#pragma unroll
  for (int e = 0; e < VW; ++e) {
    b[e] = conv_b[c + e];
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
      w[e][j] = conv_w[static_cast<int64_t>(c + e) * TAPS + j];
  }
  int s = -1;
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int t = t0 + i;
    if (t >= T) return;
    const float* cur = xs[i];
    const int sn = row_seq[t];
    if (sn != s) {
      // the inputs before this row: earlier rows of the group, then the
      // kept tail, then zeros
      s = sn;
      const int a = seq_cu[s], r = t - a;
      const int slot = seq_slots[s];
      const bool has_hist = slot >= 0 && positions[a] > 0;
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        const int e0 = r + j;       // index into [tail | new rows]
#pragma unroll
        for (int e = 0; e < VW; ++e) win[j][e] = 0.f;
        if (e0 >= TAPS - 1)
          ldv<A, VW>(x + static_cast<int64_t>(a + e0 - (TAPS - 1)) * x_stride +
                         c, win[j]);
        else if (has_hist)
          ldv<float, VW>(conv_state + (static_cast<int64_t>(slot) * hist + e0) *
                             C + c, win[j]);
      }
    }
    float y[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      float acc = b[e];
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) acc += w[e][j] * win[j][e];
      y[e] = silu_f(acc + w[e][TAPS - 1] * cur[e]);
    }
    stv<A, VW>(out + static_cast<int64_t>(t) * C + c, y);
    if constexpr (TAPS > 1) {
#pragma unroll
      for (int j = 0; j < TAPS - 2; ++j)
#pragma unroll
        for (int e = 0; e < VW; ++e) win[j][e] = win[j + 1][e];
#pragma unroll
      for (int e = 0; e < VW; ++e) win[TAPS - 2][e] = cur[e];
      // one-row groups only: nobody else reads this slot's tail
      if (keep_tail && seq_slots[s] >= 0) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
          stv<float, VW>(conv_state + (static_cast<int64_t>(seq_slots[s]) *
                                           hist + j) * C + c, win[j]);
      }
    }
  }
}

// any number of taps, one entry per thread
template <typename A>
__global__ __launch_bounds__(256) void causal_conv_silu_any_kernel(
    A* __restrict__ out, const A* __restrict__ x, int64_t x_stride,
    const float* __restrict__ conv_w, const float* __restrict__ conv_b,
    const float* __restrict__ conv_state, const int* __restrict__ seq_cu,
    const int* __restrict__ row_seq, const int* __restrict__ seq_slots,
    const int* __restrict__ positions, int C, int taps, int hist) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int s = row_seq[t];
  const int a = seq_cu[s], r = t - a;
  const int slot = seq_slots[s];
  const bool has_hist = slot >= 0 && positions[a] > 0;
  float acc = conv_b[c];
  for (int j = 0; j < taps; ++j) {
    const int e = r + j;
    float v = 0.f;
    if (e >= taps - 1)
      v = Act<A>::ld(x + static_cast<int64_t>(a + e - (taps - 1)) * x_stride +
                     c);
    else if (has_hist)
      v = conv_state[(static_cast<int64_t>(slot) * hist + e) * C + c];
    acc += conv_w[static_cast<int64_t>(c) * taps + j] * v;
  }
  Act<A>::st(out + static_cast<int64_t>(t) * C + c, silu_f(acc));
}

// ------------------------------------------------------------------- scan

// four states n0.. of channel c: decay rates in the log2 domain (0 past N)
FI_DEV void load_rates(const float* a_log, int64_t c, int N, int n0,
                       float* a2) {
#pragma unroll
  for (int i = 0; i < 4; ++i)
    a2[i] = n0 + i < N ? -kLog2e * exp2_hw(kLog2e * a_log[c * N + n0 + i])
                       : 0.f;
}

// entries n0.. of a B or C row (0 past N); vec: whole aligned vectors
template <typename A>
FI_DEV void load_vector(const A* p, int N, int n0, int vec, float* v) {
  if (vec && n0 < N) {
    ldv<A, 4>(p + n0, v);
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    v[i] = n0 + i < N ? Act<A>::ld(p + n0 + i) : 0.f;
}

FI_DEV void load_state(const float* p, int N, int n0, float* S) {
  if (N % 4 == 0 && n0 < N) {
    ldv<float, 4>(p + n0, S);
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) S[i] = n0 + i < N ? p[n0 + i] : 0.f;
}

FI_DEV void store_state(float* p, int N, int n0, const float* S) {
  if (N % 4 == 0) {
    if (n0 < N) stv<float, 4>(p + n0, S);
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (n0 + i < N) p[n0 + i] = S[i];
}

// what a launch of the portion kernel computes
enum ScanPass { kWhole = 0, kSegmentEnds = 1, kSegmentRows = 2 };

template <typename A, int LN>
__global__ __launch_bounds__(256) void selective_scan_portion_kernel(
    ScanArgs<A> a, int pass, int seg_rows, int segs,
    float* __restrict__ seg_state, float* __restrict__ seg_dt) {
  constexpr int CH = 256 / LN;             // channels per workgroup
  constexpr int NP = 4 * LN;               // padded states
  constexpr int TB = (LN == 1 || LN >= 32) ? 16 : 32;   // tokens per block
  constexpr int PT = (TB + LN - 1) / LN;   // rows a thread loads and stores
  constexpr int BR = 256 / NP;             // B / C rows per pass
  constexpr int BT = (TB + BR - 1) / BR;
  __shared__ float2 s_dt[TB][CH];          // (dt, dt * u)
  __shared__ __attribute__((aligned(16))) float s_b[TB][NP];
  __shared__ __attribute__((aligned(16))) float s_c[TB][NP];
  __shared__ float s_y[TB][CH];

  const int tid = threadIdx.x;
  const int s = blockIdx.x, seg = blockIdx.z;
  const int c0 = blockIdx.y * CH;
  const int first = a.seq_cu[s];
  const int n = a.seq_cu[s + 1] - first;
  const int r0 = seg * seg_rows;
  if (r0 >= n) return;
  const bool last = r0 + seg_rows >= n;
  // the end of the last segment is the full pass's own result
  if (pass == kSegmentEnds && last) return;
  const int rows = min(seg_rows, n - r0);
  const int64_t t0 = first + r0;
  const int slot = a.seq_slots[s];

  // role in the recurrence: channel cr, states n0 .. n0 + 3
  const int lr = tid / LN, n0 = (tid % LN) * 4;
  const int cr = c0 + lr;
  const bool live = cr < a.W;
  float a2[4] = {0.f, 0.f, 0.f, 0.f}, S[4] = {0.f, 0.f, 0.f, 0.f};
  if (live) load_rates(a.a_log, cr, a.N, n0, a2);
  const int64_t seg_row =
      (static_cast<int64_t>(s) * segs + seg) * a.W + (live ? cr : 0);
  if (live) {
    if (pass == kSegmentRows)
      ldv<float, 4>(seg_state + seg_row * NP + n0, S);
    else if (pass == kWhole && slot >= 0 && a.positions[first] > 0)
      load_state(a.state + (static_cast<int64_t>(slot) * a.W + cr) * a.N, a.N,
                 n0, S);
  }
  // role in loading and storing: channel cl, rows rl, rl + LN, ... of a
  // block. Rows and channels past the end are read from the last ones: rows
  // get a step size of zero, channels are never stored.
  const int rl = tid / CH;
  const int cl = c0 + tid % CH;
  const bool cok = cl < a.W;
  const int cm = min(cl, a.W - 1);
  const int rb = tid / NP;
  const int km = min(tid % NP, a.N - 1);
  const float bias = a.dt_bias[cm], skip = a.d_skip[cm];
  A ur[PT], dr[PT], zr[PT], br[BT], cc[BT];
  // rows r0, r0 + step, ... of a block from a uniform base pointer and
  // 32-bit offsets; offsets of rows past the last one fall back to it
  auto load_rows = [](auto& dst, const A* p, int64_t stride, int r0,
                      int step, int col, int n) {
    const unsigned sd = static_cast<unsigned>(stride);
    const unsigned end = (n - 1) * sd + col;
    unsigned off = r0 * sd + col;
#pragma unroll
    for (auto& x : dst) {
      x = p[min(off, end)];
      off += step * sd;
    }
  };
  auto load_block = [&](int base) {
    const int64_t t = t0 + base;
    const int nt = min(TB, rows - base);
    load_rows(ur, a.u + t * a.W, a.W, rl, LN, cm, nt);
    load_rows(dr, a.dt + t * a.dts, a.dts, rl, LN, cm, nt);
    load_rows(br, a.B + t * a.bs, a.bs, rb, BR, km, nt);
    load_rows(cc, a.C + t * a.cs, a.cs, rb, BR, km, nt);
  };
  float dt_sum = 0.f;
  load_block(0);
  for (int base = 0; base < rows; base += TB) {
    const int nt = min(TB, rows - base);
    float uf[PT];
#pragma unroll
    for (int i = 0; i < PT; ++i) {
      const int e = rl + LN * i;
      uf[i] = Act<A>::ld(&ur[i]);
      // rows past the end leave the state alone
      const float dt =
          e < nt ? softplus_hw(Act<A>::ld(&dr[i]) + bias) : 0.f;
      if (TB % LN == 0 || e < TB) s_dt[e][tid % CH] = float2{dt, dt * uf[i]};
    }
#pragma unroll
    for (int i = 0; i < BT; ++i) {
      const int e = rb + BR * i;
      if (TB % BR == 0 || e < TB) {
        const bool in = tid % NP < a.N;
        s_b[e][tid % NP] = in ? Act<A>::ld(&br[i]) : 0.f;
        s_c[e][tid % NP] = in ? Act<A>::ld(&cc[i]) : 0.f;
      }
    }
    __syncthreads();
    if (pass != kSegmentEnds)
      load_rows(zr, a.z + (t0 + base) * a.zs, a.zs, rl, LN, cm, nt);
    if (base + TB < rows) load_block(base + TB);

    if (pass == kSegmentEnds) {
      for (int q = 0; q < nt; q += 4) {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          const float2 d = s_dt[q + k][lr];
          float b4[4];
          ldv<float, 4>(&s_b[q + k][n0], b4);
          dt_sum += d.x;
#pragma unroll
          for (int i = 0; i < 4; ++i)
            S[i] = exp2_hw(d.x * a2[i]) * S[i] + d.y * b4[i];
        }
      }
    } else {
      // operands of four tokens are read while four others are applied
      struct Four {
        float2 d[4];
        float b[4][4], c[4][4];
      };
      auto fetch = [&](Four& f, int q) {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          f.d[k] = s_dt[q + k][lr];
          ldv<float, 4>(&s_b[q + k][n0], f.b[k]);
          ldv<float, 4>(&s_c[q + k][n0], f.c[k]);
        }
      };
      auto apply = [&](const Four& f, int q) {
        float y[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          y[k] = 0.f;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            S[i] = exp2_hw(f.d[k].x * a2[i]) * S[i] + f.d[k].y * f.b[k][i];
            y[k] += S[i] * f.c[k][i];
          }
        }
        if constexpr (LN == 4) {
          // four tokens over four lanes: lane l ends with token l's sum
          const bool o1 = tid & 1, o2 = tid & 2;
          const float u = (o1 ? y[1] : y[0]) + dpp_move<0xB1>(o1 ? y[0] : y[1]);
          const float v = (o1 ? y[3] : y[2]) + dpp_move<0xB1>(o1 ? y[2] : y[3]);
          s_y[q + tid % 4][lr] = (o2 ? v : u) + dpp_move<0x4E>(o2 ? u : v);
        } else {
#pragma unroll
          for (int k = 0; k < 4; ++k) {
            y[k] = slice_sum<LN>(y[k]);
            if (tid % LN == 0) s_y[q + k][lr] = y[k];
          }
        }
      };
      Four even, odd;
      fetch(even, 0);
      for (int q = 0; q < nt; q += 8) {
        fetch(odd, q + 4);
        apply(even, q);
        if (q + 8 < nt) fetch(even, q + 8);
        apply(odd, q + 4);
      }
    }
    __syncthreads();
    if (pass != kSegmentEnds && cok) {
      A* op = a.out + (t0 + base) * a.W;
#pragma unroll
      for (int i = 0; i < PT; ++i) {
        const int e = rl + LN * i;
        if (e < nt)
          Act<A>::st(op + static_cast<unsigned>(e * a.W + cl),
                     (s_y[e][tid % CH] + skip * uf[i]) *
                         silu_f(Act<A>::ld(&zr[i])));
      }
    }
  }
  if (!live) return;
  if (pass == kSegmentEnds) {
    stv<float, 4>(seg_state + seg_row * NP + n0, S);
    if (tid % LN == 0) seg_dt[seg_row] = dt_sum;
  } else if (last && slot >= 0) {
    store_state(a.state + (static_cast<int64_t>(slot) * a.W + cr) * a.N, a.N,
                n0, S);
  }
}

// end states of the segments -> start states, in place
template <int LN>
__global__ __launch_bounds__(256) void selective_scan_carry_kernel(
    const float* __restrict__ a_log, const float* __restrict__ state,
    const int* __restrict__ seq_cu, const int* __restrict__ seq_slots,
    const int* __restrict__ positions, int W, int N, int seg_rows, int segs,
    float* __restrict__ seg_state, const float* __restrict__ seg_dt) {
  constexpr int CH = 256 / LN, NP = 4 * LN;
  const int s = blockIdx.x;
  const int n0 = (threadIdx.x % LN) * 4;
  const int c = blockIdx.y * CH + threadIdx.x / LN;
  if (c >= W) return;
  const int first = seq_cu[s];
  const int n = seq_cu[s + 1] - first;
  const int slot = seq_slots[s];
  float a2[4], S[4] = {0.f, 0.f, 0.f, 0.f};
  load_rates(a_log, c, N, n0, a2);
  if (n > 0 && slot >= 0 && positions[first] > 0)
    load_state(state + (static_cast<int64_t>(slot) * W + c) * N, N, n0, S);
  for (int seg = 0; seg * seg_rows < n; ++seg) {
    const int64_t row = (static_cast<int64_t>(s) * segs + seg) * W + c;
    float* p = seg_state + row * NP + n0;
    if ((seg + 1) * seg_rows < n) {
      float e[4];
      ldv<float, 4>(p, e);
      const float dt = seg_dt[row];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] += exp2_hw(dt * a2[i]) * S[i];
      stv<float, 4>(p, S);
#pragma unroll
      for (int i = 0; i < 4; ++i) S[i] = e[i];
    } else {
      stv<float, 4>(p, S);
    }
  }
}

template <typename A, int LN>
__global__ __launch_bounds__(256) void selective_scan_rows_kernel(
    ScanArgs<A> a, int s0) {
  constexpr int CH = 256 / LN;
  const int s = s0 + blockIdx.x;
  const int n0 = (threadIdx.x % LN) * 4;
  const int c = blockIdx.y * CH + threadIdx.x / LN;
  if (c >= a.W) return;
  const int first = a.seq_cu[s];
  const int end = a.seq_cu[s + 1];
  if (end <= first) return;
  const int slot = a.seq_slots[s];
  float* sp = a.state + (static_cast<int64_t>(slot < 0 ? 0 : slot) * a.W + c) *
                            a.N;
  float a2[4], S[4] = {0.f, 0.f, 0.f, 0.f};
  if (slot >= 0 && a.positions[first] > 0) load_state(sp, a.N, n0, S);
  load_rates(a.a_log, c, a.N, n0, a2);
  const float bias = a.dt_bias[c], skip = a.d_skip[c];
  for (int64_t t = first; t < end; ++t) {
    const float u = Act<A>::ld(a.u + t * a.W + c);
    const float dt = softplus_hw(Act<A>::ld(a.dt + t * a.dts + c) + bias);
    const float z = Act<A>::ld(a.z + t * a.zs + c);
    float y = 0.f, b4[4], c4[4];
    load_vector(a.B + t * a.bs, a.N, n0, a.vec, b4);
    load_vector(a.C + t * a.cs, a.N, n0, a.vec, c4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      S[i] = exp2_hw(dt * a2[i]) * S[i] + dt * u * b4[i];
      y += S[i] * c4[i];
    }
    y = slice_sum<LN>(y);
    if (threadIdx.x % LN == 0)
      Act<A>::st(a.out + t * a.W + c,
                 (y + skip * u) * silu_f(z));
  }
  if (slot >= 0) store_state(sp, a.N, n0, S);
}

}  // namespace

template <typename A>
void launch_causal_conv_silu(A* out, const A* x, int64_t x_stride,
                             const float* conv_w, const float* conv_b,
                             float* conv_state, const int* seq_cu,
                             const int* row_seq, const int* seq_slots,
                             const int* positions, int T, int S, int C,
                             int taps, int hist, int max_rows,
                             hipStream_t st) {
  if (T == 0) return;
  const bool vec = C % 4 == 0 && x_stride % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(x) % (4 * sizeof(A)) == 0;
  const bool fast = taps <= 4;
  const int keep_tail = fast && max_rows == 1;
#define FI_CONV(VW_, TAPS_, ROWS_)                                             \
  hipLaunchKernelGGL((causal_conv_silu_kernel<A, VW_, TAPS_, ROWS_>),          \
                     dim3(ceil_div(T, ROWS_), ceil_div(C, 256 * VW_)),         \
                     dim3(256), 0, st, out, x, x_stride, conv_w, conv_b,       \
                     conv_state, seq_cu, row_seq, seq_slots, positions, T, C,  \
                     hist, keep_tail)
#define FI_CONV_V(TAPS_)                                                       \
  do {                                                                         \
    if (vec && T >= 1024) FI_CONV(4, TAPS_, 8);                                \
    else if (vec) FI_CONV(4, TAPS_, 1);                                        \
    else FI_CONV(1, TAPS_, 1);                                                 \
  } while (0)
  switch (taps) {
    case 1: FI_CONV_V(1); break;
    case 2: FI_CONV_V(2); break;
    case 3: FI_CONV_V(3); break;
    case 4: FI_CONV_V(4); break;
    default:
      hipLaunchKernelGGL(causal_conv_silu_any_kernel<A>,
                         dim3(T, ceil_div(C, 256)), dim3(256), 0, st, out, x,
                         x_stride, conv_w, conv_b, conv_state, seq_cu,
                         row_seq, seq_slots, positions, C, taps, hist);
  }
#undef FI_CONV_V
#undef FI_CONV
  if (!keep_tail)
    launch_conv_tail_update<A>(x, x_stride, conv_state, seq_cu, seq_slots,
                               positions, S, C, taps, hist, st);
}

int scan_lanes(int N) {
  int ln = 1;
  while (4 * ln < N) ln *= 2;
  return ln;
}

int scan_segment_rows(int groups, int max_rows, int W, int N) {
  const int wgs = groups * ceil_div(W, 256 / scan_lanes(N));
  // a cut costs the states a second time: only from a third of the chip's
  // workgroups down, into segments of at least 128 rows
  const int k = min(512 / max(wgs, 1), max_rows / 128);
  if (k < 3) return 0;
  return ceil_div(ceil_div(max_rows, k), 32) * 32;
}

#define FI_LANES(LN_RUN, ...)                                                  \
  switch (LN_RUN) {                                                            \
    case 1: { constexpr int LN = 1; __VA_ARGS__; break; }                      \
    case 2: { constexpr int LN = 2; __VA_ARGS__; break; }                      \
    case 4: { constexpr int LN = 4; __VA_ARGS__; break; }                      \
    case 8: { constexpr int LN = 8; __VA_ARGS__; break; }                      \
    case 16: { constexpr int LN = 16; __VA_ARGS__; break; }                    \
    case 32: { constexpr int LN = 32; __VA_ARGS__; break; }                    \
    default: { constexpr int LN = 64; __VA_ARGS__; break; }                    \
  }

template <typename A>
void launch_selective_scan_portions(ScanArgs<A> a, int groups, int max_rows,
                                    int seg_rows, float* seg_state,
                                    float* seg_dt, hipStream_t st) {
  if (groups == 0 || max_rows == 0) return;
  const int ln = scan_lanes(a.N);
  const int cb = ceil_div(a.W, 256 / ln);
  FI_LANES(ln, {
    auto kernel = selective_scan_portion_kernel<A, LN>;
    if (seg_rows <= 0) {
      hipLaunchKernelGGL(kernel, dim3(groups, cb, 1), dim3(256), 0, st, a,
                         static_cast<int>(kWhole), max_rows, 1, nullptr,
                         nullptr);
    } else {
      const int segs = ceil_div(max_rows, seg_rows);
      const dim3 grid(groups, cb, segs);
      hipLaunchKernelGGL(kernel, grid, dim3(256), 0, st, a,
                         static_cast<int>(kSegmentEnds), seg_rows, segs,
                         seg_state, seg_dt);
      hipLaunchKernelGGL(selective_scan_carry_kernel<LN>, dim3(groups, cb),
                         dim3(256), 0, st, a.a_log, a.state, a.seq_cu,
                         a.seq_slots, a.positions, a.W, a.N, seg_rows, segs,
                         seg_state, seg_dt);
      hipLaunchKernelGGL(kernel, grid, dim3(256), 0, st, a,
                         static_cast<int>(kSegmentRows), seg_rows, segs,
                         seg_state, seg_dt);
    }
  })
}

template <typename A>
void launch_selective_scan_rows(ScanArgs<A> a, int s0, int S, hipStream_t st) {
  if (S <= s0) return;
  auto whole = [](const A* p, int64_t stride) {
    return reinterpret_cast<uintptr_t>(p) % (4 * sizeof(A)) == 0 &&
           stride % 4 == 0;
  };
  a.vec = a.N % 4 == 0 && whole(a.B, a.bs) && whole(a.C, a.cs);
  const int ln = scan_lanes(a.N);
  FI_LANES(ln, {
    auto kernel = selective_scan_rows_kernel<A, LN>;
    hipLaunchKernelGGL(kernel, dim3(S - s0, ceil_div(a.W, 256 / LN)),
                       dim3(256), 0, st, a, s0);
  })
}

#define FI_INST(A)                                                             \
  template void launch_causal_conv_silu<A>(                                    \
      A*, const A*, int64_t, const float*, const float*, float*, const int*,   \
      const int*, const int*, const int*, int, int, int, int, int, int,        \
      hipStream_t);                                                            \
  template void launch_selective_scan_portions<A>(                             \
      ScanArgs<A>, int, int, int, float*, float*, hipStream_t);                \
  template void launch_selective_scan_rows<A>(ScanArgs<A>, int, int,           \
                                              hipStream_t);
FI_INST(float)
FI_INST(u16)
#undef FI_INST

}  // namespace fi
