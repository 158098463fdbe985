// Row kernels around sublayers with a norm on both sides (gfx950, wave64):
//
//  * norm_residual_norm: x += rms(y) * w_post (fp32 stream, in place) and
//    out = rms(x) * w_next, the next sublayer's input, in one pass over the
//    row: sublayer result and stream stay in registers.
//  * headnorm_rope_cache: every query/key head divided by its RMS, times a
//    weight shared by the heads, leading entries rotated (entry i with entry
//    i + n); processed q to a dense buffer, processed k and the (blended)
//    v to the paged caches. A workgroup takes one or four rows: the angles of
//    a row are computed once for all its heads, a head is spread over just
//    as many lanes as it has vectors.
//  * gelu_tanh: elementwise.

#include "seqmix_scan.h"

namespace fi {

namespace {

// NCH > 0: the row is held in registers (NCH chunks of 256 threads x 4
// entries, W % 4 == 0); NCH == 0: any W, the row is re-read
template <typename A, int NCH>
__global__ __launch_bounds__(256) void norm_residual_norm_kernel(
    float* __restrict__ resid, const A* __restrict__ y,
    const float* __restrict__ w_post, const float* __restrict__ w_next,
    A* __restrict__ out, float eps, int W) {
  __shared__ float scratch[8];
  const int64_t t = blockIdx.x;
  const A* yr = y + t * W;
  float* rr = resid + t * W;
  A* orow = out + t * W;
  float dummy = 0.f, sq = 0.f;
  if constexpr (NCH > 0) {
    float v[NCH][4], r[NCH][4];
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < W) {
        ldv<A, 4>(yr + i, v[c]);
        ldv<float, 4>(rr + i, r[c]);
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k) v[c][k] = r[c][k] = 0.f;
      }
#pragma unroll
      for (int k = 0; k < 4; ++k) sq += v[c][k] * v[c][k];
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float s1 = rsqrtf(sq / W + eps);
    sq = 0.f;
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      float w4[4];
      ldv<float, 4>(w_post + i, w4);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        r[c][k] += v[c][k] * s1 * w4[k];
        sq += r[c][k] * r[c][k];
      }
      stv<float, 4>(rr + i, r[c]);
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float s2 = rsqrtf(sq / W + eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      float w4[4];
      ldv<float, 4>(w_next + i, w4);
#pragma unroll
      for (int k = 0; k < 4; ++k) w4[k] *= r[c][k] * s2;
      stv<A, 4>(orow + i, w4);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += 256) {
      const float x = Act<A>::ld(yr + i);
      sq += x * x;
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float s1 = rsqrtf(sq / W + eps);
    sq = 0.f;
    for (int i = threadIdx.x; i < W; i += 256) {
      const float x = rr[i] + Act<A>::ld(yr + i) * s1 * w_post[i];
      rr[i] = x;
      sq += x * x;
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float s2 = rsqrtf(sq / W + eps);
    // the same thread wrote these entries of the stream
    for (int i = threadIdx.x; i < W; i += 256)
      Act<A>::st(orow + i, rr[i] * s2 * w_next[i]);
  }
}

// items of a head: n / VW pairs of vectors (entry i with entry i + n), then
// the vectors that pass; a group of `lph` lanes (a power of two) has up to
// SLOTS items per lane
template <typename A, int VW, int SLOTS>
__global__ __launch_bounds__(256) void headnorm_rope_cache_kernel(
    HeadRopeArgs<A> a, int rows, int lph) {
  extern __shared__ float trig[];       // [rows][n] cos, then sin
  const int tid = threadIdx.x;
  const int t0 = blockIdx.x * rows;
  const int nr = min(rows, a.T - t0);
  float* sn_t = trig + rows * a.n;
  for (int i = tid; i < nr * a.n; i += 256) {
    const float p = static_cast<float>(a.positions[t0 + i / a.n]);
    sincosf(p * a.inv_freq[i % a.n], sn_t + i, trig + i);
  }
  __syncthreads();
  const int groups = 256 / lph, gl = tid % lph;
  const int nlow = a.n / VW;
  const int items = nlow + (a.D - 2 * a.n) / VW;
  const int heads = a.H + a.G;
  for (int it = tid / lph; it < nr * heads; it += groups) {
    const int r = it / heads, hh = it % heads;
    const int64_t t = t0 + r;
    const A* src;
    const float* w;
    A* dst = nullptr;
    if (hh < a.H) {
      src = a.q + t * a.qs + static_cast<int64_t>(hh) * a.D;
      w = a.q_w;
      dst = a.q_out + (t * a.H + hh) * a.D;
    } else {
      const int g = hh - a.H;
      src = a.k + t * a.ks + static_cast<int64_t>(g) * a.D;
      w = a.k_w;
      const int slot = a.slot_mapping[t];
      if (slot >= 0)
        dst = a.k_cache + ((static_cast<int64_t>(slot / a.bs) * a.G + g) *
                               a.bs + slot % a.bs) * a.D;
    }
    float lo[SLOTS][VW], hi[SLOTS][VW];
    float ss = 0.f;
#pragma unroll
    for (int s = 0; s < SLOTS; ++s) {
      const int i = gl + s * lph;
#pragma unroll
      for (int e = 0; e < VW; ++e) lo[s][e] = hi[s][e] = 0.f;
      if (i < items) {
        ldv<A, VW>(src + (i < nlow ? i : i + nlow) * VW, lo[s]);
        if (i < nlow) ldv<A, VW>(src + a.n + i * VW, hi[s]);
      }
#pragma unroll
      for (int e = 0; e < VW; ++e)
        ss += lo[s][e] * lo[s][e] + hi[s][e] * hi[s][e];
    }
    for (int off = lph / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    const float inv = rsqrtf(ss / a.D + a.eps);
    if (dst == nullptr) continue;
#pragma unroll
    for (int s = 0; s < SLOTS; ++s) {
      const int i = gl + s * lph;
      if (i >= items) continue;
      const int d0 = (i < nlow ? i : i + nlow) * VW;
      float g4[VW];
      ldv<float, VW>(w + d0, g4);
#pragma unroll
      for (int e = 0; e < VW; ++e) lo[s][e] *= inv * g4[e];
      if (i < nlow) {
        const int d1 = a.n + i * VW;
        ldv<float, VW>(w + d1, g4);
#pragma unroll
        for (int e = 0; e < VW; ++e) {
          const float x = hi[s][e] * inv * g4[e];
          const float cs = trig[r * a.n + d0 + e];
          const float sn = sn_t[r * a.n + d0 + e];
          hi[s][e] = x * cs + lo[s][e] * sn;
          lo[s][e] = lo[s][e] * cs - x * sn;
        }
        stv<A, VW>(dst + d1, hi[s]);
      }
      stv<A, VW>(dst + d0, lo[s]);
    }
  }
  // values: blended with the first such layer's, into the cache
  const float lam = a.v_first != nullptr ? *a.lam : 0.f;
  const int nv = a.G * a.V / VW;
  for (int it = tid; it < nr * nv; it += 256) {
    const int64_t t = t0 + it / nv;
    const int i = (it % nv) * VW;
    const int slot = a.slot_mapping[t];
    if (slot < 0) continue;
    float x[VW];
    ldv<A, VW>(a.v + t * a.vs + i, x);
    if (a.v_first != nullptr) {
      float f[VW];
      ldv<A, VW>(a.v_first + t * a.fs + i, f);
#pragma unroll
      for (int e = 0; e < VW; ++e) x[e] = (1.0f - lam) * x[e] + lam * f[e];
    }
    stv<A, VW>(a.v_cache + ((static_cast<int64_t>(slot / a.bs) * a.G +
                             i / a.V) * a.bs + slot % a.bs) * a.V + i % a.V,
               x);
  }
}

template <typename A, int VW>
__global__ __launch_bounds__(256) void gelu_tanh_kernel(
    A* __restrict__ out, const A* __restrict__ x, int64_t count) {
  const int64_t i = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * VW;
  if (i >= count) return;
  float v[VW];
  ldv<A, VW>(x + i, v);
#pragma unroll
  for (int e = 0; e < VW; ++e) {
    // 0.5 (1 + tanh(a)) = sigmoid(2 a)
    const float z = v[e];
    v[e] = z * sigmoid_hw(1.5957691216057308f *
                            (z + 0.044715f * z * z * z));
  }
  stv<A, VW>(out + i, v);
}

template <typename A>
bool aligned4(const A* p, int64_t stride) {
  return p == nullptr ||
         (reinterpret_cast<uintptr_t>(p) % (4 * sizeof(A)) == 0 &&
          stride % 4 == 0);
}

}  // namespace

template <typename A>
void launch_norm_residual_norm(float* resid, const A* y, const float* w_post,
                               const float* w_next, A* out, float eps, int T,
                               int W, hipStream_t st) {
  if (T == 0) return;
  const int chunks = W % 4 == 0 ? ceil_div(W, 1024) : 0;
#define FI_NRN(N_)                                                             \
  hipLaunchKernelGGL((norm_residual_norm_kernel<A, N_>), dim3(T), dim3(256),   \
                     0, st, resid, y, w_post, w_next, out, eps, W)
  if (chunks == 1) FI_NRN(1);
  else if (chunks == 2) FI_NRN(2);
  else if (chunks > 2 && chunks <= 4) FI_NRN(4);
  else if (chunks > 4 && chunks <= 8) FI_NRN(8);
  else FI_NRN(0);
#undef FI_NRN
}

template <typename A>
void launch_headnorm_rope_cache(HeadRopeArgs<A> a, hipStream_t st) {
  if (a.T == 0) return;
  const bool vec = a.D % 4 == 0 && a.n % 4 == 0 && a.V % 4 == 0 &&
                   aligned4(a.q, a.qs) && aligned4(a.k, a.ks) &&
                   aligned4(a.v, a.vs) && aligned4(a.v_first, a.fs);
  const int items = (a.D - a.n) / (vec ? 4 : 1);
  int lph = 1;
  while (lph < items && lph < 64) lph *= 2;
  const int slots = ceil_div(items, lph);
  const int rows = a.T >= 1024 ? 4 : 1;
  const size_t lds = static_cast<size_t>(rows) * max(a.n, 1) * 2 * sizeof(float);
#define FI_HEAD(VW_, S_)                                                       \
  hipLaunchKernelGGL((headnorm_rope_cache_kernel<A, VW_, S_>),                 \
                     dim3(ceil_div(a.T, rows)), dim3(256), lds, st, a, rows,   \
                     lph)
  if (vec && slots == 1) FI_HEAD(4, 1);
  else if (vec) FI_HEAD(4, 4);
  else if (slots <= 2) FI_HEAD(1, 2);
  else FI_HEAD(1, 16);
#undef FI_HEAD
}

template <typename A>
void launch_gelu_tanh(A* out, const A* x, int T, int N, hipStream_t st) {
  const int64_t count = static_cast<int64_t>(T) * N;
  if (count == 0) return;
  auto blocks = [&](int vw) {
    return dim3(static_cast<unsigned>((count + 256 * vw - 1) / (256 * vw)));
  };
  if (count % 4 == 0 && aligned4(x, 0) && aligned4(out, 0))
    hipLaunchKernelGGL((gelu_tanh_kernel<A, 4>), blocks(4), dim3(256), 0, st,
                       out, x, count);
  else
    hipLaunchKernelGGL((gelu_tanh_kernel<A, 1>), blocks(1), dim3(256), 0, st,
                       out, x, count);
}

#define FI_INST(A)                                                             \
  template void launch_norm_residual_norm<A>(float*, const A*, const float*,   \
                                             const float*, A*, float, int,     \
                                             int, hipStream_t);                \
  template void launch_headnorm_rope_cache<A>(HeadRopeArgs<A>, hipStream_t);   \
  template void launch_gelu_tanh<A>(A*, const A*, int, int, hipStream_t);
FI_INST(float)
FI_INST(u16)
#undef FI_INST

}  // namespace fi
