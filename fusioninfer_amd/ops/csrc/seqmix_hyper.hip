// Row kernels around several copies of the residual stream and the latent
// projections (gfx950, wave64):
//
//  * hyper_start: every fp32 copy of the stream starts as embed[id]; emits
//    rms(sum_s a_s x_s) * w, the first sublayer's input.
//  * hyper_update: x_t <- sum_s M[s,t] x_s + b_t y for all copies at once,
//    y a sum of up to three sublayer terms with per-row coefficients, and
//    the next sublayer's input rms(sum_s a_s x_s) * w from the new copies:
//    the copies are read once and written once.
//  * latent_norm_cache: RMS norm of the query latent to a dense buffer; RMS
//    norm of the key/value latent and rotation of the shared key part (pairs
//    of neighbours, or entry i with entry i + n) into one paged cache row.
//    One wave per (row, part).
//  * latent_query_rope: the trailing rot_dim entries of every query head
//    rotated into the tail of the folded query buffer; one workgroup per
//    row, angles computed once for all heads.
//  * paged_rows_gather: cache rows at given slots, laid end to end.
//  * silu_and_mul.

#include <type_traits>

#include "seqmix.h"
#include "seqmix_hyper.h"

namespace fi {

namespace {

// NCH > 0: NCH chunks of 256 threads x 4 entries in registers (W % 4 == 0);
// NCH == 0: any W
template <typename A, int NCH>
__global__ __launch_bounds__(256) void hyper_start_kernel(
    float* __restrict__ xs, A* __restrict__ h, const int64_t* __restrict__ ids,
    const A* __restrict__ embed, const float* __restrict__ w_in,
    const float* __restrict__ norm_w, float eps, int S, int W) {
  __shared__ float scratch[8];
  const int64_t t = blockIdx.x;
  const A* e = embed + ids[t] * W;
  float* x = xs + t * S * W;
  A* o = h + t * W;
  float a = 0.f;
  for (int s = 0; s < S; ++s) a += w_in[s];
  float sq = 0.f, dummy = 0.f;
  if constexpr (NCH > 0) {
    float u[NCH][4];
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      ldv<A, 4>(e + i, u[c]);
      for (int s = 0; s < S; ++s)
        stv<float, 4>(x + static_cast<int64_t>(s) * W + i, u[c]);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        u[c][k] *= a;
        sq += u[c][k] * u[c][k];
      }
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float rstd = rsqrtf(sq / W + eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      float w4[4];
      ldv<float, 4>(norm_w + i, w4);
#pragma unroll
      for (int k = 0; k < 4; ++k) w4[k] *= u[c][k] * rstd;
      stv<A, 4>(o + i, w4);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += 256) {
      const float v = Act<A>::ld(e + i);
      for (int s = 0; s < S; ++s) x[static_cast<int64_t>(s) * W + i] = v;
      sq += a * v * a * v;
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float rstd = rsqrtf(sq / W + eps);
    for (int i = threadIdx.x; i < W; i += 256)
      Act<A>::st(o + i, a * Act<A>::ld(e + i) * rstd * norm_w[i]);
  }
}

// S: number of copies, or 8 for any runtime count up to 8
template <typename A, int S, int NCH>
__global__ __launch_bounds__(256) void hyper_update_kernel(
    float* __restrict__ xs, A* __restrict__ h, HyperTerms<A> terms,
    const float* __restrict__ mix, const float* __restrict__ w_out,
    const float* __restrict__ w_in, const float* __restrict__ norm_w,
    float eps, int ns, int W) {
  __shared__ float scratch[8];
  const int n = S == 8 ? ns : S;
  const int64_t t = blockIdx.x;
  float* x = xs + t * n * W;
  A* o = h + t * W;
  float coef[3];
#pragma unroll
  for (int j = 0; j < 3; ++j) {
    coef[j] = 1.f;
    if (terms.y[j] != nullptr && terms.c[j] != nullptr) {
      const float c = terms.c[j][t * terms.c_stride[j]];
      coef[j] = terms.sig[j] ? sigmoidf_acc(c) : c;
    }
  }
  float m[S][S], b[S], a[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    b[s] = s < n ? w_out[s] : 0.f;
    a[s] = s < n ? w_in[s] : 0.f;
#pragma unroll
    for (int r = 0; r < S; ++r)
      m[s][r] = s < n && r < n ? mix[s * n + r] : 0.f;
  }
  // one group of VW entries at column i: new copies written, returns the
  // weighted sum of them in u
  auto step = [&](int i, float* u, auto vw) {
    constexpr int VW = decltype(vw)::value;
    float y[VW], tmp[VW], old[S][VW];
    ldv<A, VW>(terms.y[0] + t * W + i, y);
#pragma unroll
    for (int k = 0; k < VW; ++k) y[k] *= coef[0];
#pragma unroll
    for (int j = 1; j < 3; ++j) {
      if (terms.y[j] == nullptr) continue;
      ldv<A, VW>(terms.y[j] + t * W + i, tmp);
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] += coef[j] * tmp[k];
    }
#pragma unroll
    for (int s = 0; s < S; ++s)
      if (S != 8 || s < n)
        ldv<float, VW>(x + static_cast<int64_t>(s) * W + i, old[s]);
#pragma unroll
    for (int k = 0; k < VW; ++k) u[k] = 0.f;
#pragma unroll
    for (int r = 0; r < S; ++r) {
      if (S == 8 && r >= n) continue;
      float v[VW];
#pragma unroll
      for (int k = 0; k < VW; ++k) v[k] = b[r] * y[k];
#pragma unroll
      for (int s = 0; s < S; ++s) {
        if (S == 8 && s >= n) continue;
#pragma unroll
        for (int k = 0; k < VW; ++k) v[k] += m[s][r] * old[s][k];
      }
      stv<float, VW>(x + static_cast<int64_t>(r) * W + i, v);
#pragma unroll
      for (int k = 0; k < VW; ++k) u[k] += a[r] * v[k];
    }
  };
  float sq = 0.f, dummy = 0.f;
  if constexpr (NCH > 0) {
    float u[NCH][4];
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      step(i, u[c], std::integral_constant<int, 4>{});
#pragma unroll
      for (int k = 0; k < 4; ++k) sq += u[c][k] * u[c][k];
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float rstd = rsqrtf(sq / W + eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i >= W) continue;
      float w4[4];
      ldv<float, 4>(norm_w + i, w4);
#pragma unroll
      for (int k = 0; k < 4; ++k) w4[k] *= u[c][k] * rstd;
      stv<A, 4>(o + i, w4);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += 256) {
      float u[1];
      step(i, u, std::integral_constant<int, 1>{});
      sq += u[0] * u[0];
    }
    block_reduce_sum2_256(sq, dummy, scratch);
    const float rstd = rsqrtf(sq / W + eps);
    // the same thread wrote these entries of the copies
    for (int i = threadIdx.x; i < W; i += 256) {
      float u = 0.f;
#pragma unroll
      for (int s = 0; s < S; ++s)
        if (S != 8 || s < n) u += a[s] * x[static_cast<int64_t>(s) * W + i];
      Act<A>::st(o + i, u * rstd * norm_w[i]);
    }
  }
}

// one wave: dst[i] = x[i] / rms(x) * w[i]
template <typename A, int VW>
FI_DEV void wave_rms_row(A* dst, const A* src, const float* w, int n,
                         float eps, int lane) {
  float ss = 0.f;
  for (int d = lane * VW; d < n; d += 64 * VW) {
    float x[VW];
    ldv<A, VW>(src + d, x);
#pragma unroll
    for (int k = 0; k < VW; ++k) ss += x[k] * x[k];
  }
  ss = wave_reduce_sum(ss);
  const float inv = rsqrtf(ss / n + eps);
  for (int d = lane * VW; d < n; d += 64 * VW) {
    float x[VW], g[VW];
    ldv<A, VW>(src + d, x);
    ldv<float, VW>(w + d, g);
#pragma unroll
    for (int k = 0; k < VW; ++k) x[k] *= inv * g[k];
    stv<A, VW>(dst + d, x);
  }
}

template <typename A, int VW>
__global__ __launch_bounds__(256) void latent_norm_cache_kernel(
    A* __restrict__ q_out, const A* __restrict__ dq, int64_t dq_stride, int Q,
    const A* __restrict__ dkv, int64_t dkv_stride,
    const int* __restrict__ positions, const float* __restrict__ inv_freq,
    int rot_pairs, float rot_mult, const float* __restrict__ q_w,
    const float* __restrict__ c_w, float eps, A* __restrict__ kv_cache,
    const int* __restrict__ slot_mapping, int T, int C, int R, int half) {
  const int lane = threadIdx.x % 64;
  const int64_t t = static_cast<int64_t>(blockIdx.x) * 4 + threadIdx.x / 64;
  if (t >= T) return;
  if (blockIdx.y == 0 && dq != nullptr) {
    wave_rms_row<A, VW>(q_out + t * Q, dq + t * dq_stride, q_w, Q, eps, lane);
    return;
  }
  const int slot = slot_mapping[t];
  if (slot < 0) return;
  A* row = kv_cache + static_cast<int64_t>(slot) * (C + R);
  const A* src = dkv + t * dkv_stride;
  wave_rms_row<A, VW>(row, src, c_w, C, eps, lane);
  src += C;
  row += C;
  const float pos = static_cast<float>(positions[t]);
  for (int i = lane; i < rot_pairs; i += 64) {
    const int i0 = half ? i : 2 * i, i1 = half ? i + rot_pairs : i0 + 1;
    const float u = Act<A>::ld(src + i0);
    const float w = Act<A>::ld(src + i1);
    float sn, cs;
    sincosf(pos * inv_freq[i], &sn, &cs);
    sn *= rot_mult;
    cs *= rot_mult;
    Act<A>::st(row + i0, u * cs - w * sn);
    Act<A>::st(row + i1, w * cs + u * sn);
  }
  for (int d = 2 * rot_pairs + lane; d < R; d += 64) row[d] = src[d];
}

constexpr int kMaxRotPairs = 512;

template <typename A>
__global__ __launch_bounds__(256) void latent_query_rope_kernel(
    A* q_out,                         // [T, H, C + R]; may be q itself (C = D)
    const A* q, int64_t q_stride,     // [T, H*(D+R)]
    const int* __restrict__ positions, const float* __restrict__ inv_freq,
    int rot_pairs, float rot_mult, int H, int D, int R, int C, int by_half) {
  __shared__ float cs_t[kMaxRotPairs], sn_t[kMaxRotPairs];
  const int64_t t = blockIdx.x;
  const float pos = static_cast<float>(positions[t]);
  for (int i = threadIdx.x; i < rot_pairs; i += 256) {
    float sn, cs;
    sincosf(pos * inv_freq[i], &sn, &cs);
    sn_t[i] = sn * rot_mult;
    cs_t[i] = cs * rot_mult;
  }
  __syncthreads();
  const int half = R / 2;
  for (int it = threadIdx.x; it < H * half; it += 256) {
    const int hh = it / half, i = it % half;
    const A* src = q + t * q_stride + static_cast<int64_t>(hh) * (D + R) + D;
    A* dst = q_out + (t * H + hh) * (C + R) + C;
    // pairs past the turning ones are neighbours in either pairing
    const bool apart = by_half && i < rot_pairs;
    const int i0 = apart ? i : 2 * i, i1 = apart ? i + rot_pairs : i0 + 1;
    float u = Act<A>::ld(src + i0);
    float w = Act<A>::ld(src + i1);
    if (i < rot_pairs) {
      const float a = u * cs_t[i] - w * sn_t[i];
      w = w * cs_t[i] + u * sn_t[i];
      u = a;
    }
    Act<A>::st(dst + i0, u);
    Act<A>::st(dst + i1, w);
  }
}

// rows of `words` elements from the given slots of a paged cache
template <typename V>
__global__ __launch_bounds__(256) void paged_rows_gather_kernel(
    V* __restrict__ out, const V* __restrict__ cache,
    const int* __restrict__ slots, int rows, int words) {
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (i >= static_cast<int64_t>(rows) * words) return;
  const int r = i / words, w = i % words;
  out[i] = cache[static_cast<int64_t>(slots[r]) * words + w];
}

template <typename A, int VW>
__global__ __launch_bounds__(256) void silu_and_mul_kernel(
    A* __restrict__ out, const A* __restrict__ gu, int F) {
  const int64_t t = blockIdx.y;
  const int i = (blockIdx.x * 256 + threadIdx.x) * VW;
  if (i >= F) return;
  float g[VW], u[VW];
  ldv<A, VW>(gu + t * 2 * F + i, g);
  ldv<A, VW>(gu + t * 2 * F + F + i, u);
#pragma unroll
  for (int k = 0; k < VW; ++k) g[k] = g[k] * sigmoidf_acc(g[k]) * u[k];
  stv<A, VW>(out + t * F + i, g);
}

}  // namespace

template <typename A>
void launch_hyper_start(float* xs, A* h, const int64_t* ids, const A* embed,
                        const float* w_in, const float* norm_w, float eps,
                        int T, int S, int W, hipStream_t st) {
  if (T == 0) return;
  const int chunks = W % 4 == 0 ? ceil_div(W, 1024) : 0;
#define FI_START(N_)                                                           \
  hipLaunchKernelGGL((hyper_start_kernel<A, N_>), dim3(T), dim3(256), 0, st,   \
                     xs, h, ids, embed, w_in, norm_w, eps, S, W)
  if (chunks == 1) FI_START(1);
  else if (chunks == 2) FI_START(2);
  else if (chunks > 2 && chunks <= 4) FI_START(4);
  else FI_START(0);
#undef FI_START
}

template <typename A>
void launch_hyper_update(float* xs, A* h, HyperTerms<A> terms,
                         const float* mix, const float* w_out,
                         const float* w_in, const float* norm_w, float eps,
                         int T, int S, int W, hipStream_t st) {
  if (T == 0) return;
  const int chunks = W % 4 == 0 ? ceil_div(W, 1024) : 0;
#define FI_UPD(S_, N_)                                                         \
  hipLaunchKernelGGL((hyper_update_kernel<A, S_, N_>), dim3(T), dim3(256), 0,  \
                     st, xs, h, terms, mix, w_out, w_in, norm_w, eps, S, W)
#define FI_UPD_S(S_)                                                           \
  do {                                                                         \
    if (chunks == 1) FI_UPD(S_, 1);                                            \
    else if (chunks == 2) FI_UPD(S_, 2);                                       \
    else if (chunks > 2 && chunks <= 4) FI_UPD(S_, 4);                         \
    else FI_UPD(S_, 0);                                                        \
  } while (0)
  switch (S) {
    case 1: FI_UPD_S(1); break;
    case 2: FI_UPD_S(2); break;
    case 3: FI_UPD_S(3); break;
    case 4: FI_UPD_S(4); break;
    default: FI_UPD(8, 0); break;
  }
#undef FI_UPD_S
#undef FI_UPD
}

template <typename A>
void launch_latent_norm_cache(A* q_out, const A* dq, int64_t dq_stride, int Q,
                              const A* dkv, int64_t dkv_stride,
                              const int* positions, const float* inv_freq,
                              int rot_pairs, float rot_mult, const float* q_w,
                              const float* c_w, float eps, A* kv_cache,
                              const int* slot_mapping, int T, int C, int R,
                              int half, hipStream_t st) {
  if (T == 0) return;
  auto fits = [](const void* p, int64_t stride) {
    return p == nullptr ||
           (reinterpret_cast<uintptr_t>(p) % (4 * sizeof(A)) == 0 &&
            stride % 4 == 0);
  };
  const bool vec = fits(dq, dq_stride) && fits(dkv, dkv_stride) &&
                   Q % 4 == 0 && C % 4 == 0 && R % 4 == 0;
  const dim3 grid(ceil_div(T, 4), (dq != nullptr) + (dkv != nullptr));
#define FI_LAT(VW_)                                                            \
  hipLaunchKernelGGL((latent_norm_cache_kernel<A, VW_>), grid, dim3(256), 0,   \
                     st, q_out, dq, dq_stride, Q, dkv, dkv_stride, positions,  \
                     inv_freq, rot_pairs, rot_mult, q_w, c_w, eps, kv_cache,   \
                     slot_mapping, T, C, R, half)
  if (vec) FI_LAT(4);
  else FI_LAT(1);
#undef FI_LAT
}

template <typename A>
void launch_latent_query_rope(A* q_out, const A* q, int64_t q_stride,
                              const int* positions, const float* inv_freq,
                              int rot_pairs, float rot_mult, int T, int H,
                              int D, int R, int C, int half, hipStream_t st) {
  if (T == 0 || R == 0) return;
  hipLaunchKernelGGL(latent_query_rope_kernel<A>, dim3(T), dim3(256), 0, st,
                     q_out, q, q_stride, positions, inv_freq, rot_pairs,
                     rot_mult, H, D, R, C, half);
}

void launch_paged_rows_gather(void* out, const void* cache, const int* slots,
                              int rows, int64_t row_bytes, hipStream_t st) {
  if (rows == 0) return;
  auto blocks = [&](int64_t words) {
    return dim3(static_cast<unsigned>((rows * words + 255) / 256));
  };
  if (row_bytes % 16 == 0)
    hipLaunchKernelGGL(paged_rows_gather_kernel<float4>,
                       blocks(row_bytes / 16), dim3(256), 0, st,
                       static_cast<float4*>(out),
                       static_cast<const float4*>(cache), slots, rows,
                       static_cast<int>(row_bytes / 16));
  else
    hipLaunchKernelGGL(paged_rows_gather_kernel<u16>, blocks(row_bytes / 2),
                       dim3(256), 0, st, static_cast<u16*>(out),
                       static_cast<const u16*>(cache), slots, rows,
                       static_cast<int>(row_bytes / 2));
}

template <typename A>
void launch_silu_and_mul(A* out, const A* gu, int T, int F, hipStream_t st) {
  if (T == 0) return;
  if (F % 4 == 0)
    hipLaunchKernelGGL((silu_and_mul_kernel<A, 4>), dim3(ceil_div(F, 1024), T),
                       dim3(256), 0, st, out, gu, F);
  else
    hipLaunchKernelGGL((silu_and_mul_kernel<A, 1>), dim3(ceil_div(F, 256), T),
                       dim3(256), 0, st, out, gu, F);
}

#define FI_INST(A)                                                             \
  template void launch_hyper_start<A>(float*, A*, const int64_t*, const A*,    \
                                      const float*, const float*, float, int,  \
                                      int, int, hipStream_t);                  \
  template void launch_hyper_update<A>(                                        \
      float*, A*, HyperTerms<A>, const float*, const float*, const float*,     \
      const float*, float, int, int, int, hipStream_t);                        \
  template void launch_latent_norm_cache<A>(                                   \
      A*, const A*, int64_t, int, const A*, int64_t, const int*, const float*, \
      int, float, const float*, const float*, float, A*, const int*, int, int, \
      int, int, hipStream_t);                                                  \
  template void launch_latent_query_rope<A>(A*, const A*, int64_t, const int*, \
                                            const float*, int, float, int,     \
                                            int, int, int, int, int,           \
                                            hipStream_t);                      \
  template void launch_silu_and_mul<A>(A*, const A*, int, int, hipStream_t);
FI_INST(float)
FI_INST(u16)
#undef FI_INST

}  // namespace fi
