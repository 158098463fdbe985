// PyTorch bindings of the kernels around sublayers with a norm on both sides
// and of the selective scan (part of _C_seqmix). Every entry checks operand
// shapes against what its kernel and grid assume before launching.

#include "seqmix_bind.h"
#include "seqmix_scan.h"

namespace {

using namespace fi_bind;
using OptTensor = c10::optional<at::Tensor>;

void norm_residual_norm(at::Tensor resid, at::Tensor y, at::Tensor w_post,
                        at::Tensor w_next, at::Tensor out, double eps) {
  CHECK_F32(resid);
  CHECK_ACT(y);
  CHECK_F32(w_post);
  CHECK_F32(w_next);
  TORCH_CHECK(resid.dim() == 2 && y.sizes() == resid.sizes() &&
              y.is_contiguous());
  const int64_t T = resid.size(0), W = resid.size(1);
  TORCH_CHECK(W >= 1 && w_post.numel() == W && w_next.numel() == W);
  TORCH_CHECK(out.is_cuda() && out.scalar_type() == y.scalar_type() &&
              out.is_contiguous() && out.sizes() == resid.sizes() &&
              out.data_ptr() != resid.data_ptr());
  DISPATCH_ACT(y, fi::launch_norm_residual_norm<A>(
                      resid.data_ptr<float>(), ptr<A>(y),
                      w_post.data_ptr<float>(), w_next.data_ptr<float>(),
                      ptr<A>(out), (float)eps, (int)T, (int)W, stream()));
}

void headnorm_rope_cache(at::Tensor q_out, at::Tensor q, at::Tensor k,
                         at::Tensor v, OptTensor v_first, OptTensor lam,
                         at::Tensor positions, at::Tensor q_w, at::Tensor k_w,
                         double eps, at::Tensor inv_freq, at::Tensor k_cache,
                         at::Tensor v_cache, at::Tensor slot_mapping,
                         int64_t H, int64_t G, int64_t D, int64_t V) {
  CHECK_ACT(q);
  CHECK_I32(positions);
  CHECK_I32(slot_mapping);
  CHECK_F32(q_w);
  CHECK_F32(k_w);
  CHECK_F32(inv_freq);
  const int64_t T = q.size(0), n = inv_freq.numel();
  const auto dt = q.scalar_type();
  check_rows(q, T, H * D, "q");
  check_rows(k, T, G * D, "k");
  check_rows(v, T, G * V, "v");
  TORCH_CHECK(k.is_cuda() && v.is_cuda() && k.scalar_type() == dt &&
              v.scalar_type() == dt);
  TORCH_CHECK(H >= 1 && G >= 1 && D >= 1 && D <= 1024 && V >= 1 &&
              2 * n <= D, "head size out of range");
  TORCH_CHECK(q_out.is_cuda() && q_out.scalar_type() == dt &&
              q_out.is_contiguous() && q_out.numel() == T * H * D);
  TORCH_CHECK(positions.numel() == T && slot_mapping.numel() == T &&
              q_w.numel() == D && k_w.numel() == D);
  TORCH_CHECK(k_cache.is_cuda() && v_cache.is_cuda() &&
              k_cache.is_contiguous() && v_cache.is_contiguous() &&
              k_cache.scalar_type() == dt && v_cache.scalar_type() == dt);
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 &&
              k_cache.size(0) == v_cache.size(0) && k_cache.size(1) == G &&
              v_cache.size(1) == G && k_cache.size(2) == v_cache.size(2) &&
              k_cache.size(3) == D && v_cache.size(3) == V);
  if (v_first.has_value()) {
    check_rows(*v_first, T, G * V, "first values");
    TORCH_CHECK(v_first->is_cuda() && v_first->scalar_type() == dt &&
                lam.has_value());
    CHECK_F32(*lam);
    TORCH_CHECK(lam->numel() == 1);
  }
  DISPATCH_ACT(q, {
    fi::HeadRopeArgs<A> a;
    a.q_out = ptr<A>(q_out);
    a.q = ptr<A>(q);
    a.k = ptr<A>(k);
    a.v = ptr<A>(v);
    a.v_first = v_first.has_value() ? ptr<A>(*v_first) : nullptr;
    a.qs = q.stride(0);
    a.ks = k.stride(0);
    a.vs = v.stride(0);
    a.fs = v_first.has_value() ? v_first->stride(0) : 0;
    a.lam = v_first.has_value() ? lam->data_ptr<float>() : nullptr;
    a.positions = positions.data_ptr<int>();
    a.q_w = q_w.data_ptr<float>();
    a.k_w = k_w.data_ptr<float>();
    a.inv_freq = inv_freq.data_ptr<float>();
    a.eps = (float)eps;
    a.k_cache = ptr<A>(k_cache);
    a.v_cache = ptr<A>(v_cache);
    a.slot_mapping = slot_mapping.data_ptr<int>();
    a.T = (int)T;
    a.H = (int)H;
    a.G = (int)G;
    a.D = (int)D;
    a.V = (int)V;
    a.bs = (int)k_cache.size(2);
    a.n = (int)n;
    fi::launch_headnorm_rope_cache<A>(a, stream());
  });
}

void gelu_tanh(at::Tensor out, at::Tensor x) {
  CHECK_ACT(x);
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && out.is_cuda() &&
              out.is_contiguous() && out.scalar_type() == x.scalar_type() &&
              out.sizes() == x.sizes());
  DISPATCH_ACT(x, fi::launch_gelu_tanh<A>(ptr<A>(out), ptr<A>(x),
                                          (int)x.size(0), (int)x.size(1),
                                          stream()));
}

void causal_conv_silu(at::Tensor out, at::Tensor x, at::Tensor conv_w,
                      at::Tensor conv_b, at::Tensor conv_state,
                      at::Tensor seq_cu, at::Tensor row_seq,
                      at::Tensor seq_slots, at::Tensor positions,
                      int64_t max_rows) {
  CHECK_ACT(x);
  CHECK_F32(conv_w);
  CHECK_F32(conv_b);
  CHECK_F32(conv_state);
  CHECK_I32(row_seq);
  const int64_t T = x.size(0), C = x.size(1);
  check_rows(x, T, C, "convolution input");
  TORCH_CHECK(out.is_cuda() && out.scalar_type() == x.scalar_type() &&
              out.is_contiguous() && out.sizes() == x.sizes());
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(0) == C && conv_b.numel() == C);
  const int taps = conv_w.size(1);
  TORCH_CHECK(taps >= 1 && taps <= 64);
  TORCH_CHECK(conv_state.dim() == 3 && conv_state.size(2) == C &&
              conv_state.size(1) >= std::max(taps - 1, 1));
  check_groups(seq_cu, seq_slots, positions, T);
  TORCH_CHECK(row_seq.numel() == T && max_rows >= 0);
  const int S = seq_slots.numel();
  // one row per group only if there are as many groups as rows
  TORCH_CHECK(max_rows != 1 || S == T);
  DISPATCH_ACT(x, fi::launch_causal_conv_silu<A>(
                      ptr<A>(out), ptr<A>(x), x.stride(0),
                      conv_w.data_ptr<float>(), conv_b.data_ptr<float>(),
                      conv_state.data_ptr<float>(), seq_cu.data_ptr<int>(),
                      row_seq.data_ptr<int>(), seq_slots.data_ptr<int>(),
                      positions.data_ptr<int>(), (int)T, S, (int)C, taps,
                      (int)conv_state.size(1), (int)max_rows, stream()));
}

// groups: leading multi-row groups with portion_rows rows in all, the
// longest with max_rows; the rest are one-row groups
void selective_scan(at::Tensor out, at::Tensor u, at::Tensor dt,
                    at::Tensor dt_bias, at::Tensor a_log, at::Tensor B,
                    at::Tensor C, at::Tensor d_skip, at::Tensor z,
                    at::Tensor state, at::Tensor seq_cu, at::Tensor seq_slots,
                    at::Tensor positions, int64_t groups,
                    int64_t portion_rows, int64_t max_rows) {
  CHECK_ACT(u);
  CHECK_F32(dt_bias);
  CHECK_F32(a_log);
  CHECK_F32(d_skip);
  CHECK_F32(state);
  const auto ty = u.scalar_type();
  for (const at::Tensor* t : {&dt, &B, &C, &z, &out})
    TORCH_CHECK(t->is_cuda() && t->scalar_type() == ty);
  TORCH_CHECK(u.dim() == 2 && u.is_contiguous() && out.is_contiguous() &&
              out.sizes() == u.sizes());
  TORCH_CHECK(a_log.dim() == 2);
  const int64_t T = u.size(0), W = u.size(1), N = a_log.size(1);
  check_rows(dt, T, W, "step sizes");
  check_rows(z, T, W, "gate branch");
  check_rows(B, T, N, "input vectors");
  check_rows(C, T, N, "read-out vectors");
  TORCH_CHECK(N >= 1 && N <= 256, "selective scan: 1 to 256 states a channel");
  TORCH_CHECK(a_log.size(0) == W && dt_bias.numel() == W &&
              d_skip.numel() == W);
  TORCH_CHECK(state.dim() == 3 && state.size(1) == W && state.size(2) == N);
  check_groups(seq_cu, seq_slots, positions, T);
  const int64_t S = seq_slots.numel();
  TORCH_CHECK(groups >= 0 && groups <= S && portion_rows >= 0 &&
              max_rows >= 0 && max_rows <= portion_rows &&
              T - portion_rows == S - groups,
              "rows past the portions must be one-row groups");
  // grid range, and 32-bit offsets inside a block of 32 rows
  TORCH_CHECK(W <= 65535 * 4);
  for (const at::Tensor* t : {&dt, &B, &C, &z})
    TORCH_CHECK(t->stride(0) < (int64_t{1} << 26));
  if (T == 0) return;
  int seg_rows = 0;
  at::Tensor seg_state, seg_dt;
  float *ss = nullptr, *sd = nullptr;
  if (groups > 0 && max_rows > 0) {
    seg_rows = fi::scan_segment_rows((int)groups, (int)max_rows, (int)W,
                                     (int)N);
    if (seg_rows > 0) {
      const int64_t segs = (max_rows + seg_rows - 1) / seg_rows;
      TORCH_CHECK(segs <= 65535);
      const auto f32 = u.options().dtype(at::kFloat);
      seg_state = at::empty(
          {groups * segs * W * 4 * fi::scan_lanes((int)N)}, f32);
      seg_dt = at::empty({groups * segs * W}, f32);
      ss = seg_state.data_ptr<float>();
      sd = seg_dt.data_ptr<float>();
    }
  }
  DISPATCH_ACT(u, {
    fi::ScanArgs<A> a;
    a.out = ptr<A>(out);
    a.u = ptr<A>(u);
    a.dt = ptr<A>(dt);
    a.B = ptr<A>(B);
    a.C = ptr<A>(C);
    a.z = ptr<A>(z);
    a.dts = dt.stride(0);
    a.bs = B.stride(0);
    a.cs = C.stride(0);
    a.zs = z.stride(0);
    a.dt_bias = dt_bias.data_ptr<float>();
    a.a_log = a_log.data_ptr<float>();
    a.d_skip = d_skip.data_ptr<float>();
    a.state = state.data_ptr<float>();
    a.seq_cu = seq_cu.data_ptr<int>();
    a.seq_slots = seq_slots.data_ptr<int>();
    a.positions = positions.data_ptr<int>();
    a.W = (int)W;
    a.N = (int)N;
    a.vec = 0;
    fi::launch_selective_scan_portions<A>(a, (int)groups, (int)max_rows,
                                          seg_rows, ss, sd, stream());
    fi::launch_selective_scan_rows<A>(a, (int)groups, (int)S, stream());
  });
}

}  // namespace

void register_scan_ops(pybind11::module& m) {
  m.def("norm_residual_norm", &norm_residual_norm,
        "fp32 stream += rms(y) * w_post, then rms(stream) * w_next");
  m.def("headnorm_rope_cache", &headnorm_rope_cache,
        "head RMS norms, half rotation, k and blended v into paged caches");
  m.def("gelu_tanh", &gelu_tanh, "tanh form of gelu");
  m.def("causal_conv_silu", &causal_conv_silu,
        "silu of a per-channel causal convolution, tail kept per sequence");
  m.def("selective_scan", &selective_scan,
        "selective state-space recurrence on slot state, times silu(z)");
}
