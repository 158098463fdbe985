// PyTorch bindings of the stream-copy, latent-projection and matrix-memory
// kernels (part of _C_seqmix). Every entry checks operand shapes against
// what its kernel and grid assume before launching.

#include "seqmix_bind.h"
#include "seqmix_hyper.h"

namespace {

using namespace fi_bind;
using OptTensor = c10::optional<at::Tensor>;

void hyper_start(at::Tensor xs, at::Tensor h, at::Tensor ids,
                 at::Tensor embed, at::Tensor w_in, at::Tensor norm_w,
                 double eps) {
  CHECK_F32(xs);
  CHECK_ACT(h);
  CHECK_F32(w_in);
  CHECK_F32(norm_w);
  TORCH_CHECK(ids.is_cuda() && ids.scalar_type() == at::kLong &&
              ids.is_contiguous() && ids.dim() == 1);
  TORCH_CHECK(embed.is_cuda() && embed.scalar_type() == h.scalar_type() &&
              embed.is_contiguous() && embed.dim() == 2);
  const int64_t T = ids.numel(), W = embed.size(1), S = w_in.numel();
  TORCH_CHECK(S >= 1 && S <= 8, "one to eight copies of the stream");
  TORCH_CHECK(xs.dim() == 3 && xs.size(0) == T && xs.size(1) == S &&
              xs.size(2) == W);
  TORCH_CHECK(h.is_contiguous() && h.dim() == 2 && h.size(0) == T &&
              h.size(1) == W && norm_w.numel() == W);
  DISPATCH_ACT(h, fi::launch_hyper_start<A>(
                      xs.data_ptr<float>(), ptr<A>(h),
                      ids.data_ptr<int64_t>(), ptr<A>(embed),
                      w_in.data_ptr<float>(), norm_w.data_ptr<float>(),
                      (float)eps, (int)T, (int)S, (int)W, stream()));
}

void hyper_update(at::Tensor xs, at::Tensor h, at::Tensor y1, OptTensor c1,
                  bool sig1, OptTensor y2, OptTensor c2, bool sig2,
                  OptTensor y3, OptTensor c3, bool sig3, at::Tensor mix,
                  at::Tensor w_out, at::Tensor w_in, at::Tensor norm_w,
                  double eps) {
  CHECK_F32(xs);
  CHECK_ACT(h);
  CHECK_F32(mix);
  CHECK_F32(w_out);
  CHECK_F32(w_in);
  CHECK_F32(norm_w);
  TORCH_CHECK(xs.dim() == 3);
  const int64_t T = xs.size(0), S = xs.size(1), W = xs.size(2);
  TORCH_CHECK(S >= 1 && S <= 8, "one to eight copies of the stream");
  TORCH_CHECK(mix.numel() == S * S && w_out.numel() == S &&
              w_in.numel() == S && norm_w.numel() == W);
  TORCH_CHECK(h.is_contiguous() && h.dim() == 2 && h.size(0) == T &&
              h.size(1) == W);
  const OptTensor ys[3] = {y1, y2, y3};
  const OptTensor cs[3] = {c1, c2, c3};
  const bool sg[3] = {sig1, sig2, sig3};
  DISPATCH_ACT(h, {
    fi::HyperTerms<A> terms;
    for (int j = 0; j < 3; ++j) {
      terms.y[j] = nullptr;
      terms.c[j] = nullptr;
      terms.c_stride[j] = 0;
      terms.sig[j] = sg[j];
      if (!ys[j].has_value()) continue;
      const at::Tensor& y = *ys[j];
      TORCH_CHECK(y.is_cuda() && y.scalar_type() == h.scalar_type() &&
                  y.is_contiguous() && y.dim() == 2 && y.size(0) == T &&
                  y.size(1) == W && y.data_ptr() != h.data_ptr(),
                  "sublayer term");
      terms.y[j] = ptr<A>(y);
      if (cs[j].has_value()) {
        const at::Tensor& c = *cs[j];
        TORCH_CHECK(c.is_cuda() && c.scalar_type() == at::kFloat &&
                    c.dim() == 1 && c.size(0) == T, "term coefficient");
        terms.c[j] = c.data_ptr<float>();
        terms.c_stride[j] = c.stride(0);
      }
    }
    fi::launch_hyper_update<A>(
        xs.data_ptr<float>(), ptr<A>(h), terms, mix.data_ptr<float>(),
        w_out.data_ptr<float>(), w_in.data_ptr<float>(),
        norm_w.data_ptr<float>(), (float)eps, (int)T, (int)S, (int)W,
        stream());
  });
}

void latent_norm_cache(OptTensor q_out, OptTensor dq, OptTensor dkv,
                       at::Tensor positions, at::Tensor inv_freq,
                       double rot_mult, OptTensor q_w, OptTensor c_w,
                       double eps, at::Tensor kv_cache,
                       at::Tensor slot_mapping, int64_t C, int64_t R,
                       bool half) {
  CHECK_I32(positions);
  CHECK_I32(slot_mapping);
  CHECK_F32(inv_freq);
  TORCH_CHECK(dq.has_value() || dkv.has_value());
  const at::Tensor& any = dq.has_value() ? *dq : *dkv;
  CHECK_ACT(any);
  const auto dt = any.scalar_type();
  const int64_t T = any.size(0);
  TORCH_CHECK(positions.numel() == T && slot_mapping.numel() == T);
  TORCH_CHECK(C >= 1 && R >= 0 && R % 2 == 0 && inv_freq.numel() <= R / 2);
  TORCH_CHECK(kv_cache.is_cuda() && kv_cache.is_contiguous() &&
              kv_cache.scalar_type() == dt && kv_cache.dim() == 4 &&
              kv_cache.size(1) == 1 && kv_cache.size(3) == C + R);
  int64_t Q = 0;
  if (dq.has_value()) {
    Q = dq->size(1);
    check_rows(*dq, T, Q, "query latent");
    TORCH_CHECK(q_out.has_value() && q_w.has_value());
    CHECK_F32(*q_w);
    TORCH_CHECK(q_w->numel() == Q && q_out->is_cuda() &&
                q_out->scalar_type() == dt && q_out->is_contiguous() &&
                q_out->sizes() == dq->sizes());
  }
  if (dkv.has_value()) {
    check_rows(*dkv, T, C + R, "latent projection");
    TORCH_CHECK(dkv->is_cuda() && dkv->scalar_type() == dt &&
                c_w.has_value());
    CHECK_F32(*c_w);
    TORCH_CHECK(c_w->numel() == C);
  }
  DISPATCH_ACT(any, fi::launch_latent_norm_cache<A>(
      dq.has_value() ? ptr<A>(*q_out) : nullptr,
      dq.has_value() ? ptr<A>(*dq) : nullptr,
      dq.has_value() ? dq->stride(0) : 0, (int)Q,
      dkv.has_value() ? ptr<A>(*dkv) : nullptr,
      dkv.has_value() ? dkv->stride(0) : 0, positions.data_ptr<int>(),
      inv_freq.data_ptr<float>(), (int)inv_freq.numel(), (float)rot_mult,
      dq.has_value() ? q_w->data_ptr<float>() : nullptr,
      dkv.has_value() ? c_w->data_ptr<float>() : nullptr, (float)eps,
      ptr<A>(kv_cache), slot_mapping.data_ptr<int>(), (int)T, (int)C, (int)R,
      (int)half, stream()));
}

void latent_query_rope(at::Tensor q_out, at::Tensor q, at::Tensor positions,
                       at::Tensor inv_freq, double rot_mult, int64_t H,
                       int64_t D, int64_t R, int64_t C, bool half) {
  CHECK_ACT(q);
  CHECK_I32(positions);
  CHECK_F32(inv_freq);
  const int64_t T = q.size(0);
  check_rows(q, T, H * (D + R), "queries");
  TORCH_CHECK(q_out.is_cuda() && q_out.scalar_type() == q.scalar_type() &&
              q_out.is_contiguous() && q_out.dim() == 3 &&
              q_out.size(0) == T && q_out.size(1) == H &&
              q_out.size(2) == C + R);
  TORCH_CHECK(positions.numel() == T);
  TORCH_CHECK(R % 2 == 0 && inv_freq.numel() <= R / 2 && R <= 1024);
  DISPATCH_ACT(q, fi::launch_latent_query_rope<A>(
                      ptr<A>(q_out), ptr<A>(q), q.stride(0),
                      positions.data_ptr<int>(), inv_freq.data_ptr<float>(),
                      (int)inv_freq.numel(), (float)rot_mult, (int)T, (int)H,
                      (int)D, (int)R, (int)C, (int)half, stream()));
}

void paged_rows_gather(at::Tensor out, at::Tensor cache, at::Tensor slots) {
  CHECK_ACT(cache);
  CHECK_I32(slots);
  TORCH_CHECK(cache.is_contiguous() && cache.dim() == 4 &&
              cache.size(1) == 1);
  TORCH_CHECK(out.is_cuda() && out.is_contiguous() && out.dim() == 2 &&
              out.scalar_type() == cache.scalar_type() &&
              out.size(0) == slots.numel() && out.size(1) == cache.size(3));
  fi::launch_paged_rows_gather(
      out.data_ptr(), cache.data_ptr(), slots.data_ptr<int>(),
      (int)slots.numel(), cache.size(3) * cache.element_size(), stream());
}

void silu_and_mul(at::Tensor out, at::Tensor gu) {
  CHECK_ACT(gu);
  TORCH_CHECK(gu.dim() == 2 && gu.is_contiguous() && gu.size(1) % 2 == 0);
  const int T = gu.size(0), F = gu.size(1) / 2;
  TORCH_CHECK(T <= 65535 * 16);
  TORCH_CHECK(out.is_cuda() && out.is_contiguous() &&
              out.scalar_type() == gu.scalar_type() && out.dim() == 2 &&
              out.size(0) == T && out.size(1) == F);
  DISPATCH_ACT(gu, fi::launch_silu_and_mul<A>(ptr<A>(out), ptr<A>(gu), T, F,
                                              stream()));
}

template <typename A>
fi::MemoryInputs<A> memory_inputs(const at::Tensor& q, const at::Tensor& k,
                                  const at::Tensor& v, const at::Tensor& i,
                                  const at::Tensor& f,
                                  const at::Tensor& i_bias,
                                  const at::Tensor& f_bias, double cap) {
  return {ptr<A>(q), ptr<A>(k), ptr<A>(v), ptr<A>(i), ptr<A>(f),
          q.stride(0), k.stride(0), v.stride(0), i.stride(0), f.stride(0),
          i_bias.data_ptr<float>(), f_bias.data_ptr<float>(), (float)cap};
}

void gated_memory(at::Tensor out, at::Tensor q, at::Tensor k, at::Tensor v,
                  at::Tensor i, at::Tensor f, at::Tensor i_bias,
                  at::Tensor f_bias, double cap, at::Tensor mem,
                  at::Tensor aux, at::Tensor seq_cu, at::Tensor seq_slots,
                  at::Tensor positions, int64_t H, int64_t D, int64_t V,
                  OptTensor tile_seq, OptTensor tile_row0, int64_t tile_rows) {
  CHECK_ACT(q);
  CHECK_F32(out);
  CHECK_F32(i_bias);
  CHECK_F32(f_bias);
  CHECK_F32(mem);
  CHECK_F32(aux);
  CHECK_I32(seq_cu);
  CHECK_I32(seq_slots);
  CHECK_I32(positions);
  const int64_t T = q.size(0);
  const auto dt = q.scalar_type();
  for (const at::Tensor* t : {&k, &v, &i, &f})
    TORCH_CHECK(t->is_cuda() && t->scalar_type() == dt);
  check_rows(q, T, H * D, "queries");
  check_rows(k, T, H * D, "keys");
  check_rows(v, T, H * V, "values");
  check_rows(i, T, H, "input gates");
  check_rows(f, T, H, "forget gates");
  TORCH_CHECK(D >= 1 && D <= 512, "matrix memory: key size must be <= 512");
  TORCH_CHECK(V >= 1 && cap > 0);
  TORCH_CHECK(out.numel() == T * H * V && i_bias.numel() == H &&
              f_bias.numel() == H);
  const int64_t copies = (V + fi::kMemoryCols - 1) / fi::kMemoryCols;
  TORCH_CHECK(mem.dim() == 4 && mem.size(1) == H && mem.size(2) == D &&
              mem.size(3) == V);
  TORCH_CHECK(aux.dim() == 4 && aux.size(0) == mem.size(0) &&
              aux.size(1) == H && aux.size(2) == copies &&
              aux.size(3) == D + 1);
  const int S = seq_slots.numel();
  TORCH_CHECK(seq_cu.numel() == S + 1 && positions.numel() == T);
  if (T == 0) return;
  // leading groups in chunks: all rows past tile_rows are one-row groups
  int groups = 0, tiles = 0;
  at::Tensor chunk_mem, chunk_n, meta;
  if (tile_seq.has_value() && fi::gated_memory_has_chunks((int)D)) {
    CHECK_I32(*tile_seq);
    TORCH_CHECK(tile_row0.has_value());
    CHECK_I32(*tile_row0);
    TORCH_CHECK(tile_row0->numel() == tile_seq->numel());
    TORCH_CHECK(tile_rows >= 0 && tile_rows <= T && S >= T - tile_rows);
    groups = S - (int)(T - tile_rows);
    tiles = tile_seq->numel();
    TORCH_CHECK(2 * tiles <= 65535 && groups <= 65535);
    const int64_t dp = 16 * fi::gated_memory_row_tiles((int)D);
    const auto f32 = q.options().dtype(at::kFloat);
    chunk_mem = at::empty({2 * tiles * H * copies * fi::kMemoryCols * dp}, f32);
    chunk_n = at::empty({2 * tiles * H * dp}, f32);
    meta = at::empty({2 * tiles * H * 3}, q.options().dtype(at::kDouble));
  }
  DISPATCH_ACT(q, {
    const auto in = memory_inputs<A>(q, k, v, i, f, i_bias, f_bias, cap);
    if (groups > 0)
      fi::launch_gated_memory_chunks<A>(
          out.data_ptr<float>(), chunk_mem.data_ptr<float>(),
          chunk_n.data_ptr<float>(), meta.data_ptr<double>(), in,
          mem.data_ptr<float>(), aux.data_ptr<float>(),
          seq_cu.data_ptr<int>(), seq_slots.data_ptr<int>(),
          positions.data_ptr<int>(), tile_seq->data_ptr<int>(),
          tile_row0->data_ptr<int>(), tiles, groups, (int)H, (int)D, (int)V,
          stream());
    fi::launch_gated_memory_scan<A>(
        out.data_ptr<float>(), in, mem.data_ptr<float>(),
        aux.data_ptr<float>(), seq_cu.data_ptr<int>(),
        seq_slots.data_ptr<int>(), positions.data_ptr<int>(), groups, S,
        (int)H, (int)D, (int)V, stream());
  });
}

}  // namespace

void register_hyper_ops(pybind11::module& m) {
  m.def("hyper_start", &hyper_start,
        "copies of the stream from the embedding, first normed input");
  m.def("hyper_update", &hyper_update,
        "mix the stream copies, add a sublayer's terms, emit the next "
        "sublayer's normed input");
  m.def("latent_norm_cache", &latent_norm_cache,
        "normed query latent; normed latent and rotated key part into the "
        "paged cache");
  m.def("latent_query_rope", &latent_query_rope,
        "rotated query parts into the folded query buffer");
  m.def("paged_rows_gather", &paged_rows_gather,
        "cache rows at given slots, laid end to end");
  m.def("silu_and_mul", &silu_and_mul, "silu(gate) * up");
  m.def("gated_memory", &gated_memory,
        "matrix memory with exponential gates on slot state");
}
