// torch.ops.dli.pm_* — argument checks around the launchers of kernels/postmix.hip (post-norm layers, per-head norms, differential maps).
// Included by torch_bindings.cpp inside its anonymous namespace, after gatemix_bindings.h (uses the helpers of the earlier binding
// headers).  Every shape the kernels index with is checked here.
#pragma once

// scale · table[ids] as fp32 and in the table's type
std::tuple<Tensor, Tensor> pm_embed_rows(const Tensor& ids, const Tensor& table, double scale) {
  const bool bf = act_bf16(table, "table");
  check_i32(ids, "ids");
  TORCH_CHECK(ids.dim() == 1 && table.dim() == 2 && table.is_contiguous(), "ids must be [T], table contiguous [V, W]");
  const int64_t T = ids.size(0), W = table.size(1);
  Tensor x = at::empty({T, W}, table.options().dtype(at::kFloat)), h = at::empty({T, W}, table.options());
  dli::launch_pm_embed_rows(ids.data_ptr<int>(), table.data_ptr(), bf, (int)table.size(0), (float)scale, (int)T, (int)W, x.data_ptr<float>(),
                            h.data_ptr(), cur_stream(table));
  return {x, h};
}

// x fp32 [T, W] += y / rms(y) · (1 + w); returns x (or its norm with 1 + w2) in the asked type
Tensor pm_post_norm_add(Tensor x, const Tensor& y, const Tensor& w, double eps, const c10::optional<Tensor>& w2, bool out_bf16) {
  check_f32(x, "x");
  TORCH_CHECK(x.dim() == 2, "x must be [T, W]");
  const int64_t T = x.size(0), W = x.size(1);
  const bool bf = act_bf16(y, "y");
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && y.size(0) == T && y.size(1) == W, "y must be contiguous and shaped like x");
  check_f32(w, "w", W);
  Tensor out = at::empty({T, W}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  dli::launch_pm_post_norm_add(x.data_ptr<float>(), y.data_ptr(), bf, w.data_ptr<float>(), (float)eps, opt_f32(w2, "w2", W), (int)T, (int)W,
                               out.data_ptr(), out_bf16, cur_stream(x));
  return out;
}

// per-head norm, rotation and cache write; returns the queries [T, maps · H, D] ordered (key head, map, head of its group)
Tensor pm_head_norm_rope_cache(const Tensor& proj, const c10::optional<Tensor>& qw, const c10::optional<Tensor>& kw, double eps,
                               const Tensor& positions, const c10::optional<Tensor>& freq, int64_t rot_dims, const Tensor& slot_mapping,
                               Tensor k_cache, Tensor v_cache, int64_t H, int64_t G, int64_t D, int64_t Dv, int64_t maps) {
  const bool bf = act_bf16(proj, "proj");
  check_rows(proj, "proj");
  const int64_t T = proj.size(0);
  TORCH_CHECK(G > 0 && H % G == 0 && D > 0 && Dv > 0 && maps >= 1 && proj.size(1) == (H + G) * maps * D + G * Dv,
              "proj row does not match the head sizes");
  TORCH_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= D && rot_dims * 4 <= kSmMaxLds, "rot_dims must be even and at most D");
  TORCH_CHECK((rot_dims == 0) == !freq.has_value(), "rotation comes with its frequencies");
  if (freq.has_value())
    TORCH_CHECK(freq->is_cuda() && freq->scalar_type() == at::kDouble && freq->is_contiguous() && freq->numel() == rot_dims / 2,
                "freq must be float64 [rot_dims / 2]");
  check_i32(positions, "positions");
  check_i32(slot_mapping, "slot_mapping");
  TORCH_CHECK(positions.numel() >= T && slot_mapping.numel() >= T, "step metadata shorter than the batch");
  for (const Tensor* c : {&k_cache, &v_cache}) {
    check_act_like(*c, bf, "cache");
    TORCH_CHECK(c->is_contiguous() && c->dim() == 3 && c->size(1) == kSmPageTokens && c->size(0) == k_cache.size(0), "caches must be [pages, 32, row]");
  }
  TORCH_CHECK(k_cache.size(2) == G * maps * D && v_cache.size(2) == G * Dv, "cache rows do not match the head sizes");
  Tensor q = at::empty({T, maps * H, D}, proj.options());
  dli::launch_pm_head_norm_rope_cache(proj.data_ptr(), bf, proj.stride(0), opt_f32(qw, "qw", D), opt_f32(kw, "kw", D), (float)eps,
                                      positions.data_ptr<int>(), freq.has_value() ? freq->data_ptr<double>() : nullptr, (int)rot_dims,
                                      slot_mapping.data_ptr<int>(), k_cache.data_ptr(), v_cache.data_ptr(), (int)T, (int)H, (int)G, (int)D,
                                      (int)Dv, (int)maps, q.data_ptr(), cur_stream(proj));
  return q;
}

// o fp32 [T, 2H, Dv] → out [T, H·Dv] (row-strided view)
void pm_map_combine(const Tensor& o, const Tensor& lam, double eps, double scale, int64_t G, Tensor out, const c10::optional<Tensor>& token_seq) {
  check_f32(o, "o");
  check_f32(lam, "lam", 1);
  TORCH_CHECK(o.dim() == 3 && o.size(1) % 2 == 0 && G > 0 && (o.size(1) / 2) % G == 0, "o must be [T, 2H, Dv], H a multiple of G");
  const int64_t T = o.size(0), H = o.size(1) / 2, Dv = o.size(2);
  const bool bf = act_bf16(out, "out");
  check_rows(out, "out");
  TORCH_CHECK(out.size(0) == T && out.size(1) == H * Dv, "out must be [T, H·Dv]");
  if (token_seq.has_value()) {
    check_i32(*token_seq, "token_seq");
    TORCH_CHECK(token_seq->numel() >= T, "token_seq shorter than the batch");
  }
  dli::launch_pm_map_combine(o.data_ptr<float>(), lam.data_ptr<float>(), (float)eps, (float)scale, (int)T, (int)H, (int)G, (int)Dv,
                             token_seq.has_value() ? token_seq->data_ptr<int>() : nullptr, out.data_ptr(), bf, out.stride(0), cur_stream(o));
}
