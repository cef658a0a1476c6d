// torch.ops.dli.gm_* — argument checks around the launchers of kernels/gatemix.hip (tanh norms, gated matrix states).  Included by
// torch_bindings.cpp inside its anonymous namespace, after recurmix_bindings.h (uses the helpers of the earlier binding headers).
// Every shape the kernels index with is checked here: the kernels themselves do no bounds checks.
#pragma once

// x fp32 [T, W] += mult · (y + ½ (rms(l) · wl + rms(r) · wr)); returns tanh(alpha · x) · w + b
Tensor gm_residual_tanh_norm(Tensor x, const c10::optional<Tensor>& y, const c10::optional<Tensor>& l, const c10::optional<Tensor>& r,
                             const c10::optional<Tensor>& wl, const c10::optional<Tensor>& wr, double mult, const Tensor& alpha,
                             const Tensor& w, const Tensor& b, double eps, bool out_bf16) {
  check_f32(x, "x");
  TORCH_CHECK(x.dim() == 2, "x must be [T, W]");
  const int64_t T = x.size(0), W = x.size(1);
  check_f32(alpha, "alpha", 1);
  check_f32(w, "w", W);
  check_f32(b, "b", W);
  TORCH_CHECK(l.has_value() == r.has_value() && l.has_value() == wl.has_value() && l.has_value() == wr.has_value(), "a pair comes with its weights");
  const bool bf = y.has_value() ? act_bf16(*y, "y") : l.has_value() ? act_bf16(*l, "l") : false;
  auto rows = [&](const c10::optional<Tensor>& t, const char* name) -> const void* {
    if (!t.has_value()) return nullptr;
    check_act_like(*t, bf, name);
    TORCH_CHECK(t->dim() == 2 && t->is_contiguous() && t->size(0) == T && t->size(1) == W, name, " must be contiguous and shaped like x");
    return t->data_ptr();
  };
  const void *yp = rows(y, "y"), *lp = rows(l, "l"), *rp = rows(r, "r");
  const float *wlp = opt_f32(wl, "wl", W), *wrp = opt_f32(wr, "wr", W);
  Tensor out = at::empty({T, W}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  dli::launch_gm_residual_tanh_norm(x.data_ptr<float>(), yp, lp, rp, bf, wlp, wrp, (float)mult, alpha.data_ptr<float>(), w.data_ptr<float>(),
                                    b.data_ptr<float>(), (float)eps, (int)T, (int)W, out.data_ptr(), out_bf16, cur_stream(x));
  return out;
}

Tensor gm_gelu_rows(const Tensor& x, const c10::optional<Tensor>& out_rows) {
  const bool bf = act_bf16(x, "x");
  check_rows(x, "x");
  Tensor out = out_rows.has_value() ? *out_rows : at::empty({x.size(0), x.size(1)}, x.options());
  check_act_like(out, bf, "out");
  check_rows(out, "out");
  TORCH_CHECK(out.size(0) == x.size(0) && out.size(1) == x.size(1), "out must be shaped like x");
  dli::launch_gm_gelu_rows(x.data_ptr(), bf, x.stride(0), (int)x.size(0), (int)x.size(1), out.data_ptr(), out.stride(0), cur_stream(x));
  return out;
}

// g [T, >= 2H] gate columns → log decay, input weight, exp(-m) of every token and head; state [slots, H] = running maxima
std::tuple<Tensor, Tensor, Tensor> gm_max_gates(const Tensor& g, const Tensor& bias, double cap, Tensor state, const Tensor& positions,
                                                const Tensor& qsl, const Tensor& state_slots, const Tensor& counts, int64_t num_seqs,
                                                bool chunks) {
  const bool bf = act_bf16(g, "g");
  check_rows(g, "g");
  const int64_t T = g.size(0), H = bias.numel() / 2;
  check_f32(bias, "bias", 2 * H);
  TORCH_CHECK(H >= 1 && g.size(1) >= 2 * H && cap > 0.0, "gates need 2·H columns and a positive cap");
  check_f32(state, "state");
  TORCH_CHECK(state.dim() == 2 && state.size(1) == H, "state must be [slots, H]");
  check_step_meta(positions, qsl, state_slots, counts, T, num_seqs);
  Tensor keep = at::empty({T, H}, state.options()), write = at::empty({T, H}, state.options()), floor_ = at::empty({T, H}, state.options());
  dli::launch_gm_max_gates(g.data_ptr(), bf, g.stride(0), bias.data_ptr<float>(), (float)cap, state.data_ptr<float>(),
                           positions.data_ptr<int>(), qsl.data_ptr<int>(), state_slots.data_ptr<int>(), counts.data_ptr<int>(), (int)num_seqs,
                           (int)H, keep.data_ptr<float>(), write.data_ptr<float>(), floor_.data_ptr<float>(), chunks, cur_stream(g));
  return {keep, write, floor_};
}

// the recurrence with a gated matrix state (see ops/seqmix.py: gated_scan) → (o fp32 [T, H·Dv], n · q fp32 [T, H] or empty)
std::tuple<Tensor, Tensor> gm_gated_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& decay, const Tensor& weight,
                                         Tensor state, const Tensor& positions, const Tensor& qsl, const Tensor& state_slots,
                                         const Tensor& counts, int64_t num_seqs, int64_t H, int64_t G, int64_t D, int64_t Dv, bool delta,
                                         double q_scale, bool normaliser, const c10::optional<Tensor>& tile_seq,
                                         const c10::optional<Tensor>& tile_q0, int64_t num_tiles) {
  const bool bf = act_bf16(q, "q");
  const int64_t T = q.size(0), cols = Dv + (normaliser ? 1 : 0);
  TORCH_CHECK(G >= 1 && H >= 1 && H % G == 0 && D >= 1 && Dv >= 1 && D <= dli::gm_step_max_dim() && !(delta && normaliser), "head sizes: H a multiple of G, D up to ",
              dli::gm_step_max_dim());
  check_act_like(k, bf, "k");
  check_act_like(v, bf, "v");
  check_rows(q, "q");
  check_rows(k, "k");
  check_rows(v, "v");
  TORCH_CHECK(q.size(1) == G * D && k.size(0) == T && k.size(1) == G * D && v.size(0) == T && v.size(1) == H * Dv,
              "q / k must be [T, G·D], v [T, H·Dv]");
  check_f32(decay, "decay", T * H);
  check_f32(weight, "weight", T * H);
  check_f32(state, "state");
  TORCH_CHECK(state.dim() >= 2 && state.numel() == state.size(0) * H * D * cols, "state must hold [slots][H][D · columns]");
  check_step_meta(positions, qsl, state_slots, counts, T, num_seqs);
  Tensor out = at::empty({T, H * Dv}, state.options());
  Tensor nq = at::empty({normaliser ? T : 0, H}, state.options());
  const int* tsp = nullptr;
  const int* tqp = nullptr;
  Tensor ws;
  if (num_tiles > 0 && tile_seq.has_value() && tile_q0.has_value() && D <= dli::gm_block_max_dim()) {
    check_i32(*tile_seq, "tile_seq");
    check_i32(*tile_q0, "tile_q0");
    TORCH_CHECK(tile_seq->numel() >= num_tiles && tile_q0->numel() >= num_tiles, "tile lists shorter than num_tiles");
    tsp = tile_seq->data_ptr<int>();
    tqp = tile_q0->data_ptr<int>();
    ws = at::empty({dli::gm_scan_ws_floats((int)T, (int)num_seqs, (int)H, delta)}, state.options());
  } else {
    num_tiles = 0;
  }
  dli::launch_gm_gated_scan(q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0), bf, decay.data_ptr<float>(),
                            weight.data_ptr<float>(), state.data_ptr<float>(), positions.data_ptr<int>(), qsl.data_ptr<int>(),
                            state_slots.data_ptr<int>(), counts.data_ptr<int>(), (int)num_seqs, (int)H, (int)G, (int)D, (int)Dv, delta,
                            (float)q_scale, normaliser, out.data_ptr<float>(), nq.data_ptr<float>(), tsp, tqp, (int)num_tiles,
                            num_tiles > 0 ? ws.data_ptr<float>() : nullptr, cur_stream(q));
  return {out, nq};
}

// the delta rule with a decay per key channel (see ops/seqmix.py: channel_delta_scan) → o fp32 [T, H·Dv]
Tensor gm_channel_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& z, const Tensor& rate, const Tensor& bias,
                       const Tensor& weight, Tensor state, const Tensor& positions, const Tensor& qsl, const Tensor& state_slots,
                       const Tensor& counts, int64_t num_seqs, int64_t H, int64_t G, int64_t D, int64_t Dv,
                       const c10::optional<Tensor>& tile_seq, const c10::optional<Tensor>& tile_q0, int64_t num_tiles) {
  const int64_t T = q.size(0);
  TORCH_CHECK(G >= 1 && H >= 1 && H % G == 0 && D >= 1 && Dv >= 1 && D <= dli::gm_step_max_dim(), "head sizes: H a multiple of G, D up to ",
              dli::gm_step_max_dim());
  check_act_like(q, false, "q");
  check_act_like(k, false, "k");
  check_act_like(v, false, "v");
  const bool zb = act_bf16(z, "z");
  check_rows(q, "q");
  check_rows(k, "k");
  check_rows(v, "v");
  check_rows(z, "z");
  TORCH_CHECK(q.size(1) == G * D && k.size(0) == T && k.size(1) == G * D && v.size(0) == T && v.size(1) == H * Dv && z.size(0) == T &&
                  z.size(1) == H * D, "q / k must be [T, G·D], v [T, H·Dv], z [T, H·D]");
  check_f32(rate, "rate", H);
  check_f32(bias, "bias", H * D);
  check_f32(weight, "weight", T * H);
  check_f32(state, "state");
  TORCH_CHECK(state.dim() >= 2 && state.numel() == state.size(0) * H * D * Dv, "state must hold [slots][H][D · Dv]");
  check_step_meta(positions, qsl, state_slots, counts, T, num_seqs);
  Tensor out = at::empty({T, H * Dv}, state.options());
  const int* tsp = nullptr;
  const int* tqp = nullptr;
  Tensor ws;
  if (num_tiles > 0 && tile_seq.has_value() && tile_q0.has_value() && D <= dli::gm_block_max_dim()) {
    check_i32(*tile_seq, "tile_seq");
    check_i32(*tile_q0, "tile_q0");
    TORCH_CHECK(tile_seq->numel() >= num_tiles && tile_q0->numel() >= num_tiles, "tile lists shorter than num_tiles");
    tsp = tile_seq->data_ptr<int>();
    tqp = tile_q0->data_ptr<int>();
    ws = at::empty({dli::gm_channel_ws_floats((int)T, (int)num_seqs, (int)H, (int)D)}, state.options());
  } else {
    num_tiles = 0;
  }
  dli::launch_gm_channel_scan(q.data_ptr<float>(), q.stride(0), k.data_ptr<float>(), k.stride(0), v.data_ptr<float>(), v.stride(0), z.data_ptr(),
                              zb, z.stride(0), rate.data_ptr<float>(), bias.data_ptr<float>(), weight.data_ptr<float>(), state.data_ptr<float>(),
                              positions.data_ptr<int>(), qsl.data_ptr<int>(), state_slots.data_ptr<int>(), counts.data_ptr<int>(), (int)num_seqs,
                              (int)H, (int)G, (int)D, (int)Dv, out.data_ptr<float>(), tsp, tqp, (int)num_tiles,
                              num_tiles > 0 ? ws.data_ptr<float>() : nullptr, cur_stream(q));
  return out;
}
