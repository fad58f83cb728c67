// torch.ops.hipserve_delta.* — window attention (with a sink, chunked, or differential with two maps per head), the
// delta-rule and decayed linear-attention recurrences, token shift, the softmax router and the experts' GEMMs, and
// the elementwise activations of the layer-list decoders (csrc/kernels/seq/window_attention*.hip, delta_scan.hip,
// router.hip, expert_ffn.hip), plus the residual + norm kernels (group_norm.hip, sandwich.hip); built as their own library (hipserve/_C_delta.so) so a model compiles only
// what it runs.
// All ops write into caller-provided outputs (no allocation except moe_align's scratch, no host sync).
#include <torch/library.h>
#include <ATen/ATen.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>

#include "hipserve/seq_kernels.h"
#include "hipserve/seq_shared_bindings.h"
#include "hipserve/seq_window_bindings.h"

namespace {

using namespace hipserve_shared;

void scaled_add_group_rmsnorm(at::Tensor& out, at::Tensor& residual, const at::Tensor& w, int64_t groups, double eps,
                              const c10::optional<at::Tensor>& mix, const c10::optional<at::Tensor>& ls1,
                              const c10::optional<at::Tensor>& y, const c10::optional<at::Tensor>& pair_slot,
                              int64_t top, const c10::optional<at::Tensor>& ls2,
                              const c10::optional<at::Tensor>& extra) {
  CHECK_DEV(out); CHECK_CONTIG(out); CHECK_F32(residual); CHECK_F32(w);
  const bool f32 = is_f32(out, "scaled_add_group_rmsnorm");
  TORCH_CHECK(residual.dim() == 2 && out.sizes() == residual.sizes());
  const long T = residual.size(0), H = residual.size(1);
  TORCH_CHECK(groups >= 1 && H % groups == 0 && w.numel() == H && H + groups <= 15000, "group norm shape");
  if (mix.has_value()) {
    TORCH_CHECK(mix->scalar_type() == out.scalar_type() && mix->is_contiguous() && mix->sizes() == residual.sizes());
    TORCH_CHECK(!ls1.has_value() || (ls1->scalar_type() == at::kFloat && ls1->is_contiguous() && ls1->numel() == H));
  }
  if (y.has_value()) {
    TORCH_CHECK(y->scalar_type() == out.scalar_type() && y->is_contiguous() && y->dim() == 2 && y->size(1) == H);
    TORCH_CHECK(top >= 1 && pair_slot.has_value() && pair_slot->scalar_type() == at::kInt &&
                pair_slot->is_contiguous() && pair_slot->numel() >= T * top);
    TORCH_CHECK(ls2.has_value() && ls2->scalar_type() == at::kFloat && ls2->numel() == H);
  }
  if (extra.has_value())
    TORCH_CHECK(extra->scalar_type() == out.scalar_type() && extra->is_contiguous() && extra->sizes() == residual.sizes());
  c10::hip::HIPGuardMasqueradingAsCUDA g(out.device());
  hipserve::launch_scaled_add_group_rmsnorm(
      out.data_ptr(), residual.data_ptr<float>(), w.data_ptr<float>(), T, H, groups, (float)eps, opt_ptr(mix),
      (const float*)opt_ptr(ls1), opt_ptr(y), (const int*)opt_ptr(pair_slot), y.has_value() ? top : 0,
      (const float*)opt_ptr(ls2), opt_ptr(extra), f32, cur_stream());
}


// What both gated-rule ops check and pass on; `step`: every sequence brings one row.
hipserve::GatedDelta gated_args(at::Tensor& y, at::Tensor& S, at::Tensor& conv_state, const at::Tensor& proj,
                                const at::Tensor& conv_w, const at::Tensor& a_log, const at::Tensor& dt_bias,
                                const at::Tensor& norm_w, const at::Tensor& seq_cu, const at::Tensor& seq_ctx,
                                const at::Tensor& seq_state, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim,
                                int64_t taps, double eps, int64_t off_a, int64_t off_g, int64_t off_b, bool channel,
                                bool silu) {
  CHECK_DEV(proj); CHECK_F32(S); CHECK_F32(conv_state); CHECK_F32(conv_w); CHECK_F32(a_log);
  CHECK_F32(dt_bias); CHECK_F32(norm_w); CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  TORCH_CHECK(y.scalar_type() == proj.scalar_type());
  TORCH_CHECK(heads >= 1 && kv_heads >= 1 && heads % kv_heads == 0 && dim >= 1 && dim <= hipserve::delta_max_dim() &&
              vdim >= 1 && taps >= 1 && taps <= hipserve::delta_max_taps(), "gated_delta: sizes");
  const long T = proj.size(0), nseq = seq_ctx.numel(), C = 2 * kv_heads * dim + heads * vdim;
  TORCH_CHECK(rows2d(proj) && rows2d(y) && y.size(0) == T && y.size(1) == heads * vdim);
  TORCH_CHECK(off_b >= C && proj.size(1) >= off_b + heads && off_a >= C && off_g >= C, "gated_delta: columns");
  TORCH_CHECK(channel || (proj.size(1) >= off_a + heads && proj.size(1) >= off_g + heads * vdim), "gated_delta: columns");
  TORCH_CHECK(S.dim() == 4 && S.size(1) == heads && S.size(2) == dim && S.size(3) == vdim);
  TORCH_CHECK(conv_state.dim() == 3 && conv_state.size(0) == S.size(0) && conv_state.size(2) == C &&
              conv_state.size(1) == (taps > 1 ? taps - 1 : 1));
  TORCH_CHECK(conv_w.numel() == C * taps && a_log.numel() == heads && norm_w.numel() == vdim &&
              dt_bias.numel() == (channel ? heads * dim : heads));
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535);
  hipserve::GatedDelta p{};
  p.y = y.data_ptr(); p.y_ld = y.stride(0);
  p.S = S.data_ptr<float>(); p.conv_state = conv_state.data_ptr<float>();
  p.proj = proj.data_ptr(); p.ld = proj.stride(0);
  p.conv_w = conv_w.data_ptr<float>(); p.a_log = a_log.data_ptr<float>();
  p.dt_bias = dt_bias.data_ptr<float>(); p.norm_w = norm_w.data_ptr<float>();
  p.seq_cu = seq_cu.data_ptr<int>(); p.seq_ctx = seq_ctx.data_ptr<int>(); p.seq_state = seq_state.data_ptr<int>();
  p.nseq = nseq; p.T = T; p.heads = heads; p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim; p.taps = taps;
  p.off_a = off_a; p.off_g = off_g; p.off_b = off_b; p.eps = (float)eps; p.channel = channel; p.silu = silu;
  return p;
}

void gated_delta(at::Tensor& y, at::Tensor& S, at::Tensor& conv_state, const at::Tensor& proj,
                 const at::Tensor& conv_w, const at::Tensor& a_log, const at::Tensor& dt_bias,
                 const at::Tensor& norm_w, const c10::optional<at::Tensor>& decay,
                 const c10::optional<at::Tensor>& gate, const at::Tensor& seq_cu, const at::Tensor& seq_ctx,
                 const at::Tensor& seq_state, at::Tensor& scratch, int64_t heads, int64_t kv_heads, int64_t dim,
                 int64_t vdim, int64_t taps, double eps, int64_t off_a, int64_t off_g, int64_t off_b, bool channel,
                 bool silu, const c10::optional<at::Tensor>& chunks) {
  auto p = gated_args(y, S, conv_state, proj, conv_w, a_log, dt_bias, norm_w, seq_cu, seq_ctx, seq_state, heads, kv_heads,
                      dim, vdim, taps, eps, off_a, off_g, off_b, channel, silu);
  CHECK_F32(scratch);
  TORCH_CHECK(scratch.numel() >= (long)p.T * (2 * kv_heads * dim + 2 * heads * vdim + heads * (1 + (channel ? dim : 1))) + 64);
  TORCH_CHECK(channel == decay.has_value() && channel == gate.has_value(), "gated_delta: bottlenecks' results");
  if (channel) {
    CHECK_F32(*decay); CHECK_CONTIG(*gate);
    TORCH_CHECK(decay->numel() == (long)p.T * heads * dim && gate->scalar_type() == proj.scalar_type() &&
                gate->numel() == (long)p.T * heads * vdim, "gated_delta: bottlenecks' results");
    p.decay = decay->data_ptr<float>();
    p.gate = gate->data_ptr();
  }
  if (chunks.has_value()) {
    CHECK_F32(*chunks);
    TORCH_CHECK(dim <= hipserve::delta_chunk_max_dim() &&
                chunks->numel() >= hipserve::delta_chunk_floats(p.T, p.nseq, heads, dim, vdim) && p.T / 16 + p.nseq <= 65535,
                "gated_delta: room for the chunks");
    p.chunks = chunks->data_ptr<float>();
  }
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_gated_delta(p, scratch.data_ptr<float>(), is_f32(proj, "gated_delta"), cur_stream());
}

int64_t delta_chunk_floats(int64_t T, int64_t nseq, int64_t heads, int64_t dim, int64_t vdim) {
  return dim > hipserve::delta_chunk_max_dim() ? 0 : hipserve::delta_chunk_floats(T, nseq, heads, dim, vdim);
}

void gated_delta_step(at::Tensor& y, at::Tensor& S, at::Tensor& conv_state, const at::Tensor& proj,
                      const at::Tensor& conv_w, const at::Tensor& a_log, const at::Tensor& dt_bias,
                      const at::Tensor& norm_w, const c10::optional<at::Tensor>& a2, const c10::optional<at::Tensor>& g2,
                      const at::Tensor& seq_cu, const at::Tensor& seq_ctx, const at::Tensor& seq_state, int64_t heads,
                      int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps, double eps, int64_t off_a, int64_t off_g,
                      int64_t off_b, bool channel, bool silu) {
  auto p = gated_args(y, S, conv_state, proj, conv_w, a_log, dt_bias, norm_w, seq_cu, seq_ctx, seq_state, heads, kv_heads,
                      dim, vdim, taps, eps, off_a, off_g, off_b, channel, silu);
  TORCH_CHECK(vdim <= 256, "gated_delta_step: value size");
  TORCH_CHECK(channel == a2.has_value() && channel == g2.has_value(), "gated_delta_step: bottlenecks");
  if (channel) {
    CHECK_CONTIG(*a2); CHECK_CONTIG(*g2);
    TORCH_CHECK(a2->scalar_type() == proj.scalar_type() && g2->scalar_type() == proj.scalar_type() && a2->dim() == 2 &&
                g2->dim() == 2 && a2->size(0) == heads * dim && g2->size(0) == heads * vdim, "gated_delta_step: bottlenecks");
    p.a2 = a2->data_ptr(); p.g2 = g2->data_ptr();
    p.ra = a2->size(1); p.rg = g2->size(1);
    TORCH_CHECK(p.ra + p.rg <= hipserve::gated_delta_step_max_rank() && proj.size(1) >= off_a + p.ra &&
                proj.size(1) >= off_g + p.rg, "gated_delta_step: bottleneck columns");
  }
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_gated_delta_step(p, is_f32(proj, "gated_delta_step"), cur_stream());
}

void sandwich_update(at::Tensor& out, at::Tensor& residual, const at::Tensor& w_next, double eps,
                     const c10::optional<at::Tensor>& w_post, double mult, const c10::optional<at::Tensor>& table,
                     const c10::optional<at::Tensor>& ids, double table_scale, const c10::optional<at::Tensor>& a,
                     const c10::optional<at::Tensor>& a_w, const c10::optional<at::Tensor>& b,
                     const c10::optional<at::Tensor>& b_w, double a_scale, double b_scale,
                     const c10::optional<at::Tensor>& ye, const c10::optional<at::Tensor>& pair_slot,
                     const c10::optional<at::Tensor>& wts, const c10::optional<at::Tensor>& shared,
                     const c10::optional<at::Tensor>& gate) {
  CHECK_DEV(out); CHECK_CONTIG(out); CHECK_F32(residual); CHECK_F32(w_next);
  const bool f32 = is_f32(out, "sandwich_update");
  TORCH_CHECK(residual.dim() == 2 && out.sizes() == residual.sizes());
  const long T = residual.size(0), H = residual.size(1);
  TORCH_CHECK(H >= 1 && H <= hipserve::sandwich_update_max_width() && w_next.numel() == H, "sandwich_update: width");
  auto rows = [&](const at::Tensor& x) {
    TORCH_CHECK(x.scalar_type() == out.scalar_type() && x.is_contiguous() && x.sizes() == residual.sizes(),
                "sandwich_update: rows of the activation type");
  };
  auto weight = [&](const c10::optional<at::Tensor>& x) {
    TORCH_CHECK(x.has_value() && x->scalar_type() == at::kFloat && x->is_contiguous() && x->numel() == H,
                "sandwich_update: a weight per channel");
  };
  hipserve::SandwichUpdate p{};
  p.out = out.data_ptr(); p.residual = residual.data_ptr<float>(); p.w_next = w_next.data_ptr<float>();
  p.T = T; p.H = H; p.eps = (float)eps; p.mult = (float)mult;
  p.table_scale = (float)table_scale; p.a_scale = (float)a_scale; p.b_scale = (float)b_scale;
  if (table.has_value()) {
    TORCH_CHECK(table->scalar_type() == out.scalar_type() && table->is_contiguous() && table->dim() == 2 &&
                table->size(1) == H && table->size(0) >= 1 && ids.has_value() && ids->scalar_type() == at::kLong &&
                ids->is_contiguous() && ids->numel() >= T, "sandwich_update: table [vocab, H] and one id per row");
    p.table = table->data_ptr(); p.ids = ids->data_ptr<long>(); p.vocab = table->size(0);
  }
  TORCH_CHECK(!(a.has_value() && ye.has_value()) && (a.has_value() || !b.has_value()), "sandwich_update: one addend");
  if (a.has_value() || ye.has_value()) {
    weight(w_post);
    p.w_post = w_post->data_ptr<float>();
  }
  if (a.has_value()) {
    rows(*a);
    p.a = a->data_ptr();
    if (b.has_value()) {
      rows(*b); weight(a_w); weight(b_w);
      p.b = b->data_ptr(); p.a_w = a_w->data_ptr<float>(); p.b_w = b_w->data_ptr<float>();
    }
  }
  if (ye.has_value()) {
    TORCH_CHECK(ye->scalar_type() == out.scalar_type() && ye->is_contiguous() && ye->dim() == 2 && ye->size(1) == H &&
                pair_slot.has_value() && wts.has_value(), "sandwich_update: a mixture's parts");
    CHECK_I32(*pair_slot); CHECK_F32(*wts);
    TORCH_CHECK(wts->dim() == 2 && wts->size(0) == T && pair_slot->numel() >= wts->numel());
    p.ye = ye->data_ptr(); p.pair_slot = pair_slot->data_ptr<int>(); p.wts = wts->data_ptr<float>(); p.top = wts->size(1);
    if (shared.has_value()) { rows(*shared); p.shared = shared->data_ptr(); }
    if (gate.has_value()) {
      TORCH_CHECK(shared.has_value() && gate->scalar_type() == at::kFloat && gate->dim() == 2 && gate->size(0) == T &&
                  gate->size(1) == 1, "sandwich_update: the shared expert's gate is fp32 [T, 1]");
      p.gate = gate->data_ptr<float>(); p.gate_ld = gate->stride(0);
    }
  }
  c10::hip::HIPGuardMasqueradingAsCUDA g(out.device());
  hipserve::launch_sandwich_update(p, f32, cur_stream());
}

void delta_rule(at::Tensor& out, at::Tensor& S, const at::Tensor& proj, const at::Tensor& wl, const at::Tensor& a_b,
                const at::Tensor& w0, const at::Tensor& norm_w, const at::Tensor& seq_cu, const at::Tensor& seq_ctx,
                const at::Tensor& seq_state, at::Tensor& scratch, int64_t heads, int64_t dim, double eps,
                double out_scale) {
  CHECK_DEV(proj); CHECK_F32(S); CHECK_F32(wl); CHECK_F32(a_b); CHECK_F32(w0); CHECK_F32(norm_w); CHECK_F32(scratch);
  CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  const bool f32 = is_f32(proj, "delta_rule");
  TORCH_CHECK(out.scalar_type() == proj.scalar_type());
  TORCH_CHECK(heads >= 1 && dim >= 1 && dim <= hipserve::delta_max_dim(), "delta_rule: sizes");
  const long T = proj.size(0), nseq = seq_ctx.numel(), N = heads * dim;
  TORCH_CHECK(rows2d(proj) && proj.size(1) >= 5 * N && rows2d(out) && out.size(0) == T && out.size(1) == N);
  TORCH_CHECK(S.dim() == 4 && S.size(1) == heads && S.size(2) == dim && S.size(3) == dim);
  TORCH_CHECK(wl.numel() == T * N && a_b.numel() == N && w0.numel() == N && norm_w.numel() == N);
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535 &&
              scratch.numel() >= T * 7 * N);
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_delta_rule(out.data_ptr(), out.stride(0), S.data_ptr<float>(), proj.data_ptr(), proj.stride(0),
                              wl.data_ptr<float>(), a_b.data_ptr<float>(), w0.data_ptr<float>(),
                              norm_w.data_ptr<float>(), seq_cu.data_ptr<int>(), seq_ctx.data_ptr<int>(),
                              seq_state.data_ptr<int>(), nseq, T, scratch.data_ptr<float>(), heads, dim, (float)eps,
                              (float)out_scale, f32, cur_stream());
}

void add_normed(at::Tensor& out, at::Tensor& residual, const at::Tensor& w, double eps,
                const c10::optional<at::Tensor>& y, const c10::optional<at::Tensor>& ye,
                const c10::optional<at::Tensor>& pair_slot, const c10::optional<at::Tensor>& ids,
                const c10::optional<at::Tensor>& wts, int64_t E, const c10::optional<at::Tensor>& h,
                const c10::optional<at::Tensor>& shared) {
  CHECK_DEV(out); CHECK_CONTIG(out); CHECK_F32(residual); CHECK_F32(w);
  const bool f32 = is_f32(out, "add_normed");
  TORCH_CHECK(residual.dim() == 2 && out.sizes() == residual.sizes());
  const long T = residual.size(0), H = residual.size(1);
  TORCH_CHECK(w.numel() == H && H <= 15000, "add_normed shape");
  auto same = [&](const at::Tensor& t) { return t.scalar_type() == out.scalar_type() && t.is_contiguous(); };
  long top = 0;
  if (y.has_value()) {
    TORCH_CHECK(same(*y) && y->sizes() == residual.sizes());
  } else {
    TORCH_CHECK(ye.has_value() && pair_slot.has_value() && ids.has_value() && wts.has_value() && h.has_value(),
                "add_normed: an addend or the parts of a mixture's output");
    CHECK_I32(*pair_slot); CHECK_I32(*ids); CHECK_F32(*wts);
    TORCH_CHECK(ids->dim() == 2 && ids->size(0) == T && wts->sizes() == ids->sizes());
    top = ids->size(1);
    TORCH_CHECK(same(*ye) && ye->dim() == 2 && ye->size(1) == H && pair_slot->numel() >= T * top);
    TORCH_CHECK(same(*h) && h->sizes() == residual.sizes() && h->data_ptr() != out.data_ptr());
    if (shared.has_value()) TORCH_CHECK(same(*shared) && shared->sizes() == residual.sizes());
  }
  c10::hip::HIPGuardMasqueradingAsCUDA g(out.device());
  hipserve::launch_add_normed(out.data_ptr(), residual.data_ptr<float>(), w.data_ptr<float>(), T, H, (float)eps,
                              opt_ptr(y), opt_ptr(ye), (const int*)opt_ptr(pair_slot), (const int*)opt_ptr(ids),
                              (const float*)opt_ptr(wts), top, E, opt_ptr(h), y.has_value() ? nullptr : opt_ptr(shared),
                              f32, cur_stream());
}

void token_shift(at::Tensor& out, const at::Tensor& x, at::Tensor& state, const at::Tensor& mu,
                 const at::Tensor& seq_cu, const at::Tensor& seq_ctx, const at::Tensor& seq_state) {
  CHECK_DEV(x); CHECK_CONTIG(out); CHECK_F32(x); CHECK_F32(state); CHECK_F32(mu);
  CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  const bool f32 = is_f32(out, "token_shift");
  TORCH_CHECK(x.dim() == 2 && out.dim() == 3 && mu.dim() == 2 && state.dim() == 2);
  const long T = x.size(0), H = x.size(1), nb = out.size(0), nseq = seq_ctx.numel();
  TORCH_CHECK(out.size(1) == T && out.size(2) == H && mu.size(0) == nb && mu.size(1) == H && state.size(1) == H);
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535);
  c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  hipserve::launch_token_shift(out.data_ptr(), x.data_ptr<float>(), state.data_ptr<float>(), mu.data_ptr<float>(),
                               seq_cu.data_ptr<int>(), seq_ctx.data_ptr<int>(), seq_state.data_ptr<int>(), nseq, T, H,
                               nb, f32, cur_stream());
}

void wkv(at::Tensor& out, at::Tensor& S, const at::Tensor& proj, const at::Tensor& wl, const at::Tensor& w0,
         const at::Tensor& u, const at::Tensor& norm_w, const at::Tensor& seq_cu, const at::Tensor& seq_ctx,
         const at::Tensor& seq_state, at::Tensor& scratch, int64_t heads, int64_t dim, double eps) {
  CHECK_DEV(proj); CHECK_CONTIG(proj); CHECK_CONTIG(out); CHECK_F32(S); CHECK_F32(wl); CHECK_F32(w0); CHECK_F32(u);
  CHECK_F32(norm_w); CHECK_F32(scratch); CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  const bool f32 = is_f32(proj, "wkv");
  TORCH_CHECK(out.scalar_type() == proj.scalar_type());
  TORCH_CHECK(heads >= 1 && dim >= 1 && dim <= hipserve::delta_max_dim(), "wkv: sizes");
  const long N = heads * dim, nseq = seq_ctx.numel();
  TORCH_CHECK(proj.dim() == 3 && proj.size(0) == 4 && proj.size(2) == N);
  const long T = proj.size(1);
  TORCH_CHECK(out.numel() == T * N && wl.numel() == T * N && w0.numel() == N && u.numel() == N && norm_w.numel() == N);
  TORCH_CHECK(S.dim() == 4 && S.size(1) == heads && S.size(2) == dim && S.size(3) == dim);
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535 &&
              scratch.numel() >= T * (5 * N + heads));
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_wkv(out.data_ptr(), S.data_ptr<float>(), proj.data_ptr(), wl.data_ptr<float>(),
                       w0.data_ptr<float>(), u.data_ptr<float>(), norm_w.data_ptr<float>(), seq_cu.data_ptr<int>(),
                       seq_ctx.data_ptr<int>(), seq_state.data_ptr<int>(), nseq, T, scratch.data_ptr<float>(), heads,
                       dim, (float)eps, f32, cur_stream());
}

void wkv_step(at::Tensor& out, at::Tensor& S, const at::Tensor& proj, const at::Tensor& low, const at::Tensor& w2,
              const at::Tensor& w0, const at::Tensor& u, const at::Tensor& norm_w, const at::Tensor& seq_cu,
              const at::Tensor& seq_ctx, const at::Tensor& seq_state, int64_t heads, int64_t dim, double eps) {
  CHECK_DEV(proj); CHECK_CONTIG(proj); CHECK_CONTIG(out); CHECK_CONTIG(low); CHECK_CONTIG(w2); CHECK_F32(S); CHECK_F32(w0);
  CHECK_F32(u); CHECK_F32(norm_w); CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  const bool f32 = is_f32(proj, "wkv_step");
  TORCH_CHECK(out.scalar_type() == proj.scalar_type() && low.scalar_type() == proj.scalar_type() &&
              w2.scalar_type() == proj.scalar_type());
  TORCH_CHECK(heads >= 1 && dim >= 1 && dim <= 256, "wkv_step: sizes");
  const long N = heads * dim, nseq = seq_ctx.numel();
  TORCH_CHECK(proj.dim() == 3 && proj.size(0) == 4 && proj.size(2) == N);
  const long T = proj.size(1);
  TORCH_CHECK(low.dim() == 2 && low.size(0) == T && w2.dim() == 2 && w2.size(0) == N && w2.size(1) == low.size(1));
  const long rank = low.size(1);
  TORCH_CHECK((rank + 3 * dim) * 4 <= 60 * 1024, "wkv_step: bottleneck too wide");
  TORCH_CHECK(out.numel() == T * N && w0.numel() == N && u.numel() == N && norm_w.numel() == N);
  TORCH_CHECK(S.dim() == 4 && S.size(1) == heads && S.size(2) == dim && S.size(3) == dim);
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535);
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_wkv_step(out.data_ptr(), S.data_ptr<float>(), proj.data_ptr(), T, low.data_ptr(), w2.data_ptr(), rank,
                            w0.data_ptr<float>(), u.data_ptr<float>(), norm_w.data_ptr<float>(),
                            seq_cu.data_ptr<int>(), seq_ctx.data_ptr<int>(), seq_state.data_ptr<int>(), nseq, heads,
                            dim, (float)eps, f32, cur_stream());
}

}  // namespace

TORCH_LIBRARY(hipserve_delta, m) {
  def_window_ops(m);
  m.def("scaled_add_group_rmsnorm(Tensor(a!) out, Tensor(b!) residual, Tensor w, int groups, float eps, Tensor? mix, "
        "Tensor? ls1, Tensor? y, Tensor? pair_slot, int top, Tensor? ls2, Tensor? extra) -> ()");
  m.def("gated_delta(Tensor(a!) y, Tensor(b!) S, Tensor(c!) conv_state, Tensor proj, Tensor conv_w, Tensor a_log, "
        "Tensor dt_bias, Tensor norm_w, Tensor? decay, Tensor? gate, Tensor seq_cu, Tensor seq_ctx, Tensor seq_state, "
        "Tensor(d!) scratch, int heads, int kv_heads, int dim, int vdim, int taps, float eps, int off_a, int off_g, int off_b, "
        "bool channel, bool silu, Tensor(e!)? chunks=None) -> ()");
  m.def("delta_chunk_floats(int T, int nseq, int heads, int dim, int vdim) -> int", &delta_chunk_floats);
  m.def("gated_delta_step(Tensor(a!) y, Tensor(b!) S, Tensor(c!) conv_state, Tensor proj, Tensor conv_w, Tensor a_log, "
        "Tensor dt_bias, Tensor norm_w, Tensor? a2, Tensor? g2, Tensor seq_cu, Tensor seq_ctx, Tensor seq_state, int heads, "
        "int kv_heads, int dim, int vdim, int taps, float eps, int off_a, int off_g, int off_b, bool channel, bool silu) -> ()");
  m.def("sandwich_update(Tensor(a!) out, Tensor(b!) residual, Tensor w_next, float eps, Tensor? w_post, float mult, "
        "Tensor? table, Tensor? ids, float table_scale, Tensor? a, Tensor? a_w, Tensor? b, Tensor? b_w, float a_scale, "
        "float b_scale, Tensor? ye, Tensor? pair_slot, Tensor? wts, Tensor? shared, Tensor? gate) -> ()");
  m.def("delta_rule(Tensor(a!) out, Tensor(b!) S, Tensor proj, Tensor wl, Tensor a_b, Tensor w0, Tensor norm_w, "
        "Tensor seq_cu, Tensor seq_ctx, Tensor seq_state, Tensor(c!) scratch, int heads, int dim, float eps, "
        "float out_scale) -> ()");
  m.def("add_normed(Tensor(a!) out, Tensor(b!) residual, Tensor w, float eps, Tensor? y, Tensor? ye, Tensor? pair_slot, "
        "Tensor? ids, Tensor? wts, int E, Tensor? h, Tensor? shared) -> ()");
  m.def("token_shift(Tensor(a!) out, Tensor x, Tensor(b!) state, Tensor mu, Tensor seq_cu, Tensor seq_ctx, "
        "Tensor seq_state) -> ()");
  m.def("wkv(Tensor(a!) out, Tensor(b!) S, Tensor proj, Tensor wl, Tensor w0, Tensor u, Tensor norm_w, Tensor seq_cu, "
        "Tensor seq_ctx, Tensor seq_state, Tensor(c!) scratch, int heads, int dim, float eps) -> ()");
  m.def("wkv_step(Tensor(a!) out, Tensor(b!) S, Tensor proj, Tensor low, Tensor w2, Tensor w0, Tensor u, Tensor norm_w, "
        "Tensor seq_cu, Tensor seq_ctx, Tensor seq_state, int heads, int dim, float eps) -> ()");
}

TORCH_LIBRARY_IMPL(hipserve_delta, CUDA, m) {
  impl_window_ops(m);
  m.impl("scaled_add_group_rmsnorm", &scaled_add_group_rmsnorm);
  m.impl("gated_delta", &gated_delta);
  m.impl("gated_delta_step", &gated_delta_step);
  m.impl("sandwich_update", &sandwich_update);
  m.impl("delta_rule", &delta_rule);
  m.impl("add_normed", &add_normed);
  m.impl("token_shift", &token_shift);
  m.impl("wkv", &wkv);
  m.impl("wkv_step", &wkv_step);
}
