// torch.ops.hipserve_stream.* — the kernels of layer-list decoders with several residual streams: the streams' update
// fused with the next sublayer's input and norm (streams.hip), lightning attention (lightning.hip), window attention
// (window_attention*.hip), the router (router.hip), the experts' GEMMs (expert_ffn.hip, moe.hip) and the activations
// (elementwise.hip). Built as their own library (hipserve/_C_stream.so) so that a model compiles only what it runs.
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

void stream_update(at::Tensor& out, const c10::optional<at::Tensor>& dst, const c10::optional<at::Tensor>& src,
                   const c10::optional<at::Tensor>& table, const c10::optional<at::Tensor>& ids, double table_scale,
                   const at::Tensor& coef,
                   const at::Tensor& w, double eps, const c10::optional<at::Tensor>& y1,
                   const c10::optional<at::Tensor>& y2, const c10::optional<at::Tensor>& ye,
                   const c10::optional<at::Tensor>& pair_slot, const c10::optional<at::Tensor>& wts, int64_t top,
                   const c10::optional<at::Tensor>& shared, const c10::optional<at::Tensor>& gate) {
  CHECK_DEV(out); CHECK_CONTIG(out); CHECK_F32(coef); CHECK_F32(w);
  const bool f32 = is_f32(out, "stream_update");
  TORCH_CHECK(out.dim() == 2 && src.has_value() != table.has_value(), "stream_update: streams or an embedding table");
  const long T = out.size(0), H = out.size(1);
  const bool one_row = !src.has_value() || src->dim() == 2;
  long S = 1;
  while (S * S + 3 * S < coef.numel()) ++S;
  TORCH_CHECK(S * S + 3 * S == coef.numel() && S <= hipserve::stream_update_max_streams(),
              "stream_update: coefficients of at most ", hipserve::stream_update_max_streams(), " streams");
  TORCH_CHECK(H <= hipserve::stream_update_max_width(), "stream_update: width");
  TORCH_CHECK(w.numel() == H);
  if (src.has_value()) {
    CHECK_F32(*src);
    TORCH_CHECK((src->dim() == 2 || src->dim() == 3) && src->size(0) == T && src->size(-1) == H &&
                (one_row || src->size(1) == S), "stream_update: src [T, S, H] or [T, H]");
  } else {
    TORCH_CHECK(table->scalar_type() == out.scalar_type() && table->is_contiguous() && table->dim() == 2 &&
                table->size(1) == H && table->size(0) >= 1 && ids.has_value() && ids->scalar_type() == at::kLong &&
                ids->is_contiguous() && ids->numel() >= T, "stream_update: table [vocab, H] and one id per row");
  }
  if (dst.has_value()) {
    CHECK_F32(*dst);
    TORCH_CHECK(dst->dim() == 3 && dst->size(0) == T && dst->size(1) == S && dst->size(2) == H);
  }
  auto same = [&](const at::Tensor& t) { return t.scalar_type() == out.scalar_type() && t.is_contiguous(); };
  if (y1.has_value()) TORCH_CHECK(same(*y1) && y1->sizes() == out.sizes());
  if (y2.has_value()) TORCH_CHECK(same(*y2) && y2->sizes() == out.sizes() && !ye.has_value());
  if (ye.has_value()) {
    TORCH_CHECK(pair_slot.has_value() && top >= 1 && same(*ye) && ye->dim() == 2 && ye->size(1) == H);
    CHECK_I32(*pair_slot);
    TORCH_CHECK(pair_slot->numel() >= T * top);
    if (wts.has_value()) {
      CHECK_F32(*wts);
      TORCH_CHECK(wts->numel() == T * top);
    }
    if (shared.has_value()) TORCH_CHECK(same(*shared) && shared->sizes() == out.sizes());
    if (gate.has_value())
      TORCH_CHECK(shared.has_value() && gate->scalar_type() == at::kFloat && gate->dim() == 2 && gate->size(0) == T &&
                  gate->size(1) == 1, "stream_update: the shared expert's gate is fp32 [T, 1]");
  }
  c10::hip::HIPGuardMasqueradingAsCUDA g(out.device());
  hipserve::launch_stream_update(
      out.data_ptr(), dst.has_value() ? dst->data_ptr<float>() : nullptr, (const float*)opt_ptr(src), one_row,
      opt_ptr(table), table.has_value() ? ids->data_ptr<long>() : nullptr, table.has_value() ? table->size(0) : 0,
      (float)table_scale, coef.data_ptr<float>(), S, w.data_ptr<float>(), T, H, (float)eps, opt_ptr(y1), opt_ptr(y2), opt_ptr(ye),
      (const int*)opt_ptr(pair_slot), (const float*)opt_ptr(wts), top, ye.has_value() ? opt_ptr(shared) : nullptr,
      ye.has_value() ? (const float*)opt_ptr(gate) : nullptr, gate.has_value() ? gate->stride(0) : 0, f32, cur_stream());
}

bool lightning_mfma_ok(int64_t dim, int64_t vdim, int64_t ld, int64_t offset) {
  return hipserve::lightning_mfma_ok(dim, vdim, ld, offset);
}

void lightning(at::Tensor& out, at::Tensor& S, const at::Tensor& proj, const at::Tensor& powers,
               const at::Tensor& norm_w, const at::Tensor& seq_cu, const at::Tensor& seq_ctx,
               const at::Tensor& seq_state, at::Tensor& scratch, int64_t npf, int64_t pf_rows, int64_t heads, int64_t dim,
               int64_t vdim, double eps, double out_scale, bool mfma, int64_t nseg, int64_t seg_len,
               int64_t max_q) {
  CHECK_DEV(proj); CHECK_F32(S); CHECK_F32(powers); CHECK_F32(norm_w); CHECK_F32(scratch);
  CHECK_I32(seq_cu); CHECK_I32(seq_ctx); CHECK_I32(seq_state);
  const bool f32 = is_f32(proj, "lightning");
  TORCH_CHECK(heads >= 1 && dim >= 1 && dim <= hipserve::lightning_max_dim() && vdim >= 1, "lightning: sizes");
  const long T = proj.size(0), nseq = seq_ctx.numel(), N = heads * vdim;
  TORCH_CHECK(rows2d(proj) && proj.size(1) >= 2 * heads * dim + 2 * N);
  TORCH_CHECK(out.scalar_type() == proj.scalar_type() && rows2d(out) && out.size(0) == T && out.size(1) == N);
  TORCH_CHECK(powers.dim() == 2 && powers.size(0) == heads && powers.size(1) == hipserve::lightning_powers());
  TORCH_CHECK(norm_w.numel() == N && S.dim() == 4 && S.size(1) == heads && S.size(2) == dim && S.size(3) == vdim);
  TORCH_CHECK(seq_cu.numel() == nseq + 1 && seq_state.numel() >= nseq && nseq <= 65535);
  TORCH_CHECK(0 <= npf && npf <= nseq && 0 <= pf_rows && pf_rows + (nseq - npf) <= T,
              "lightning: prompt portions first, then one row per sequence");
  TORCH_CHECK(!mfma || (!f32 && hipserve::lightning_mfma_ok(dim, vdim, proj.stride(0), proj.storage_offset())),
              "lightning: the chunk kernel takes bf16 and heads of multiples of 8 elements, keys up to 128");
  TORCH_CHECK(nseg >= 1 && (nseg == 1 || (seg_len > 0 && seg_len % 64 == 0 && nseg * seg_len >= max_q)) && npf * nseg <= 65535,
              "lightning: segments of a multiple of 64 tokens that cover the longest portion");
  TORCH_CHECK(npf == 0 || scratch.numel() >= T * N + (!mfma ? pf_rows * heads * (2 * dim + vdim)
                                                          : nseg > 1 ? npf * nseg * heads * dim * vdim : 0));
  TORCH_CHECK(scratch.numel() >= T * N);
  c10::hip::HIPGuardMasqueradingAsCUDA g(proj.device());
  hipserve::launch_lightning(out.data_ptr(), out.stride(0), S.data_ptr<float>(), proj.data_ptr(), proj.stride(0),
                             powers.data_ptr<float>(), norm_w.data_ptr<float>(), seq_cu.data_ptr<int>(),
                             seq_ctx.data_ptr<int>(), seq_state.data_ptr<int>(), nseq, npf, T, pf_rows,
                             scratch.data_ptr<float>(), heads, dim, vdim, (float)eps, (float)out_scale, mfma, nseg, seg_len, f32,
                             cur_stream());
}

}  // namespace

TORCH_LIBRARY(hipserve_stream, m) {
  def_window_ops(m);
  m.def("stream_update(Tensor(a!) out, Tensor(b!)? dst, Tensor? src, Tensor? table, Tensor? ids, float table_scale, Tensor coef, Tensor w, float eps, Tensor? y1, "
        "Tensor? y2, Tensor? ye, Tensor? pair_slot, Tensor? wts, int top, Tensor? shared, Tensor? gate) -> ()");
  m.def("lightning(Tensor(a!) out, Tensor(b!) S, Tensor proj, Tensor powers, Tensor norm_w, Tensor seq_cu, "
        "Tensor seq_ctx, Tensor seq_state, Tensor(c!) scratch, int npf, int pf_rows, int heads, int dim, int vdim, "
        "float eps, float out_scale, bool mfma, int nseg, int seg_len, int max_q) -> ()");
  m.def("lightning_mfma_ok(int dim, int vdim, int ld, int offset) -> bool", &lightning_mfma_ok);
}

TORCH_LIBRARY_IMPL(hipserve_stream, CUDA, m) {
  impl_window_ops(m);
  m.impl("stream_update", &stream_update);
  m.impl("lightning", &lightning);
}
