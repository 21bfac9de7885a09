// Torch bindings (part of `_C_seq`): tanh norms around sublayers, attention
// inputs normed over the whole projection, soft-capped attention of any shape,
// the gated delta rule, clamped gates, f32 router products.  Every shape the
// kernels assume is checked here, on the host, before a launch.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <hip/hip_bf16.h>

template <typename T>
void launch_stream_add_tanh_norm(float*, const T*, const T*, float, const float*, const float*,
                                 float, const float*, const float*, T*, int, int, hipStream_t);
template <typename T>
void launch_wide_norm(T*, const T*, long, const float*, const float*, const float*, const T*,
                      float, T*, T*, const long*, int, int, int, int, float, hipStream_t);
template <typename T>
void launch_clamped_glu(T*, const T*, float, const float*, int, long, hipStream_t);
template <typename T, typename W>
void launch_router_logits(float*, const T*, long, const W*, int, int, int, hipStream_t);
template <typename T, typename W>
void launch_route_experts(float*, int*, float*, const T*, long, const W*, const float*, int,
                          int, int, int, int, int, int, float, hipStream_t);
template <typename T>
void launch_scale_logits(float*, const T*, float, long, hipStream_t);
template <typename T>
void launch_capped_attention(T*, long, const T*, long, const T*, const T*, const int*, int,
                             const int*, const int*, int, float, int, int, int, int, int, int,
                             int, int, const float*, float, hipStream_t);
template <typename T>
void launch_delta_scan(float*, const T*, long, const T*, long, const T*, long, const T*, long,
                       const T*, long, const float*, const float*, float, float*, const int*,
                       const int*, const int*, int, int, int, int, int, int, float*, float*,
                       int, hipStream_t);
int delta_fused_columns(int dim, int vdim);
template <typename T>
void launch_delta_fused(T*, const T*, long, const T*, long, const T*, long, const T*, long,
                        const T*, long, const float*, const float*, const T*, long,
                        const float*, float, float, float*, const int*, const int*, const int*,
                        int, int, int, int, int, int, hipStream_t);
template <typename T>
void launch_gated_group_norm(T*, const float*, const T*, long, const float*, float, int, int,
                             int, int, hipStream_t);

namespace {

using OptTensor = c10::optional<torch::Tensor>;

hipStream_t stream() { return at::hip::getCurrentHIPStream().stream(); }

template <typename T>
T* ptr(const torch::Tensor& t) {
  return reinterpret_cast<T*>(t.data_ptr());
}
template <typename T>
T* optr(const OptTensor& t) {
  return t.has_value() ? ptr<T>(t.value()) : nullptr;
}

#define DISPATCH_F32_BF16(DTYPE, BODY)                                  \
  switch (DTYPE) {                                                      \
    case at::ScalarType::BFloat16: {                                    \
      using scalar_t = __hip_bfloat16;                                  \
      BODY;                                                             \
      break;                                                            \
    }                                                                   \
    case at::ScalarType::Float: {                                       \
      using scalar_t = float;                                           \
      BODY;                                                             \
      break;                                                            \
    }                                                                   \
    default:                                                            \
      TORCH_CHECK(false, "this op takes float32 or bfloat16 tensors");  \
  }

void check_type(const torch::Tensor& t, at::ScalarType dt, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == dt && t.is_contiguous(), what,
              " must be a contiguous GPU tensor of the expected type");
}
void check_f32(const torch::Tensor& t, long numel, const char* what) {
  check_type(t, at::ScalarType::Float, what);
  TORCH_CHECK(numel < 0 || t.numel() == numel, what, " has the wrong size");
}
void check_f32(const OptTensor& t, long numel, const char* what) {
  if (t.has_value()) check_f32(t.value(), numel, what);
}
bool aligned16(const torch::Tensor& t) {
  return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0;
}

// rows with unit stride, strided one after the other
void check_rows(const torch::Tensor& t, at::ScalarType dt, long rows, long cols,
                const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.scalar_type() == dt && t.size(0) == rows &&
                  t.size(1) == cols && (cols == 1 || t.stride(1) == 1), what,
              " must be rows of the expected type and size");
}

// heads of one row laid out [heads, size] with unit stride, rows strided
void check_heads_view(const torch::Tensor& t, at::ScalarType dt, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 3 && t.stride(2) == 1 &&
                  t.stride(1) == t.size(2) && t.scalar_type() == dt, what,
              " must be [rows, heads, size] rows");
}

int check_seqs(const torch::Tensor& loc, const torch::Tensor& seq_lens,
               const torch::Tensor& slots) {
  check_type(loc, at::ScalarType::Int, "seq_start_loc");
  check_type(seq_lens, at::ScalarType::Int, "seq_lens");
  check_type(slots, at::ScalarType::Int, "state_slots");
  const int nseq = seq_lens.numel();
  TORCH_CHECK(loc.numel() == nseq + 1 && slots.numel() == nseq,
              "seq_start_loc / seq_lens / state_slots do not fit each other");
  return nseq;
}

void check_cache(const torch::Tensor& k, const torch::Tensor& v, at::ScalarType dt) {
  check_type(k, dt, "k_cache");
  check_type(v, dt, "v_cache");
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.size(0) == v.size(0) &&
              k.size(1) == v.size(1) && k.size(2) == v.size(2) && k.size(1) >= 1,
              "key and value caches do not fit each other");
}

void stream_add_tanh_norm(torch::Tensor x, OptTensor a, OptTensor b, double alpha, OptTensor w,
                          OptTensor bias, double next_alpha, OptTensor next_w,
                          OptTensor next_bias, OptTensor next_out) {
  check_f32(x, -1, "x");
  TORCH_CHECK(x.dim() == 2);
  const int rows = x.size(0), width = x.size(1);
  for (const OptTensor* t : {&w, &bias, &next_w, &next_bias}) check_f32(*t, width, "norm");
  TORCH_CHECK(a.has_value() || !b.has_value());
  TORCH_CHECK(a.has_value() || next_out.has_value(), "nothing to do");
  TORCH_CHECK(!a.has_value() || (w.has_value() && bias.has_value()), "norm missing");
  TORCH_CHECK(!next_out.has_value() || (next_w.has_value() && next_bias.has_value()),
              "next norm missing");
  const auto dt = a.has_value() ? a.value().scalar_type() : next_out.value().scalar_type();
  for (const OptTensor* t : {&a, &b, &next_out})
    if (t->has_value()) {
      check_type(t->value(), dt, "rows");
      TORCH_CHECK(t->value().numel() == x.numel(), "rows must match x");
    }
  TORCH_CHECK(rows < 4 * 65535, "too many rows");
  if (rows == 0) return;
  DISPATCH_F32_BF16(dt, {
    launch_stream_add_tanh_norm<scalar_t>(
        ptr<float>(x), optr<scalar_t>(a), optr<scalar_t>(b), (float)alpha, optr<float>(w),
        optr<float>(bias), (float)next_alpha, optr<float>(next_w), optr<float>(next_bias),
        optr<scalar_t>(next_out), rows, width, stream());
  });
}

void wide_norm_cache_write(torch::Tensor q_out, torch::Tensor proj, OptTensor bias,
                           int64_t kv_heads, int64_t vdim, double eps, torch::Tensor qw,
                           torch::Tensor kw, OptTensor v_first, double v_mix,
                           torch::Tensor k_cache, torch::Tensor v_cache,
                           torch::Tensor slot_mapping) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  const auto dt = proj.scalar_type();
  check_type(q_out, dt, "q_out");
  TORCH_CHECK(q_out.dim() == 3 && q_out.size(0) == proj.size(0));
  const int rows = proj.size(0);
  const long dim = q_out.size(2), nq = q_out.size(1) * dim, nk = kv_heads * dim;
  const long nv = kv_heads * vdim;
  TORCH_CHECK(nq >= 1 && nk >= 1 && nv >= 1 && proj.size(1) == nq + nk + nv,
              "projected rows are [q | k | v]");
  check_f32(bias, nq + nk + nv, "bias");
  check_f32(qw, nq, "query norm");
  check_f32(kw, nk, "key norm");
  check_cache(k_cache, v_cache, dt);
  TORCH_CHECK(k_cache.size(2) == kv_heads && k_cache.size(3) == dim &&
              v_cache.size(3) == vdim, "cache shape");
  if (v_first.has_value()) {
    check_type(v_first.value(), dt, "v_first");
    TORCH_CHECK(v_first.value().sizes() == v_cache.sizes(),
                "the earlier layer's value cache must have this layer's shape");
  }
  check_type(slot_mapping, at::ScalarType::Long, "slot_mapping");
  TORCH_CHECK(slot_mapping.numel() == rows);
  if (rows == 0) return;
  DISPATCH_F32_BF16(dt, {
    launch_wide_norm<scalar_t>(
        ptr<scalar_t>(q_out), ptr<scalar_t>(proj), (long)proj.stride(0), optr<float>(bias),
        ptr<float>(qw), ptr<float>(kw), optr<scalar_t>(v_first), (float)v_mix,
        ptr<scalar_t>(k_cache), ptr<scalar_t>(v_cache), ptr<long>(slot_mapping), rows, (int)nq,
        (int)nk, (int)nv, (float)eps, stream());
  });
}

void capped_attention(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                      torch::Tensor v_cache, torch::Tensor block_tables,
                      OptTensor query_start_loc, torch::Tensor seq_lens, double scale,
                      int64_t window, OptTensor sinks, double softcap) {
  const auto dt = q.scalar_type();
  check_heads_view(q, dt, "q");
  check_heads_view(out, dt, "out");
  check_cache(k_cache, v_cache, dt);
  TORCH_CHECK(window >= 0 && softcap >= 0.0, "window and softcap");
  const int rows = q.size(0), heads = q.size(1), dim = q.size(2);
  const int kv_heads = k_cache.size(2), vdim = v_cache.size(3);
  TORCH_CHECK(k_cache.size(3) == dim && kv_heads >= 1 && heads % kv_heads == 0,
              "cache shape");
  TORCH_CHECK(vdim <= 1024, "value size above 1024 is not supported");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads && out.size(2) == vdim);
  check_f32(sinks, heads, "sinks");
  check_type(seq_lens, at::ScalarType::Int, "seq_lens");
  const int nseq = seq_lens.numel();
  TORCH_CHECK(block_tables.is_cuda() && block_tables.scalar_type() == at::ScalarType::Int &&
              block_tables.dim() == 2 && block_tables.stride(1) == 1 &&
              block_tables.size(0) >= nseq, "block tables");
  if (query_start_loc.has_value()) {
    check_type(query_start_loc.value(), at::ScalarType::Int, "query_start_loc");
    TORCH_CHECK(query_start_loc.value().numel() == nseq + 1);
  } else {
    TORCH_CHECK(rows == nseq, "one query row per sequence expected");
  }
  if (rows == 0 || nseq == 0) return;
  const int vec_ok = dim % (dt == at::ScalarType::Float ? 4 : 8) == 0 && aligned16(k_cache);
  DISPATCH_F32_BF16(dt, {
    launch_capped_attention<scalar_t>(
        ptr<scalar_t>(out), (long)out.stride(0), ptr<scalar_t>(q), (long)q.stride(0),
        ptr<scalar_t>(k_cache), ptr<scalar_t>(v_cache), ptr<int>(block_tables),
        (int)block_tables.stride(0), optr<int>(query_start_loc), ptr<int>(seq_lens), nseq,
        (float)scale, rows, heads, kv_heads, dim, vdim, (int)k_cache.size(1), vec_ok,
        (int)window, optr<float>(sinks), (float)softcap, stream());
  });
}

// shapes shared by the two delta-rule entries; returns the number of sequences
int check_delta(const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                const torch::Tensor& b_pre, const torch::Tensor& a_pre,
                const torch::Tensor& a_log, const torch::Tensor& dt_bias,
                const torch::Tensor& state, const torch::Tensor& loc,
                const torch::Tensor& seq_lens, const torch::Tensor& slots) {
  const auto dt = q.scalar_type();
  check_heads_view(q, dt, "q");
  check_heads_view(k, dt, "k");
  check_heads_view(v, dt, "v");
  const long rows = q.size(0), groups = q.size(1), dim = q.size(2);
  const long heads = v.size(1), vdim = v.size(2);
  TORCH_CHECK(k.sizes() == q.sizes() && v.size(0) == rows && groups >= 1 &&
              heads % groups == 0, "q / k heads must divide the value heads");
  TORCH_CHECK(dim >= 1 && dim <= 1024 && vdim >= 1 && vdim <= 4096, "head size");
  check_rows(b_pre, dt, rows, heads, "b_pre");
  check_rows(a_pre, dt, rows, heads, "a_pre");
  check_f32(a_log, heads, "a_log");
  check_f32(dt_bias, heads, "dt_bias");
  check_f32(state, -1, "state");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == heads && state.size(2) == vdim &&
              state.size(3) == dim, "state must be [slots, heads, vdim, dim]");
  return check_seqs(loc, seq_lens, slots);
}

void delta_scan(torch::Tensor o, torch::Tensor q, torch::Tensor k, torch::Tensor v,
                torch::Tensor b_pre, torch::Tensor a_pre, torch::Tensor a_log,
                torch::Tensor dt_bias, torch::Tensor state, torch::Tensor loc,
                torch::Tensor seq_lens, torch::Tensor slots) {
  const int nseq =
      check_delta(q, k, v, b_pre, a_pre, a_log, dt_bias, state, loc, seq_lens, slots);
  const auto dt = q.scalar_type();
  const int rows = q.size(0), groups = q.size(1), dim = q.size(2);
  const int heads = v.size(1), vdim = v.size(2);
  check_f32(o, (long)rows * heads * vdim, "o");
  if (rows == 0 || nseq == 0) return;
  auto kq = torch::empty({(long)rows, 2L * groups * dim}, o.options());
  auto gates = torch::empty({(long)rows, (long)heads, 4L}, o.options());
  const int vec_ok = dim % 4 == 0 && aligned16(state) && aligned16(kq);
  DISPATCH_F32_BF16(dt, {
    launch_delta_scan<scalar_t>(
        ptr<float>(o), ptr<scalar_t>(q), (long)q.stride(0), ptr<scalar_t>(k),
        (long)k.stride(0), ptr<scalar_t>(v), (long)v.stride(0), ptr<scalar_t>(b_pre),
        (long)b_pre.stride(0), ptr<scalar_t>(a_pre), (long)a_pre.stride(0), ptr<float>(a_log),
        ptr<float>(dt_bias), 1.0f / std::sqrt((float)dim), ptr<float>(state), ptr<int>(loc),
        ptr<int>(seq_lens), ptr<int>(slots), nseq, heads, groups, dim, vdim, vec_ok,
        ptr<float>(kq), ptr<float>(gates), rows, stream());
  });
}

// the scan followed by the per-head norm, its weight and silu(gate): one kernel
// where the shape fits, three otherwise
void delta_gated(torch::Tensor out, torch::Tensor q, torch::Tensor k, torch::Tensor v,
                 torch::Tensor b_pre, torch::Tensor a_pre, torch::Tensor a_log,
                 torch::Tensor dt_bias, torch::Tensor gate, torch::Tensor norm, double eps,
                 torch::Tensor state, torch::Tensor loc, torch::Tensor seq_lens,
                 torch::Tensor slots, bool general) {
  const int nseq =
      check_delta(q, k, v, b_pre, a_pre, a_log, dt_bias, state, loc, seq_lens, slots);
  const auto dt = q.scalar_type();
  const int rows = q.size(0), groups = q.size(1), dim = q.size(2);
  const int heads = v.size(1), vdim = v.size(2);
  check_rows(gate, dt, rows, (long)heads * vdim, "gate");
  check_f32(norm, (long)heads * vdim, "norm");
  check_type(out, dt, "out");
  TORCH_CHECK(out.numel() == (long)rows * heads * vdim);
  if (rows == 0 || nseq == 0) return;
  bool fits = !general && delta_fused_columns(dim, vdim) > 0 && aligned16(state);
  for (const torch::Tensor* t : {&q, &k, &v})
    fits = fits && t->stride(0) % 8 == 0 && aligned16(*t);
  if (!fits) {
    auto o = torch::empty({(long)rows, (long)heads * vdim}, state.options());
    delta_scan(o, q, k, v, b_pre, a_pre, a_log, dt_bias, state, loc, seq_lens, slots);
    DISPATCH_F32_BF16(dt, {
      launch_gated_group_norm<scalar_t>(ptr<scalar_t>(out), ptr<float>(o), ptr<scalar_t>(gate),
                                        (long)gate.stride(0), ptr<float>(norm), (float)eps,
                                        rows, heads * vdim, heads, 2, stream());
    });
    return;
  }
  DISPATCH_F32_BF16(dt, {
    launch_delta_fused<scalar_t>(
        ptr<scalar_t>(out), ptr<scalar_t>(q), (long)q.stride(0), ptr<scalar_t>(k),
        (long)k.stride(0), ptr<scalar_t>(v), (long)v.stride(0), ptr<scalar_t>(b_pre),
        (long)b_pre.stride(0), ptr<scalar_t>(a_pre), (long)a_pre.stride(0), ptr<float>(a_log),
        ptr<float>(dt_bias), ptr<scalar_t>(gate), (long)gate.stride(0), ptr<float>(norm),
        1.0f / std::sqrt((float)dim), (float)eps, ptr<float>(state), ptr<int>(loc),
        ptr<int>(seq_lens), ptr<int>(slots), nseq, heads, groups, dim, vdim, rows, stream());
  });
}

void clamped_glu(torch::Tensor out, torch::Tensor gu, double limit, OptTensor col_scale) {
  TORCH_CHECK(gu.is_cuda() && gu.is_contiguous() && gu.dim() == 2);
  const long rows = gu.size(0);
  const long experts = col_scale.has_value() ? col_scale.value().size(1) : 1;
  check_f32(col_scale, rows * experts, "col_scale");
  TORCH_CHECK(experts >= 1 && gu.size(1) % (2 * experts) == 0,
              "columns must divide into the experts' gate and up parts");
  check_type(out, gu.scalar_type(), "out");
  TORCH_CHECK(out.numel() * 2 == gu.numel());
  if (out.numel() == 0) return;
  DISPATCH_F32_BF16(gu.scalar_type(), {
    launch_clamped_glu<scalar_t>(ptr<scalar_t>(out), ptr<scalar_t>(gu), (float)limit,
                                 optr<float>(col_scale), (int)(gu.size(1) / (2 * experts)),
                                 (long)out.numel(), stream());
  });
}

// router weights are f32 or bf16 whatever the rows are
template <typename F>
void with_router(const torch::Tensor& w, F launch) {
  if (w.scalar_type() == at::ScalarType::Float) launch(ptr<const float>(w));
  else launch(ptr<const __hip_bfloat16>(w));
}

void router_logits(torch::Tensor out, torch::Tensor h, torch::Tensor w) {
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.stride(1) == 1 && w.dim() == 2 &&
              w.size(1) == h.size(1), "rows and router width");
  TORCH_CHECK(w.is_cuda() && w.is_contiguous() &&
              (w.scalar_type() == at::ScalarType::Float ||
               w.scalar_type() == at::ScalarType::BFloat16), "router: f32 or bf16 weights");
  const int rows = h.size(0), width = h.size(1), experts = w.size(0);
  check_f32(out, (long)rows * experts, "out");
  if (rows == 0 || experts == 0) return;
  DISPATCH_F32_BF16(h.scalar_type(), {
    with_router(w, [&](auto* wp) {
      launch_router_logits(ptr<float>(out), ptr<scalar_t>(h), (long)h.stride(0), wp, rows,
                           experts, width, stream());
    });
  });
}

void route_experts(torch::Tensor dense, torch::Tensor ids, torch::Tensor wts, torch::Tensor h,
                   torch::Tensor w, OptTensor correction, int64_t groups, int64_t keep,
                   bool renormalise, double scale) {
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.stride(1) == 1 && w.dim() == 2 &&
              w.size(1) == h.size(1), "rows and router width");
  TORCH_CHECK(w.is_cuda() && w.is_contiguous() &&
              (w.scalar_type() == at::ScalarType::Float ||
               w.scalar_type() == at::ScalarType::BFloat16), "router: f32 or bf16 weights");
  const int rows = h.size(0), width = h.size(1), experts = w.size(0);
  TORCH_CHECK(experts >= 1 && experts <= 64 && width % 32 == 0 && h.stride(0) % 8 == 0 &&
              aligned16(h) && aligned16(w), "shape off the fused router");
  check_f32(correction, experts, "correction");
  check_f32(dense, (long)rows * experts, "dense");
  check_f32(wts, -1, "weights");
  check_type(ids, at::ScalarType::Int, "ids");
  TORCH_CHECK(ids.dim() == 2 && ids.size(0) == rows && wts.sizes() == ids.sizes());
  const int top = ids.size(1);
  TORCH_CHECK(groups >= 1 && experts % groups == 0 && keep >= 1 && keep <= groups && top >= 1 &&
              top <= keep * (experts / groups), "expert groups");
  if (rows == 0) return;
  DISPATCH_F32_BF16(h.scalar_type(), {
    with_router(w, [&](auto* wp) {
      launch_route_experts(ptr<float>(dense), ptr<int>(ids), ptr<float>(wts), ptr<scalar_t>(h),
                           (long)h.stride(0), wp, optr<float>(correction), rows, experts, width,
                           top, (int)groups, (int)keep, renormalise ? 1 : 0, (float)scale,
                           stream());
    });
  });
}

void scale_logits(torch::Tensor out, torch::Tensor x, double scale) {
  check_type(x, x.scalar_type(), "logits");
  check_f32(out, (long)x.numel(), "out");
  if (x.numel() == 0) return;
  DISPATCH_F32_BF16(x.scalar_type(), {
    launch_scale_logits<scalar_t>(ptr<float>(out), ptr<scalar_t>(x), (float)scale,
                                  (long)x.numel(), stream());
  });
}

}  // namespace

void register_row_ops(pybind11::module& m) {
  m.def("stream_add_tanh_norm", &stream_add_tanh_norm);
  m.def("wide_norm_cache_write", &wide_norm_cache_write);
  m.def("capped_attention", &capped_attention);
  m.def("delta_scan", &delta_scan);
  m.def("delta_gated", &delta_gated);
  m.def("clamped_glu", &clamped_glu);
  m.def("router_logits", &router_logits);
  m.def("route_experts", &route_experts);
  m.def("scale_logits", &scale_logits);
}
