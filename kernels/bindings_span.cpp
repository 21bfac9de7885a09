// Torch bindings (part of `_C_seq`): grouped norms around sublayers, rotation
// tables, attention inputs in one pass, pooled key/value blocks, attention over
// a window plus a prefix, gated linear attention and the biased silu gate.
// Every shape the kernels assume is checked here, on the host, before a launch.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <hip/hip_bf16.h>

template <typename T>
void launch_stream_add_group_norm(float*, const T*, const float*, const T*, const float*,
                                  const float*, const float*, const float*, T*, float,
                                  float, int, int, int, hipStream_t);
void launch_rotary_table(float*, const long*, const float*, int, int, hipStream_t);
template <typename T>
void launch_attn_inputs(T*, const T*, long, const float*, const float*, const float*,
                        const float*, T*, int, const float*, int, const float*, int, T*,
                        T*, const long*, const int*, const int*, const int*, int, int, int,
                        int, int, int, float, int, hipStream_t);
template <typename T>
void launch_pool_cache_write(const T*, const T*, T*, T*, int, int, const int*, int,
                             const int*, const int*, int, int, int, int, int, hipStream_t);
template <typename T>
void launch_silu_mul_bias(T*, const T*, const float*, int, long, hipStream_t);
template <typename T>
void launch_span_attention(T*, long, const T*, long, const T*, const T*, const T*,
                           const T*, const int*, int, const int*, const int*, int, float,
                           int, int, int, int, int, int, int, int, int, int, int,
                           const float*, hipStream_t);
template <typename T>
void launch_gla_scan(float*, const T*, long, const T*, long, const T*, long, const T*,
                     long, const float*, const float*, float, float, float*, const int*,
                     const int*, const int*, int, int, int, int, int, int, float*, int,
                     hipStream_t);
int gla_fused_columns(int dim, int vdim);
template <typename T>
void launch_gla_fused(T*, const T*, long, const T*, long, const T*, long, const T*, long,
                      const T*, long, const float*, const float*, float, float,
                      const float*, float, float*, const int*, const int*, const int*, int,
                      int, int, int, int, int, hipStream_t);
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

// heads of one row laid out [heads, size] with unit stride, rows strided
void check_heads_view(const torch::Tensor& t, at::ScalarType dt, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 3 && t.stride(2) == 1 &&
                  t.stride(1) == t.size(2) && t.scalar_type() == dt, what,
              " must be [rows, heads, size] rows");
}

void check_cache(const torch::Tensor& k, const torch::Tensor& v, at::ScalarType dt) {
  check_type(k, dt, "k_cache");
  check_type(v, dt, "v_cache");
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.size(0) == v.size(0) &&
              k.size(1) == v.size(1) && k.size(2) == v.size(2) && k.size(1) >= 1,
              "key and value caches do not fit each other");
}

// pooled blocks beside the caches; returns how many a cache block has room for
int check_pool(const torch::Tensor& k_cache, const torch::Tensor& v_cache,
               const OptTensor& k_pool, const OptTensor& v_pool, int64_t pool) {
  TORCH_CHECK(pool >= 0, "pool");
  if (pool == 0) return 0;
  TORCH_CHECK(k_pool.has_value() && v_pool.has_value(), "pooled caches missing");
  const auto &kp = k_pool.value(), &vp = v_pool.value();
  check_cache(kp, vp, k_cache.scalar_type());
  const int64_t per_block = (k_cache.size(1) + pool - 1) / pool;
  TORCH_CHECK(kp.size(0) == k_cache.size(0) && kp.size(1) == per_block &&
              kp.size(2) == k_cache.size(2) && kp.size(3) == k_cache.size(3) &&
              vp.size(3) == v_cache.size(3), "pooled caches do not fit the caches");
  return (int)per_block;
}

void check_tables(const torch::Tensor& t, int nseq) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::ScalarType::Int && t.dim() == 2 &&
              t.stride(1) == 1 && t.size(0) >= nseq, "block tables");
}

void stream_add_group_norm(torch::Tensor x, OptTensor a, OptTensor a_bias, OptTensor b,
                           OptTensor wa, OptTensor wb, OptTensor w_out, int64_t groups,
                           double eps, double mix, OptTensor next_w, OptTensor next_out) {
  check_f32(x, -1, "x");
  TORCH_CHECK(x.dim() == 2);
  const int rows = x.size(0), width = x.size(1);
  TORCH_CHECK(groups >= 1 && width % groups == 0, "groups must divide the width");
  check_f32(a_bias, width, "a_bias");
  check_f32(wa, width, "wa");
  check_f32(wb, width, "wb");
  check_f32(w_out, width, "w_out");
  check_f32(next_w, width, "next_w");
  TORCH_CHECK(a.has_value() || !b.has_value());
  TORCH_CHECK(!a.has_value() || w_out.has_value(), "w_out missing");
  TORCH_CHECK(!b.has_value() || (wa.has_value() && wb.has_value()), "wa / wb missing");
  TORCH_CHECK(next_w.has_value() == next_out.has_value());
  TORCH_CHECK(a.has_value() || next_out.has_value(), "nothing to do");
  const auto dt = a.has_value() ? a.value().scalar_type() : next_out.value().scalar_type();
  for (const OptTensor* t : {&a, &b, &next_out})
    if (t->has_value()) {
      check_type(t->value(), dt, "rows");
      TORCH_CHECK(t->value().numel() == x.numel(), "rows must match x");
    }
  if (rows == 0) return;
  DISPATCH_F32_BF16(dt, {
    launch_stream_add_group_norm<scalar_t>(
        ptr<float>(x), optr<scalar_t>(a), optr<float>(a_bias), optr<scalar_t>(b),
        optr<float>(wa), optr<float>(wb), optr<float>(w_out), optr<float>(next_w),
        optr<scalar_t>(next_out), (float)eps, (float)mix, rows, width, (int)groups,
        stream());
  });
}

void rotary_table(torch::Tensor out, torch::Tensor positions, torch::Tensor inv_freq) {
  check_type(positions, at::ScalarType::Long, "positions");
  check_f32(inv_freq, -1, "inv_freq");
  const int rows = positions.numel(), pairs = inv_freq.numel();
  check_f32(out, 2L * rows * pairs, "out");
  if (rows == 0 || pairs == 0) return;
  launch_rotary_table(ptr<float>(out), ptr<long>(positions), ptr<float>(inv_freq), rows,
                      pairs, stream());
}

void attn_inputs_cache_write(torch::Tensor q_out, torch::Tensor proj, OptTensor bias,
                             int64_t kv_heads, int64_t vdim, double eps, OptTensor qw,
                             OptTensor kw, OptTensor conv_weight, OptTensor conv_state,
                             OptTensor rot_table, OptTensor v_table, torch::Tensor k_cache,
                             torch::Tensor v_cache, torch::Tensor slot_mapping,
                             OptTensor loc, OptTensor seq_lens, OptTensor slots,
                             bool has_portions) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  const auto dt = proj.scalar_type();
  check_type(q_out, dt, "q_out");
  TORCH_CHECK(q_out.dim() == 3 && q_out.size(0) == proj.size(0));
  const int rows = proj.size(0), heads = q_out.size(1), dim = q_out.size(2);
  TORCH_CHECK(kv_heads >= 1 && vdim >= 1 && dim <= 2048 && vdim <= 2048, "head sizes");
  const long channels = (long)heads * dim + kv_heads * (dim + vdim);
  TORCH_CHECK(proj.size(1) == channels, "projected rows are [q | k | v]");
  check_cache(k_cache, v_cache, dt);
  TORCH_CHECK(k_cache.size(2) == kv_heads && k_cache.size(3) == dim &&
              v_cache.size(3) == vdim, "cache shape");
  check_type(slot_mapping, at::ScalarType::Long, "slot_mapping");
  TORCH_CHECK(slot_mapping.numel() == rows);
  check_f32(bias, channels, "bias");
  check_f32(qw, dim, "q weight");
  check_f32(kw, dim, "k weight");
  int rot = 0, vrot = 0, taps = 0, nseq = 0;
  if (rot_table.has_value()) {
    TORCH_CHECK(rot_table.value().dim() == 3);
    rot = 2 * rot_table.value().size(1);
    check_f32(rot_table, (long)rows * rot, "rot_table");
    TORCH_CHECK(rot <= dim, "rotated dims");
  }
  if (v_table.has_value()) {
    TORCH_CHECK(v_table.value().dim() == 3);
    vrot = 2 * v_table.value().size(1);
    check_f32(v_table, (long)rows * vrot, "v_table");
    TORCH_CHECK(vrot <= vdim, "rotated dims");
  }
  if (conv_weight.has_value()) {
    TORCH_CHECK(conv_weight.value().dim() == 2 && conv_weight.value().size(1) == channels);
    check_f32(conv_weight, -1, "conv_weight");
    taps = conv_weight.value().size(0);
    TORCH_CHECK(taps >= 1 && conv_state.has_value() && loc.has_value() &&
                seq_lens.has_value() && slots.has_value(), "convolution state");
    const auto& st = conv_state.value();
    check_type(st, dt, "conv_state");
    TORCH_CHECK(st.dim() == 3 && st.size(1) == taps - 1 && st.size(2) == channels,
                "conv_state must be [slots, taps - 1, channels]");
    nseq = check_seqs(loc.value(), seq_lens.value(), slots.value());
    if (nseq == 0) return;
    TORCH_CHECK(has_portions || nseq == rows, "one row per sequence expected");
  }
  if (rows == 0) return;
  DISPATCH_F32_BF16(dt, {
    launch_attn_inputs<scalar_t>(
        ptr<scalar_t>(q_out), ptr<scalar_t>(proj), (long)proj.stride(0), optr<float>(bias),
        optr<float>(qw), optr<float>(kw), optr<float>(conv_weight),
        optr<scalar_t>(conv_state), taps, optr<float>(rot_table), rot, optr<float>(v_table),
        vrot, ptr<scalar_t>(k_cache), ptr<scalar_t>(v_cache), ptr<long>(slot_mapping),
        optr<int>(loc), optr<int>(seq_lens), optr<int>(slots), nseq, rows, heads,
        (int)kv_heads, dim, (int)vdim, (float)eps, has_portions ? 1 : 0, stream());
  });
}

void pool_cache_write(torch::Tensor k_cache, torch::Tensor v_cache, torch::Tensor k_pool,
                      torch::Tensor v_pool, int64_t pool, torch::Tensor block_tables,
                      OptTensor query_start_loc, torch::Tensor seq_lens, int64_t rows) {
  const auto dt = k_cache.scalar_type();
  check_cache(k_cache, v_cache, dt);
  TORCH_CHECK(pool >= 1, "pool");
  const int per_block = check_pool(k_cache, v_cache, k_pool, v_pool, pool);
  check_type(seq_lens, at::ScalarType::Int, "seq_lens");
  const int nseq = seq_lens.numel();
  check_tables(block_tables, nseq);
  if (query_start_loc.has_value()) {
    check_type(query_start_loc.value(), at::ScalarType::Int, "query_start_loc");
    TORCH_CHECK(query_start_loc.value().numel() == nseq + 1);
  } else {
    TORCH_CHECK(rows == nseq, "one row per sequence expected");
  }
  if (rows <= 0 || nseq == 0) return;
  DISPATCH_F32_BF16(dt, {
    launch_pool_cache_write<scalar_t>(
        ptr<scalar_t>(k_cache), ptr<scalar_t>(v_cache), ptr<scalar_t>(k_pool),
        ptr<scalar_t>(v_pool), (int)pool, per_block, ptr<int>(block_tables),
        (int)block_tables.stride(0), optr<int>(query_start_loc), ptr<int>(seq_lens), nseq,
        (int)rows, (int)k_cache.size(1), (int)(k_cache.size(2) * k_cache.size(3)),
        (int)(v_cache.size(2) * v_cache.size(3)), stream());
  });
}

void span_attention(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                    torch::Tensor v_cache, OptTensor k_pool, OptTensor v_pool,
                    torch::Tensor block_tables, OptTensor query_start_loc,
                    torch::Tensor seq_lens, double scale, int64_t window,
                    int64_t keep_first, int64_t pool, OptTensor back_table) {
  const auto dt = q.scalar_type();
  check_heads_view(q, dt, "q");
  check_heads_view(out, dt, "out");
  check_cache(k_cache, v_cache, dt);
  TORCH_CHECK(window >= 0 && keep_first >= 0 && !(keep_first && pool), "mask");
  const int per_block = check_pool(k_cache, v_cache, k_pool, v_pool, pool);
  const int rows = q.size(0), heads = q.size(1), dim = q.size(2);
  const int kv_heads = k_cache.size(2), vdim = v_cache.size(3);
  TORCH_CHECK(k_cache.size(3) == dim && kv_heads >= 1 && heads % kv_heads == 0,
              "cache shape");
  TORCH_CHECK(vdim <= 1024, "value size above 1024 is not supported");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads && out.size(2) == vdim);
  check_type(seq_lens, at::ScalarType::Int, "seq_lens");
  const int nseq = seq_lens.numel();
  check_tables(block_tables, nseq);
  if (query_start_loc.has_value()) {
    check_type(query_start_loc.value(), at::ScalarType::Int, "query_start_loc");
    TORCH_CHECK(query_start_loc.value().numel() == nseq + 1);
  } else {
    TORCH_CHECK(rows == nseq, "one query row per sequence expected");
  }
  TORCH_CHECK(!back_table.has_value() || vdim % 2 == 0);
  check_f32(back_table, (long)rows * vdim, "back_table");
  if (rows == 0 || nseq == 0) return;
  const int elems16 = dt == at::ScalarType::Float ? 4 : 8;
  const int vec_ok = dim % elems16 == 0 && aligned16(k_cache) &&
                     (pool == 0 || aligned16(k_pool.value()));
  DISPATCH_F32_BF16(dt, {
    launch_span_attention<scalar_t>(
        ptr<scalar_t>(out), (long)out.stride(0), ptr<scalar_t>(q), (long)q.stride(0),
        ptr<scalar_t>(k_cache), ptr<scalar_t>(v_cache), optr<scalar_t>(k_pool),
        optr<scalar_t>(v_pool), ptr<int>(block_tables), (int)block_tables.stride(0),
        optr<int>(query_start_loc), ptr<int>(seq_lens), nseq, (float)scale, rows, heads,
        kv_heads, dim, vdim, (int)k_cache.size(1), per_block, vec_ok, (int)window,
        (int)keep_first, (int)pool, optr<float>(back_table), stream());
  });
}

void gla_scan(torch::Tensor o, torch::Tensor q, torch::Tensor k, torch::Tensor v,
              torch::Tensor a1, torch::Tensor a2, torch::Tensor a2_bias, double inv_tau,
              double q_scale, torch::Tensor state, torch::Tensor loc,
              torch::Tensor seq_lens, torch::Tensor slots) {
  const int nseq = check_seqs(loc, seq_lens, slots);
  const auto dt = q.scalar_type();
  check_heads_view(q, dt, "q");
  check_heads_view(k, dt, "k");
  check_heads_view(v, dt, "v");
  const int rows = q.size(0), heads = q.size(1), dim = q.size(2), vdim = v.size(2);
  TORCH_CHECK(k.sizes() == q.sizes() && v.size(0) == rows && v.size(1) == heads);
  TORCH_CHECK(dim >= 1 && dim <= 1024, "gla_scan: head size");
  TORCH_CHECK(a1.is_cuda() && a1.dim() == 2 && a1.size(0) == rows && a1.stride(1) == 1 &&
              a1.scalar_type() == dt, "a1 is [rows, rank]");
  const int rank = a1.size(1);
  TORCH_CHECK(rank >= 1 && rank <= 512, "gla_scan: rank");
  check_f32(a2, (long)rank * heads * dim, "a2");
  check_f32(a2_bias, (long)heads * dim, "a2_bias");
  check_f32(o, (long)rows * heads * vdim, "o");
  check_f32(state, -1, "state");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == heads && state.size(2) == vdim &&
              state.size(3) == dim, "gla_scan: state must be [slots, heads, vdim, dim]");
  if (rows == 0 || nseq == 0) return;
  auto decay = torch::empty({(long)rows, (long)heads * dim}, o.options());
  const int vec_ok = dim % 8 == 0 && q.stride(0) % 8 == 0 && k.stride(0) % 8 == 0 &&
                     aligned16(q) && aligned16(k) && aligned16(state) && aligned16(decay);
  DISPATCH_F32_BF16(dt, {
    launch_gla_scan<scalar_t>(
        ptr<float>(o), ptr<scalar_t>(q), (long)q.stride(0), ptr<scalar_t>(k),
        (long)k.stride(0), ptr<scalar_t>(v), (long)v.stride(0), ptr<scalar_t>(a1),
        (long)a1.stride(0), ptr<float>(a2), ptr<float>(a2_bias), (float)inv_tau,
        (float)q_scale, ptr<float>(state), ptr<int>(loc), ptr<int>(seq_lens),
        ptr<int>(slots), nseq, heads, dim, vdim, rank, vec_ok, ptr<float>(decay), rows,
        stream());
  });
}

// the scan followed by the per-head norm, its weight and silu(gate): one kernel
// where the shape fits, three otherwise
void gla_gated(torch::Tensor out, torch::Tensor q, torch::Tensor k, torch::Tensor v,
               torch::Tensor g, torch::Tensor a1, torch::Tensor a2, torch::Tensor a2_bias,
               double inv_tau, double q_scale, torch::Tensor norm, double eps,
               torch::Tensor state, torch::Tensor loc, torch::Tensor seq_lens,
               torch::Tensor slots, bool general) {
  const auto dt = q.scalar_type();
  check_heads_view(q, dt, "q");
  check_heads_view(k, dt, "k");
  check_heads_view(v, dt, "v");
  const int rows = q.size(0), heads = q.size(1), dim = q.size(2), vdim = v.size(2);
  TORCH_CHECK(g.is_cuda() && g.dim() == 2 && g.size(0) == rows && g.stride(1) == 1 &&
              g.size(1) == (long)heads * vdim && g.scalar_type() == dt,
              "the gate is [rows, heads * vdim]");
  check_f32(norm, (long)heads * vdim, "norm");
  check_type(out, dt, "out");
  TORCH_CHECK(out.numel() == (long)rows * heads * vdim);
  const int nseq = check_seqs(loc, seq_lens, slots);
  if (rows == 0 || nseq == 0) return;
  const int64_t rank = a1.dim() == 2 ? a1.size(1) : 0;
  bool fits = !general && gla_fused_columns(dim, vdim) > 0 && rank <= 64 && aligned16(state);
  for (const torch::Tensor* t : {&q, &k, &v})
    fits = fits && t->stride(0) % 8 == 0 && aligned16(*t);
  if (!fits) {
    auto o = torch::empty({(long)rows, (long)heads * vdim}, state.options());
    gla_scan(o, q, k, v, a1, a2, a2_bias, inv_tau, q_scale, state, loc, seq_lens, slots);
    DISPATCH_F32_BF16(dt, {
      launch_gated_group_norm<scalar_t>(ptr<scalar_t>(out), ptr<float>(o), ptr<scalar_t>(g),
                                        (long)g.stride(0), ptr<float>(norm), (float)eps,
                                        rows, heads * vdim, heads, 2, stream());
    });
    return;
  }
  TORCH_CHECK(k.sizes() == q.sizes() && v.size(0) == rows && v.size(1) == heads);
  TORCH_CHECK(a1.is_cuda() && a1.size(0) == rows && a1.stride(1) == 1 && rank >= 1 &&
              a1.scalar_type() == dt, "a1 is [rows, rank]");
  check_f32(a2, (long)rank * heads * dim, "a2");
  check_f32(a2_bias, (long)heads * dim, "a2_bias");
  check_f32(state, -1, "state");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == heads && state.size(2) == vdim &&
              state.size(3) == dim, "state must be [slots, heads, vdim, dim]");
  DISPATCH_F32_BF16(dt, {
    launch_gla_fused<scalar_t>(
        ptr<scalar_t>(out), ptr<scalar_t>(q), (long)q.stride(0), ptr<scalar_t>(k),
        (long)k.stride(0), ptr<scalar_t>(v), (long)v.stride(0), ptr<scalar_t>(g),
        (long)g.stride(0), ptr<scalar_t>(a1), (long)a1.stride(0), ptr<float>(a2),
        ptr<float>(a2_bias), (float)inv_tau, (float)q_scale, ptr<float>(norm), (float)eps,
        ptr<float>(state), ptr<int>(loc), ptr<int>(seq_lens), ptr<int>(slots), nseq, heads,
        dim, vdim, (int)rank, rows, stream());
  });
}

void silu_mul_bias(torch::Tensor out, torch::Tensor gu, OptTensor bias) {
  TORCH_CHECK(gu.is_cuda() && gu.is_contiguous() && gu.dim() == 2 && gu.size(1) % 2 == 0);
  const long rows = gu.size(0);
  const int ff = gu.size(1) / 2;
  check_f32(bias, 2L * ff, "bias");
  check_type(out, gu.scalar_type(), "out");
  TORCH_CHECK(out.numel() == rows * ff);
  if (out.numel() == 0) return;
  DISPATCH_F32_BF16(gu.scalar_type(), {
    launch_silu_mul_bias<scalar_t>(ptr<scalar_t>(out), ptr<scalar_t>(gu), optr<float>(bias),
                                   ff, rows, stream());
  });
}

}  // namespace

void register_span_ops(pybind11::module& m) {
  m.def("stream_add_group_norm", &stream_add_group_norm);
  m.def("rotary_table", &rotary_table);
  m.def("attn_inputs_cache_write", &attn_inputs_cache_write);
  m.def("pool_cache_write", &pool_cache_write);
  m.def("span_attention", &span_attention);
  m.def("gla_scan", &gla_scan);
  m.def("gla_gated", &gla_gated);
  m.def("silu_mul_bias", &silu_mul_bias);
}
