// Torch bindings of the paged grouped-query attention kernels (generic f32 /
// f16 / bf16, bf16 MFMA decode and prefill, fp8 cache variants).  Compiled
// into `_C` and, with module_attn.cpp, into the small `_C_attn` extension for
// models that need nothing else of `_C`.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <hip/hip_bf16.h>
#include <hip/hip_fp16.h>

template <typename T>
void launch_paged_decode(T*, const T*, const T*, const T*, const int*,
                         const int*, float, int, int, int, int, int, int,
                         hipStream_t);
template <typename T>
void launch_paged_prefill(T*, const T*, const T*, const T*, const int*,
                          const int*, const int*, float, int, int, int, int,
                          int, int, int, hipStream_t);
void launch_paged_prefill_mfma_v2(__hip_bfloat16*, const __hip_bfloat16*,
                                  const __hip_bfloat16*, const __hip_bfloat16*,
                                  const int*, const int*, const int*, float,
                                  int, int, int, int, int, int, int,
                                  hipStream_t);
void launch_paged_prefill_mfma(__hip_bfloat16*, const __hip_bfloat16*,
                               const __hip_bfloat16*, const __hip_bfloat16*,
                               const int*, const int*, const int*, float, int,
                               int, int, int, int, int, int, hipStream_t);
void launch_paged_prefill_mfma_v2_capped(__hip_bfloat16*, const __hip_bfloat16*,
                                         const __hip_bfloat16*, const __hip_bfloat16*,
                                         const int*, const int*, const int*, float, int, int,
                                         int, int, int, int, int, int, int, const float*, float,
                                         hipStream_t);
void launch_paged_decode_mfma_capped(__hip_bfloat16*, float*, float*, const __hip_bfloat16*,
                                     const __hip_bfloat16*, const __hip_bfloat16*, const int*,
                                     const int*, float, int, int, int, int, int, int, int, int,
                                     int, const float*, float, hipStream_t);
int decode_mfma_num_partitions(int nseq, int kvh, int max_context);
void launch_paged_decode_mfma_fp8(__hip_bfloat16*, float*, float*,
                                  const __hip_bfloat16*, const unsigned char*,
                                  const unsigned char*, const int*,
                                  const int*, float, int, int, int, int, int,
                                  int, int, hipStream_t);
void launch_paged_prefill_mfma_v2_fp8(__hip_bfloat16*, const __hip_bfloat16*,
                                      const unsigned char*,
                                      const unsigned char*, const int*,
                                      const int*, const int*, float, int, int,
                                      int, int, int, int, int, hipStream_t);
void launch_paged_decode_mfma(__hip_bfloat16*, float*, float*,
                              const __hip_bfloat16*, const __hip_bfloat16*,
                              const __hip_bfloat16*, const int*, const int*,
                              float, int, int, int, int, int, int, int,
                              hipStream_t);

void launch_paged_prefill_mfma_v2_ws(__hip_bfloat16*, const __hip_bfloat16*,
                                     const __hip_bfloat16*, const __hip_bfloat16*,
                                     const int*, const int*, const int*, float,
                                     int, int, int, int, int, int, int, int, int,
                                     float, hipStream_t);
void launch_paged_prefill_mfma_v2_chunk(float*, const __hip_bfloat16*,
                                        const __hip_bfloat16*, const __hip_bfloat16*,
                                        const int*, const int*, const int*, float,
                                        int, int, int, int, int, int, int, int,
                                        hipStream_t);
void launch_paged_decode_mfma_chunk(float*, float*, float*, const __hip_bfloat16*,
                                    const __hip_bfloat16*, const __hip_bfloat16*,
                                    const int*, const int*, float, int, int, int,
                                    int, int, int, int, int, int, hipStream_t);
void launch_paged_prefill_mfma_v2_span(__hip_bfloat16*, const __hip_bfloat16*,
                                       const __hip_bfloat16*, const __hip_bfloat16*,
                                       const __hip_bfloat16*, const __hip_bfloat16*,
                                       const int*, const int*, const int*, float, int,
                                       int, int, int, int, int, int, int, int, int,
                                       const float*, hipStream_t);
void launch_paged_decode_mfma_span(__hip_bfloat16*, float*, float*, const __hip_bfloat16*,
                                   const __hip_bfloat16*, const __hip_bfloat16*,
                                   const __hip_bfloat16*, const __hip_bfloat16*,
                                   const int*, const int*, float, int, int, int, int, int,
                                   int, int, int, int, int, int, const float*,
                                   hipStream_t);
void launch_paged_decode_mfma_ws(__hip_bfloat16*, float*, float*,
                                 const __hip_bfloat16*, const __hip_bfloat16*,
                                 const __hip_bfloat16*, const int*, const int*,
                                 float, int, int, int, int, int, int, int, int,
                                 int, float, hipStream_t);

namespace {

hipStream_t current_stream() {
  return at::hip::getCurrentHIPStream().stream();
}

template <typename T>
T* ptr(torch::Tensor& t) {
  return reinterpret_cast<T*>(t.data_ptr());
}
template <typename T>
const T* cptr(const torch::Tensor& t) {
  return reinterpret_cast<const T*>(t.data_ptr());
}

#define DISPATCH_FLOATING(DTYPE, BODY)                                   \
  switch (DTYPE) {                                                       \
    case at::ScalarType::BFloat16: {                                     \
      using scalar_t = __hip_bfloat16;                                   \
      BODY;                                                              \
      break;                                                             \
    }                                                                    \
    case at::ScalarType::Half: {                                         \
      using scalar_t = __half;                                           \
      BODY;                                                              \
      break;                                                             \
    }                                                                    \
    case at::ScalarType::Float: {                                        \
      using scalar_t = float;                                            \
      BODY;                                                              \
      break;                                                             \
    }                                                                    \
    default:                                                             \
      TORCH_CHECK(false, "unsupported dtype");                           \
  }

void paged_attention_decode(torch::Tensor out, torch::Tensor q,
                            torch::Tensor k_cache, torch::Tensor v_cache,
                            torch::Tensor block_tables, torch::Tensor seq_lens,
                            double scale) {
  const int nseq = q.size(0);
  const int nheads = q.size(1);
  const int head_dim = q.size(2);
  const int kvh = k_cache.size(2);
  const int block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  TORCH_CHECK(block_tables.scalar_type() == at::ScalarType::Int);
  TORCH_CHECK(seq_lens.scalar_type() == at::ScalarType::Int);
  const int group = nheads / kvh;
  static const bool force_valu = [] {
    const char* e = getenv("VTA_DECODE_VALU");
    return e && e[0] == '1';
  }();
  const bool kv_fp8 = k_cache.scalar_type() == at::ScalarType::Byte;
  if (kv_fp8) {
    TORCH_CHECK(q.scalar_type() == at::ScalarType::BFloat16 &&
                    (head_dim == 64 || head_dim == 128) && group >= 1 &&
                    group <= 8,
                "fp8 KV cache requires the bf16 MFMA decode path");
    const int npart = decode_mfma_num_partitions(nseq, kvh, max_blocks * block_size);
    const int P = npart * 4;
    auto opts = q.options().dtype(at::ScalarType::Float);
    auto part_acc = at::empty({nseq, nheads, P, head_dim}, opts);
    auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
    launch_paged_decode_mfma_fp8(
        reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
        part_acc.data_ptr<float>(), part_ml.data_ptr<float>(),
        reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
        reinterpret_cast<const unsigned char*>(k_cache.data_ptr()),
        reinterpret_cast<const unsigned char*>(v_cache.data_ptr()),
        block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (float)scale,
        nseq, nheads, kvh, head_dim, block_size, max_blocks, npart,
        current_stream());
    return;
  }
  if (!force_valu && q.scalar_type() == at::ScalarType::BFloat16 &&
      (head_dim == 64 || head_dim == 128) && group >= 1 && group <= 8 &&
      nheads == kvh * group && nseq > 0) {
    const int npart = decode_mfma_num_partitions(nseq, kvh, max_blocks * block_size);
    const int P = npart * 4;
    auto opts = q.options().dtype(at::ScalarType::Float);
    auto part_acc = at::empty({nseq, nheads, P, head_dim}, opts);
    auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
    launch_paged_decode_mfma(
        reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
        part_acc.data_ptr<float>(), part_ml.data_ptr<float>(),
        reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
        block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (float)scale,
        nseq, nheads, kvh, head_dim, block_size, max_blocks, npart,
        current_stream());
    return;
  }
  DISPATCH_FLOATING(q.scalar_type(), {
    launch_paged_decode<scalar_t>(
        ptr<scalar_t>(out), cptr<scalar_t>(q), cptr<scalar_t>(k_cache),
        cptr<scalar_t>(v_cache), block_tables.data_ptr<int>(),
        seq_lens.data_ptr<int>(), (float)scale, nseq, nheads, kvh, head_dim,
        block_size, max_blocks, current_stream());
  });
}

void paged_attention_prefill(torch::Tensor out, torch::Tensor q,
                             torch::Tensor k_cache, torch::Tensor v_cache,
                             torch::Tensor block_tables,
                             torch::Tensor query_start_loc,
                             torch::Tensor seq_lens, double scale,
                             int64_t max_query_len) {
  const int nseq = seq_lens.size(0);
  const int nheads = q.size(1);
  const int head_dim = q.size(2);
  const int kvh = k_cache.size(2);
  const int block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  static const bool force_valu = [] {
    const char* e = getenv("VTA_PREFILL_VALU");
    return e && e[0] == '1';
  }();
  static const bool force_v1 = [] {
    const char* e = getenv("VTA_PREFILL_V1");
    return e && e[0] == '1';
  }();
  if (k_cache.scalar_type() == at::ScalarType::Byte) {
    TORCH_CHECK(q.scalar_type() == at::ScalarType::BFloat16 && head_dim == 128,
                "fp8 KV cache requires the bf16 v2 prefill path (hd=128)");
    launch_paged_prefill_mfma_v2_fp8(
        reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
        reinterpret_cast<const unsigned char*>(k_cache.data_ptr()),
        reinterpret_cast<const unsigned char*>(v_cache.data_ptr()),
        block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
        seq_lens.data_ptr<int>(), (float)scale, nseq, nheads, kvh, head_dim,
        block_size, max_blocks, (int)max_query_len, current_stream());
    return;
  }
  if (!force_valu && !force_v1 &&
      q.scalar_type() == at::ScalarType::BFloat16 && head_dim == 128) {
    launch_paged_prefill_mfma_v2(
        reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
        block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
        seq_lens.data_ptr<int>(), (float)scale, nseq, nheads, kvh, head_dim,
        block_size, max_blocks, (int)max_query_len, current_stream());
    return;
  }
  if (!force_valu && q.scalar_type() == at::ScalarType::BFloat16 &&
      (head_dim == 64 || head_dim == 128)) {
    launch_paged_prefill_mfma(
        reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
        reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
        block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
        seq_lens.data_ptr<int>(), (float)scale, nseq, nheads, kvh, head_dim,
        block_size, max_blocks, (int)max_query_len, current_stream());
    return;
  }
  DISPATCH_FLOATING(q.scalar_type(), {
    launch_paged_prefill<scalar_t>(
        ptr<scalar_t>(out), cptr<scalar_t>(q), cptr<scalar_t>(k_cache),
        cptr<scalar_t>(v_cache), block_tables.data_ptr<int>(),
        query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(),
        (float)scale, nseq, nheads, kvh, head_dim, block_size, max_blocks,
        (int)max_query_len, current_stream());
  });
}

// Window + sink variants of the bf16 MFMA kernels: position i sees keys j with
// 0 <= i - j < window (0: all j <= i); has_sink: exp(sink) joins the softmax
// denominator.  Key size = value size = 128 (prompt portions) or 64 / 128
// (single queries), up to 8 query heads per key head.
void check_windowed(const torch::Tensor& out, const torch::Tensor& q,
                    const torch::Tensor& k_cache, const torch::Tensor& v_cache,
                    const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                    int64_t window) {
  TORCH_CHECK(q.is_cuda() && q.dim() == 3 && q.is_contiguous() && out.is_contiguous() &&
              out.sizes() == q.sizes(), "q / out must be contiguous [rows, heads, dim]");
  TORCH_CHECK(q.scalar_type() == at::ScalarType::BFloat16 &&
              out.scalar_type() == at::ScalarType::BFloat16 &&
              k_cache.scalar_type() == at::ScalarType::BFloat16 &&
              v_cache.scalar_type() == at::ScalarType::BFloat16, "bf16 only");
  TORCH_CHECK(k_cache.is_contiguous() && v_cache.is_contiguous() && k_cache.dim() == 4 &&
              k_cache.sizes() == v_cache.sizes() && k_cache.size(3) == q.size(2),
              "cache shape");
  const int nheads = q.size(1), kvh = k_cache.size(2);
  TORCH_CHECK(kvh >= 1 && nheads % kvh == 0 && nheads / kvh <= 8, "heads per key head");
  TORCH_CHECK(block_tables.is_cuda() && block_tables.scalar_type() == at::ScalarType::Int &&
              block_tables.dim() == 2 && block_tables.is_contiguous() &&
              block_tables.size(0) >= seq_lens.numel());
  TORCH_CHECK(seq_lens.is_cuda() && seq_lens.scalar_type() == at::ScalarType::Int &&
              seq_lens.is_contiguous());
  TORCH_CHECK(window >= 0, "window");
}

void windowed_attention_prefill(torch::Tensor out, torch::Tensor q,
                                torch::Tensor k_cache, torch::Tensor v_cache,
                                torch::Tensor block_tables,
                                torch::Tensor query_start_loc,
                                torch::Tensor seq_lens, double scale,
                                int64_t max_query_len, int64_t window,
                                bool has_sink, double sink) {
  check_windowed(out, q, k_cache, v_cache, block_tables, seq_lens, window);
  TORCH_CHECK(q.size(2) == 128, "prompt portions need key size 128");
  const int nseq = seq_lens.numel();
  TORCH_CHECK(query_start_loc.is_cuda() && query_start_loc.is_contiguous() &&
              query_start_loc.scalar_type() == at::ScalarType::Int &&
              query_start_loc.numel() == nseq + 1 && max_query_len >= 1);
  if (q.size(0) == 0 || nseq == 0) return;
  launch_paged_prefill_mfma_v2_ws(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
      seq_lens.data_ptr<int>(), (float)scale, nseq, (int)q.size(1),
      (int)k_cache.size(2), 128, (int)k_cache.size(1), (int)block_tables.size(1),
      (int)max_query_len, (int)window, has_sink ? 1 : 0, (float)sink,
      current_stream());
}

void windowed_attention_decode(torch::Tensor out, torch::Tensor q,
                               torch::Tensor k_cache, torch::Tensor v_cache,
                               torch::Tensor block_tables, torch::Tensor seq_lens,
                               double scale, int64_t window, bool has_sink,
                               double sink) {
  check_windowed(out, q, k_cache, v_cache, block_tables, seq_lens, window);
  const int nseq = q.size(0), nheads = q.size(1), head_dim = q.size(2);
  TORCH_CHECK(head_dim == 64 || head_dim == 128, "key size 64 or 128");
  TORCH_CHECK(seq_lens.numel() == nseq, "one query row per sequence expected");
  if (nseq == 0) return;
  const int kvh = k_cache.size(2), block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  // shape-pure split count; a window bounds the keys a query reads
  int span = max_blocks * block_size;
  if (window > 0 && window + 32 < span) span = (int)window + 32;
  const int npart = decode_mfma_num_partitions(nseq, kvh, span);
  const int P = npart * 4;
  auto opts = q.options().dtype(at::ScalarType::Float);
  auto part_acc = at::empty({nseq, nheads, P, head_dim}, opts);
  auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
  launch_paged_decode_mfma_ws(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()), part_acc.data_ptr<float>(),
      part_ml.data_ptr<float>(), reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (float)scale, nseq,
      nheads, kvh, head_dim, block_size, max_blocks, npart, (int)window,
      has_sink ? 1 : 0, (float)sink, current_stream());
}

// Capped variants: scores softcap * tanh(score / softcap) (0: as they are), sinks
// per head or none; window and types as for the window variants, key / value sizes
// 64/64, 96/64, 128/128 or 192/128.
void check_capped(const torch::Tensor& out, const torch::Tensor& q,
                  const torch::Tensor& k_cache, const torch::Tensor& v_cache,
                  const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                  int64_t window, const c10::optional<torch::Tensor>& sinks, double softcap) {
  TORCH_CHECK(softcap >= 0.0 && window >= 0, "softcap and window");
  for (const auto* t : {&out, &q, &k_cache, &v_cache})
    TORCH_CHECK(t->is_cuda() && t->is_contiguous() &&
                t->scalar_type() == at::ScalarType::BFloat16, "contiguous bf16 tensors");
  TORCH_CHECK(q.dim() == 3 && out.dim() == 3 && k_cache.dim() == 4 && v_cache.dim() == 4);
  const int64_t heads = q.size(1), dim = q.size(2), kvh = k_cache.size(2);
  const int64_t vdim = v_cache.size(3);
  TORCH_CHECK((dim == 64 && vdim == 64) || (dim == 96 && vdim == 64) ||
              (dim == 128 && vdim == 128) || (dim == 192 && vdim == 128), "head sizes");
  TORCH_CHECK(out.size(0) == q.size(0) && out.size(1) == heads && out.size(2) == vdim, "out");
  TORCH_CHECK(k_cache.size(3) == dim && v_cache.size(0) == k_cache.size(0) &&
              v_cache.size(1) == k_cache.size(1) && v_cache.size(2) == kvh, "cache shape");
  TORCH_CHECK(kvh >= 1 && heads % kvh == 0 && heads / kvh <= 8, "at most 8 heads per key head");
  TORCH_CHECK(seq_lens.is_cuda() && seq_lens.is_contiguous() &&
              seq_lens.scalar_type() == at::ScalarType::Int);
  TORCH_CHECK(block_tables.is_cuda() && block_tables.is_contiguous() && block_tables.dim() == 2 &&
              block_tables.scalar_type() == at::ScalarType::Int &&
              block_tables.size(0) >= seq_lens.numel(), "block tables");
  if (!sinks.has_value()) return;
  const auto& t = sinks.value();
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::ScalarType::Float &&
              t.numel() == heads, "one f32 sink per head");
}

void capped_attention_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                              torch::Tensor v_cache, torch::Tensor block_tables,
                              torch::Tensor query_start_loc, torch::Tensor seq_lens,
                              double scale, int64_t max_query_len, int64_t window,
                              c10::optional<torch::Tensor> sinks, double softcap) {
  check_capped(out, q, k_cache, v_cache, block_tables, seq_lens, window, sinks, softcap);
  const int nseq = seq_lens.numel();
  TORCH_CHECK(query_start_loc.is_cuda() && query_start_loc.is_contiguous() &&
              query_start_loc.scalar_type() == at::ScalarType::Int &&
              query_start_loc.numel() == nseq + 1 && max_query_len >= 1);
  if (q.size(0) == 0 || nseq == 0) return;
  launch_paged_prefill_mfma_v2_capped(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
      seq_lens.data_ptr<int>(), (float)scale, nseq, (int)q.size(1), (int)k_cache.size(2),
      (int)q.size(2), (int)v_cache.size(3), (int)k_cache.size(1), (int)block_tables.size(1), (int)max_query_len, (int)window,
      sinks.has_value() ? sinks.value().data_ptr<float>() : nullptr, (float)softcap,
      current_stream());
}

void capped_attention_decode(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                             torch::Tensor v_cache, torch::Tensor block_tables,
                             torch::Tensor seq_lens, double scale, int64_t window,
                             c10::optional<torch::Tensor> sinks, double softcap) {
  check_capped(out, q, k_cache, v_cache, block_tables, seq_lens, window, sinks, softcap);
  const int nseq = q.size(0), nheads = q.size(1), dim = q.size(2), vdim = v_cache.size(3);
  TORCH_CHECK(seq_lens.numel() == nseq, "one query row per sequence expected");
  if (nseq == 0) return;
  const int kvh = k_cache.size(2), block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  int span = max_blocks * block_size;
  if (window > 0 && window + 32 < span) span = (int)window + 32;
  const int npart = decode_mfma_num_partitions(nseq, kvh, span);
  const int P = npart * 4;
  auto opts = q.options().dtype(at::ScalarType::Float);
  auto part_acc = at::empty({nseq, nheads, P, vdim}, opts);
  auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
  launch_paged_decode_mfma_capped(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()), part_acc.data_ptr<float>(),
      part_ml.data_ptr<float>(), reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (float)scale, nseq, nheads, kvh,
      dim, vdim, block_size, max_blocks, npart, (int)window,
      sinks.has_value() ? sinks.value().data_ptr<float>() : nullptr, (float)softcap,
      current_stream());
}

// Chunk variants of the bf16 MFMA kernels: position i sees keys j <= i with
// floor(j / chunk) = floor(i / chunk) (0: all j <= i); the value cache may hold
// fewer heads than the key cache (key head g reads value head g mod Gv); the
// output is f32.  Sizes as for the window variants.
void check_chunked(const torch::Tensor& out, const torch::Tensor& q,
                   const torch::Tensor& k_cache, const torch::Tensor& v_cache,
                   const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                   int64_t chunk) {
  TORCH_CHECK(q.is_cuda() && q.dim() == 3 && q.is_contiguous() && out.is_cuda() &&
              out.is_contiguous() && out.sizes() == q.sizes(),
              "q / out must be contiguous [rows, heads, dim]");
  TORCH_CHECK(q.scalar_type() == at::ScalarType::BFloat16 &&
              out.scalar_type() == at::ScalarType::Float &&
              k_cache.scalar_type() == at::ScalarType::BFloat16 &&
              v_cache.scalar_type() == at::ScalarType::BFloat16, "bf16 in, f32 out");
  TORCH_CHECK(k_cache.is_cuda() && v_cache.is_cuda() && k_cache.is_contiguous() &&
              v_cache.is_contiguous() && k_cache.dim() == 4 && v_cache.dim() == 4 &&
              k_cache.size(0) == v_cache.size(0) && k_cache.size(1) == v_cache.size(1) &&
              k_cache.size(3) == q.size(2) && v_cache.size(3) == q.size(2),
              "cache shape");
  const int nheads = q.size(1), kvh = k_cache.size(2), vh = v_cache.size(2);
  TORCH_CHECK(kvh >= 1 && nheads % kvh == 0 && nheads / kvh <= 8, "heads per key head");
  TORCH_CHECK(vh >= 1 && kvh % vh == 0, "key heads per value head");
  TORCH_CHECK(block_tables.is_cuda() && block_tables.scalar_type() == at::ScalarType::Int &&
              block_tables.dim() == 2 && block_tables.is_contiguous() &&
              block_tables.size(0) >= seq_lens.numel());
  TORCH_CHECK(seq_lens.is_cuda() && seq_lens.scalar_type() == at::ScalarType::Int &&
              seq_lens.is_contiguous());
  TORCH_CHECK(chunk >= 0, "chunk");
}

void chunk_attention_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                             torch::Tensor v_cache, torch::Tensor block_tables,
                             torch::Tensor query_start_loc, torch::Tensor seq_lens,
                             double scale, int64_t max_query_len, int64_t chunk) {
  check_chunked(out, q, k_cache, v_cache, block_tables, seq_lens, chunk);
  TORCH_CHECK(q.size(2) == 128, "prompt portions need key size 128");
  const int nseq = seq_lens.numel();
  TORCH_CHECK(query_start_loc.is_cuda() && query_start_loc.is_contiguous() &&
              query_start_loc.scalar_type() == at::ScalarType::Int &&
              query_start_loc.numel() == nseq + 1 && max_query_len >= 1);
  if (q.size(0) == 0 || nseq == 0) return;
  launch_paged_prefill_mfma_v2_chunk(
      out.data_ptr<float>(), reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
      seq_lens.data_ptr<int>(), (float)scale, nseq, (int)q.size(1),
      (int)k_cache.size(2), (int)v_cache.size(2), (int)k_cache.size(1),
      (int)block_tables.size(1), (int)max_query_len, (int)chunk, current_stream());
}

void chunk_attention_decode(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                            torch::Tensor v_cache, torch::Tensor block_tables,
                            torch::Tensor seq_lens, double scale, int64_t chunk) {
  check_chunked(out, q, k_cache, v_cache, block_tables, seq_lens, chunk);
  const int nseq = q.size(0), nheads = q.size(1), head_dim = q.size(2);
  TORCH_CHECK(head_dim == 64 || head_dim == 128, "key size 64 or 128");
  TORCH_CHECK(seq_lens.numel() == nseq, "one query row per sequence expected");
  if (nseq == 0) return;
  const int kvh = k_cache.size(2), block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  // shape-pure split count; a chunk bounds the keys a query reads
  int span = max_blocks * block_size;
  if (chunk > 0 && chunk + 32 < span) span = (int)chunk + 32;
  const int npart = decode_mfma_num_partitions(nseq, kvh, span);
  const int P = npart * 4;
  auto opts = q.options().dtype(at::ScalarType::Float);
  auto part_acc = at::empty({nseq, nheads, P, head_dim}, opts);
  auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
  launch_paged_decode_mfma_chunk(
      out.data_ptr<float>(), part_acc.data_ptr<float>(), part_ml.data_ptr<float>(),
      reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()),
      block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (float)scale, nseq,
      nheads, kvh, (int)v_cache.size(2), head_dim, block_size, max_blocks, npart,
      (int)chunk, current_stream());
}

// Prefix variants of the bf16 MFMA kernels: a window (> 0) and, beside it, the
// first `keep` tokens or one pooled key and value per block of `pool` positions
// that ends at or before the window (pooled block b lives in the cache block of
// its last token).  back_table [rows, dim/2, 2] f32: the output's dims m and
// m + dim/2 are turned back by the row's angles.  Sizes as for the window
// variants.  Returns the places per cache block.
int check_span(const torch::Tensor& out, const torch::Tensor& q,
               const torch::Tensor& k_cache, const torch::Tensor& v_cache,
               const c10::optional<torch::Tensor>& k_pool,
               const c10::optional<torch::Tensor>& v_pool,
               const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
               int64_t window, int64_t keep, int64_t pool,
               const c10::optional<torch::Tensor>& back) {
  check_windowed(out, q, k_cache, v_cache, block_tables, seq_lens, window);
  TORCH_CHECK(window > 0 && keep >= 0 && pool >= 0 && !(keep && pool), "mask");
  if (back.has_value()) {
    const auto& b = back.value();
    TORCH_CHECK(b.is_cuda() && b.is_contiguous() &&
                b.scalar_type() == at::ScalarType::Float &&
                b.numel() == q.size(0) * q.size(2), "back_table is [rows, dim / 2, 2]");
  }
  if (pool == 0) return 0;
  TORCH_CHECK(k_pool.has_value() && v_pool.has_value(), "pooled caches missing");
  const auto &kp = k_pool.value(), &vp = v_pool.value();
  const int64_t per_block = (k_cache.size(1) + pool - 1) / pool;
  TORCH_CHECK(kp.is_cuda() && kp.is_contiguous() && vp.is_cuda() && vp.is_contiguous() &&
              kp.scalar_type() == at::ScalarType::BFloat16 &&
              vp.scalar_type() == at::ScalarType::BFloat16 && kp.dim() == 4 &&
              kp.sizes() == vp.sizes() && kp.size(0) == k_cache.size(0) &&
              kp.size(1) == per_block && kp.size(2) == k_cache.size(2) &&
              kp.size(3) == k_cache.size(3), "pooled caches do not fit the caches");
  return (int)per_block;
}

const __hip_bfloat16* bf16_or_null(const c10::optional<torch::Tensor>& t) {
  return t.has_value() ? reinterpret_cast<const __hip_bfloat16*>(t.value().data_ptr())
                       : nullptr;
}

void span_attention_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                            torch::Tensor v_cache, c10::optional<torch::Tensor> k_pool,
                            c10::optional<torch::Tensor> v_pool,
                            torch::Tensor block_tables, torch::Tensor query_start_loc,
                            torch::Tensor seq_lens, double scale, int64_t max_query_len,
                            int64_t window, int64_t keep, int64_t pool,
                            c10::optional<torch::Tensor> back) {
  const int per_block = check_span(out, q, k_cache, v_cache, k_pool, v_pool, block_tables,
                                   seq_lens, window, keep, pool, back);
  TORCH_CHECK(q.size(2) == 128, "prompt portions need key size 128");
  const int nseq = seq_lens.numel();
  TORCH_CHECK(query_start_loc.is_cuda() && query_start_loc.is_contiguous() &&
              query_start_loc.scalar_type() == at::ScalarType::Int &&
              query_start_loc.numel() == nseq + 1 && max_query_len >= 1);
  if (q.size(0) == 0 || nseq == 0) return;
  launch_paged_prefill_mfma_v2_span(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()), bf16_or_null(k_pool),
      bf16_or_null(v_pool), block_tables.data_ptr<int>(), query_start_loc.data_ptr<int>(),
      seq_lens.data_ptr<int>(), (float)scale, nseq, (int)q.size(1), (int)k_cache.size(2),
      (int)k_cache.size(1), per_block, (int)block_tables.size(1), (int)max_query_len,
      (int)window, (int)keep, (int)pool,
      back.has_value() ? back.value().data_ptr<float>() : nullptr, current_stream());
}

void span_attention_decode(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                           torch::Tensor v_cache, c10::optional<torch::Tensor> k_pool,
                           c10::optional<torch::Tensor> v_pool, torch::Tensor block_tables,
                           torch::Tensor seq_lens, double scale, int64_t window,
                           int64_t keep, int64_t pool, c10::optional<torch::Tensor> back) {
  const int per_block = check_span(out, q, k_cache, v_cache, k_pool, v_pool, block_tables,
                                   seq_lens, window, keep, pool, back);
  const int nseq = q.size(0), nheads = q.size(1), head_dim = q.size(2);
  TORCH_CHECK(head_dim == 64 || head_dim == 128, "key size 64 or 128");
  TORCH_CHECK(seq_lens.numel() == nseq, "one query row per sequence expected");
  if (nseq == 0) return;
  const int kvh = k_cache.size(2), block_size = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  // shape-pure split count: window and prefix bound the keys a query reads
  const int64_t ctx = (int64_t)max_blocks * block_size;
  const int64_t span = std::min(ctx, window + 32) +
                       (pool > 0 ? ctx / pool + 32 : std::min(ctx, keep + 32));
  const int npart = decode_mfma_num_partitions(nseq, kvh, (int)span);
  const int P = npart * 4;
  auto opts = q.options().dtype(at::ScalarType::Float);
  auto part_acc = at::empty({nseq, nheads, P, head_dim}, opts);
  auto part_ml = at::empty({nseq, nheads, P, 2}, opts);
  launch_paged_decode_mfma_span(
      reinterpret_cast<__hip_bfloat16*>(out.data_ptr()), part_acc.data_ptr<float>(),
      part_ml.data_ptr<float>(), reinterpret_cast<const __hip_bfloat16*>(q.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(k_cache.data_ptr()),
      reinterpret_cast<const __hip_bfloat16*>(v_cache.data_ptr()), bf16_or_null(k_pool),
      bf16_or_null(v_pool), block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(),
      (float)scale, nseq, nheads, kvh, head_dim, block_size, per_block, max_blocks, npart,
      (int)window, (int)keep, (int)pool,
      back.has_value() ? back.value().data_ptr<float>() : nullptr, current_stream());
}

}  // namespace

void register_attention_ops(pybind11::module& m) {
  m.def("span_attention_prefill", &span_attention_prefill,
        "paged prefill attention over a window plus a prefix (CDNA4)");
  m.def("span_attention_decode", &span_attention_decode,
        "paged decode attention over a window plus a prefix (CDNA4)");
  m.def("chunk_attention_prefill", &chunk_attention_prefill,
        "paged chunk-masked prefill attention, f32 out (CDNA4)");
  m.def("chunk_attention_decode", &chunk_attention_decode,
        "paged chunk-masked decode attention, f32 out (CDNA4)");
  m.def("windowed_attention_prefill", &windowed_attention_prefill,
        "paged windowed prefill attention with a softmax sink (CDNA4)");
  m.def("capped_attention_prefill", &capped_attention_prefill,
        "paged windowed prefill attention, soft-capped scores, sinks per head (CDNA4)");
  m.def("capped_attention_decode", &capped_attention_decode,
        "paged windowed decode attention, soft-capped scores, sinks per head (CDNA4)");
  m.def("windowed_attention_decode", &windowed_attention_decode,
        "paged windowed decode attention with a softmax sink (CDNA4)");
  m.def("paged_attention_decode", &paged_attention_decode,
        "paged decode attention (CDNA4)");
  m.def("paged_attention_prefill", &paged_attention_prefill,
        "paged causal prefill attention (CDNA4)");
}
