// Row kernels of layers whose norms keep no statistics and whose attention norms
// queries and keys over the whole projection.
//
//   stream_add_tanh_norm  x += F(a + b), then F' of the updated x, with F(y) =
//                         tanh(alpha y) w + bias
//   wide_norm             projected rows [q | k | v] -> bias, RMS norm over all
//                         query heads and over all key heads, values mixed with
//                         an earlier layer's cached values, paged cache write
//   clamped_glu           g sigmoid(1.702 g) (u + 1), g = min(gate, limit), u = up
//                         clamped to +-limit, times a weight per expert
//   router_logits         rows times a small f32 matrix, in f32 on the matrix cores;
//                         route_experts: and the choice of experts from them
//   scale_logits          f32 copy times a constant
//
// All memory-bound.  Statistics, tanh, gates, mixing and the stream are f32
// whatever the storage type; every result is rounded once.

#include "moe_route.h"

namespace {

// eight elements as they are stored
template <typename T> struct Raw8;
template <> struct Raw8<__hip_bfloat16> { uint4 u; };
template <> struct Raw8<float> { float4 a, b; };
template <typename T>
DEVINLINE Raw8<T> ldraw(const T* p) { return *reinterpret_cast<const Raw8<T>*>(p); }
DEVINLINE void unpack8(const Raw8<float>& r, float* f) {
  f[0] = r.a.x; f[1] = r.a.y; f[2] = r.a.z; f[3] = r.a.w;
  f[4] = r.b.x; f[5] = r.b.y; f[6] = r.b.z; f[7] = r.b.w;
}
DEVINLINE void unpack8(const Raw8<__hip_bfloat16>& r, float* f) {
  const unsigned u[4] = {r.u.x, r.u.y, r.u.z, r.u.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f[2 * i] = __uint_as_float(u[i] << 16);
    f[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u);
  }
}
template <typename T>
DEVINLINE void ld8(const T* p, float* f) { unpack8(ldraw<T>(p), f); }
template <typename T> DEVINLINE void st8(T* p, const float* f);
template <> DEVINLINE void st8<float>(float* p, const float* f) {
  reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
  reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
}
template <> DEVINLINE void st8<__hip_bfloat16>(__hip_bfloat16* p, const float* f) {
  union { __hip_bfloat16 h[8]; uint4 u; } o;
#pragma unroll
  for (int i = 0; i < 8; ++i) o.h[i] = __float2bfloat16(f[i]);
  *reinterpret_cast<uint4*>(p) = o.u;
}

// ---------------------------------------------------------------------------
// stream_add_tanh_norm.  A thread owns N neighbouring columns of ROWS rows, so
// that the norms' vectors are read once for all of them.
// ---------------------------------------------------------------------------
template <typename T, int N> struct Cols;
template <typename T> struct Cols<T, 4> {
  static DEVINLINE void load(const T* p, float* f);
  static DEVINLINE void store(T* p, const float* f);
};
template <> DEVINLINE void Cols<float, 4>::load(const float* p, float* f) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  f[0] = t.x; f[1] = t.y; f[2] = t.z; f[3] = t.w;
}
template <> DEVINLINE void Cols<float, 4>::store(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
}
template <> DEVINLINE void Cols<__hip_bfloat16, 4>::load(const __hip_bfloat16* p, float* f) {
  const uint2 t = *reinterpret_cast<const uint2*>(p);
  f[0] = __uint_as_float(t.x << 16); f[1] = __uint_as_float(t.x & 0xffff0000u);
  f[2] = __uint_as_float(t.y << 16); f[3] = __uint_as_float(t.y & 0xffff0000u);
}
template <> DEVINLINE void Cols<__hip_bfloat16, 4>::store(__hip_bfloat16* p, const float* f) {
  union { __hip_bfloat16 h[4]; uint2 u; } o;
#pragma unroll
  for (int i = 0; i < 4; ++i) o.h[i] = __float2bfloat16(f[i]);
  *reinterpret_cast<uint2*>(p) = o.u;
}
template <typename T> struct Cols<T, 1> {
  static DEVINLINE void load(const T* p, float* f) { f[0] = ScalarOps<T>::to_f32(*p); }
  static DEVINLINE void store(T* p, const float* f) { *p = ScalarOps<T>::from_f32(f[0]); }
};

template <typename T, int N, int ROWS>
__global__ __launch_bounds__(256) void stream_add_tanh_norm_kernel(
    float* __restrict__ x, const T* __restrict__ a, const T* __restrict__ b, float alpha,
    const float* __restrict__ w, const float* __restrict__ bias, float next_alpha,
    const float* __restrict__ next_w, const float* __restrict__ next_bias,
    T* __restrict__ next_out, int rows, int width) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * N;
  if (c >= width) return;
  const int r0 = blockIdx.y * ROWS;
  float xv[ROWS][N], y[ROWS][N];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    if (r0 + r >= rows) break;
    const long at = (long)(r0 + r) * width + c;
    Cols<float, N>::load(x + at, xv[r]);
    if (a != nullptr) {
      Cols<T, N>::load(a + at, y[r]);
      if (b != nullptr) {
        float z[N];
        Cols<T, N>::load(b + at, z);
#pragma unroll
        for (int k = 0; k < N; ++k) y[r][k] += z[k];
      }
    }
  }
  float wv[N], bv[N], nw[N], nb[N];
  if (a != nullptr) {
    Cols<float, N>::load(w + c, wv);
    Cols<float, N>::load(bias + c, bv);
  }
  if (next_out != nullptr) {
    Cols<float, N>::load(next_w + c, nw);
    Cols<float, N>::load(next_bias + c, nb);
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    if (r0 + r >= rows) break;
    const long at = (long)(r0 + r) * width + c;
    if (a != nullptr) {
#pragma unroll
      for (int k = 0; k < N; ++k) xv[r][k] += tanh_f32(alpha * y[r][k]) * wv[k] + bv[k];
      Cols<float, N>::store(x + at, xv[r]);
    }
    if (next_out != nullptr) {
#pragma unroll
      for (int k = 0; k < N; ++k) y[r][k] = tanh_f32(next_alpha * xv[r][k]) * nw[k] + nb[k];
      Cols<T, N>::store(next_out + at, y[r]);
    }
  }
}

// ---------------------------------------------------------------------------
// wide_norm.  Channel order [H * dim queries | G * dim keys | G * vdim values].
// ---------------------------------------------------------------------------
template <typename T>
struct WideIn {
  const T* proj; long st;
  const float* bias;                 // [C] or null
  const float* qw; const float* kw;  // [nq], [nk]
  const T* v_first; float v_mix;     // the earlier layer's value cache or null
  T* q_out; T* k_cache; T* v_cache;
  const long* slot_mapping;
  int rows, nq, nk, nv;
  float eps;
};

// NV vectors of eight per thread, a row in registers from read to write; the
// biases and weights of a thread's channels serve ROWS rows.
template <typename T, int NV, int ROWS>
__global__ __launch_bounds__(256) void wide_norm_vec_kernel(WideIn<T> p) {
  __shared__ float red[2][2][4];
  const int lane = threadIdx.x & (WAVE_SIZE - 1), wave = threadIdx.x / WAVE_SIZE;
  const int total = p.nq + p.nk + p.nv;
  const int row_end = min(p.rows, (int)(blockIdx.x + 1) * ROWS);
  float bias[NV][8], w[NV][8];
  auto chan = [&](int i) { return (threadIdx.x + i * 256) * 8; };
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = chan(i);
#pragma unroll
    for (int k = 0; k < 8; ++k) { bias[i][k] = 0.f; w[i][k] = 1.f; }
    if (c < total && p.bias != nullptr) ld8<float>(p.bias + c, bias[i]);
    if (c < p.nq) ld8<float>(p.qw + c, w[i]);
    else if (c < p.nq + p.nk) ld8<float>(p.kw + c - p.nq, w[i]);
  }
  Raw8<T> cur[NV];
  auto fetch = [&](int row) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (chan(i) < total) cur[i] = ldraw<T>(p.proj + (long)row * p.st + chan(i));
  };
  fetch(blockIdx.x * ROWS);
  for (int row = blockIdx.x * ROWS, par = 0; row < row_end; ++row, par ^= 1) {
    const long slot = p.slot_mapping[row];
    float y[NV][8];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = chan(i);
      if (c >= total) continue;
      unpack8(cur[i], y[i]);
      float s = 0.f;
#pragma unroll
      for (int k = 0; k < 8; ++k) { y[i][k] += bias[i][k]; s += y[i][k] * y[i][k]; }
      if (c < p.nq) sq += s;
      else if (c < p.nq + p.nk) sk += s;
    }
    if (row + 1 < row_end) fetch(row + 1);
    sq = wave_reduce_sum(sq);
    sk = wave_reduce_sum(sk);
    if (lane == 0) { red[par][0][wave] = sq; red[par][1][wave] = sk; }
    __syncthreads();   // the other half of red is free again after this one
    sq = sk = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) { sq += red[par][0][i]; sk += red[par][1][i]; }
    const float iq = 1.0f / sqrtf(sq / p.nq + p.eps), ik = 1.0f / sqrtf(sk / p.nk + p.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = chan(i);
      if (c >= total) continue;
      if (c < p.nq) {
#pragma unroll
        for (int k = 0; k < 8; ++k) y[i][k] *= iq * w[i][k];
        st8<T>(p.q_out + (long)row * p.nq + c, y[i]);
      } else if (slot >= 0 && c < p.nq + p.nk) {
#pragma unroll
        for (int k = 0; k < 8; ++k) y[i][k] *= ik * w[i][k];
        st8<T>(p.k_cache + slot * p.nk + c - p.nq, y[i]);
      } else if (slot >= 0) {
        const int cv = c - p.nq - p.nk;
        if (p.v_first != nullptr) {
          float f[8];
          ld8<T>(p.v_first + slot * p.nv + cv, f);
#pragma unroll
          for (int k = 0; k < 8; ++k) y[i][k] = (1.0f - p.v_mix) * y[i][k] + p.v_mix * f[k];
        }
        st8<T>(p.v_cache + slot * p.nv + cv, y[i]);
      }
    }
  }
}

// any sizes: inputs re-read from cache between statistic and output
template <typename T>
__global__ __launch_bounds__(256) void wide_norm_kernel(WideIn<T> p) {
  __shared__ float red[8];
  const long row = blockIdx.x;
  const long slot = p.slot_mapping[row];
  const T* src = p.proj + row * p.st;
  auto at = [&](int c) {
    return ScalarOps<T>::to_f32(src[c]) + (p.bias != nullptr ? p.bias[c] : 0.f);
  };
  auto inv_rms = [&](int c0, int n) {
    float s = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) { const float y = at(c0 + c); s += y * y; }
    const float tot = block_reduce_sum(s, red);
    __syncthreads();   // red is used again
    return 1.0f / sqrtf(tot / n + p.eps);
  };
  const float iq = inv_rms(0, p.nq), ik = inv_rms(p.nq, p.nk);
  for (int c = threadIdx.x; c < p.nq; c += 256)
    p.q_out[row * p.nq + c] = ScalarOps<T>::from_f32(at(c) * iq * p.qw[c]);
  if (slot < 0) return;
  for (int c = threadIdx.x; c < p.nk; c += 256)
    p.k_cache[slot * p.nk + c] = ScalarOps<T>::from_f32(at(p.nq + c) * ik * p.kw[c]);
  for (int c = threadIdx.x; c < p.nv; c += 256) {
    float v = at(p.nq + p.nk + c);
    if (p.v_first != nullptr)
      v = (1.0f - p.v_mix) * v + p.v_mix * ScalarOps<T>::to_f32(p.v_first[slot * p.nv + c]);
    p.v_cache[slot * p.nv + c] = ScalarOps<T>::from_f32(v);
  }
}

// ---------------------------------------------------------------------------
// clamped_glu.  gu [T, E, 2, ff] -> out [T, E, ff]; n counts groups of N outputs.
// ---------------------------------------------------------------------------
template <typename T, int N>
__global__ void clamped_glu_kernel(T* __restrict__ out, const T* __restrict__ gu, float limit,
                                   const float* __restrict__ col_scale, int ff, long n) {
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < n;
       i += (long)gridDim.x * blockDim.x) {
    const long e = i * N;
    const long te = e / ff;          // token * E + expert
    const T* gp = gu + te * 2 * ff + (e - te * ff);
    const float sc = col_scale != nullptr ? col_scale[te] : 1.0f;
    float g[N], u[N];
    if constexpr (N == 8) {
      ld8<T>(gp, g);
      ld8<T>(gp + ff, u);
    } else {
      g[0] = ScalarOps<T>::to_f32(gp[0]);
      u[0] = ScalarOps<T>::to_f32(gp[ff]);
    }
#pragma unroll
    for (int k = 0; k < N; ++k) g[k] = clamped_gate(g[k], u[k], limit) * sc;
    if constexpr (N == 8) st8<T>(out + e, g);
    else out[e] = ScalarOps<T>::from_f32(g[0]);
  }
}

// ---------------------------------------------------------------------------
// router_logits: out [T, E] = h [T, W] . w [E, W]^T in f32.  A workgroup has 16
// rows and NT tiles of 16 experts; its waves split the width in interleaved pieces
// of 32 and are summed through LDS.  A lane loads eight consecutive elements of row
// (or expert) lane % 16, the eight of slot lane / 16.  bf16 rows and weights go
// straight to v_mfma_f32_16x16x32_bf16, whose products are exact in f32; with f32 on
// either side they are fed one by one to v_mfma_f32_16x16x4_f32, slot s of
// instruction j being element 8 s + j on both sides.
// ---------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(8))) short bf16x8_t;
constexpr int RL_WAVES = 16;

DEVINLINE f32x4_t router_mfma(const Raw8<__hip_bfloat16>& a, const Raw8<__hip_bfloat16>& b,
                              f32x4_t acc) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a.u),
                                                 __builtin_bit_cast(bf16x8_t, b.u), acc, 0, 0, 0);
}
template <typename A, typename B>
DEVINLINE f32x4_t router_mfma(const Raw8<A>& a, const Raw8<B>& b, f32x4_t acc) {
  float x[8], y[8];
  unpack8(a, x);
  unpack8(b, y);
#pragma unroll
  for (int j = 0; j < 8; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], y[j], acc, 0, 0, 0);
  return acc;
}

// z_s [16][NT * 16]: the logits of rows row0 .. row0 + 15, experts e0 ..
template <typename T, typename W, int NT>
DEVINLINE void router_tile(float* z_s, float* part, const T* __restrict__ h, long h_st,
                           const W* __restrict__ w, int row0, int e0, int rows, int experts,
                           int width) {
  // pieces loaded ahead of the products
  constexpr int FLY = (sizeof(T) == 2 && sizeof(W) == 2 ? 8 : 4) / NT;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int i = lane & 15, s = lane >> 4;
  // rows and experts past the end are clamped: they compute and are not used
  const T* hp = h + (long)min(row0 + i, rows - 1) * h_st + s * 8;
  const W* wp[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
    wp[t] = w + (long)min(e0 + t * 16 + i, experts - 1) * width + s * 8;
  f32x4_t acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4_t{};
  for (int c0 = wave * 32; c0 < width; c0 += FLY * RL_WAVES * 32) {
    Raw8<T> a[FLY];
    Raw8<W> b[FLY][NT];
#pragma unroll
    for (int f = 0; f < FLY; ++f) {
      const int c = c0 + f * RL_WAVES * 32;
      a[f] = Raw8<T>{};
#pragma unroll
      for (int t = 0; t < NT; ++t) b[f][t] = Raw8<W>{};
      if (c < width) {               // uniform over the wave
        a[f] = ldraw<T>(hp + c);
#pragma unroll
        for (int t = 0; t < NT; ++t) b[f][t] = ldraw<W>(wp[t] + c);
      }
    }
#pragma unroll
    for (int f = 0; f < FLY; ++f)
#pragma unroll
      for (int t = 0; t < NT; ++t) acc[t] = router_mfma(a[f], b[f][t], acc[t]);
  }
  // lane holds element [4 * (lane / 16) + r][lane % 16] of a tile
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      part[wave * NT * 256 + (4 * s + r) * NT * 16 + t * 16 + i] = acc[t][r];
  __syncthreads();
  for (int x = threadIdx.x; x < NT * 256; x += RL_WAVES * 64) {
    float z = 0.f;
#pragma unroll
    for (int k = 0; k < RL_WAVES; ++k) z += part[k * NT * 256 + x];
    z_s[x] = z;
  }
  __syncthreads();
}

template <typename T, typename W, int NT>
__global__ __launch_bounds__(RL_WAVES * 64) void router_logits_kernel(
    float* __restrict__ out, const T* __restrict__ h, long h_st,
    const W* __restrict__ w, int rows, int experts, int width) {
  __shared__ float part[RL_WAVES * NT * 256], z_s[NT * 256];
  const int row0 = blockIdx.x * 16, e0 = blockIdx.y * NT * 16;
  router_tile<T, W, NT>(z_s, part, h, h_st, w, row0, e0, rows, experts, width);
  for (int x = threadIdx.x; x < NT * 256; x += RL_WAVES * 64) {
    const int r = row0 + x / (NT * 16), e = e0 + x % (NT * 16);
    if (r < rows && e < experts) out[(long)r * experts + e] = z_s[x];
  }
}

// a wave per row chooses from the logits in LDS (at most NT * 16 experts)
template <typename T, typename W, int NT>
__global__ __launch_bounds__(RL_WAVES * 64) void route_experts_kernel(
    float* __restrict__ dense, int* __restrict__ ids, float* __restrict__ wts,
    const T* __restrict__ h, long h_st, const W* __restrict__ w, int rows, int width,
    RouteRule rule) {
  __shared__ float part[RL_WAVES * NT * 256], z_s[NT * 256];
  const int row0 = blockIdx.x * 16, wave = threadIdx.x >> 6;
  router_tile<T, W, NT>(z_s, part, h, h_st, w, row0, 0, rows, rule.n, width);
  const long t = row0 + wave;
  if (t >= rows) return;
  moe_route_lanes<1>(z_s + wave * NT * 16, rule, dense + t * rule.n, nullptr, ids + t * rule.top,
                     wts + t * rule.top);
}

// any width: one wave per (row, expert)
template <typename T, typename W>
__global__ __launch_bounds__(256) void router_logits_any_kernel(
    float* __restrict__ out, const T* __restrict__ h, long h_st,
    const W* __restrict__ w, int rows, int experts, int width) {
  const long id = blockIdx.x * 4L + threadIdx.x / WAVE_SIZE;
  if (id >= (long)rows * experts) return;
  const long row = id / experts;
  const int e = (int)(id - row * experts);
  float z = 0.f;
  for (int c = threadIdx.x & (WAVE_SIZE - 1); c < width; c += WAVE_SIZE)
    z += ScalarOps<T>::to_f32(h[row * h_st + c]) * ScalarOps<W>::to_f32(w[(long)e * width + c]);
  z = wave_reduce_sum(z);
  if ((threadIdx.x & (WAVE_SIZE - 1)) == 0) out[id] = z;
}

template <typename T>
__global__ void scale_logits_kernel(float* __restrict__ out, const T* __restrict__ x, float scale,
                                    int vec, long n) {
  const long i = (blockIdx.x * (long)blockDim.x + threadIdx.x) * 8;
  if (i >= n) return;
  if (vec && i + 8 <= n) {
    float f[8];
    ld8<T>(x + i, f);
#pragma unroll
    for (int k = 0; k < 8; ++k) f[k] *= scale;
    st8<float>(out + i, f);
  } else {
    for (long k = i; k < min(i + 8, n); ++k) out[k] = ScalarOps<T>::to_f32(x[k]) * scale;
  }
}

bool al(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

}  // namespace

template <typename T>
void launch_stream_add_tanh_norm(float* x, const T* a, const T* b, float alpha, const float* w,
                                 const float* bias, float next_alpha, const float* next_w,
                                 const float* next_bias, T* next_out, int rows, int width,
                                 hipStream_t s) {
  const size_t tb = 4 * sizeof(T);
  const bool vec = width % 4 == 0 && al(x, 16) && al(a, tb) && al(b, tb) && al(w, 16) &&
                   al(bias, 16) && al(next_w, 16) && al(next_bias, 16) && al(next_out, tb);
#define TANH_LAUNCH(N, R)                                                                     \
  stream_add_tanh_norm_kernel<T, N, R>                                                        \
      <<<dim3((width + 256 * N - 1) / (256 * N), (rows + R - 1) / R), 256, 0, s>>>(           \
          x, a, b, alpha, w, bias, next_alpha, next_w, next_bias, next_out, rows, width)
  if (!vec && rows < 65536) TANH_LAUNCH(1, 1);
  else if (!vec) TANH_LAUNCH(1, 4);
  else if (rows < 1024) TANH_LAUNCH(4, 1);
  else TANH_LAUNCH(4, 4);
#undef TANH_LAUNCH
}

template <typename T>
void launch_wide_norm(T* q_out, const T* proj, long st, const float* bias, const float* qw,
                      const float* kw, const T* v_first, float v_mix, T* k_cache, T* v_cache,
                      const long* slot_mapping, int rows, int nq, int nk, int nv, float eps,
                      hipStream_t s) {
  WideIn<T> p;
  p.proj = proj; p.st = st; p.bias = bias; p.qw = qw; p.kw = kw;
  p.v_first = v_first; p.v_mix = v_mix;
  p.q_out = q_out; p.k_cache = k_cache; p.v_cache = v_cache; p.slot_mapping = slot_mapping;
  p.rows = rows; p.nq = nq; p.nk = nk; p.nv = nv; p.eps = eps;
  const int vecs = (nq + nk + nv) / 8, per = (vecs + 255) / 256;
  const bool vec = nq % 8 == 0 && nk % 8 == 0 && nv % 8 == 0 && st % 8 == 0 && per <= 8 &&
                   al(proj, 16) && al(bias, 16) && al(qw, 16) && al(kw, 16) && al(v_first, 16) &&
                   al(q_out, 16) && al(k_cache, 16) && al(v_cache, 16);
#define WIDE_LAUNCH(NV)                                                                \
  if (rows < 2048) wide_norm_vec_kernel<T, NV, 1><<<rows, 256, 0, s>>>(p);             \
  else wide_norm_vec_kernel<T, NV, 4><<<(rows + 3) / 4, 256, 0, s>>>(p)
  if (!vec) wide_norm_kernel<T><<<rows, 256, 0, s>>>(p);
  else if (per == 1) { WIDE_LAUNCH(1); }
  else if (per == 2) { WIDE_LAUNCH(2); }
  else if (per == 3) { WIDE_LAUNCH(3); }
  else if (per == 4) { WIDE_LAUNCH(4); }
  else { WIDE_LAUNCH(8); }
#undef WIDE_LAUNCH
}

template <typename T>
void launch_clamped_glu(T* out, const T* gu, float limit, const float* col_scale, int ff,
                        long n, hipStream_t s) {
  const bool vec = ff % 8 == 0 && al(out, 16) && al(gu, 16);
  const long work = vec ? n / 8 : n;
  const int blocks = (int)((work + 255) / 256 > 65536 ? 65536 : (work + 255) / 256);
  if (vec) clamped_glu_kernel<T, 8><<<blocks, 256, 0, s>>>(out, gu, limit, col_scale, ff, work);
  else clamped_glu_kernel<T, 1><<<blocks, 256, 0, s>>>(out, gu, limit, col_scale, ff, work);
}

template <typename T, typename W>
void launch_router_logits(float* out, const T* h, long h_st, const W* w, int rows,
                          int experts, int width, hipStream_t s) {
  const int tiles = (experts + 15) / 16;
#define ROUTER_LAUNCH(NT)                                                              \
  router_logits_kernel<T, W, NT><<<dim3((rows + 15) / 16, (tiles + NT - 1) / NT),         \
                                RL_WAVES * 64, 0, s>>>(out, h, h_st, w, rows, experts, width)
  if (width % 32 || h_st % 8 || !al(h, 16) || !al(w, 16))
    router_logits_any_kernel<T, W><<<(int)(((long)rows * experts + 3) / 4), 256, 0, s>>>(
        out, h, h_st, w, rows, experts, width);
  else if (tiles == 1) ROUTER_LAUNCH(1);
  else if (tiles == 2) ROUTER_LAUNCH(2);
  else ROUTER_LAUNCH(4);
#undef ROUTER_LAUNCH
}

// at most 64 experts, width a multiple of 32, 16-byte aligned rows
template <typename T, typename W>
void launch_route_experts(float* dense, int* ids, float* wts, const T* h, long h_st,
                          const W* w, const float* correction, int rows, int experts,
                          int width, int top, int groups, int keep, int renorm, float scale,
                          hipStream_t s) {
  const RouteRule rule{correction, experts, experts, top, 1, groups, keep, renorm, scale};
#define ROUTE_LAUNCH(NT)                                                               \
  route_experts_kernel<T, W, NT><<<(rows + 15) / 16, RL_WAVES * 64, 0, s>>>(              \
      dense, ids, wts, h, h_st, w, rows, width, rule)
  if (experts <= 16) ROUTE_LAUNCH(1);
  else if (experts <= 32) ROUTE_LAUNCH(2);
  else ROUTE_LAUNCH(4);
#undef ROUTE_LAUNCH
}

template <typename T>
void launch_scale_logits(float* out, const T* x, float scale, long n, hipStream_t s) {
  scale_logits_kernel<T><<<(int)((n + 2047) / 2048), 256, 0, s>>>(
      out, x, scale, al(out, 16) && al(x, 16), n);
}

#define INSTANTIATE(T)                                                                   \
  template void launch_stream_add_tanh_norm<T>(float*, const T*, const T*, float,        \
                                               const float*, const float*, float,        \
                                               const float*, const float*, T*, int, int, \
                                               hipStream_t);                             \
  template void launch_wide_norm<T>(T*, const T*, long, const float*, const float*,      \
                                    const float*, const T*, float, T*, T*, const long*,  \
                                    int, int, int, int, float, hipStream_t);             \
  template void launch_clamped_glu<T>(T*, const T*, float, const float*, int, long,      \
                                      hipStream_t);                                      \
  template void launch_scale_logits<T>(float*, const T*, float, long, hipStream_t);
INSTANTIATE(float)
INSTANTIATE(__hip_bfloat16)

#define INSTANTIATE_ROUTER(T, W)                                                         \
  template void launch_router_logits<T, W>(float*, const T*, long, const W*, int, int,   \
                                           int, hipStream_t);                            \
  template void launch_route_experts<T, W>(float*, int*, float*, const T*, long,         \
                                           const W*, const float*, int, int, int, int,   \
                                           int, int, int, float, hipStream_t);
INSTANTIATE_ROUTER(float, float)
INSTANTIATE_ROUTER(float, __hip_bfloat16)
INSTANTIATE_ROUTER(__hip_bfloat16, float)
INSTANTIATE_ROUTER(__hip_bfloat16, __hip_bfloat16)
