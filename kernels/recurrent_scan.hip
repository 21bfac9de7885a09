// Recurrences with per-sequence f32 state, advanced over the rows a step
// brings for each sequence (a prompt portion or one decoded token).
//
// A step brings, for sequence s, rows [loc[s], loc[s+1]) that continue it at
// position start = seq_len[s] - n.  State lives in slot-indexed f32 tensors;
// a sequence with start == 0 starts from zero state whatever its slot holds
// (slots are reused without clearing), slot < 0 marks a padding row of a
// captured decode bucket (zeros out, no state touched).
//
// matrix_scan<KIND>: state S [vdim, N] per (sequence, head), one column of
// the value axis per thread group:
//     S_t[j, :] = alpha_t * S_(t-1)[j, :] + beta_t * v_t[j] * k_t[:]
//     y_t[j]    = S_t[j, :] . q_t
//   KIND_SSD    alpha = exp(-exp(A_log) dt), beta = dt = softplus(raw + bias),
//               k = B, q = C (shared by the heads of a group), v = x,
//               y += D * x
//   KIND_MLSTM  log gates i, f (capped), running maximum m: alpha = exp(f + m
//               - m'), beta = exp(i - m'), a normaliser n_t = alpha n + beta k,
//               y = S q / (max(|n . q|, exp(-m')) + 1e-6)
//   KIND_HGRN2  a forget gate per state channel that also sets what is
//               written: S_t[j, i] = g_t[i] S_(t-1)[j, i] + (1 - g_t[i]) v_t[j],
//               g = l + (1 - l) sigmoid(f + b) with a lower bound l per
//               channel, y = S silu(q); a pointwise kernel ahead of the scan
//               writes g and silu(q) in f32 once per (row, head, channel)
//   KIND_DELTA  gated delta rule, alpha = g per head: u_t[j] = beta_t (v_t[j] -
//               g_t S_(t-1)[j, :] . k_t), S_t[j, :] = g_t S_(t-1)[j, :] + u_t[j] k_t,
//               y = g_t S_(t-1) . q_t + (k_t . q_t) u_t (the read-out sees the write);
//               unit keys and scaled unit queries come in f32 from a pre-pass
//               together with g, beta and k . q per (row, head)
//   KIND_GLA    a decay per key channel: S_t[j, i] = alpha_t[i] S_(t-1)[j, i] +
//               k_t[i] v_t[j], y = S q * q_scale; alpha = sigmoid(z)^(1/tau) with z
//               from a low-rank product, written by a pre-pass in f32 once per
//               (row, head, channel)
// alpha, beta (and exp(-m')) are computed once per (row, head) by small gate
// kernels ahead of the scan (for the mLSTM a sequential pass over the rows
// carries the maximum), not by every thread of it.
// The N axis is split over NSP adjacent lanes, 16 state values per lane in
// registers (N <= 1024); a workgroup of 256 threads owns 256 / NSP value
// columns of one (sequence, head), or four times as many with four columns
// per thread (the key / query slices a thread loads then serve four columns).  State rows are stored [vdim, N] so that a
// wave loads and stores them as one contiguous run.  The value columns are
// independent of each other, so there is no barrier in the token loop: per
// token a thread does 32 FMAs per column and log2(NSP) DPP adds for its dot
// product.
//
// rglru_scan: elementwise linear recurrence, one thread per (sequence,
// channel), gates and decay computed in f32 on the fly.

#include "scan_common.h"

#include <type_traits>

namespace {

enum { KIND_SSD = 0, KIND_MLSTM = 1, KIND_HGRN2 = 2, KIND_GLA = 3, KIND_DELTA = 4 };

struct ScanArgs {
  // rows
  const void* q; const void* k; const void* v;
  long q_st, k_st, v_st;             // row strides (elements)
  const void* g0; const void* g1;    // SSD: raw dt; mLSTM: i_pre, f_pre  [T, H] strided
  long g0_st, g1_st;
  const float* p0; const float* p1; const float* p2;  // SSD: dt_bias, A_log, D; mLSTM: i_bias, f_bias
  float cap, q_scale;
  float4* gates; int rows;           // per (row, head): alpha, beta, exp(-m), -  (f32)
  float* y; long y_st;               // [T, H*vdim] f32
  float* s_state; float* n_state; float* m_state;
  const int* loc; const int* seq_lens; const int* slots;
  const float* decay;                // GLA: [T, H*nk] f32
  int heads, vdim, nk, per_group;    // nk = N (SSD) or dim (mLSTM); heads per k/q group
  int vec_ok;
};

// Gates per (row, head), computed once instead of by every thread of the scan.
// Pointwise part: SSD alpha = exp(-exp(A_log) dt), beta = dt; mLSTM the capped
// log gates (i in .x, f in .y) that the sequential pass below turns into
// alpha, beta and exp(-m).
template <typename T, int KIND>
__global__ void scan_gates_pointwise_kernel(ScanArgs a) {
  const long idx = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (idx >= (long)a.rows * a.heads) return;
  const long row = idx / a.heads;
  const int h = (int)(idx - row * a.heads);
  const float g0 = ScalarOps<T>::to_f32(reinterpret_cast<const T*>(a.g0)[row * a.g0_st + h]);
  float4 out = make_float4(0.f, 0.f, 1.f, 0.f);
  if (KIND == KIND_SSD) {
    const float dt = softplus_f(g0 + a.p0[h]);
    out.x = expf(-expf(a.p1[h]) * dt);
    out.y = dt;
  } else {
    const float g1 = ScalarOps<T>::to_f32(reinterpret_cast<const T*>(a.g1)[row * a.g1_st + h]);
    out.x = a.cap * tanhf((g0 + a.p0[h]) / a.cap);
    out.y = logsigmoid_f(a.cap * tanhf((g1 + a.p1[h]) / a.cap));
  }
  a.gates[idx] = out;
}

// mLSTM: one thread per (sequence, head) walks the step's rows with the
// running maximum (0 at position 0): m' = max(f + m, i), alpha = exp(f + m -
// m'), beta = exp(i - m'), and stores exp(-m') for the output's denominator.
// Leaves the new maximum in m_state; nothing else reads m_state in the step.
__global__ void mlstm_gates_scan_kernel(ScanArgs a, int nseq) {
  const int idx = blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= nseq * a.heads) return;
  const int s = idx / a.heads;
  const int h = idx - s * a.heads;
  const int row0 = a.loc[s];
  const int n = a.loc[s + 1] - row0;
  const int slot = a.slots[s];
  if (n <= 0 || slot < 0) return;
  float* mp = a.m_state + (long)slot * a.heads + h;
  float m = (a.seq_lens[s] - n) > 0 ? *mp : 0.f;
  for (int r = 0; r < n; ++r) {
    float4* g = a.gates + (long)(row0 + r) * a.heads + h;
    const float ig = g->x, fg = g->y;
    const float m_new = fmaxf(fg + m, ig);
    *g = make_float4(expf(fg + m - m_new), expf(ig - m_new), expf(-m_new), 0.f);
    m = m_new;
  }
  *mp = m;
}

template <typename T, int KIND, int NSP, int VPT>
__global__ __launch_bounds__(256) void matrix_scan_kernel(ScanArgs a) {
  constexpr int JW = 256 / NSP;            // thread groups per workgroup
  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int ns = threadIdx.x % NSP;
  const int jbase = (blockIdx.y * JW + threadIdx.x / NSP) * VPT;   // first value column
  const int row0 = a.loc[s];
  const int n = a.loc[s + 1] - row0;
  if (n <= 0) return;
  const int slot = a.slots[s];
  if (slot < 0) {
    if (ns == 0)
      for (int r = 0; r < n; ++r)
#pragma unroll
        for (int c = 0; c < VPT; ++c)
          if (jbase + c < a.vdim)
            a.y[(long)(row0 + r) * a.y_st + (long)h * a.vdim + jbase + c] = 0.f;
    return;
  }
  const int start = a.seq_lens[s] - n;
  const int n0 = ns * NPT;
  const int grp = h / a.per_group;
  const bool vec = a.vec_ok != 0;

  // columns past vdim are clamped: they compute and never store
  int jc[VPT];
#pragma unroll
  for (int c = 0; c < VPT; ++c) jc[c] = min(jbase + c, a.vdim - 1);

  float S[VPT][NPT], nst[NPT];
  float* sbase = a.s_state + ((long)slot * a.heads + h) * a.vdim * a.nk;
  const float* nrow = KIND == KIND_MLSTM ? a.n_state + ((long)slot * a.heads + h) * a.nk : nullptr;
  if (start > 0) {
#pragma unroll
    for (int c = 0; c < VPT; ++c) load_slice<float>(sbase + (long)jc[c] * a.nk, n0, a.nk, vec, S[c]);
    if (KIND == KIND_MLSTM) load_slice<float>(nrow, n0, a.nk, vec, nst);
  } else {
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
      nst[i] = 0.f;
#pragma unroll
      for (int c = 0; c < VPT; ++c) S[c][i] = 0.f;
    }
  }

  const float c2 = KIND == KIND_SSD ? a.p2[h] : 0.f;   // D
  const float4* gp = a.gates + h;
  // HGRN2 reads its gate and activated query, the delta rule its unit keys and
  // queries from the f32 rows of a pre-pass
  using KQ =
      typename std::conditional<KIND == KIND_HGRN2 || KIND == KIND_DELTA, float, T>::type;
  const KQ* qp = reinterpret_cast<const KQ*>(a.q) + (long)grp * a.nk;
  const KQ* kp = reinterpret_cast<const KQ*>(a.k) + (long)grp * a.nk;
  const T* vp = reinterpret_cast<const T*>(a.v) + (long)h * a.vdim;

  // the next row's inputs are loaded while this row is computed: with two
  // waves per SIMD the load latency is otherwise paid once per token
  // constant subscripts only, so that the decay slices of the other kinds vanish
  constexpr int ND = KIND == KIND_GLA ? NPT : 1;
  const float* dp = KIND == KIND_GLA ? a.decay + (long)h * a.nk : nullptr;
  const long d_st = (long)a.heads * a.nk;
  float kk[NPT], qq[NPT], vj[VPT], dd[ND];
  float4 gt;
  auto load_row = [&](long row, float* k_, float* q_, float* v_, float* d_, float4& g_) {
    if constexpr (KIND == KIND_GLA) load_slice<float>(dp + row * d_st, n0, a.nk, vec, d_);
    load_slice<KQ>(kp + row * a.k_st, n0, a.nk, vec, k_);
    load_slice<KQ>(qp + row * a.q_st, n0, a.nk, vec, q_);
#pragma unroll
    for (int c = 0; c < VPT; ++c) v_[c] = ScalarOps<T>::to_f32(vp[row * a.v_st + jc[c]]);
    g_ = KIND == KIND_HGRN2 || KIND == KIND_GLA ? make_float4(0.f, 0.f, 0.f, 0.f) : gp[row * a.heads];
  };
  load_row(row0, kk, qq, vj, dd, gt);
  for (int r = 0; r < n; ++r) {
    const long row = row0 + r;
    float kn[NPT], qn[NPT], vn[VPT], dn[ND];
    float4 gn;
    const bool more = r + 1 < n;       // uniform over the workgroup
    if (more) load_row(row + 1, kn, qn, vn, dn, gn);
    const float alpha = gt.x, beta = gt.y;
    if constexpr (KIND == KIND_DELTA) {
      float dk[VPT], dq[VPT], u[VPT];
#pragma unroll
      for (int c = 0; c < VPT; ++c) {
        dk[c] = dq[c] = 0.f;
#pragma unroll
        for (int i = 0; i < NPT; ++i) {
          dk[c] += S[c][i] * kk[i];
          dq[c] += S[c][i] * qq[i];
        }
        u[c] = beta * (vj[c] - alpha * lanes_sum<NSP>(dk[c]));
        const float yv = alpha * lanes_sum<NSP>(dq[c]) + gt.z * u[c];
        if (ns == 0 && jbase + c < a.vdim)
          a.y[row * a.y_st + (long)h * a.vdim + jbase + c] = yv;
#pragma unroll
        for (int i = 0; i < NPT; ++i) S[c][i] = alpha * S[c][i] + u[c] * kk[i];
      }
    } else {
      float dot[VPT], ndot = 0.f;
#pragma unroll
      for (int c = 0; c < VPT; ++c) dot[c] = 0.f;
#pragma unroll
      for (int i = 0; i < NPT; ++i) {
        const float al = KIND == KIND_HGRN2 ? kk[i] : KIND == KIND_GLA ? dd[i < ND ? i : 0] : alpha;
        const float bk = KIND == KIND_HGRN2 ? 1.0f - kk[i] : KIND == KIND_GLA ? kk[i] : beta * kk[i];
        if (KIND == KIND_MLSTM) {
          nst[i] = alpha * nst[i] + bk;
          ndot += nst[i] * qq[i];
        }
#pragma unroll
        for (int c = 0; c < VPT; ++c) {
          S[c][i] = al * S[c][i] + bk * vj[c];
          dot[c] += S[c][i] * qq[i];
        }
      }
      float den = 1.f;    // mLSTM: the query scale is applied to the two sums
      if (KIND == KIND_MLSTM) {
        ndot = lanes_sum<NSP>(ndot) * a.q_scale;
        den = a.q_scale / (fmaxf(fabsf(ndot), gt.z) + 1e-6f);
      }
#pragma unroll
      for (int c = 0; c < VPT; ++c) {
        const float d = lanes_sum<NSP>(dot[c]);
        const float yv = KIND == KIND_MLSTM ? d * den
                         : KIND == KIND_GLA ? d * a.q_scale : d + c2 * vj[c];
        if (ns == 0 && jbase + c < a.vdim)
          a.y[row * a.y_st + (long)h * a.vdim + jbase + c] = yv;
      }
    }
    if (more) {
#pragma unroll
      for (int i = 0; i < NPT; ++i) { kk[i] = kn[i]; qq[i] = qn[i]; }
      if constexpr (KIND == KIND_GLA) {
#pragma unroll
        for (int i = 0; i < ND; ++i) dd[i] = dn[i];
      }
#pragma unroll
      for (int c = 0; c < VPT; ++c) vj[c] = vn[c];
      gt = gn;
    }
  }

#pragma unroll
  for (int c = 0; c < VPT; ++c) {
    if (jbase + c >= a.vdim) continue;
    float* srow = sbase + (long)(jbase + c) * a.nk;
    if (vec && n0 + NPT <= a.nk) {
#pragma unroll
      for (int i = 0; i < NPT; i += 4)
        *reinterpret_cast<float4*>(srow + n0 + i) =
            make_float4(S[c][i], S[c][i + 1], S[c][i + 2], S[c][i + 3]);
    } else {
#pragma unroll
      for (int i = 0; i < NPT; ++i)
        if (n0 + i < a.nk) srow[n0 + i] = S[c][i];
    }
  }
  // the normaliser n is read by every workgroup of this (sequence, head) and
  // therefore advanced by a kernel of its own, after this one, on the same
  // stream
}

// Advances the mLSTM normaliser n [slots, H, dim] over the step's rows with the
// precomputed gates: one workgroup per (sequence, head), one thread per key dim.
template <typename T>
__global__ __launch_bounds__(256) void mlstm_norm_state_kernel(ScanArgs a) {
  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int row0 = a.loc[s];
  const int n = a.loc[s + 1] - row0;
  const int slot = a.slots[s];
  if (n <= 0 || slot < 0) return;
  const int start = a.seq_lens[s] - n;
  const T* kp = reinterpret_cast<const T*>(a.k) + (long)h * a.nk;
  const float4* gp = a.gates + h;
  float* nrow = a.n_state + ((long)slot * a.heads + h) * a.nk;
  for (int d = threadIdx.x; d < a.nk; d += blockDim.x) {
    float nv = start > 0 ? nrow[d] : 0.f;
    for (int r = 0; r < n; ++r) {
      const long row = row0 + r;
      const float4 gt = gp[row * a.heads];
      nv = gt.x * nv + gt.y * ScalarOps<T>::to_f32(kp[row * a.k_st + d]);
    }
    nrow[d] = nv;
  }
}

// HGRN2 pre-pass: gq [T, 2, H * dim] f32 = (l + (1 - l) sigmoid(f + b), silu(q))
template <typename T>
__global__ __launch_bounds__(256) void hgrn2_gates_kernel(
    float* __restrict__ gq, const T* __restrict__ q, long q_st,
    const T* __restrict__ f, long f_st, const float* __restrict__ f_bias,
    const float* __restrict__ lower, long rows, int hd) {
  const long idx = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (idx >= rows * hd) return;
  const long row = idx / hd;
  const int c = (int)(idx - row * hd);
  const float lo = lower[c];
  const float fv = ScalarOps<T>::to_f32(f[row * f_st + c]) + f_bias[c];
  const float qv = ScalarOps<T>::to_f32(q[row * q_st + c]);
  gq[row * 2 * hd + c] = lo + (1.0f - lo) * sigmoid_f(fv);
  gq[row * 2 * hd + hd + c] = qv * sigmoid_f(qv);
}

// Delta-rule pre-pass, one workgroup per row: kq [T, 2, G * dim] f32 = (k / |k|,
// q / |q| * q_scale) per head of the short-convolved rows, gates (g, beta,
// k . q, -) per head of the values.
template <typename T>
__global__ __launch_bounds__(256) void delta_inputs_kernel(
    float* __restrict__ kq, float4* __restrict__ gates, const T* __restrict__ q, long q_st,
    const T* __restrict__ k, long k_st, const T* __restrict__ b_pre, long b_st,
    const T* __restrict__ a_pre, long a_st, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, float q_scale, int heads, int groups, int dim) {
  extern __shared__ float both[];   // [groups] k . q
  const long row = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1), wave = threadIdx.x / WAVE_SIZE;
  const int gd = groups * dim;
  for (int g = wave; g < groups; g += 256 / WAVE_SIZE) {
    float sk = 0.f, sq = 0.f, kqs = 0.f;
    for (int c = lane; c < dim; c += WAVE_SIZE) {
      const float kv = ScalarOps<T>::to_f32(k[row * k_st + g * dim + c]);
      const float qv = ScalarOps<T>::to_f32(q[row * q_st + g * dim + c]);
      sk += kv * kv; sq += qv * qv; kqs += kv * qv;
    }
    sk = wave_reduce_sum(sk); sq = wave_reduce_sum(sq); kqs = wave_reduce_sum(kqs);
    const float ik = 1.0f / sqrtf(sk + kUnitEps), iq = q_scale / sqrtf(sq + kUnitEps);
    for (int c = lane; c < dim; c += WAVE_SIZE) {
      kq[row * 2 * gd + g * dim + c] = ScalarOps<T>::to_f32(k[row * k_st + g * dim + c]) * ik;
      kq[row * 2 * gd + gd + g * dim + c] =
          ScalarOps<T>::to_f32(q[row * q_st + g * dim + c]) * iq;
    }
    if (lane == 0) both[g] = kqs * ik * iq;
  }
  __syncthreads();
  for (int h = threadIdx.x; h < heads; h += 256)
    gates[row * heads + h] = make_float4(
        delta_decay(ScalarOps<T>::to_f32(a_pre[row * a_st + h]), a_log[h], dt_bias[h]),
        sigmoid_f(ScalarOps<T>::to_f32(b_pre[row * b_st + h])), both[h / (heads / groups)], 0.f);
}

// exp(logsigmoid(z) * inv_tau) on the hardware's exp2 / log2: log1p through
// log(u), u = 1 + e, with what the rounding of u lost added back
DEVINLINE float gla_decay_of(float z, float inv_tau) {
  const float e = __expf(-fabsf(z));
  const float u = 1.0f + e;
  const float l = __logf(u) + (e - (u - 1.0f)) * __builtin_amdgcn_rcpf(u);
  return __expf((fminf(z, 0.f) - l) * inv_tau);
}

// GLA pre-pass: decay [T, channels] f32 = exp(logsigmoid(a1 . a2[:, c] + b) / tau).
// One thread per channel and GLA_ROWS rows; the rows' inner projections are
// broadcast from LDS, a channel's column of a2 [rank, channels] is read once.
constexpr int GLA_ROWS = 16;

template <typename T>
__global__ __launch_bounds__(256) void gla_decay_kernel(
    float* __restrict__ decay, const T* __restrict__ a1, long a1_st,
    const float* __restrict__ a2, const float* __restrict__ bias, float inv_tau, int rows,
    int channels, int rank) {
  extern __shared__ float inner[];   // [rank][GLA_ROWS]
  const int r0 = blockIdx.x * GLA_ROWS;
  const int n = min(GLA_ROWS, rows - r0);
  for (int i = threadIdx.x; i < rank * GLA_ROWS; i += blockDim.x) {
    const int r = i / rank, k = i - r * rank;
    inner[k * GLA_ROWS + r] =
        r < n ? ScalarOps<T>::to_f32(a1[(long)(r0 + r) * a1_st + k]) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= channels) return;
  float z[GLA_ROWS];
  const float b = bias[c];
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r) z[r] = b;
  for (int k = 0; k < rank; ++k) {
    const float w = a2[(long)k * channels + c];
#pragma unroll
    for (int r = 0; r < GLA_ROWS; ++r) z[r] += inner[k * GLA_ROWS + r] * w;
  }
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r)
    if (r < n) decay[(long)(r0 + r) * channels + c] = gla_decay_of(z[r], inv_tau);
}

// GLA in one kernel where a workgroup can own all value columns of a head: per
// chunk of GLA_ROWS rows the projected rows go through registers (loaded while
// the previous chunk is computed) into LDS as f32, the decays are computed
// there from the inner projections, the recurrence runs on them, and the
// chunk's outputs, kept in LDS where the values were, are normed per head,
// gated with silu and rounded once.  Key-channel rows in LDS are laid out so
// that the NSP lanes of a column read neighbouring 16-byte pieces.
struct GlaArgs {
  const void* q; const void* k; const void* v; const void* g; const void* a1;
  long q_st, k_st, v_st, g_st, a1_st;
  const float* a2; const float* a2_bias; const float* norm;
  float inv_tau, q_scale, eps;
  void* out;                       // [T, heads * vdim]
  float* state;
  const int* loc; const int* seq_lens; const int* slots;
  int heads, dim, vdim, rank;
};

template <typename T, int NSP, int VPT>
__global__ __launch_bounds__(256) void gla_fused_kernel(GlaArgs a) {
  constexpr int R = GLA_ROWS;
  constexpr int DP = NSP * NPT;                 // key channels, padded
  constexpr int NV = 256 / NSP * VPT;           // value columns, padded
  constexpr int KU = (R * DP / 8 + 255) / 256;  // pieces of a chunk per thread
  constexpr int VU = (R * NV / 8 + 255) / 256;
  constexpr int GV = (NV + 63) / 64;
  constexpr int CH = DP < 256 ? DP : 256;       // channels side by side in the decay step
  constexpr int SETS = 256 / CH, RPS = R / SETS;
  constexpr int GR = R / 4;               // rows per wave in the norm step
  extern __shared__ float smem[];
  float* dec_s = smem;              // [R][DP], interleaved
  float* k_s = dec_s + R * DP;
  float* q_s = k_s + R * DP;
  float* v_s = q_s + R * DP;        // [R][NV]; outputs replace the values
  float* a1_s = v_s + R * NV;       // [R][rank_p]
  const int rank_p = (a.rank + 15) & ~15;

  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int tid = threadIdx.x;
  const int ns = tid % NSP, jg = tid / NSP;
  const int lane = tid & (WAVE_SIZE - 1), wave = tid / WAVE_SIZE;
  const int row0 = a.loc[s];
  const int n = a.loc[s + 1] - row0;
  if (n <= 0) return;
  const int slot = a.slots[s];
  const long out_st = (long)a.heads * a.vdim;
  T* outp = reinterpret_cast<T*>(a.out) + (long)h * a.vdim;
  if (slot < 0) {
    for (int r = 0; r < n; ++r)
      for (int c = tid; c < a.vdim; c += 256)
        outp[(row0 + r) * out_st + c] = ScalarOps<T>::from_f32(0.f);
    return;
  }
  const T* kp = reinterpret_cast<const T*>(a.k) + (long)h * a.dim;
  const T* qp = reinterpret_cast<const T*>(a.q) + (long)h * a.dim;
  const T* vp = reinterpret_cast<const T*>(a.v) + (long)h * a.vdim;
  const T* gp = reinterpret_cast<const T*>(a.g) + (long)h * a.vdim;
  const T* a1p = reinterpret_cast<const T*>(a.a1);
  const long hd = (long)a.heads * a.dim;

  // state columns of this thread
  const int n0 = ns * NPT;
  float S[VPT][NPT];
  float* sbase = a.state + ((long)slot * a.heads + h) * a.vdim * a.dim;
  const bool carry = a.seq_lens[s] - n > 0;
#pragma unroll
  for (int c = 0; c < VPT; ++c) {
    const int j = jg * VPT + c;
    if (carry && j < a.vdim) {
      load_slice<float>(sbase + (long)j * a.dim, n0, a.dim, true, S[c]);
    } else {
#pragma unroll
      for (int i = 0; i < NPT; ++i) S[c][i] = 0.f;
    }
  }

  RowPiece<T> rk[KU], rq[KU], rv[VU];
  float ra1 = 0.f;
  auto fetch = [&](int r0) {
    const int nr = min(R, n - r0);
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int idx = tid + u * 256, r = idx / (DP / 8), c = idx % (DP / 8) * 8;
      rk[u] = rq[u] = RowPiece<T>{};
      if (r < nr && c < a.dim) {
        const long row = row0 + r0 + r;
        rk[u] = *reinterpret_cast<const RowPiece<T>*>(kp + row * a.k_st + c);
        rq[u] = *reinterpret_cast<const RowPiece<T>*>(qp + row * a.q_st + c);
      }
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int idx = tid + u * 256, r = idx / (NV / 8), c = idx % (NV / 8) * 8;
      rv[u] = RowPiece<T>{};
      if (r < nr && c < a.vdim)
        rv[u] = *reinterpret_cast<const RowPiece<T>*>(vp + (row0 + r0 + r) * a.v_st + c);
    }
    const int r = tid / rank_p, i = tid % rank_p;
    ra1 = r < nr && i < a.rank
              ? ScalarOps<T>::to_f32(a1p[(row0 + r0 + r) * a.a1_st + i]) : 0.f;
  };

  fetch(0);
  for (int r0 = 0; r0 < n; r0 += R) {
    const int nr = min(R, n - r0);
    // ---- this chunk into LDS ------------------------------------------------
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int idx = tid + u * 256, r = idx / (DP / 8), c = idx % (DP / 8) * 8;
      if (r < R) {
        const int at = r * DP + (c % NPT) / 4 * (NSP * 4) + c / NPT * 4;
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          const int e = half * 4;
          *reinterpret_cast<float4*>(k_s + at + half * NSP * 4) =
              make_float4(rk[u].at(e), rk[u].at(e + 1), rk[u].at(e + 2), rk[u].at(e + 3));
          *reinterpret_cast<float4*>(q_s + at + half * NSP * 4) =
              make_float4(rq[u].at(e) * a.q_scale, rq[u].at(e + 1) * a.q_scale,
                          rq[u].at(e + 2) * a.q_scale, rq[u].at(e + 3) * a.q_scale);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int idx = tid + u * 256, r = idx / (NV / 8), c = idx % (NV / 8) * 8;
      if (r < R) {
#pragma unroll
        for (int e = 0; e < 8; e += 4)
          *reinterpret_cast<float4*>(v_s + r * NV + c + e) =
              make_float4(rv[u].at(e), rv[u].at(e + 1), rv[u].at(e + 2), rv[u].at(e + 3));
      }
    }
    if (tid < R * rank_p) a1_s[tid] = ra1;
    for (int idx = tid + 256; idx < R * rank_p; idx += 256) {
      const int r = idx / rank_p, i = idx % rank_p;
      a1_s[idx] = r < nr && i < a.rank
                      ? ScalarOps<T>::to_f32(a1p[(row0 + r0 + r) * a.a1_st + i]) : 0.f;
    }
    __syncthreads();
    if (r0 + R < n) fetch(r0 + R);
    // the gates of this chunk, needed after the recurrence: rows wave, wave + 4, ..
    float gv[GR][GV];
#pragma unroll
    for (int i = 0; i < GR; ++i)
#pragma unroll
      for (int j = 0; j < GV; ++j) {
        const int r = wave + 4 * i, c = lane + 64 * j;
        gv[i][j] = r < nr && c < a.vdim
                       ? ScalarOps<T>::to_f32(gp[(row0 + r0 + r) * a.g_st + c]) : 0.f;
      }
    // ---- decays: a thread has one channel of RPS rows ------------------------
#pragma unroll
    for (int cb = 0; cb < DP; cb += CH) {
      const int c = cb + tid % CH, rb = tid / CH * RPS;
      if (c < a.dim && rb < nr) {
        float z[RPS];
        const float* w2 = a.a2 + (long)h * a.dim + c;
        const float bias = a.a2_bias[(long)h * a.dim + c];
#pragma unroll
        for (int r = 0; r < RPS; ++r) z[r] = bias;
        for (int i0 = 0; i0 < a.rank; i0 += 16) {
          float w[16];
#pragma unroll
          for (int i = 0; i < 16; ++i) w[i] = i0 + i < a.rank ? w2[(i0 + i) * hd] : 0.f;
#pragma unroll
          for (int r = 0; r < RPS; ++r)
#pragma unroll
            for (int i = 0; i < 16; i += 4) {
              const float4 x =
                  *reinterpret_cast<const float4*>(a1_s + (rb + r) * rank_p + i0 + i);
              z[r] += (x.x * w[i] + x.y * w[i + 1]) + (x.z * w[i + 2] + x.w * w[i + 3]);
            }
        }
        float* d = dec_s + rb * DP + (c % NPT) / 4 * (NSP * 4) + c / NPT * 4 + c % 4;
#pragma unroll
        for (int r = 0; r < RPS; ++r) d[r * DP] = gla_decay_of(z[r], a.inv_tau);
      } else if (c >= a.dim) {
        float* d = dec_s + rb * DP + (c % NPT) / 4 * (NSP * 4) + c / NPT * 4 + c % 4;
#pragma unroll
        for (int r = 0; r < RPS; ++r) d[r * DP] = 0.f;   // padding channels stay zero
      }
    }
    __syncthreads();
    // ---- the recurrence --------------------------------------------------------
    for (int r = 0; r < nr; ++r) {
      float vj[VPT], dot[VPT];
#pragma unroll
      for (int c = 0; c < VPT; ++c) {
        vj[c] = v_s[r * NV + jg * VPT + c];
        dot[c] = 0.f;
      }
#pragma unroll
      for (int i4 = 0; i4 < NPT / 4; ++i4) {
        const int at = r * DP + i4 * (NSP * 4) + ns * 4;
        const float4 d4 = *reinterpret_cast<const float4*>(dec_s + at);
        const float4 k4 = *reinterpret_cast<const float4*>(k_s + at);
        const float4 q4 = *reinterpret_cast<const float4*>(q_s + at);
        const float dd[4] = {d4.x, d4.y, d4.z, d4.w};
        const float kk[4] = {k4.x, k4.y, k4.z, k4.w};
        const float qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int c = 0; c < VPT; ++c) {
            float& st = S[c][i4 * 4 + e];
            st = dd[e] * st + kk[e] * vj[c];
            dot[c] += st * qq[e];
          }
      }
#pragma unroll
      for (int c = 0; c < VPT; ++c) dot[c] = lanes_sum<NSP>(dot[c]);
      // only the lanes of this column group read these values, all before now
      if (ns == 0) {
#pragma unroll
        for (int c = 0; c < VPT; ++c) v_s[r * NV + jg * VPT + c] = dot[c];
      }
    }
    __syncthreads();
    // ---- norm and gate ----------------------------------------------------------
#pragma unroll
    for (int i = 0; i < GR; ++i) {
      const int r = wave + 4 * i;
      if (r >= nr) continue;                 // uniform over the wave
      float y[GV];
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < GV; ++j) {
        const int c = lane + 64 * j;
        y[j] = c < a.vdim ? v_s[r * NV + c] : 0.f;
        ss += y[j] * y[j];
      }
      ss = wave_reduce_sum(ss);
      const float inv = 1.0f / sqrtf(ss / a.vdim + a.eps);
#pragma unroll
      for (int j = 0; j < GV; ++j) {
        const int c = lane + 64 * j;
        if (c < a.vdim)
          outp[(row0 + r0 + r) * out_st + c] = ScalarOps<T>::from_f32(
              y[j] * inv * a.norm[(long)h * a.vdim + c] * gv[i][j] * sigmoid_f(gv[i][j]));
      }
    }
    __syncthreads();   // the next chunk overwrites LDS
  }

#pragma unroll
  for (int c = 0; c < VPT; ++c) {
    const int j = jg * VPT + c;
    if (j >= a.vdim) continue;
    float* srow = sbase + (long)j * a.dim;
#pragma unroll
    for (int i = 0; i < NPT; i += 4)
      if (n0 + i < a.dim)      // dim is a multiple of 8
        *reinterpret_cast<float4*>(srow + n0 + i) =
            make_float4(S[c][i], S[c][i + 1], S[c][i + 2], S[c][i + 3]);
  }
}

// GLA for steps in which the sequences bring single rows: the state is the
// traffic, so it is streamed column by column (LW lanes per column, a lane
// holding eight of its elements as two 16-byte pieces) with the row's decays,
// keys and queries in registers; few registers and many resident waves keep
// the loads in flight.  Correct for
// any number of rows: each row reads back what the one before stored.
template <typename T, int LW>
__global__ __launch_bounds__(256) void gla_row_kernel(GlaArgs a) {
  constexpr int COLS = 256 / LW;    // columns side by side
  constexpr int FLY = 2;            // column groups in flight
  extern __shared__ float smem[];
  float* dec_s = smem;              // [LW * 8]
  float* y_s = dec_s + LW * 8;      // [vdim]
  float* v_s = y_s + a.vdim;        // [vdim]
  float* a1_s = v_s + a.vdim;       // [rank]
  __shared__ float red[8];
  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int tid = threadIdx.x, l = tid % LW, jg = tid / LW;
  const int row0 = a.loc[s];
  const int n = a.loc[s + 1] - row0;
  if (n <= 0) return;
  const int slot = a.slots[s];
  const long out_st = (long)a.heads * a.vdim;
  T* outp = reinterpret_cast<T*>(a.out) + (long)h * a.vdim;
  if (slot < 0) {
    for (int r = 0; r < n; ++r)
      for (int c = tid; c < a.vdim; c += 256)
        outp[(row0 + r) * out_st + c] = ScalarOps<T>::from_f32(0.f);
    return;
  }
  float* sbase = a.state + ((long)slot * a.heads + h) * a.vdim * a.dim;
  const int p0 = l * 4, p1 = (LW + l) * 4;      // the lane's two pieces of a column
  const bool in0 = p0 < a.dim, in1 = p1 < a.dim;
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  bool carry = a.seq_lens[s] - n > 0;
  for (int r = 0; r < n; ++r) {
    const long row = row0 + r;
    const T* kp = reinterpret_cast<const T*>(a.k) + row * a.k_st + (long)h * a.dim;
    const T* qp = reinterpret_cast<const T*>(a.q) + row * a.q_st + (long)h * a.dim;
    const T* vp = reinterpret_cast<const T*>(a.v) + row * a.v_st + (long)h * a.vdim;
    const T* gp = reinterpret_cast<const T*>(a.g) + row * a.g_st + (long)h * a.vdim;
    const T* a1p = reinterpret_cast<const T*>(a.a1) + row * a.a1_st;
    float k[8], q[8], d[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int c = (i < 4 ? p0 : p1 - 4) + i;
      const bool in = i < 4 ? in0 : in1;
      k[i] = in ? ScalarOps<T>::to_f32(kp[c]) : 0.f;
      q[i] = in ? ScalarOps<T>::to_f32(qp[c]) * a.q_scale : 0.f;
    }
    for (int i = tid; i < a.rank; i += 256) a1_s[i] = ScalarOps<T>::to_f32(a1p[i]);
    // through LDS: a load inside the column loop would wait for the columns ahead
    for (int c = tid; c < a.vdim; c += 256) v_s[c] = ScalarOps<T>::to_f32(vp[c]);
    __syncthreads();
    for (int c = tid; c < LW * 8; c += 256) {
      float dv = 0.f;
      if (c < a.dim) {
        const float* w2 = a.a2 + (long)h * a.dim + c;
        const long hd = (long)a.heads * a.dim;
        float z = a.a2_bias[(long)h * a.dim + c];
#pragma unroll 8
        for (int i = 0; i < a.rank; ++i) z += a1_s[i] * w2[i * hd];
        dv = gla_decay_of(z, a.inv_tau);
      }
      dec_s[c] = dv;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; ++i) d[i] = dec_s[(i < 4 ? p0 : p1 - 4) + i];
    for (int j0 = jg; j0 < a.vdim; j0 += FLY * COLS) {
      float4 cur[FLY][2];
#pragma unroll
      for (int f = 0; f < FLY; ++f) {
        const int j = j0 + f * COLS;
        const float* p = sbase + (long)j * a.dim;
        cur[f][0] = carry && in0 && j < a.vdim ? *reinterpret_cast<const float4*>(p + p0) : zero;
        cur[f][1] = carry && in1 && j < a.vdim ? *reinterpret_cast<const float4*>(p + p1) : zero;
      }
#pragma unroll
      for (int f = 0; f < FLY; ++f) {
        const int j = j0 + f * COLS;
        const bool live = j < a.vdim;
        const float v = live ? v_s[j] : 0.f;
        float x[8] = {cur[f][0].x, cur[f][0].y, cur[f][0].z, cur[f][0].w,
                      cur[f][1].x, cur[f][1].y, cur[f][1].z, cur[f][1].w};
        float dot = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          x[i] = d[i] * x[i] + k[i] * v;
          dot += x[i] * q[i];
        }
        float* p = sbase + (long)j * a.dim;
        if (live && in0) *reinterpret_cast<float4*>(p + p0) = make_float4(x[0], x[1], x[2], x[3]);
        if (live && in1) *reinterpret_cast<float4*>(p + p1) = make_float4(x[4], x[5], x[6], x[7]);
        dot = lanes_sum<LW>(dot);
        if (live && l == 0) y_s[j] = dot;
      }
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = tid; c < a.vdim; c += 256) ss += y_s[c] * y_s[c];
    ss = block_reduce_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / a.vdim + a.eps);
    for (int c = tid; c < a.vdim; c += 256) {
      const float g = ScalarOps<T>::to_f32(gp[c]);
      outp[row * out_st + c] = ScalarOps<T>::from_f32(
          y_s[c] * inv * a.norm[(long)h * a.vdim + c] * g * sigmoid_f(g));
    }
    __syncthreads();   // LDS is rewritten by the next row
    carry = true;
  }
}

template <typename T, int KIND>
void launch_matrix_scan(const ScanArgs& a, int nseq, hipStream_t stream) {
  const int nslices = (a.nk + NPT - 1) / NPT;
  int nsp = 1;
  while (nsp < nslices) nsp <<= 1;
  // four (or two) value columns per thread when that still fills a workgroup: the key
  // and query slices a thread loads then serve four state columns
#define SCAN_CASE(P)                                                           \
  case P: {                                                                    \
    constexpr int JW = 256 / P;                                                \
    if (a.vdim >= 4 * JW) {                                                    \
      dim3 grid(nseq * a.heads, (a.vdim + 4 * JW - 1) / (4 * JW));             \
      matrix_scan_kernel<T, KIND, P, 4><<<grid, 256, 0, stream>>>(a);          \
    } else if (a.vdim >= 2 * JW) {                                             \
      dim3 grid(nseq * a.heads, (a.vdim + 2 * JW - 1) / (2 * JW));             \
      matrix_scan_kernel<T, KIND, P, 2><<<grid, 256, 0, stream>>>(a);          \
    } else {                                                                   \
      dim3 grid(nseq * a.heads, (a.vdim + JW - 1) / JW);                       \
      matrix_scan_kernel<T, KIND, P, 1><<<grid, 256, 0, stream>>>(a);          \
    }                                                                          \
    break;                                                                     \
  }
  switch (nsp) {
    SCAN_CASE(1) SCAN_CASE(2) SCAN_CASE(4) SCAN_CASE(8) SCAN_CASE(16)
    SCAN_CASE(32) SCAN_CASE(64)
    default: break;   // the binding refuses N > 1024
  }
#undef SCAN_CASE
}

template <typename T>
__global__ __launch_bounds__(256) void rglru_scan_kernel(
    T* __restrict__ out, const T* __restrict__ u, const T* __restrict__ r_pre,
    const T* __restrict__ i_pre, const float* __restrict__ r_bias,
    const float* __restrict__ i_bias, const float* __restrict__ lam, float gate_c,
    const T* __restrict__ y_branch, float* __restrict__ state,
    const int* __restrict__ loc, const int* __restrict__ seq_lens,
    const int* __restrict__ slots, int width) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= width) return;
  const int row0 = loc[s];
  const int n = loc[s + 1] - row0;
  if (n <= 0) return;
  const int slot = slots[s];
  if (slot < 0) {
    for (int r = 0; r < n; ++r) out[(long)(row0 + r) * width + c] = ScalarOps<T>::from_f32(0.f);
    return;
  }
  const int start = seq_lens[s] - n;
  float S = start > 0 ? state[(long)slot * width + c] : 0.f;
  const float rb = r_bias[c], ib = i_bias[c];
  const float sp = -gate_c * softplus_f(lam[c]);
  for (int r = 0; r < n; ++r) {
    const long o = (long)(row0 + r) * width + c;
    const float uv = ScalarOps<T>::to_f32(u[o]);
    const float rg = sigmoid_f(ScalarOps<T>::to_f32(r_pre[o]) + rb);
    const float ig = sigmoid_f(ScalarOps<T>::to_f32(i_pre[o]) + ib);
    const float av = expf(sp * rg);
    S = av * S + sqrtf(1.0f - av * av) * ig * uv;
    out[o] = ScalarOps<T>::from_f32(S * ScalarOps<T>::to_f32(y_branch[o]));
  }
  state[(long)slot * width + c] = S;
}

}  // namespace

template <typename T>
void launch_ssd_scan(float* y, const T* xbc, long xbc_st, const T* dt, long dt_st,
                     const float* dt_bias, const float* a_log, const float* d_skip,
                     float* state, const int* loc, const int* seq_lens,
                     const int* slots, int nseq, int heads, int vdim, int nstate,
                     int groups, int vec_ok, float* gates, int rows,
                     hipStream_t stream) {
  const int inner = heads * vdim;
  ScanArgs a{};
  a.gates = reinterpret_cast<float4*>(gates); a.rows = rows;
  a.v = xbc;                                  a.v_st = xbc_st;
  a.k = xbc + inner;                          a.k_st = xbc_st;
  a.q = xbc + inner + (long)groups * nstate;  a.q_st = xbc_st;
  a.g0 = dt; a.g0_st = dt_st;
  a.p0 = dt_bias; a.p1 = a_log; a.p2 = d_skip;
  a.y = y; a.y_st = inner;
  a.s_state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.vdim = vdim; a.nk = nstate; a.per_group = heads / groups;
  a.vec_ok = vec_ok;
  const long ng = (long)rows * heads;
  scan_gates_pointwise_kernel<T, KIND_SSD><<<(int)((ng + 255) / 256), 256, 0, stream>>>(a);
  launch_matrix_scan<T, KIND_SSD>(a, nseq, stream);
}

template <typename T>
void launch_mlstm_scan(float* o, const T* q, long q_st, const T* k, long k_st,
                       const T* v, long v_st, const T* i_pre, long i_st,
                       const T* f_pre, long f_st, const float* i_bias,
                       const float* f_bias, float cap, float q_scale,
                       float* s_state, float* n_state, float* m_state,
                       const int* loc, const int* seq_lens, const int* slots,
                       int nseq, int heads, int dim, int vdim, int vec_ok,
                       float* gates, int rows, hipStream_t stream) {
  ScanArgs a{};
  a.gates = reinterpret_cast<float4*>(gates); a.rows = rows;
  a.q = q; a.q_st = q_st; a.k = k; a.k_st = k_st; a.v = v; a.v_st = v_st;
  a.g0 = i_pre; a.g0_st = i_st; a.g1 = f_pre; a.g1_st = f_st;
  a.p0 = i_bias; a.p1 = f_bias;
  a.cap = cap; a.q_scale = q_scale;
  a.y = o; a.y_st = (long)heads * vdim;
  a.s_state = s_state; a.n_state = n_state; a.m_state = m_state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.vdim = vdim; a.nk = dim; a.per_group = 1;
  a.vec_ok = vec_ok;
  const long ng = (long)rows * heads;
  scan_gates_pointwise_kernel<T, KIND_MLSTM><<<(int)((ng + 255) / 256), 256, 0, stream>>>(a);
  mlstm_gates_scan_kernel<<<(nseq * heads + 63) / 64, 64, 0, stream>>>(a, nseq);
  launch_matrix_scan<T, KIND_MLSTM>(a, nseq, stream);
  const int block = dim >= 256 ? 256 : ((dim + 63) / 64) * 64;
  mlstm_norm_state_kernel<T><<<nseq * heads, block, 0, stream>>>(a);
}

template <typename T>
void launch_hgrn2_scan(float* o, const T* q, long q_st, const T* f, long f_st,
                       const T* v, long v_st, const float* f_bias,
                       const float* lower, float* state, const int* loc,
                       const int* seq_lens, const int* slots, int nseq, int heads,
                       int dim, int vdim, int vec_ok, float* gq, int rows,
                       hipStream_t stream) {
  const int hd = heads * dim;
  const long total = (long)rows * hd;
  hgrn2_gates_kernel<T><<<(int)((total + 255) / 256), 256, 0, stream>>>(
      gq, q, q_st, f, f_st, f_bias, lower, rows, hd);
  ScanArgs a{};
  a.rows = rows;
  a.k = gq;      a.k_st = 2L * hd;
  a.q = gq + hd; a.q_st = 2L * hd;
  a.v = v;       a.v_st = v_st;
  a.y = o; a.y_st = (long)heads * vdim;
  a.s_state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.vdim = vdim; a.nk = dim; a.per_group = 1;
  a.vec_ok = vec_ok;
  launch_matrix_scan<T, KIND_HGRN2>(a, nseq, stream);
}

template <typename T>
void launch_gla_scan(float* o, const T* q, long q_st, const T* k, long k_st, const T* v,
                     long v_st, const T* a1, long a1_st, const float* a2,
                     const float* a2_bias, float inv_tau, float q_scale, float* state,
                     const int* loc, const int* seq_lens, const int* slots, int nseq,
                     int heads, int dim, int vdim, int rank, int vec_ok, float* decay,
                     int rows, hipStream_t stream) {
  const int hd = heads * dim;
  const dim3 grid((rows + GLA_ROWS - 1) / GLA_ROWS, (hd + 255) / 256);
  gla_decay_kernel<T><<<grid, 256, sizeof(float) * GLA_ROWS * rank, stream>>>(
      decay, a1, a1_st, a2, a2_bias, inv_tau, rows, hd, rank);
  ScanArgs a{};
  a.rows = rows;
  a.q = q; a.q_st = q_st; a.k = k; a.k_st = k_st; a.v = v; a.v_st = v_st;
  a.decay = decay;
  a.q_scale = q_scale;
  a.y = o; a.y_st = (long)heads * vdim;
  a.s_state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.vdim = vdim; a.nk = dim; a.per_group = 1;
  a.vec_ok = vec_ok;
  launch_matrix_scan<T, KIND_GLA>(a, nseq, stream);
}

template <typename T>
void launch_delta_scan(float* o, const T* q, long q_st, const T* k, long k_st, const T* v,
                       long v_st, const T* b_pre, long b_st, const T* a_pre, long a_st,
                       const float* a_log, const float* dt_bias, float q_scale, float* state,
                       const int* loc, const int* seq_lens, const int* slots, int nseq,
                       int heads, int groups, int dim, int vdim, int vec_ok, float* kq,
                       float* gates, int rows, hipStream_t stream) {
  const int gd = groups * dim;
  ScanArgs a{};
  a.gates = reinterpret_cast<float4*>(gates); a.rows = rows;
  delta_inputs_kernel<T><<<rows, 256, sizeof(float) * groups, stream>>>(
      kq, a.gates, q, q_st, k, k_st, b_pre, b_st, a_pre, a_st, a_log, dt_bias, q_scale, heads,
      groups, dim);
  a.k = kq;      a.k_st = 2L * gd;
  a.q = kq + gd; a.q_st = 2L * gd;
  a.v = v;       a.v_st = v_st;
  a.y = o; a.y_st = (long)heads * vdim;
  a.s_state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.vdim = vdim; a.nk = dim; a.per_group = heads / groups;
  a.vec_ok = vec_ok;
  launch_matrix_scan<T, KIND_DELTA>(a, nseq, stream);
}

// value columns per thread of the one-kernel form, 0 when the shape does not fit
int gla_fused_columns(int dim, int vdim) {
  if (dim % 8 || vdim % 8 || dim > 256) return 0;
  const int nsp = dim <= 32 ? 2 : dim <= 64 ? 4 : dim <= 128 ? 8 : 16;
  for (int vpt = 1; vpt <= 4; vpt *= 2)
    if (256 / nsp * vpt >= vdim) return vpt;
  return 0;
}

template <typename T>
void launch_gla_fused(T* out, const T* q, long q_st, const T* k, long k_st, const T* v,
                      long v_st, const T* g, long g_st, const T* a1, long a1_st,
                      const float* a2, const float* a2_bias, float inv_tau, float q_scale,
                      const float* norm, float eps, float* state, const int* loc,
                      const int* seq_lens, const int* slots, int nseq, int heads, int dim,
                      int vdim, int rank, int rows, hipStream_t stream) {
  GlaArgs a;
  a.q = q; a.k = k; a.v = v; a.g = g; a.a1 = a1;
  a.q_st = q_st; a.k_st = k_st; a.v_st = v_st; a.g_st = g_st; a.a1_st = a1_st;
  a.a2 = a2; a.a2_bias = a2_bias; a.norm = norm;
  a.inv_tau = inv_tau; a.q_scale = q_scale; a.eps = eps;
  a.out = out; a.state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.dim = dim; a.vdim = vdim; a.rank = rank;
  const int vpt = gla_fused_columns(dim, vdim);
  const int rank_p = (rank + 15) & ~15;
  if (rows <= nseq) {   // a handful of rows per sequence at most: stream the state
    const int lw = dim <= 32 ? 4 : dim <= 64 ? 8 : dim <= 128 ? 16 : 32;
    const size_t smem = sizeof(float) * (lw * 8 + 2 * vdim + rank);
    if (lw == 4) gla_row_kernel<T, 4><<<nseq * heads, 256, smem, stream>>>(a);
    else if (lw == 8) gla_row_kernel<T, 8><<<nseq * heads, 256, smem, stream>>>(a);
    else if (lw == 16) gla_row_kernel<T, 16><<<nseq * heads, 256, smem, stream>>>(a);
    else gla_row_kernel<T, 32><<<nseq * heads, 256, smem, stream>>>(a);
    return;
  }
#define GLA_LAUNCH(N, V)                                                               \
  gla_fused_kernel<T, N, V><<<nseq * heads, 256,                                       \
                              sizeof(float) * GLA_ROWS *                               \
                                  (3 * N * NPT + 256 / N * V + rank_p), stream>>>(a)
#define GLA_CASE(N)                                                                    \
  if (vpt == 1) GLA_LAUNCH(N, 1);                                                      \
  else if (vpt == 2) GLA_LAUNCH(N, 2);                                                 \
  else GLA_LAUNCH(N, 4)
  if (dim <= 32) { GLA_CASE(2); }
  else if (dim <= 64) { GLA_CASE(4); }
  else if (dim <= 128) { GLA_CASE(8); }
  else { GLA_CASE(16); }
#undef GLA_CASE
#undef GLA_LAUNCH
}

template <typename T>
void launch_rglru_scan(T* out, const T* u, const T* r_pre, const T* i_pre,
                       const float* r_bias, const float* i_bias, const float* lam,
                       float gate_c, const T* y_branch, float* state,
                       const int* loc, const int* seq_lens, const int* slots,
                       int nseq, int width, hipStream_t stream) {
  const int block = width >= 256 ? 256 : ((width + 63) / 64) * 64;
  dim3 grid(nseq, (width + block - 1) / block);
  rglru_scan_kernel<T><<<grid, block, 0, stream>>>(
      out, u, r_pre, i_pre, r_bias, i_bias, lam, gate_c, y_branch, state, loc,
      seq_lens, slots, width);
}

#define INSTANTIATE(T)                                                          \
  template void launch_ssd_scan<T>(float*, const T*, long, const T*, long,      \
                                   const float*, const float*, const float*,    \
                                   float*, const int*, const int*, const int*,  \
                                   int, int, int, int, int, int, float*, int,   \
                                   hipStream_t);                                \
  template void launch_mlstm_scan<T>(                                           \
      float*, const T*, long, const T*, long, const T*, long, const T*, long,   \
      const T*, long, const float*, const float*, float, float, float*, float*, \
      float*, const int*, const int*, const int*, int, int, int, int, int,      \
      float*, int, hipStream_t);                                                \
  template void launch_hgrn2_scan<T>(float*, const T*, long, const T*, long,    \
                                     const T*, long, const float*, const float*,\
                                     float*, const int*, const int*, const int*,\
                                     int, int, int, int, int, float*, int,      \
                                     hipStream_t);                              \
  template void launch_gla_scan<T>(float*, const T*, long, const T*, long,      \
                                   const T*, long, const T*, long, const float*, \
                                   const float*, float, float, float*,          \
                                   const int*, const int*, const int*, int, int, \
                                   int, int, int, int, float*, int, hipStream_t); \
  template void launch_delta_scan<T>(float*, const T*, long, const T*, long,    \
                                     const T*, long, const T*, long, const T*,  \
                                     long, const float*, const float*, float,   \
                                     float*, const int*, const int*, const int*, \
                                     int, int, int, int, int, int, float*,      \
                                     float*, int, hipStream_t);                 \
  template void launch_gla_fused<T>(T*, const T*, long, const T*, long,         \
                                    const T*, long, const T*, long, const T*,   \
                                    long, const float*, const float*, float,    \
                                    float, const float*, float, float*,         \
                                    const int*, const int*, const int*, int,    \
                                    int, int, int, int, int, hipStream_t);      \
  template void launch_rglru_scan<T>(T*, const T*, const T*, const T*,          \
                                     const float*, const float*, const float*,  \
                                     float, const T*, float*, const int*,       \
                                     const int*, const int*, int, int,          \
                                     hipStream_t);
INSTANTIATE(float)
INSTANTIATE(__hip_bfloat16)
