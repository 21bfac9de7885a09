// Gated delta rule with per-sequence f32 state, everything between the short
// convolution and the output projection in one kernel.  Per head, S [vdim, dim]:
//     S <- g S,  u = beta (v - S k),  S <- S + u k^T,  o = S q
// with unit keys and scaled unit queries, g = exp(-exp(A_log) softplus(a +
// dt_bias)) and beta = sigmoid(b); then o is RMS-normed over vdim, times a weight,
// times silu(gate), rounded once.  Head h uses query / key head h / per_group.
//
// Both dot products of a token read the state as the token before left it,
//     o = g (S q) + (k . q) u,
// so one pass over the registers serves S k and S q, and k . q is a scalar that
// is formed while the row is staged.
//
// delta_fused  prompt portions: a workgroup owns all value columns of a
//              (sequence, head).  The state is kept divided by the product G of
//              the decays since G was last one, T = S / G, which makes the update
//              a single multiply-add, T += (u / G) k; G is multiplied back in
//              before it gets small (and at the end), so nothing under- or
//              overflows however strong the decay is.
// delta_row    steps of single rows: the state is the traffic and is streamed
//              through registers column by column.
// A sequence that starts in a step starts from zero state whatever its slot
// holds; slot < 0 marks a padding row (zeros out, no state touched).

#include "scan_common.h"

namespace {

constexpr int DL_ROWS = 16;          // rows per chunk
constexpr float kSmallG = 1e-12f;

struct DeltaArgs {
  const void* q; const void* k; const void* v; const void* gate;
  const void* b_pre; const void* a_pre;
  long q_st, k_st, v_st, gate_st, b_st, a_st;
  const float* a_log; const float* dt_bias; const float* norm;
  float q_scale, eps;
  void* out;                       // [T, heads * vdim]
  float* state;                    // [slots, heads, vdim, dim]
  const int* loc; const int* seq_lens; const int* slots;
  int heads, per_group, dim, vdim;
};

// Key-channel rows in LDS are laid out so that the NSP lanes of a column read
// neighbouring 16-byte pieces.
template <int NSP>
DEVINLINE int key_place(int c) { return (c % NPT) / 4 * (NSP * 4) + c / NPT * 4 + c % 4; }

template <typename T, int NSP, int VPT>
__global__ __launch_bounds__(256) void delta_fused_kernel(DeltaArgs a) {
  constexpr int R = DL_ROWS;
  constexpr int DP = NSP * NPT;                 // key channels, padded
  constexpr int NV = 256 / NSP * VPT;           // value columns, padded
  constexpr int KL = DP / 8;                    // pieces (and lanes) per key row
  constexpr int KU = (R * KL + 255) / 256;      // pieces of a chunk per thread
  constexpr int VU = (R * NV / 8 + 255) / 256;
  constexpr int GV = (NV + 63) / 64;
  constexpr int GR = R / 4;                     // rows per wave in the norm step
  extern __shared__ float smem[];
  float* k_s = smem;                // [R][DP], interleaved
  float* q_s = k_s + R * DP;
  float* v_s = q_s + R * DP;        // [R][NV]; outputs replace the values
  float* kq_s = v_s + R * NV;       // [R]
  float* g_s = kq_s + R;            // [R]
  float* beta_s = g_s + R;          // [R]

  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int grp = h / a.per_group;
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
  const T* kp = reinterpret_cast<const T*>(a.k) + (long)grp * a.dim;
  const T* qp = reinterpret_cast<const T*>(a.q) + (long)grp * a.dim;
  const T* vp = reinterpret_cast<const T*>(a.v) + (long)h * a.vdim;
  const T* gp = reinterpret_cast<const T*>(a.gate) + (long)h * a.vdim;
  const T* bp = reinterpret_cast<const T*>(a.b_pre) + h;
  const T* ap = reinterpret_cast<const T*>(a.a_pre) + h;
  const float a_log = a.a_log[h], dt_bias = a.dt_bias[h];

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
  float rb = 0.f, ra = 0.f;
  auto fetch = [&](int r0) {
    const int nr = min(R, n - r0);
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int idx = tid + u * 256, r = idx / KL, c = idx % KL * 8;
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
    if (tid < nr) {
      rb = ScalarOps<T>::to_f32(bp[(row0 + r0 + tid) * a.b_st]);
      ra = ScalarOps<T>::to_f32(ap[(row0 + r0 + tid) * a.a_st]);
    }
  };

  float G = 1.f;     // S = G * (what the registers hold)
  fetch(0);
  for (int r0 = 0; r0 < n; r0 += R) {
    const int nr = min(R, n - r0);
    // ---- this chunk into LDS, keys and queries as unit vectors ---------------
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int idx = tid + u * 256, r = idx / KL, c = idx % KL * 8;
      if (r < R) {                    // uniform over the wave
        float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float kv = rk[u].at(e), qv = rq[u].at(e);
          sk += kv * kv; sq += qv * qv; kq += kv * qv;
        }
        sk = lanes_sum<KL>(sk); sq = lanes_sum<KL>(sq); kq = lanes_sum<KL>(kq);
        const float ik = 1.0f / sqrtf(sk + kUnitEps), iq = a.q_scale / sqrtf(sq + kUnitEps);
        const int at = r * DP + key_place<NSP>(c);
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          const int e = half * 4;
          *reinterpret_cast<float4*>(k_s + at + half * NSP * 4) =
              make_float4(rk[u].at(e) * ik, rk[u].at(e + 1) * ik, rk[u].at(e + 2) * ik,
                          rk[u].at(e + 3) * ik);
          *reinterpret_cast<float4*>(q_s + at + half * NSP * 4) =
              make_float4(rq[u].at(e) * iq, rq[u].at(e + 1) * iq, rq[u].at(e + 2) * iq,
                          rq[u].at(e + 3) * iq);
        }
        if (c == 0) kq_s[r] = kq * ik * iq;
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
    if (tid < R) {
      g_s[tid] = delta_decay(ra, a_log, dt_bias);
      beta_s[tid] = sigmoid_f(rb);
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
                       ? ScalarOps<T>::to_f32(gp[(row0 + r0 + r) * a.gate_st + c]) : 0.f;
      }
    // ---- the recurrence --------------------------------------------------------
    for (int r = 0; r < nr; ++r) {
      G *= g_s[r];
      if (G < kSmallG) {              // uniform over the workgroup
#pragma unroll
        for (int c = 0; c < VPT; ++c)
#pragma unroll
          for (int i = 0; i < NPT; ++i) S[c][i] *= G;
        G = 1.f;
      }
      float vj[VPT], dk[VPT], dq[VPT], kk[NPT];
#pragma unroll
      for (int c = 0; c < VPT; ++c) {
        vj[c] = v_s[r * NV + jg * VPT + c];
        dk[c] = dq[c] = 0.f;
      }
#pragma unroll
      for (int i4 = 0; i4 < NPT / 4; ++i4) {
        const int at = r * DP + i4 * (NSP * 4) + ns * 4;
        const float4 k4 = *reinterpret_cast<const float4*>(k_s + at);
        const float4 q4 = *reinterpret_cast<const float4*>(q_s + at);
        const float qq[4] = {q4.x, q4.y, q4.z, q4.w};
        kk[i4 * 4] = k4.x; kk[i4 * 4 + 1] = k4.y; kk[i4 * 4 + 2] = k4.z; kk[i4 * 4 + 3] = k4.w;
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int c = 0; c < VPT; ++c) {
            dk[c] += S[c][i4 * 4 + e] * kk[i4 * 4 + e];
            dq[c] += S[c][i4 * 4 + e] * qq[e];
          }
      }
      const float beta = beta_s[r], kq = kq_s[r], inv_g = 1.0f / G;
#pragma unroll
      for (int c = 0; c < VPT; ++c) {
        dk[c] = lanes_sum<NSP>(dk[c]);
        dq[c] = lanes_sum<NSP>(dq[c]);
        const float u = beta * (vj[c] - G * dk[c]);
        dq[c] = G * dq[c] + kq * u;
        const float w = u * inv_g;
#pragma unroll
        for (int i = 0; i < NPT; ++i) S[c][i] += w * kk[i];
      }
      // only the lanes of this column group read these values, all before now
      if (ns == 0) {
#pragma unroll
        for (int c = 0; c < VPT; ++c) v_s[r * NV + jg * VPT + c] = dq[c];
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
            make_float4(S[c][i] * G, S[c][i + 1] * G, S[c][i + 2] * G, S[c][i + 3] * G);
  }
}

// Steps of single rows (correct for any number: each row reads back what the one
// before stored).  LW lanes per column, a lane holding eight of its elements as
// two 16-byte pieces; key and query of the row in registers.
template <typename T, int LW>
__global__ __launch_bounds__(256) void delta_row_kernel(DeltaArgs a) {
  constexpr int COLS = 256 / LW;    // columns side by side
  constexpr int FLY = 2;            // column groups in flight
  extern __shared__ float smem[];
  float* y_s = smem;                // [vdim]
  float* v_s = y_s + a.vdim;        // [vdim]
  __shared__ float red[8];
  const int s = blockIdx.x / a.heads;
  const int h = blockIdx.x % a.heads;
  const int grp = h / a.per_group;
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
  const float a_log = a.a_log[h], dt_bias = a.dt_bias[h];
  bool carry = a.seq_lens[s] - n > 0;
  for (int r = 0; r < n; ++r) {
    const long row = row0 + r;
    const T* kp = reinterpret_cast<const T*>(a.k) + row * a.k_st + (long)grp * a.dim;
    const T* qp = reinterpret_cast<const T*>(a.q) + row * a.q_st + (long)grp * a.dim;
    const T* vp = reinterpret_cast<const T*>(a.v) + row * a.v_st + (long)h * a.vdim;
    const T* gp = reinterpret_cast<const T*>(a.gate) + row * a.gate_st + (long)h * a.vdim;
    float k[8], q[8];
    float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int c = (i < 4 ? p0 : p1 - 4) + i;
      const bool in = i < 4 ? in0 : in1;
      k[i] = in ? ScalarOps<T>::to_f32(kp[c]) : 0.f;
      q[i] = in ? ScalarOps<T>::to_f32(qp[c]) : 0.f;
      sk += k[i] * k[i]; sq += q[i] * q[i]; kq += k[i] * q[i];
    }
    // through LDS: a load inside the column loop would wait for the columns ahead
    for (int c = tid; c < a.vdim; c += 256) v_s[c] = ScalarOps<T>::to_f32(vp[c]);
    const float g = delta_decay(
        ScalarOps<T>::to_f32(reinterpret_cast<const T*>(a.a_pre)[row * a.a_st + h]), a_log, dt_bias);
    const float beta =
        sigmoid_f(ScalarOps<T>::to_f32(reinterpret_cast<const T*>(a.b_pre)[row * a.b_st + h]));
    sk = lanes_sum<LW>(sk); sq = lanes_sum<LW>(sq); kq = lanes_sum<LW>(kq);
    const float ik = 1.0f / sqrtf(sk + kUnitEps), iq = a.q_scale / sqrtf(sq + kUnitEps);
    kq *= ik * iq;
#pragma unroll
    for (int i = 0; i < 8; ++i) { k[i] *= ik; q[i] *= iq; }
    __syncthreads();
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
        float dk = 0.f, dq = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          x[i] *= g;
          dk += x[i] * k[i];
          dq += x[i] * q[i];
        }
        dk = lanes_sum<LW>(dk);
        dq = lanes_sum<LW>(dq);
        const float u = beta * (v - dk);
#pragma unroll
        for (int i = 0; i < 8; ++i) x[i] += u * k[i];
        float* p = sbase + (long)j * a.dim;
        if (live && in0) *reinterpret_cast<float4*>(p + p0) = make_float4(x[0], x[1], x[2], x[3]);
        if (live && in1) *reinterpret_cast<float4*>(p + p1) = make_float4(x[4], x[5], x[6], x[7]);
        if (live && l == 0) y_s[j] = dq + kq * u;
      }
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = tid; c < a.vdim; c += 256) ss += y_s[c] * y_s[c];
    ss = block_reduce_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / a.vdim + a.eps);
    for (int c = tid; c < a.vdim; c += 256) {
      const float gt = ScalarOps<T>::to_f32(gp[c]);
      outp[row * out_st + c] = ScalarOps<T>::from_f32(
          y_s[c] * inv * a.norm[(long)h * a.vdim + c] * gt * sigmoid_f(gt));
    }
    __syncthreads();   // LDS is rewritten by the next row
    carry = true;
  }
}

}  // namespace

// value columns per thread of the one-kernel form, 0 when the shape does not fit
int delta_fused_columns(int dim, int vdim) {
  if (dim % 8 || vdim % 8 || dim > 256) return 0;
  const int nsp = dim <= 32 ? 2 : dim <= 64 ? 4 : dim <= 128 ? 8 : 16;
  for (int vpt = 1; vpt <= 4; vpt *= 2)
    if (256 / nsp * vpt >= vdim) return vpt;
  return 0;
}

template <typename T>
void launch_delta_fused(T* out, const T* q, long q_st, const T* k, long k_st, const T* v,
                        long v_st, const T* b_pre, long b_st, const T* a_pre, long a_st,
                        const float* a_log, const float* dt_bias, const T* gate, long gate_st,
                        const float* norm, float q_scale, float eps, float* state,
                        const int* loc, const int* seq_lens, const int* slots, int nseq,
                        int heads, int groups, int dim, int vdim, int rows,
                        hipStream_t stream) {
  DeltaArgs a;
  a.q = q; a.k = k; a.v = v; a.gate = gate; a.b_pre = b_pre; a.a_pre = a_pre;
  a.q_st = q_st; a.k_st = k_st; a.v_st = v_st; a.gate_st = gate_st; a.b_st = b_st; a.a_st = a_st;
  a.a_log = a_log; a.dt_bias = dt_bias; a.norm = norm;
  a.q_scale = q_scale; a.eps = eps;
  a.out = out; a.state = state;
  a.loc = loc; a.seq_lens = seq_lens; a.slots = slots;
  a.heads = heads; a.per_group = heads / groups; a.dim = dim; a.vdim = vdim;
  if (rows <= nseq) {   // a handful of rows per sequence at most: stream the state
    const size_t smem = sizeof(float) * 2 * vdim;
    if (dim <= 32) delta_row_kernel<T, 4><<<nseq * heads, 256, smem, stream>>>(a);
    else if (dim <= 64) delta_row_kernel<T, 8><<<nseq * heads, 256, smem, stream>>>(a);
    else if (dim <= 128) delta_row_kernel<T, 16><<<nseq * heads, 256, smem, stream>>>(a);
    else delta_row_kernel<T, 32><<<nseq * heads, 256, smem, stream>>>(a);
    return;
  }
  const int vpt = delta_fused_columns(dim, vdim);
#define DELTA_LAUNCH(N, V)                                                             \
  delta_fused_kernel<T, N, V><<<nseq * heads, 256,                                     \
                                sizeof(float) * DL_ROWS *                              \
                                    (2 * N * NPT + 256 / N * V + 3), stream>>>(a)
#define DELTA_CASE(N)                                                                  \
  if (vpt == 1) DELTA_LAUNCH(N, 1);                                                    \
  else if (vpt == 2) DELTA_LAUNCH(N, 2);                                               \
  else DELTA_LAUNCH(N, 4)
  if (dim <= 32) { DELTA_CASE(2); }
  else if (dim <= 64) { DELTA_CASE(4); }
  else if (dim <= 128) { DELTA_CASE(8); }
  else { DELTA_CASE(16); }
#undef DELTA_CASE
#undef DELTA_LAUNCH
}

#define INSTANTIATE(T)                                                                 \
  template void launch_delta_fused<T>(                                                 \
      T*, const T*, long, const T*, long, const T*, long, const T*, long, const T*,    \
      long, const float*, const float*, const T*, long, const float*, float, float,    \
      float*, const int*, const int*, const int*, int, int, int, int, int, int,        \
      hipStream_t);
INSTANTIATE(float)
INSTANTIATE(__hip_bfloat16)
