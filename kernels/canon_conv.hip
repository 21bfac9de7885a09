// Short depthwise causal convolution over time with per-sequence state.
//
//   out_t = act([h_t +] sum_j w[:, j] * h_(t - taps + 1 + j) [+ bias])
//
// act is the identity or silu; the input rows may be a column slice of a wider
// matrix (row stride in_st), output and state rows are dense.
//
// A step brings, for each sequence, rows [loc[s], loc[s+1]) of new inputs that
// continue the sequence at position start = seq_len - n.  Inputs older than the
// step's rows come from state[slot] (the last taps-1 inputs, row j holding
// position start - (taps-1) + j); positions before 0 are zero and are never
// read from the state, so a reused slot needs no clearing.  A second kernel on
// the same stream advances the state past the new rows: row j of the new state
// is position end - (taps-1) + j, taken from the step's rows or, when the step
// is shorter than taps-1, from old state row j + n — each thread walks j
// upwards, so it reads row j + n before that row is overwritten.
//
// Two kernels.  The row-walking one: a thread owns 8 channels and walks up to
// CW_ROWS consecutive rows with their weights and the last taps-1 inputs in
// registers, so every input is read once, the next rows' while these are
// computed; where every sequence of the step brings a single row it also
// advances the state itself (nobody else reads that sequence's rows).  The other
// takes any tap count and width: one thread per (row, 4 channels) — or one channel when the width is not a
// multiple of 4.  Consecutive threads take consecutive channels,
// every load and store is coalesced; accumulation is f32.

#include "common.h"

template <typename T, int CH>
DEVINLINE void load_ch(const T* p, float* v) {
  if (CH == 4) {
    if (sizeof(T) == 4) {
      const float4 t = *reinterpret_cast<const float4*>(p);
      v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
    } else {
      const uint2 t = *reinterpret_cast<const uint2*>(p);
      v[0] = __uint_as_float(t.x << 16);
      v[1] = __uint_as_float(t.x & 0xffff0000u);
      v[2] = __uint_as_float(t.y << 16);
      v[3] = __uint_as_float(t.y & 0xffff0000u);
    }
  } else {
    v[0] = ScalarOps<T>::to_f32(p[0]);
  }
}

template <typename T, int CH>
DEVINLINE void store_ch(T* p, const float* v) {
#pragma unroll
  for (int k = 0; k < CH; ++k) p[k] = ScalarOps<T>::from_f32(v[k]);
}

// eight channels as they are stored
template <typename T> struct Vec8;
template <> struct Vec8<__hip_bfloat16> {
  uint4 u;
  static DEVINLINE Vec8 load(const __hip_bfloat16* p) {
    return Vec8{*reinterpret_cast<const uint4*>(p)};
  }
  DEVINLINE void unpack(float* f) const {
    const unsigned t[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[2 * i] = __uint_as_float(t[i] << 16);
      f[2 * i + 1] = __uint_as_float(t[i] & 0xffff0000u);
    }
  }
  static DEVINLINE void store(__hip_bfloat16* p, const float* f) {
    union { __hip_bfloat16 h[8]; uint4 u; } o;
#pragma unroll
    for (int i = 0; i < 8; ++i) o.h[i] = __float2bfloat16(f[i]);
    *reinterpret_cast<uint4*>(p) = o.u;
  }
};
template <> struct Vec8<float> {
  float4 a, b;
  static DEVINLINE Vec8 load(const float* p) {
    return Vec8{reinterpret_cast<const float4*>(p)[0], reinterpret_cast<const float4*>(p)[1]};
  }
  DEVINLINE void unpack(float* f) const {
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
    f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
  }
  static DEVINLINE void store(float* p, const float* f) {
    reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
    reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
  }
};

DEVINLINE int find_seq(const int* __restrict__ loc, int nseq, int row) {
  int lo = 0, hi = nseq;  // largest s with loc[s] <= row
  while (hi - lo > 1) {
    const int mid = (lo + hi) >> 1;
    if (loc[mid] <= row) lo = mid; else hi = mid;
  }
  return lo;
}

// CH channels per thread: 4 (8/16-byte accesses) when width % 4 == 0, else 1.
// TAPS > 0: tap count known at compile time — the thread's CH x TAPS weights
// are one contiguous run fetched with 16-byte loads into registers; TAPS == 0
// reads them one by one for any tap count.
template <typename T, int CH, int TAPS>
__global__ void causal_conv_kernel(T* __restrict__ out, const T* __restrict__ h,
                                   const float* __restrict__ w,   // [W, taps]
                                   const T* __restrict__ state,   // [slots, taps-1, W]
                                   const int* __restrict__ loc,
                                   const int* __restrict__ seq_lens,
                                   const int* __restrict__ slots, int nseq,
                                   int width, int taps, int add_input,
                                   long in_st, const float* __restrict__ bias,
                                   int act) {
  const int row = blockIdx.x;
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * CH;
  if (c >= width) return;
  const int s = find_seq(loc, nseq, row);
  const int slot = slots[s];
  const long o = (long)row * width + c;
  float acc[CH];
  if (slot < 0) {  // padding row of a captured bucket
#pragma unroll
    for (int k = 0; k < CH; ++k) acc[k] = 0.f;
    store_ch<T, CH>(out + o, acc);
    return;
  }
  const int n = loc[s + 1] - loc[s];
  const int start = seq_lens[s] - n;
  const int p = start + (row - loc[s]);
  const T* st = state + (long)slot * (taps - 1) * width;
  float wreg[CH * (TAPS > 0 ? TAPS : 1)];
  if (TAPS > 0 && CH == 4) {
#pragma unroll
    for (int i = 0; i < TAPS; ++i) {
      const float4 t = reinterpret_cast<const float4*>(w + (long)c * TAPS)[i];
      wreg[4 * i] = t.x; wreg[4 * i + 1] = t.y; wreg[4 * i + 2] = t.z; wreg[4 * i + 3] = t.w;
    }
  }
  if (add_input) {
    load_ch<T, CH>(h + (long)row * in_st + c, acc);
  } else {
#pragma unroll
    for (int k = 0; k < CH; ++k) acc[k] = 0.f;
  }
#pragma unroll
  for (int j = 0; j < (TAPS > 0 ? TAPS : taps); ++j) {
    const int pj = p - (taps - 1) + j;
    if (pj < 0) continue;
    float v[CH];
    if (pj >= start)
      load_ch<T, CH>(h + (long)(loc[s] + pj - start) * in_st + c, v);
    else
      load_ch<T, CH>(st + (long)(pj - (start - (taps - 1))) * width + c, v);
#pragma unroll
    for (int k = 0; k < CH; ++k) {
      const float wk = (TAPS > 0 && CH == 4) ? wreg[k * TAPS + j] : w[(c + k) * taps + j];
      acc[k] += wk * v[k];
    }
  }
  if (bias != nullptr) {
#pragma unroll
    for (int k = 0; k < CH; ++k) acc[k] += bias[c + k];
  }
  if (act == 1) {
#pragma unroll
    for (int k = 0; k < CH; ++k) acc[k] = acc[k] / (1.0f + expf(-acc[k]));
  }
  store_ch<T, CH>(out + o, acc);
}

constexpr int CW_ROWS = 16;

template <typename T, int TAPS, int ROWS>
__global__ __launch_bounds__(256) void causal_conv_walk_kernel(
    T* __restrict__ out, const T* __restrict__ h, const float* __restrict__ w,
    T* __restrict__ state, const int* __restrict__ loc, const int* __restrict__ seq_lens,
    const int* __restrict__ slots, int nseq, int rows, int width, int add_input, long in_st,
    const float* __restrict__ bias, int act, int single_rows) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= width) return;
  constexpr int AHEAD = ROWS < 4 ? ROWS : 4;   // rows loaded ahead of the ones computed
  const int r0 = blockIdx.x * ROWS, r1 = min(r0 + ROWS, rows);
  Vec8<T> nxt[AHEAD];
  auto fetch = [&](int row) {
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
      if (row + u < r1) nxt[u] = Vec8<T>::load(h + (long)(row + u) * in_st + c);
  };
  fetch(r0);
  float wv[TAPS][8], bv[8], hist[TAPS][8];   // hist[TAPS - 1]: the current row
#pragma unroll
  for (int k = 0; k < 8; ++k) {
    bv[k] = bias != nullptr ? bias[c + k] : 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) wv[j][k] = w[(long)(c + k) * TAPS + j];
  }
  int s = find_seq(loc, nseq, r0);
  bool fresh = true;             // the history registers do not hold this sequence's rows
  for (int g0 = r0; g0 < r1; g0 += AHEAD) {
    Vec8<T> now[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) now[u] = nxt[u];
    if (g0 + AHEAD < r1) fetch(g0 + AHEAD);
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      const int row = g0 + u;
      if (row >= r1) break;
      while (s + 1 < nseq && row >= loc[s + 1]) { ++s; fresh = true; }
      const int slot = slots[s], first = loc[s];
      const int start = seq_lens[s] - (loc[s + 1] - first);
      const int p = start + row - first;
      if (fresh) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
          const int pj = p - (TAPS - 1) + j;
#pragma unroll
          for (int k = 0; k < 8; ++k) hist[j][k] = 0.f;
          if (pj >= start)
            Vec8<T>::load(h + (long)(first + pj - start) * in_st + c).unpack(hist[j]);
          else if (pj >= 0 && slot >= 0)
            Vec8<T>::load(state + ((long)slot * (TAPS - 1) + pj - start + TAPS - 1) * width + c)
                .unpack(hist[j]);
        }
        fresh = false;
      }
      now[u].unpack(hist[TAPS - 1]);
      float acc[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        acc[k] = bv[k] + (add_input ? hist[TAPS - 1][k] : 0.f);
#pragma unroll
        for (int j = 0; j < TAPS; ++j) acc[k] += wv[j][k] * hist[j][k];
        if (act == 1) acc[k] = acc[k] / (1.0f + __expf(-acc[k]));
        if (slot < 0) acc[k] = 0.f;           // padding row of a captured bucket
      }
      Vec8<T>::store(out + (long)row * width + c, acc);
      if (single_rows && slot >= 0) {
        T* st = state + (long)slot * (TAPS - 1) * width + c;
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) Vec8<T>::store(st + (long)j * width, hist[j + 1]);
      }
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
        for (int k = 0; k < 8; ++k) hist[j][k] = hist[j + 1][k];
    }
  }
}

template <typename T>
__global__ void conv_state_update_kernel(T* __restrict__ state,
                                         const T* __restrict__ h,
                                         const int* __restrict__ loc,
                                         const int* __restrict__ seq_lens,
                                         const int* __restrict__ slots,
                                         int width, int taps, long in_st) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= width) return;
  const int slot = slots[s];
  if (slot < 0) return;
  const int n = loc[s + 1] - loc[s];
  if (n <= 0) return;
  const int end = seq_lens[s];
  const int start = end - n;
  T* st = state + (long)slot * (taps - 1) * width;
  for (int j = 0; j < taps - 1; ++j) {
    const int pj = end - (taps - 1) + j;
    T v = ScalarOps<T>::from_f32(0.f);
    if (pj >= start)
      v = h[(long)(loc[s] + pj - start) * in_st + c];
    else if (pj >= 0)
      v = st[(long)(j + n) * width + c];
    st[(long)j * width + c] = v;
  }
}

// advances the kept inputs of every sequence past its new rows (taps > 1)
template <typename T>
void launch_conv_state_update(T* state, const T* h, const int* loc, const int* seq_lens,
                              const int* slots, int nseq, int width, int taps, long in_st,
                              hipStream_t stream) {
  const int block = 256;
  dim3 g2(nseq, (width + block - 1) / block);
  conv_state_update_kernel<T><<<g2, block, 0, stream>>>(state, h, loc, seq_lens, slots,
                                                       width, taps, in_st);
}

template <typename T>
void launch_causal_conv_state(T* out, const T* h, const float* w, T* state,
                              const int* loc, const int* seq_lens,
                              const int* slots, int rows, int nseq, int width,
                              int taps, int add_input, long in_st,
                              const float* bias, int act, int single_rows,
                              hipStream_t stream) {
  const int block = 256;
  const bool walk = taps >= 2 && taps <= 4 && width % 8 == 0 && in_st % 8 == 0 &&
                    reinterpret_cast<uintptr_t>(h) % 16 == 0 &&
                    reinterpret_cast<uintptr_t>(out) % 16 == 0 &&
                    reinterpret_cast<uintptr_t>(state) % 16 == 0;
  if (walk) {
    const int gy = (width / 8 + block - 1) / block;
#define WALK_LAUNCH(TP, R)                                                         \
    causal_conv_walk_kernel<T, TP, R><<<dim3((rows + R - 1) / R, gy), block, 0, stream>>>( \
        out, h, w, state, loc, seq_lens, slots, nseq, rows, width, add_input, in_st, bias, act, \
        single_rows)
#define WALK_CASE(TP)                                                              \
    if (single_rows || rows < 1024) WALK_LAUNCH(TP, 1); else WALK_LAUNCH(TP, CW_ROWS)
    if (taps == 2) { WALK_CASE(2); }
    else if (taps == 3) { WALK_CASE(3); }
    else { WALK_CASE(4); }
#undef WALK_CASE
#undef WALK_LAUNCH
    if (!single_rows)
      launch_conv_state_update<T>(state, h, loc, seq_lens, slots, nseq, width, taps, in_st,
                                  stream);
    return;
  }
  const bool vec = width % 4 == 0 && in_st % 4 == 0 &&
                   (bias == nullptr || reinterpret_cast<uintptr_t>(bias) % 16 == 0) &&
                   reinterpret_cast<uintptr_t>(h) % (4 * sizeof(T)) == 0 &&
                   reinterpret_cast<uintptr_t>(state) % (4 * sizeof(T)) == 0 &&
                   reinterpret_cast<uintptr_t>(w) % 16 == 0;
  if (vec) {
    dim3 g1(rows, (width / 4 + block - 1) / block);
#define CONV_LAUNCH(TP)                                                        \
    causal_conv_kernel<T, 4, TP><<<g1, block, 0, stream>>>(                    \
        out, h, w, state, loc, seq_lens, slots, nseq, width, taps, add_input, \
        in_st, bias, act)
    switch (taps) {
      case 2: CONV_LAUNCH(2); break;
      case 3: CONV_LAUNCH(3); break;
      case 4: CONV_LAUNCH(4); break;
      default: CONV_LAUNCH(0); break;
    }
#undef CONV_LAUNCH
  } else {
    dim3 g1(rows, (width + block - 1) / block);
    causal_conv_kernel<T, 1, 0><<<g1, block, 0, stream>>>(
        out, h, w, state, loc, seq_lens, slots, nseq, width, taps, add_input,
        in_st, bias, act);
  }
  if (taps > 1)
    launch_conv_state_update<T>(state, h, loc, seq_lens, slots, nseq, width, taps, in_st,
                                stream);
}

template void launch_causal_conv_state<float>(float*, const float*, const float*,
                                              float*, const int*, const int*,
                                              const int*, int, int, int, int,
                                              int, long, const float*, int, int,
                                              hipStream_t);
template void launch_causal_conv_state<__hip_bfloat16>(
    __hip_bfloat16*, const __hip_bfloat16*, const float*, __hip_bfloat16*,
    const int*, const int*, const int*, int, int, int, int, int, long,
    const float*, int, int, hipStream_t);
template void launch_conv_state_update<float>(float*, const float*, const int*,
                                              const int*, const int*, int, int, int,
                                              long, hipStream_t);
template void launch_conv_state_update<__hip_bfloat16>(
    __hip_bfloat16*, const __hip_bfloat16*, const int*, const int*, const int*, int,
    int, int, long, hipStream_t);
