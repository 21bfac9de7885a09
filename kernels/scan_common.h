// Helpers shared by the recurrence kernels with per-sequence matrix state.
#pragma once

#include "common.h"

namespace {

constexpr int NPT = 16;   // state values per thread along the key axis

DEVINLINE float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
DEVINLINE float logsigmoid_f(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
DEVINLINE float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }

// decay of the gated delta rule, and what unit vectors add under the root
constexpr float kUnitEps = 1e-6f;
DEVINLINE float delta_decay(float a_pre, float a_log, float dt_bias) {
  return expf(-expf(a_log) * softplus_f(a_pre + dt_bias));
}

// Sum over NSP adjacent lanes (NSP a power of two, groups aligned), result in
// every lane.  Up to 16 lanes the partner values come through DPP modifiers on
// the adds (quad permutes, then the half-row and row mirrors — each mirror
// pairs a lane with one from the other, already uniform, half), which costs no
// LDS-crossbar round trip; wider groups finish with two shuffles.
template <int CTRL>
DEVINLINE float dpp_move(float v) {
  return __int_as_float(
      __builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
template <int NSP>
DEVINLINE float lanes_sum(float x) {
  if (NSP >= 2) x += dpp_move<0xB1>(x);    // quad_perm [1,0,3,2]
  if (NSP >= 4) x += dpp_move<0x4E>(x);    // quad_perm [2,3,0,1]
  if (NSP >= 8) x += dpp_move<0x141>(x);   // row_half_mirror
  if (NSP >= 16) x += dpp_move<0x140>(x);  // row_mirror
  if (NSP >= 32) x += __shfl_xor(x, 16, WAVE_SIZE);
  if (NSP >= 64) x += __shfl_xor(x, 32, WAVE_SIZE);
  return x;
}

// 16 consecutive values p[n0 .. n0+16) of a row of length n_total as f32,
// zeros past the end
template <typename T>
DEVINLINE void load_slice(const T* __restrict__ p, int n0, int n_total, bool vec,
                          float* dst) {
  if (vec && n0 + NPT <= n_total) {
    constexpr int V = Vec16<T>::kElems;
#pragma unroll
    for (int i = 0; i < NPT; i += V) {
      const Vec16<T> v = load16(p + n0 + i);
#pragma unroll
      for (int u = 0; u < V; ++u) dst[i + u] = ScalarOps<T>::to_f32(v.data[u]);
    }
  } else {
#pragma unroll
    for (int i = 0; i < NPT; ++i)
      dst[i] = (n0 + i < n_total) ? ScalarOps<T>::to_f32(p[n0 + i]) : 0.f;
  }
}

template <typename T> struct RowPiece;    // eight elements as stored
template <> struct RowPiece<__hip_bfloat16> {
  uint4 u;
  DEVINLINE float at(int i) const {
    const unsigned w[4] = {u.x, u.y, u.z, u.w};
    return __uint_as_float(i & 1 ? w[i / 2] & 0xffff0000u : w[i / 2] << 16);
  }
};
template <> struct RowPiece<float> {
  float f[8];
  DEVINLINE float at(int i) const { return f[i]; }
};

}  // namespace
