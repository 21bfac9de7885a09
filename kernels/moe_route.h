// Choice of experts for one token by one wave, shared by the router kernels.
#pragma once

#include "common.h"

namespace {

// scores: softmax of the logits, or (sigmoid) their sigmoid; choice scores: plus
// the correction, which the sigmoid form may lack.  groups > 1 (at most 64): only
// the experts of the `keep` groups of neighbours with the largest sum of their two
// best choice scores stay open.  The `top` largest choice scores are chosen (ties:
// the lower index); their weights are the scores, renorm: divided by their sum,
// times scale.  Outputs past num_real are identity experts.
struct RouteRule {
  const float* correction;
  int n, num_real, top, sigmoid, groups, keep, renorm;
  float scale;
};

constexpr int RT_MAX = 8;   // experts per lane at most

// best score and its index over `span` lanes (a power of two), ties to the lower
DEVINLINE void best_of(float& best, int& at, int span) {
  for (int off = span >> 1; off > 0; off >>= 1) {
    const float ob = __shfl_xor(best, off, WAVE_SIZE);
    const int oa = __shfl_xor(at, off, WAVE_SIZE);
    if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
  }
}

// Lane l owns experts l, l + 64, ... (RT of them); with at most 32 experts or
// groups the reductions stay inside the lanes that have any.
template <int RT>
DEVINLINE void moe_route_lanes(const float* z, const RouteRule& rule, float* dense, float* ident,
                               int* ids, float* wts) {
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const int n = rule.n;
  int span = WAVE_SIZE;
  while (span > 1 && span / 2 >= n && span / 2 >= rule.groups) span >>= 1;
  float s[RT], ch[RT];
  bool taken[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int e = lane + i * WAVE_SIZE;
    s[i] = (e < n) ? z[e] : -INFINITY;
    taken[i] = false;
  }
  if (!rule.sigmoid) {
    float m = -INFINITY, den = 0.f;
#pragma unroll
    for (int i = 0; i < RT; ++i) m = fmaxf(m, s[i]);
    m = wave_reduce_max(m);
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      s[i] = (lane + i * WAVE_SIZE < n) ? expf(s[i] - m) : 0.f;
      den += s[i];
    }
    den = wave_reduce_sum(den);
#pragma unroll
    for (int i = 0; i < RT; ++i) s[i] = s[i] / den;
  } else {
#pragma unroll
    for (int i = 0; i < RT; ++i)
      s[i] = (lane + i * WAVE_SIZE < n) ? 1.0f / (1.0f + expf(-s[i])) : 0.f;
  }
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int e = lane + i * WAVE_SIZE;
    ch[i] = -INFINITY;
    if (e < n) ch[i] = s[i] + (rule.correction != nullptr ? rule.correction[e] : 0.f);
  }

  if (rule.groups > 1) {
    const int size = n / rule.groups;
    float score = -INFINITY;       // lane g: group g's
    if (RT == 1 && (size & (size - 1)) == 0) {
      // groups are aligned runs of lanes: all of them at once
      float b1 = ch[0], b2 = -INFINITY;
      for (int off = 1; off < size; off <<= 1) {
        const float o1 = __shfl_xor(b1, off, WAVE_SIZE), o2 = __shfl_xor(b2, off, WAVE_SIZE);
        b2 = fmaxf(fmaxf(b2, o2), fminf(b1, o1));
        b1 = fmaxf(b1, o1);
      }
      const float both = size > 1 ? b1 + b2 : b1;
      const float mine = __shfl(both, (lane * size) & (WAVE_SIZE - 1), WAVE_SIZE);
      if (lane < rule.groups) score = mine;
    } else {
      for (int g = 0; g < rule.groups; ++g) {
        float b1 = -INFINITY, b2 = -INFINITY;   // this lane's two best in the group
#pragma unroll
        for (int i = 0; i < RT; ++i) {
          const int e = lane + i * WAVE_SIZE;
          if (e >= g * size && e < (g + 1) * size) {
            b2 = fmaxf(b2, fminf(b1, ch[i]));
            b1 = fmaxf(b1, ch[i]);
          }
        }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) {
          const float o1 = __shfl_xor(b1, off, WAVE_SIZE), o2 = __shfl_xor(b2, off, WAVE_SIZE);
          b2 = fmaxf(fmaxf(b2, o2), fminf(b1, o1));
          b1 = fmaxf(b1, o1);
        }
        if (lane == g) score = size > 1 ? b1 + b2 : b1;
      }
    }
    unsigned long long open = 0;
    for (int k = 0; k < rule.keep; ++k) {
      const bool free = lane < rule.groups && !((open >> lane) & 1);
      float best = free ? score : -INFINITY;
      int at = free ? lane : 0x7fffffff;
      best_of(best, at, span);
      if (at < rule.groups) open |= 1ull << at;
    }
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int e = lane + i * WAVE_SIZE;
      if (e < n && !((open >> (e / size)) & 1)) ch[i] = -INFINITY;
    }
  }

  float total = 0.f, id_sum = 0.f;
  for (int k = 0; k < rule.top; ++k) {
    float best = -INFINITY;
    int best_e = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int e = lane + i * WAVE_SIZE;
      if (e < n && !taken[i] && (ch[i] > best || (ch[i] == best && e < best_e))) {
        best = ch[i];
        best_e = e;
      }
    }
    best_of(best, best_e, span);
    // the owner marks it and tells the others its score
    float sv = 0.f;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      if (lane + i * WAVE_SIZE == best_e) taken[i] = true;
      if (best_e / WAVE_SIZE == i) sv = s[i];
    }
    sv = __shfl(sv, best_e & (WAVE_SIZE - 1), WAVE_SIZE);
    total += sv;
    if (best_e >= rule.num_real) id_sum += sv;
    if (lane == 0) {
      ids[k] = best_e;
      wts[k] = sv;
    }
  }
  const float inv = (rule.renorm ? 1.0f / (total + 1e-20f) : 1.0f) * rule.scale;
  if (dense != nullptr) {
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int e = lane + i * WAVE_SIZE;
      if (e < rule.num_real) dense[e] = taken[i] ? s[i] * inv : 0.f;
    }
  }
  // lane 0 wrote wts itself, so it may rescale them in place
  if (lane == 0) {
    if (rule.renorm || rule.scale != 1.0f)
      for (int k = 0; k < rule.top; ++k) wts[k] *= inv;
    if (ident != nullptr) *ident = id_sum * inv;
  }
}

DEVINLINE void moe_route_token(const float* z, const RouteRule& rule, float* dense, float* ident,
                               int* ids, float* wts) {
  if (rule.n <= WAVE_SIZE) moe_route_lanes<1>(z, rule, dense, ident, ids, wts);
  else moe_route_lanes<RT_MAX>(z, rule, dense, ident, ids, wts);
}

}  // namespace
