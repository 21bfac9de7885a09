// Row kernels of layers with a grouped RMS norm before and after every sublayer
// and attention over a window plus a prefix.
//
//   stream_add_group_norm  x += N(y) w, N an RMS norm in equal groups, y one
//                          sublayer output (+ bias) or the scaled sum of two
//                          RMS-normed ones; then the norm that reads x next
//   rotary_table           cos, sin of position * frequency, once per step
//   attn_inputs            projected rows [q | k | v] -> bias, short causal
//                          convolution, query/key norm, rotation of queries,
//                          keys and values, paged cache write
//   pool_cache_write       means of completed blocks of cached keys / values
//   silu_mul_bias          silu(gate + b) * (up + b)
//
// All memory-bound.  Statistics, angles, convolution sums, means, gates and
// the stream are f32 whatever the storage type; every result is rounded once.

#include "common.h"

namespace {

struct F4 { float v[4]; };
template <typename T> DEVINLINE F4 ld4(const T* p);
template <> DEVINLINE F4 ld4<float>(const float* p) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  return F4{{t.x, t.y, t.z, t.w}};
}
template <> DEVINLINE F4 ld4<__hip_bfloat16>(const __hip_bfloat16* p) {
  const uint2 t = *reinterpret_cast<const uint2*>(p);
  return F4{{__uint_as_float(t.x << 16), __uint_as_float(t.x & 0xffff0000u),
             __uint_as_float(t.y << 16), __uint_as_float(t.y & 0xffff0000u)}};
}
template <typename T> DEVINLINE void st4(T* p, const F4& f);
template <> DEVINLINE void st4<float>(float* p, const F4& f) {
  *reinterpret_cast<float4*>(p) = make_float4(f.v[0], f.v[1], f.v[2], f.v[3]);
}
template <> DEVINLINE void st4<__hip_bfloat16>(__hip_bfloat16* p, const F4& f) {
  union { __hip_bfloat16 h[4]; uint2 u; } o;
#pragma unroll
  for (int i = 0; i < 4; ++i) o.h[i] = __float2bfloat16(f.v[i]);
  *reinterpret_cast<uint2*>(p) = o.u;
}

template <typename T>
DEVINLINE void ld8(const T* p, float* f) {
  const F4 a = ld4<T>(p), b = ld4<T>(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) { f[i] = a.v[i]; f[4 + i] = b.v[i]; }
}
template <>
DEVINLINE void ld8<__hip_bfloat16>(const __hip_bfloat16* p, float* f) {
  const uint4 t = *reinterpret_cast<const uint4*>(p);
  const unsigned u[4] = {t.x, t.y, t.z, t.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f[2 * i] = __uint_as_float(u[i] << 16);
    f[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u);
  }
}
// eight elements as they are stored
template <typename T> struct Raw8;
template <> struct Raw8<__hip_bfloat16> { uint4 u; };
template <> struct Raw8<float> { float4 a, b; };
template <typename T>
DEVINLINE Raw8<T> ldraw(const T* p) { return *reinterpret_cast<const Raw8<T>*>(p); }
template <typename T>
DEVINLINE void straw(T* p, const Raw8<T>& r) { *reinterpret_cast<Raw8<T>*>(p) = r; }
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
DEVINLINE void st8(T* p, const float* f) {
  st4<T>(p, F4{{f[0], f[1], f[2], f[3]}});
  st4<T>(p + 4, F4{{f[4], f[5], f[6], f[7]}});
}
template <>
DEVINLINE void st8<__hip_bfloat16>(__hip_bfloat16* p, const float* f) {
  union { __hip_bfloat16 h[8]; uint4 u; } o;
#pragma unroll
  for (int i = 0; i < 8; ++i) o.h[i] = __float2bfloat16(f[i]);
  *reinterpret_cast<uint4*>(p) = o.u;
}

// ---------------------------------------------------------------------------
// stream_add_group_norm.  Register variant: one workgroup per row, `wpg` waves
// per group of the norm, so that a wave's elements lie in one group and the row
// stays in registers from the first read to the last write (NV vectors of four
// per thread).
// ---------------------------------------------------------------------------
template <typename T, int NV>
__global__ __launch_bounds__(1024) void stream_add_group_norm_reg_kernel(
    float* __restrict__ x, const T* __restrict__ a, const float* __restrict__ a_bias,
    const T* __restrict__ b, const float* __restrict__ wa,
    const float* __restrict__ wb, const float* __restrict__ w_out,
    const float* __restrict__ next_w, T* __restrict__ next_out, float eps, float mix,
    int width, int gsize, int wpg) {
  __shared__ float r0[16], r1[16], r2[16], r3[16];
  const long row = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const int wave = threadIdx.x / WAVE_SIZE;
  const int nwaves = blockDim.x / WAVE_SIZE;
  const int g = wave / wpg;
  const int t = (wave - g * wpg) * WAVE_SIZE + lane;
  const int step = wpg * WAVE_SIZE;
  const int c0 = g * gsize;
  F4 xv[NV], wo[NV], wn[NV];
  auto col = [&](int i) { return (t + i * step) * 4; };
  // everything a reduction does not decide is loaded ahead of it
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    xv[i] = wo[i] = wn[i] = F4{{0.f, 0.f, 0.f, 0.f}};
    if (col(i) < gsize) {
      xv[i] = ld4<float>(x + row * width + c0 + col(i));
      if (w_out != nullptr) wo[i] = ld4<float>(w_out + c0 + col(i));
      if (next_w != nullptr) wn[i] = ld4<float>(next_w + c0 + col(i));
    }
  }
  auto group_sum = [&](float s, float* r) {
    s = wave_reduce_sum(s);
    if (lane == 0) r[wave] = s;
    __syncthreads();
    float tot = 0.f;
    for (int i = 0; i < wpg; ++i) tot += r[g * wpg + i];
    return tot;
  };
  if (a != nullptr) {
    F4 y[NV];
    if (b == nullptr) {
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        y[i] = F4{{0.f, 0.f, 0.f, 0.f}};
        if (col(i) < gsize) {
          y[i] = ld4<T>(a + row * width + c0 + col(i));
          if (a_bias != nullptr) {
            const F4 ab = ld4<float>(a_bias + c0 + col(i));
#pragma unroll
            for (int k = 0; k < 4; ++k) y[i].v[k] += ab.v[k];
          }
        }
      }
    } else {
      F4 z[NV];
      float sa = 0.f, sb = 0.f;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        y[i] = z[i] = F4{{0.f, 0.f, 0.f, 0.f}};
        if (col(i) < gsize) {
          y[i] = ld4<T>(a + row * width + c0 + col(i));
          z[i] = ld4<T>(b + row * width + c0 + col(i));
          if (a_bias != nullptr) {
            const F4 ab = ld4<float>(a_bias + c0 + col(i));
#pragma unroll
            for (int k = 0; k < 4; ++k) y[i].v[k] += ab.v[k];
          }
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          sa += y[i].v[k] * y[i].v[k];
          sb += z[i].v[k] * z[i].v[k];
        }
      }
      sa = wave_reduce_sum(sa);
      sb = wave_reduce_sum(sb);
      if (lane == 0) { r0[wave] = sa; r1[wave] = sb; }
      __syncthreads();
      sa = sb = 0.f;
      for (int i = 0; i < nwaves; ++i) { sa += r0[i]; sb += r1[i]; }
      const float ia = mix / sqrtf(sa / width + eps), ib = mix / sqrtf(sb / width + eps);
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (col(i) < gsize) {
          const F4 ua = ld4<float>(wa + c0 + col(i)), ub = ld4<float>(wb + c0 + col(i));
#pragma unroll
          for (int k = 0; k < 4; ++k)
            y[i].v[k] = y[i].v[k] * ia * ua.v[k] + z[i].v[k] * ib * ub.v[k];
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k) ss += y[i].v[k] * y[i].v[k];
    const float inv = 1.0f / sqrtf(group_sum(ss, r2) / gsize + eps);
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (col(i) < gsize) {
#pragma unroll
        for (int k = 0; k < 4; ++k) xv[i].v[k] += y[i].v[k] * inv * wo[i].v[k];
        st4<float>(x + row * width + c0 + col(i), xv[i]);
      }
  }
  if (next_w == nullptr) return;
  float sx = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int k = 0; k < 4; ++k) sx += xv[i].v[k] * xv[i].v[k];
  const float inv = 1.0f / sqrtf(group_sum(sx, r3) / gsize + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (col(i) < gsize) {
      F4 o;
#pragma unroll
      for (int k = 0; k < 4; ++k) o.v[k] = xv[i].v[k] * inv * wn[i].v[k];
      st4<T>(next_out + row * width + c0 + col(i), o);
    }
}

// Any width and group count: the groups one after the other, inputs re-read
// from cache between statistic and output.
template <typename T>
__global__ __launch_bounds__(256) void stream_add_group_norm_kernel(
    float* __restrict__ x, const T* __restrict__ a, const float* __restrict__ a_bias,
    const T* __restrict__ b, const float* __restrict__ wa,
    const float* __restrict__ wb, const float* __restrict__ w_out,
    const float* __restrict__ next_w, T* __restrict__ next_out, float eps, float mix,
    int width, int gsize) {
  __shared__ float red[8];
  const long row = blockIdx.x;
  float* xr = x + row * width;
  const T* ar = a + row * width;
  const T* br = b + row * width;
  auto reduce = [&](float s) {
    const float tot = block_reduce_sum(s, red);
    __syncthreads();   // red is used again
    return tot;
  };
  auto a_at = [&](int c) {
    return ScalarOps<T>::to_f32(ar[c]) + (a_bias != nullptr ? a_bias[c] : 0.f);
  };
  float ia = 1.f, ib = 0.f;
  if (a != nullptr && b != nullptr) {
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      const float u = a_at(c), v = ScalarOps<T>::to_f32(br[c]);
      sa += u * u;
      sb += v * v;
    }
    ia = mix / sqrtf(reduce(sa) / width + eps);
    ib = mix / sqrtf(reduce(sb) / width + eps);
  }
  auto y_at = [&](int c) {
    if (b == nullptr) return a_at(c);
    return a_at(c) * ia * wa[c] + ScalarOps<T>::to_f32(br[c]) * ib * wb[c];
  };
  for (int c0 = 0; c0 < width; c0 += gsize) {
    if (a != nullptr) {
      float ss = 0.f;
      for (int c = c0 + threadIdx.x; c < c0 + gsize; c += blockDim.x) {
        const float y = y_at(c);
        ss += y * y;
      }
      const float inv = 1.0f / sqrtf(reduce(ss) / gsize + eps);
      // every thread re-reads below only what it wrote itself
      for (int c = c0 + threadIdx.x; c < c0 + gsize; c += blockDim.x)
        xr[c] += y_at(c) * inv * w_out[c];
    }
    if (next_w != nullptr) {
      float sx = 0.f;
      for (int c = c0 + threadIdx.x; c < c0 + gsize; c += blockDim.x) sx += xr[c] * xr[c];
      const float inv = 1.0f / sqrtf(reduce(sx) / gsize + eps);
      for (int c = c0 + threadIdx.x; c < c0 + gsize; c += blockDim.x)
        next_out[row * width + c] = ScalarOps<T>::from_f32(xr[c] * inv * next_w[c]);
    }
  }
}

__global__ void rotary_table_kernel(float2* __restrict__ out, const long* __restrict__ pos,
                                    const float* __restrict__ inv_freq, int pairs, long n) {
  const long i = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (i >= n) return;
  const long t = i / pairs;
  float sn, cs;
  sincosf((float)pos[t] * inv_freq[i - t * pairs], &sn, &cs);
  out[i] = make_float2(cs, sn);
}

// ---------------------------------------------------------------------------
// attn_inputs.  Channel order [H*dim queries | G*dim keys | G*vdim values].
// The convolution's state keeps projected rows before the bias, as stored, so
// that a row read back from it is bit for bit the row a longer portion reads.
// ---------------------------------------------------------------------------
template <typename T>
struct AttnIn {
  const T* proj; long st;
  const float* bias;               // [C] or null
  const float* qw; const float* kw;  // [dim] or null
  const float* cw; T* conv_state; int taps;   // [taps, C]; [slots, taps-1, C]
  const float2* rot_tab; int rot;    // [rows, rot/2]
  const float2* v_tab; int vrot;     // [rows, vrot/2]
  T* q_out; T* k_cache; T* v_cache;
  const long* slot_mapping;
  const int* loc; const int* lens; const int* slots; int nseq;
  int rows, heads, kv_heads, dim, vdim, channels;
  float eps;
  int update_state;                  // every sequence brings one row
};

DEVINLINE int seq_of_row(const int* __restrict__ loc, int nseq, int row) {
  int lo = 0, hi = nseq;
  while (hi - lo > 1) {
    const int mid = (lo + hi) >> 1;
    if (loc[mid] <= row) lo = mid; else hi = mid;
  }
  return lo;
}

// one head of a row: which unit it is, where its channels start and go
template <typename T>
struct Unit {
  int size, rot, chan;
  const float* w;
  const float2* tab;
  bool norm;
  T* dst;
};
template <typename T>
DEVINLINE Unit<T> unit_of(const AttnIn<T>& p, int hh, long row, long slot) {
  Unit<T> u;
  const int nq = p.heads * p.dim, nk = p.kv_heads * p.dim;
  if (hh < p.heads + p.kv_heads) {
    const bool q = hh < p.heads;
    u.size = p.dim; u.rot = p.rot; u.norm = true;
    u.w = q ? p.qw : p.kw;
    u.tab = p.rot_tab + row * (p.rot / 2);
    u.chan = hh * p.dim;
    u.dst = q ? p.q_out + (row * p.heads + hh) * p.dim
              : (slot >= 0 ? p.k_cache + (slot * p.kv_heads + (hh - p.heads)) * p.dim : nullptr);
  } else {
    const int g = hh - p.heads - p.kv_heads;
    u.size = p.vdim; u.rot = p.vrot; u.norm = false;
    u.w = nullptr;
    u.tab = p.v_tab + row * (p.vrot / 2);
    u.chan = nq + nk + g * p.vdim;
    u.dst = slot >= 0 ? p.v_cache + (slot * p.kv_heads + g) * p.vdim : nullptr;
  }
  return u;
}

// Any sizes: one workgroup per row, one wave per head at a time, the head's
// values in LDS between the convolution and the rotation.
template <typename T>
__global__ __launch_bounds__(256) void attn_inputs_kernel(AttnIn<T> p) {
  extern __shared__ float smem[];
  const int row = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const int wave = threadIdx.x / WAVE_SIZE;
  float* buf = smem + wave * max(p.dim, p.vdim);
  const long slot = p.slot_mapping[row];
  int row0 = row, start = 0, state_slot = -1;
  if (p.cw != nullptr) {
    const int s = seq_of_row(p.loc, p.nseq, row);
    row0 = p.loc[s];
    start = p.lens[s] - (p.loc[s + 1] - row0);
    state_slot = p.slots[s];
  }
  const int pos = start + row - row0;
  T* state = p.conv_state + (long)max(state_slot, 0) * (p.taps - 1) * p.channels;
  const int total = p.heads + 2 * p.kv_heads;
  const int rounds = (total + 3) / 4;
  for (int r = 0; r < rounds; ++r) {
    const int hh = r * 4 + wave;
    float ss = 0.f;
    Unit<T> u{};
    if (hh < total) {
      u = unit_of(p, hh, row, slot);
      for (int c = lane; c < u.size; c += WAVE_SIZE) {
        const int ch = u.chan + c;
        const T raw = p.proj[row * p.st + ch];
        const float bias = p.bias != nullptr ? p.bias[ch] : 0.f;
        float y = ScalarOps<T>::to_f32(raw) + bias;
        if (p.cw != nullptr) {
          y *= p.cw[(long)(p.taps - 1) * p.channels + ch];
          for (int j = 0; j < p.taps - 1; ++j) {
            const int pj = pos - (p.taps - 1) + j;
            if (pj < 0 || (pj < start && state_slot < 0)) continue;
            const T h = pj >= start ? p.proj[(long)(row0 + pj - start) * p.st + ch]
                                    : state[(long)(pj - start + p.taps - 1) * p.channels + ch];
            y += p.cw[(long)j * p.channels + ch] * (ScalarOps<T>::to_f32(h) + bias);
          }
          if (p.update_state && state_slot >= 0) {
            for (int j = 0; j + 2 < p.taps; ++j)
              state[(long)j * p.channels + ch] = state[(long)(j + 1) * p.channels + ch];
            if (p.taps > 1) state[(long)(p.taps - 2) * p.channels + ch] = raw;
          }
        }
        buf[c] = y;
        ss += y * y;
      }
    }
    ss = wave_reduce_sum(ss);
    __syncthreads();
    if (hh < total && u.dst != nullptr) {
      const float inv = u.norm ? 1.0f / sqrtf(ss / u.size + p.eps) : 1.f;
      const int half = u.rot / 2;
      auto val = [&](int c) { return buf[c] * inv * (u.w != nullptr ? u.w[c] : 1.f); };
      for (int c = lane; c < u.size; c += WAVE_SIZE) {
        float y;
        if (c < half) {
          const float2 cs = u.tab[c];
          y = val(c) * cs.x - val(c + half) * cs.y;
        } else if (c < u.rot) {
          const float2 cs = u.tab[c - half];
          y = val(c) * cs.x + val(c - half) * cs.y;
        } else {
          y = val(c);
        }
        u.dst[c] = ScalarOps<T>::from_f32(y);
      }
    }
    __syncthreads();   // buf is rewritten by the next round
  }
}

// 16-byte accesses: eight lanes per head, a lane owning chunks of eight
// consecutive channels (for a rotated pair also the partner chunk).  A
// workgroup walks up to AI_ROWS consecutive rows per head, so that bias and convolution
// weights are read once for all of them and earlier rows stay in registers; the
// next row is loaded while the current one is computed.  PC pair chunks and TC unrotated chunks per lane at most.
constexpr int AI_ROWS = 16;

template <typename T, int TAPS, int PC, int TC>
__global__ __launch_bounds__(256) void attn_inputs_vec_kernel(AttnIn<T> p, int tb) {
  constexpr int NC = 2 * PC + TC;
  constexpr int HIST = TAPS > 1 ? TAPS - 1 : 1;
  constexpr int NW = TAPS > 0 ? TAPS : 1;
  __shared__ int s_row0[AI_ROWS], s_start[AI_ROWS], s_slot[AI_ROWS];
  __shared__ long s_cache[AI_ROWS];
  // last rows first: a step's single-row sequences lie there and, each with
  // earlier rows of its own to fetch, take longest
  const int t0 = (gridDim.x - 1 - blockIdx.x) * tb;
  const int n = min(tb, p.rows - t0);
  if (threadIdx.x < n) {
    s_cache[threadIdx.x] = p.slot_mapping[t0 + threadIdx.x];
    if (TAPS > 0) {
      const int s = seq_of_row(p.loc, p.nseq, t0 + threadIdx.x);
      s_row0[threadIdx.x] = p.loc[s];
      s_start[threadIdx.x] = p.lens[s] - (p.loc[s + 1] - p.loc[s]);
      s_slot[threadIdx.x] = p.slots[s];
    }
  }
  __syncthreads();
  const int sub = threadIdx.x & 7;
  const int total = p.heads + 2 * p.kv_heads;
  for (int hh = blockIdx.y * 32 + threadIdx.x / 8; hh < total; hh += gridDim.y * 32) {
    // the lane's chunks: offset inside the head, -1 = none
    int off[NC];
    {
      const Unit<T> u = unit_of(p, hh, 0, 0);
      const int npc = u.rot / 16, ntc = (u.size - u.rot) / 8;
#pragma unroll
      for (int j = 0; j < PC; ++j) {
        const int ch = sub + j * 8;
        off[2 * j] = ch < npc ? ch * 8 : -1;
        off[2 * j + 1] = ch < npc ? u.rot / 2 + ch * 8 : -1;
      }
#pragma unroll
      for (int j = 0; j < TC; ++j) {
        const int ch = sub + j * 8;
        off[2 * PC + j] = ch < ntc ? u.rot + ch * 8 : -1;
      }
    }
    const int chan = unit_of(p, hh, 0, 0).chan;
    float bias[NC][8], wn[NC][8], w[NC][NW][8], hist[NC][HIST][8];
    const float* norm_w = unit_of(p, hh, 0, 0).w;
#pragma unroll
    for (int i = 0; i < NC; ++i) {
#pragma unroll
      for (int k = 0; k < 8; ++k) { bias[i][k] = 0.f; wn[i][k] = 1.f; }
      if (off[i] >= 0) {
        if (norm_w != nullptr) ld8<float>(norm_w + off[i], wn[i]);
        if (p.bias != nullptr) ld8<float>(p.bias + chan + off[i], bias[i]);
        if (TAPS > 0) {
#pragma unroll
          for (int j = 0; j < TAPS; ++j)
            ld8<float>(p.cw + (long)j * p.channels + chan + off[i], w[i][j]);
        }
      }
    }
    // the next row and its angles, both ahead of this row's stores: loads and
    // stores retire in order, so a later load would wait for the stores too
    Raw8<T> next[NC];
    float next_cs[PC > 0 ? PC : 1][16];
    // ... and the rows ahead of it where they are not the ones just computed
    Raw8<T> before[NC][HIST];
    auto fetch = [&](int tt) {
      const long row = t0 + tt;
      const float2* tab = unit_of(p, hh, row, 0).tab;
      if (TAPS > 1 && (tt == 0 || row == s_row0[tt])) {
        const int row0 = s_row0[tt], start = s_start[tt], state_slot = s_slot[tt];
        const int pos = start + (int)row - row0;
        const T* state = p.conv_state + (long)max(state_slot, 0) * (TAPS - 1) * p.channels;
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
          const int pj = pos - (TAPS - 1) + j;
          if (pj < 0 || (pj < start && state_slot < 0)) continue;
          const T* src = pj >= start ? p.proj + (long)(row0 + pj - start) * p.st
                                     : state + (long)(pj - start + TAPS - 1) * p.channels;
#pragma unroll
          for (int i = 0; i < NC; ++i)
            if (off[i] >= 0) before[i][j] = ldraw<T>(src + chan + off[i]);
        }
      }
#pragma unroll
      for (int i = 0; i < NC; ++i)
        if (off[i] >= 0) next[i] = ldraw<T>(p.proj + row * p.st + chan + off[i]);
#pragma unroll
      for (int j = 0; j < PC; ++j)
        if (off[2 * j] >= 0) {
          ld8<float>(reinterpret_cast<const float*>(tab + off[2 * j]), next_cs[j]);
          ld8<float>(reinterpret_cast<const float*>(tab + off[2 * j] + 4), next_cs[j] + 8);
        }
    };
    fetch(0);
    for (int tt = 0; tt < n; ++tt) {
      const long row = t0 + tt;
      const long slot = s_cache[tt];
      Raw8<T> raw[NC];
      float cs[PC > 0 ? PC : 1][16];
#pragma unroll
      for (int i = 0; i < NC; ++i) raw[i] = next[i];
#pragma unroll
      for (int j = 0; j < PC; ++j)
#pragma unroll
        for (int k = 0; k < 16; ++k) cs[j][k] = next_cs[j][k];
      int state_slot = -1;
      T* state = nullptr;
      if (TAPS > 1) {
        state_slot = s_slot[tt];
        state = p.conv_state + (long)max(state_slot, 0) * (TAPS - 1) * p.channels;
        if (tt == 0 || row == s_row0[tt]) {
          const int start = s_start[tt], pos = start + (int)row - s_row0[tt];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) {
            const int pj = pos - (TAPS - 1) + j;
            const bool none = pj < 0 || (pj < start && state_slot < 0);
#pragma unroll
            for (int i = 0; i < NC; ++i) {
              if (off[i] < 0) continue;
              float f[8];
              unpack8(before[i][j], f);
#pragma unroll
              for (int k = 0; k < 8; ++k) hist[i][j][k] = none ? 0.f : f[k] + bias[i][k];
            }
          }
        }
      }
      if (tt + 1 < n) fetch(tt + 1);
      const Unit<T> u = unit_of(p, hh, row, slot);
      float y[NC][8];
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        if (off[i] < 0) continue;
        float cur[8];
        unpack8(raw[i], cur);
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          cur[k] += bias[i][k];
          y[i][k] = cur[k];
          if (TAPS > 0) {
            y[i][k] *= w[i][NW - 1][k];
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) y[i][k] += w[i][j][k] * hist[i][j][k];
          }
          ss += y[i][k] * y[i][k];
        }
        if (TAPS > 1) {
          if (p.update_state && state_slot >= 0) {
            T* sc = state + chan + off[i];
#pragma unroll
            for (int j = 0; j < TAPS - 2; ++j)
              straw<T>(sc + (long)j * p.channels, ldraw<T>(sc + (long)(j + 1) * p.channels));
            straw<T>(sc + (long)(TAPS - 2) * p.channels, raw[i]);
          }
#pragma unroll
          for (int j = 0; j < TAPS - 2; ++j)
#pragma unroll
            for (int k = 0; k < 8; ++k) hist[i][j][k] = hist[i][j + 1][k];
#pragma unroll
          for (int k = 0; k < 8; ++k) hist[i][HIST - 1][k] = cur[k];
        }
      }
      ss = group_reduce_sum<8>(ss);
      if (u.dst == nullptr) continue;
      const float inv = u.norm ? 1.0f / sqrtf(ss / u.size + p.eps) : 1.f;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        if (off[i] < 0) continue;
#pragma unroll
        for (int k = 0; k < 8; ++k) y[i][k] *= inv * wn[i][k];
      }
#pragma unroll
      for (int j = 0; j < PC; ++j) {
        if (off[2 * j] < 0) continue;
        float oa[8], ob[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          oa[k] = y[2 * j][k] * cs[j][2 * k] - y[2 * j + 1][k] * cs[j][2 * k + 1];
          ob[k] = y[2 * j + 1][k] * cs[j][2 * k] + y[2 * j][k] * cs[j][2 * k + 1];
        }
        st8<T>(u.dst + off[2 * j], oa);
        st8<T>(u.dst + off[2 * j + 1], ob);
      }
#pragma unroll
      for (int j = 0; j < TC; ++j)
        if (off[2 * PC + j] >= 0) st8<T>(u.dst + off[2 * PC + j], y[2 * PC + j]);
    }
  }
}

// ---------------------------------------------------------------------------
// pool_cache_write: one workgroup per `chunk` new rows (<= 256).  Rows that
// complete a block are found first, one row per thread; for each of them the
// workgroup writes the means of the block's cached keys and values to the place
// of that block inside the cache block that holds its last token.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void pool_cache_write_kernel(
    const T* __restrict__ k_cache, const T* __restrict__ v_cache, T* __restrict__ k_pool,
    T* __restrict__ v_pool, int pool, int per_block, const int* __restrict__ block_tables,
    int bt_stride, const int* __restrict__ qsl, const int* __restrict__ seq_lens, int nseq,
    int rows, int chunk, int block_size, int kn, int vn, int vec) {
  __shared__ int done_seq[256], done_end[256], count;
  if (threadIdx.x == 0) count = 0;
  __syncthreads();
  const int row = blockIdx.x * chunk + threadIdx.x;
  if (threadIdx.x < chunk && row < rows) {
    int seq = row, end;
    if (qsl != nullptr) {
      seq = seq_of_row(qsl, nseq, row);
      end = seq_lens[seq] - (qsl[seq + 1] - row) + 1;   // row's position + 1
    } else {
      end = seq_lens[seq];
    }
    if (end > 0 && end % pool == 0) {
      const int i = atomicAdd(&count, 1);
      done_seq[i] = seq;
      done_end[i] = end;
    }
  }
  __syncthreads();
  const int found = count;
  const float inv = 1.0f / pool;
  for (int i = 0; i < found; ++i) {
    const int end = done_end[i], first = end - pool, b = end / pool - 1;
    const int page = (end - 1) / block_size;
    const int* bt = block_tables + (long)done_seq[i] * bt_stride;
    const long dst = (long)bt[page] * per_block + (b - page * block_size / pool);
    auto tok = [&](int j) { return (long)bt[j / block_size] * block_size + j % block_size; };
    if (vec) {   // eight elements per thread
      for (int c = threadIdx.x * 8; c < kn + vn; c += blockDim.x * 8) {
        const bool isk = c < kn;
        const T* src = isk ? k_cache + c : v_cache + (c - kn);
        const long n = isk ? kn : vn;
        float s[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) s[u] = 0.f;
#pragma unroll 8
        for (int j = first; j < end; ++j) {
          float f[8];
          ld8<T>(src + tok(j) * n, f);
#pragma unroll
          for (int u = 0; u < 8; ++u) s[u] += f[u];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) s[u] *= inv;
        st8<T>(isk ? k_pool + dst * kn + c : v_pool + dst * vn + (c - kn), s);
      }
      continue;
    }
    for (int c = threadIdx.x; c < kn + vn; c += blockDim.x) {
      const bool isk = c < kn;
      const T* src = isk ? k_cache + c : v_cache + (c - kn);
      const long n = isk ? kn : vn;
      float s = 0.f;
      for (int j = first; j < end; ++j) s += ScalarOps<T>::to_f32(src[tok(j) * n]);
      *(isk ? k_pool + dst * kn + c : v_pool + dst * vn + (c - kn)) =
          ScalarOps<T>::from_f32(s * inv);
    }
  }
}

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void silu_mul_bias_kernel(
    T* __restrict__ out, const T* __restrict__ gu, const float* __restrict__ bias, int ff,
    long n) {
  constexpr int S = VEC ? 8 : 1;
  const long i = (blockIdx.x * (long)blockDim.x + threadIdx.x) * S;
  if (i >= n) return;
  const long row = i / ff;
  const int c = (int)(i - row * ff);
  const T* gp = gu + row * 2 * ff + c;
  float g[S], u[S];
  if constexpr (VEC) {
    ld8<T>(gp, g);
    ld8<T>(gp + ff, u);
    if (bias != nullptr) {
      float bg[8], bu[8];
      ld8<float>(bias + c, bg);
      ld8<float>(bias + ff + c, bu);
#pragma unroll
      for (int k = 0; k < 8; ++k) { g[k] += bg[k]; u[k] += bu[k]; }
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) g[k] = g[k] / (1.0f + expf(-g[k])) * u[k];
    st8<T>(out + i, g);
  } else {
    g[0] = ScalarOps<T>::to_f32(gp[0]);
    u[0] = ScalarOps<T>::to_f32(gp[ff]);
    if (bias != nullptr) { g[0] += bias[c]; u[0] += bias[ff + c]; }
    out[i] = ScalarOps<T>::from_f32(g[0] / (1.0f + expf(-g[0])) * u[0]);
  }
}

bool al16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

}  // namespace

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
template <typename T>
void launch_stream_add_group_norm(float* x, const T* a, const float* a_bias, const T* b,
                                  const float* wa, const float* wb, const float* w_out,
                                  const float* next_w, T* next_out, float eps, float mix,
                                  int rows, int width, int groups, hipStream_t s) {
  const int gsize = width / groups;
  bool vec = gsize % 4 == 0 && groups <= 16;
  for (const void* p : {(const void*)x, (const void*)a, (const void*)a_bias, (const void*)b,
                        (const void*)wa, (const void*)wb, (const void*)w_out,
                        (const void*)next_w, (const void*)next_out})
    vec = vec && al16(p);
  const int lanes = (gsize / 4 + WAVE_SIZE - 1) / WAVE_SIZE;   // waves a group can use
  int wpg = 4 / groups;
  if (width > 4096) wpg = 8 / groups;
  wpg = wpg < 1 ? 1 : (wpg > lanes ? lanes : wpg);
  const int nv = vec ? (gsize / 4 + wpg * WAVE_SIZE - 1) / (wpg * WAVE_SIZE) : 99;
#define GN_CASE(N)                                                                    \
  stream_add_group_norm_reg_kernel<T, N><<<rows, groups * wpg * WAVE_SIZE, 0, s>>>(   \
      x, a, a_bias, b, wa, wb, w_out, next_w, next_out, eps, mix, width, gsize, wpg)
  if (nv <= 1) GN_CASE(1);
  else if (nv <= 2) GN_CASE(2);
  else if (nv <= 4) GN_CASE(4);
  else if (nv <= 8) GN_CASE(8);
  else
    stream_add_group_norm_kernel<T><<<rows, 256, 0, s>>>(x, a, a_bias, b, wa, wb, w_out,
                                                         next_w, next_out, eps, mix, width,
                                                         gsize);
#undef GN_CASE
}

void launch_rotary_table(float* out, const long* pos, const float* inv_freq, int rows,
                         int pairs, hipStream_t s) {
  const long n = (long)rows * pairs;
  rotary_table_kernel<<<(int)((n + 255) / 256), 256, 0, s>>>(
      reinterpret_cast<float2*>(out), pos, inv_freq, pairs, n);
}

template <typename T>
void launch_conv_state_update(T*, const T*, const int*, const int*, const int*, int, int,
                              int, long, hipStream_t);

template <typename T>
void launch_attn_inputs(T* q_out, const T* proj, long st, const float* bias,
                        const float* qw, const float* kw, const float* cw, T* conv_state,
                        int taps, const float* rot_tab, int rot, const float* v_tab,
                        int vrot, T* k_cache, T* v_cache, const long* slot_mapping,
                        const int* loc, const int* lens, const int* slots, int nseq,
                        int rows, int heads, int kv_heads, int dim, int vdim, float eps,
                        int has_portions, hipStream_t s) {
  AttnIn<T> p;
  p.proj = proj; p.st = st; p.bias = bias; p.qw = qw; p.kw = kw;
  p.cw = cw; p.conv_state = conv_state; p.taps = taps;
  p.rot_tab = reinterpret_cast<const float2*>(rot_tab); p.rot = rot;
  p.v_tab = reinterpret_cast<const float2*>(v_tab); p.vrot = vrot;
  p.q_out = q_out; p.k_cache = k_cache; p.v_cache = v_cache; p.slot_mapping = slot_mapping;
  p.loc = loc; p.lens = lens; p.slots = slots; p.nseq = nseq;
  p.rows = rows; p.heads = heads; p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim;
  p.channels = heads * dim + kv_heads * (dim + vdim);
  p.eps = eps;
  p.update_state = cw != nullptr && taps > 1 && !has_portions;
  constexpr int E = 16 / sizeof(T);
  const int t = cw != nullptr ? taps : 0;
  bool vec = rot % 16 == 0 && (dim - rot) % 8 == 0 && vrot % 16 == 0 &&
             (vdim - vrot) % 8 == 0 && st % E == 0 && t <= 4;
  for (const void* q : {(const void*)proj, (const void*)bias, (const void*)qw, (const void*)kw,
                        (const void*)cw, (const void*)conv_state, (const void*)rot_tab,
                        (const void*)v_tab, (const void*)q_out, (const void*)k_cache,
                        (const void*)v_cache})
    vec = vec && al16(q);
  const int pmax = rot > vrot ? rot : vrot;
  const int tmax = dim - rot > vdim - vrot ? dim - rot : vdim - vrot;
  vec = vec && pmax <= 128 && tmax <= 128;
  if (vec) {
    const int tb = rows >= 4096 ? AI_ROWS : rows >= 2048 ? 8 : 1;
    const int total = heads + 2 * kv_heads;
    const dim3 grid((rows + tb - 1) / tb, (total + 31) / 32);
#define AI_LAUNCH(TP)                                                                   \
    if (tmax == 0) attn_inputs_vec_kernel<T, TP, 1, 0><<<grid, 256, 0, s>>>(p, tb);     \
    else if (pmax == 0) attn_inputs_vec_kernel<T, TP, 0, 2><<<grid, 256, 0, s>>>(p, tb); \
    else attn_inputs_vec_kernel<T, TP, 1, 2><<<grid, 256, 0, s>>>(p, tb)
    switch (t) {
      case 0: AI_LAUNCH(0); break;
      case 1: AI_LAUNCH(1); break;
      case 2: AI_LAUNCH(2); break;
      case 3: AI_LAUNCH(3); break;
      default: AI_LAUNCH(4); break;
    }
#undef AI_LAUNCH
  } else {
    const size_t smem = sizeof(float) * 4 * (dim > vdim ? dim : vdim);
    attn_inputs_kernel<T><<<rows, 256, smem, s>>>(p);
  }
  if (cw != nullptr && taps > 1 && has_portions)
    launch_conv_state_update<T>(conv_state, proj, loc, lens, slots, nseq, p.channels, taps,
                                st, s);
}

template <typename T>
void launch_pool_cache_write(const T* k_cache, const T* v_cache, T* k_pool, T* v_pool,
                             int pool, int per_block, const int* block_tables, int bt_stride,
                             const int* qsl, const int* seq_lens, int nseq, int rows,
                             int block_size, int kn, int vn, hipStream_t s) {
  const int vec = kn % 8 == 0 && vn % 8 == 0 && al16(k_cache) && al16(v_cache) &&
                  al16(k_pool) && al16(v_pool);
  // about one completed block per workgroup
  const int chunk = qsl == nullptr ? 1 : (pool < 256 ? pool : 256);
  pool_cache_write_kernel<T><<<(rows + chunk - 1) / chunk, 256, 0, s>>>(
      k_cache, v_cache, k_pool, v_pool, pool, per_block, block_tables, bt_stride, qsl,
      seq_lens, nseq, rows, chunk, block_size, kn, vn, vec);
}

template <typename T>
void launch_silu_mul_bias(T* out, const T* gu, const float* bias, int ff, long rows,
                          hipStream_t s) {
  const long n = rows * ff;
  if (ff % 8 == 0 && al16(out) && al16(gu) && al16(bias))
    silu_mul_bias_kernel<T, true><<<(int)((n / 8 + 255) / 256), 256, 0, s>>>(out, gu, bias,
                                                                            ff, n);
  else
    silu_mul_bias_kernel<T, false><<<(int)((n + 255) / 256), 256, 0, s>>>(out, gu, bias, ff,
                                                                         n);
}

#define INSTANTIATE(T)                                                                  \
  template void launch_stream_add_group_norm<T>(                                        \
      float*, const T*, const float*, const T*, const float*, const float*,             \
      const float*, const float*, T*, float, float, int, int, int, hipStream_t);        \
  template void launch_attn_inputs<T>(                                                  \
      T*, const T*, long, const float*, const float*, const float*, const float*, T*,   \
      int, const float*, int, const float*, int, T*, T*, const long*, const int*,       \
      const int*, const int*, int, int, int, int, int, int, float, int, hipStream_t);   \
  template void launch_pool_cache_write<T>(const T*, const T*, T*, T*, int, int,        \
                                           const int*, int, const int*, const int*,     \
                                           int, int, int, int, int, hipStream_t);       \
  template void launch_silu_mul_bias<T>(T*, const T*, const float*, int, long,          \
                                        hipStream_t);
INSTANTIATE(float)
INSTANTIATE(__hip_bfloat16)
