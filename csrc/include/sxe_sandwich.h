// Decode prologue of the norm on both sides of a sublayer (residual_norm.hip sandwich_norm, few rows): a
// workgroup builds the next product's input in LDS,
//   v = x + rms(y) wp [+ add],  input = rms(v) wn,   y = one row, or the sum of k rows picked by slots.
// Rows live in registers between the two reductions: M * K <= 8 U NT elements.
#pragma once
#include "sxe_common.h"

namespace sxe {
namespace sw {

constexpr int kMaxM = 4;

struct Args {
  const unsigned short *y, *wp, *wn;  // y [rows, K] bf16
  const float *x, *add;               // [M, K]; add may be null
  const int* slots;                   // [M, k] rows of y, or null (row m)
  int k;
  float eps;
  float* xo;                          // [M, K] v, written by the workgroup with `writer`
};

// NORM: act = bf16(v rinv wn), else act = bf16(v wn) and the caller scales by rinv[m]. red: LDS [NT / 64][kMaxM].
// Ends with a barrier.
template <int NT, int U, bool NORM>
__device__ __forceinline__ void build(const Args& a, int M, int K, bool writer, unsigned short* act, float* rinv,
                                      float (*red)[kMaxM]) {
  const int per = K / 8, n = M * per, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float v[U][8];
  f32x4 r0[U], r1[U];
  u16x8 gp[U];
  float ss[kMaxM] = {0.f, 0.f, 0.f, 0.f};
  const int k = a.slots != nullptr ? a.k : 1;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int idx = min(u * NT + (int)threadIdx.x, n - 1), m = idx / per, c = (idx - m * per) * 8;
    r0[u] = *reinterpret_cast<const f32x4*>(a.x + (int64_t)m * K + c);
    r1[u] = *reinterpret_cast<const f32x4*>(a.x + (int64_t)m * K + c + 4);
    gp[u] = *reinterpret_cast<const u16x8*>(a.wp + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[u][e] = 0.f;
  }
  for (int j0 = 0; j0 < k; j0 += 4) {  // every load of four rows is in flight before the first use
    u16x8 t[4][U];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int idx = min(u * NT + (int)threadIdx.x, n - 1), m = idx / per, c = (idx - m * per) * 8;
        t[j][u] = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
        if (j0 + j < k) {
          const int64_t row = a.slots != nullptr ? a.slots[m * a.k + j0 + j] : m;
          t[j][u] = *reinterpret_cast<const u16x8*>(a.y + row * K + c);
        }
      }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int e = 0; e < 8; ++e) v[u][e] += bf16_to_f32(t[j][u][e]);
  }
  auto reduce = [&]() {  // ss -> rinv-style factor per row in the return of factor()
#pragma unroll
    for (int m = 0; m < kMaxM; ++m) {
      const float t = wave_sum(ss[m]);
      if (lane == 0) red[wave][m] = t;
    }
    __syncthreads();
  };
  auto factor = [&](int m) {
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; ++w) t += red[w][m];
    return 1.f / sqrtf(t / (float)K + a.eps);
  };
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int idx = u * NT + threadIdx.x, m = min(idx, n - 1) / per;
    float q = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) q += v[u][e] * v[u][e];
#pragma unroll
    for (int mm = 0; mm < kMaxM; ++mm)
      if (mm == m && idx < n) ss[mm] += q;
  }
  reduce();
  float f[kMaxM];
#pragma unroll
  for (int m = 0; m < kMaxM; ++m) f[m] = factor(m);
  __syncthreads();  // red is free again
#pragma unroll
  for (int m = 0; m < kMaxM; ++m) ss[m] = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int idx = u * NT + threadIdx.x, cl = min(idx, n - 1), m = cl / per, c = (cl - m * per) * 8;
    float fm = f[0];
#pragma unroll
    for (int mm = 1; mm < kMaxM; ++mm) fm = mm == m ? f[mm] : fm;
    f32x4 a0 = {0.f, 0.f, 0.f, 0.f}, a1 = a0;
    if (a.add != nullptr) {
      a0 = *reinterpret_cast<const f32x4*>(a.add + (int64_t)m * K + c);
      a1 = *reinterpret_cast<const f32x4*>(a.add + (int64_t)m * K + c + 4);
    }
    float q = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      v[u][e] = v[u][e] * fm * bf16_to_f32(gp[u][e]) + (e < 4 ? r0[u][e & 3] + a0[e & 3] : r1[u][e & 3] + a1[e & 3]);
      q += v[u][e] * v[u][e];
    }
    if (idx < n) {
      if (writer) {
        *reinterpret_cast<f32x4*>(a.xo + (int64_t)m * K + c) = f32x4{v[u][0], v[u][1], v[u][2], v[u][3]};
        *reinterpret_cast<f32x4*>(a.xo + (int64_t)m * K + c + 4) = f32x4{v[u][4], v[u][5], v[u][6], v[u][7]};
      }
      if constexpr (!NORM) {
        float o[8];
        const u16x8 gn = *reinterpret_cast<const u16x8*>(a.wn + c);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = v[u][e] * bf16_to_f32(gn[e]);
        store8<DT::BF16>(act + (int64_t)m * K + c, o);
      }
#pragma unroll
      for (int mm = 0; mm < kMaxM; ++mm)
        if (mm == m) ss[mm] += q;
    }
  }
  reduce();
  if constexpr (NORM) {
#pragma unroll
    for (int m = 0; m < kMaxM; ++m) f[m] = factor(m);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int idx = u * NT + threadIdx.x, m = idx / per, c = (idx - m * per) * 8;
      if (idx >= n) continue;
      float fm = f[0], o[8];
      const u16x8 gn = *reinterpret_cast<const u16x8*>(a.wn + c);
#pragma unroll
      for (int mm = 1; mm < kMaxM; ++mm) fm = mm == m ? f[mm] : fm;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = v[u][e] * fm * bf16_to_f32(gn[e]);
      store8<DT::BF16>(act + (int64_t)m * K + c, o);
    }
  } else if (threadIdx.x < kMaxM) {
    rinv[threadIdx.x] = factor(threadIdx.x);
  }
  __syncthreads();
}

}  // namespace sw
}  // namespace sxe
