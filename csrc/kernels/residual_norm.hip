// Row kernels of decoders that keep a 32-bit residual stream (gfx950).
//
//  * embed_scale: x = table[id] * scale, fp32, plus its 16-bit copy for the next projection;
//  * residual_rms_norm: x' = rms(alpha * x + y) * (offset + w) -- the norm AFTER a scaled residual sum
//    (alpha and the weight's offset are parameters: offset 1 = a weight stored around zero, 0 = a plain
//    weight). x, x' and every intermediate are fp32, y is the sublayer's output in the compute
//    dtype; the 16-bit copy of x' the next projection reads is written in the same pass. Rows may be
//    picked by index (the last-token rows before the LM head);
//  * sandwich_norm: a sublayer with a norm on both sides and the next one's input in one pass,
//    x' = x + rms(y) * wp [+ add], h = rms(x') * wn (plain weights); y may be the sum of several rows
//    (expert outputs, one row per (token, expert));
//  * embed_norm: x = rms(table[id]) * w and h = rms(x) * wn;
//  * gated_rms_norm: rms(x) * w * sigmoid(gate) over whole rows;
//  * qkv_norm_append: RMS norm over a token's WHOLE query projection and whole key projection (all
//    heads at once, plain weights), the normalised q to [T, nq, Dq] and k, v to their paged cache
//    slots, head rows zero-padded to the cache's row length.
// One workgroup per row; a thread keeps its share of the row in registers between the reduction and the
// scaling pass when the row allows 4-wide accesses (any other width takes the scalar re-reading form).
#include "sxe_common.h"
#include <torch/library.h>

namespace sxe {
namespace rn {

constexpr int kThreads = 256;

template <DT T>
__device__ __forceinline__ f32x4 load4(const typename dt_traits<T>::storage* p) {
  if constexpr (T == DT::F32) {
    return *reinterpret_cast<const f32x4*>(p);
  } else {
    const u16x4 a = *reinterpret_cast<const u16x4*>(p);
    return f32x4{to_f32<T>(a[0]), to_f32<T>(a[1]), to_f32<T>(a[2]), to_f32<T>(a[3])};
  }
}
template <DT T>
__device__ __forceinline__ void store4(typename dt_traits<T>::storage* p, f32x4 v) {
  if constexpr (T == DT::F32) {
    *reinterpret_cast<f32x4*>(p) = v;
  } else {
    u16x4 a;
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] = from_f32<T>(v[i]);
    *reinterpret_cast<u16x4*>(p) = a;
  }
}

template <DT T, bool VEC>
__global__ __launch_bounds__(kThreads) void embed_scale_kernel(const typename dt_traits<T>::storage* __restrict table,
                                                               const int64_t* __restrict ids, int rows, int W,
                                                               float scale, float* __restrict x,
                                                               typename dt_traits<T>::storage* __restrict xb) {
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const bool ok = id >= 0 && id < rows;
  const auto* src = table + (ok ? id : 0) * W;
  if constexpr (VEC) {
    for (int c = threadIdx.x * 4; c < W; c += kThreads * 4) {
      f32x4 v = load4<T>(src + c) * scale;
      if (!ok) v = f32x4{0.f, 0.f, 0.f, 0.f};
      *reinterpret_cast<f32x4*>(x + t * W + c) = v;
      if (xb != nullptr) store4<T>(xb + t * W + c, v);
    }
    return;
  }
  for (int c = threadIdx.x; c < W; c += kThreads) {
    const float v = ok ? to_f32<T>(src[c]) * scale : 0.f;
    x[t * W + c] = v;
    if (xb != nullptr) xb[t * W + c] = from_f32<T>(v);
  }
}

// C > 0: 4-wide, C chunks of 4 x 256 elements in registers; C == 0: scalar, the row is read twice
template <DT T, int C>
__global__ __launch_bounds__(kThreads) void residual_rms_norm_kernel(
    const float* __restrict x, const typename dt_traits<T>::storage* __restrict y,
    const typename dt_traits<T>::storage* __restrict w, const int64_t* __restrict index, int W, float alpha, float eps,
    float offset, float* __restrict xo, typename dt_traits<T>::storage* __restrict xb) {
  __shared__ float red[kThreads / 64];
  const int64_t o = blockIdx.x, r = index != nullptr ? index[o] : o;
  const float* xr = x + r * W;
  const auto* yr = y != nullptr ? y + r * W : nullptr;
  float ss = 0.f;
  if constexpr (C > 0) {
    f32x4 h[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      h[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (c < W) {
        h[i] = *reinterpret_cast<const f32x4*>(xr + c) * alpha;
        if (yr != nullptr) h[i] += load4<T>(yr + c);
      }
    }
#pragma unroll
    for (int i = 0; i < C; ++i) ss += h[i][0] * h[i][0] + h[i][1] * h[i][1] + h[i][2] * h[i][2] + h[i][3] * h[i][3];
    ss = block_sum<kThreads / 64>(ss, red);
    const float rs = 1.f / sqrtf(ss / (float)W + eps);
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      if (c >= W) continue;
      const f32x4 g = load4<T>(w + c);
      f32x4 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = h[i][j] * rs * (offset + g[j]);
      if (xo != nullptr) *reinterpret_cast<f32x4*>(xo + o * W + c) = v;
      if (xb != nullptr) store4<T>(xb + o * W + c, v);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float v = xr[c] * alpha + (yr != nullptr ? to_f32<T>(yr[c]) : 0.f);
      ss += v * v;
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rs = 1.f / sqrtf(ss / (float)W + eps);
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float v = (xr[c] * alpha + (yr != nullptr ? to_f32<T>(yr[c]) : 0.f)) * rs * (offset + to_f32<T>(w[c]));
      if (xo != nullptr) xo[o * W + c] = v;
      if (xb != nullptr) xb[o * W + c] = from_f32<T>(v);
    }
  }
}

struct SandwichArgs {
  const float* x;        // [T, W] or nullptr (zero: embed_norm)
  const void* y;         // [T, W], rows picked by ids (table) or summed over slots
  const void *wp, *wn;   // norm weights after y and for h
  const float* add;      // [T, W] or nullptr
  const int* slots;      // [T, k] or nullptr
  const int64_t* ids;    // rows of y, or nullptr
  const int64_t* index;  // which rows to produce, or nullptr
  float* xo;             // nullptr: not wanted
  void* h;
  int W, k, rows;        // rows: of y, for ids
  float eps;
};

// C as in residual_rms_norm_kernel; C == 0 recomputes the sums in every pass
template <DT T, int C>
__global__ __launch_bounds__(kThreads) void sandwich_norm_kernel(SandwichArgs a) {
  using S = typename dt_traits<T>::storage;
  __shared__ float red[kThreads / 64];
  const int W = a.W;
  const int64_t o = blockIdx.x, r = a.index != nullptr ? a.index[o] : o;
  const float* xr = a.x != nullptr ? a.x + r * W : nullptr;
  const float* ar = a.add != nullptr ? a.add + r * W : nullptr;
  int64_t y0 = r;
  bool ok = true;
  if (a.ids != nullptr) {
    y0 = a.ids[r];
    ok = y0 >= 0 && y0 < a.rows;
    if (!ok) y0 = 0;
  }
  const S* yb = static_cast<const S*>(a.y);
  const S *wp = static_cast<const S*>(a.wp), *wn = static_cast<const S*>(a.wn);
  S* hr = static_cast<S*>(a.h) + o * W;
  float ss = 0.f;
  if constexpr (C > 0) {
    // everything the row needs is in flight before the first reduction
    f32x4 v[C], x0[C], g[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = min((i * kThreads + (int)threadIdx.x) * 4, W - 4);
      v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      x0[i] = xr != nullptr ? *reinterpret_cast<const f32x4*>(xr + c) : v[i];
      g[i] = load4<T>(wp + c);
    }
    if (a.slots == nullptr) {
#pragma unroll
      for (int i = 0; i < C; ++i) {
        const int c = (i * kThreads + threadIdx.x) * 4;
        if (c < W && ok) v[i] = load4<T>(yb + y0 * W + c);
      }
    } else {
      constexpr int J = 4;  // rows in flight
      for (int j0 = 0; j0 < a.k; j0 += J) {
        const S* yr[J];
#pragma unroll
        for (int j = 0; j < J; ++j) yr[j] = yb + (int64_t)a.slots[r * a.k + min(j0 + j, a.k - 1)] * W;
#pragma unroll
        for (int i = 0; i < C; ++i) {
          const int c = (i * kThreads + threadIdx.x) * 4;
          if (c >= W) continue;
          f32x4 t[J];
#pragma unroll
          for (int j = 0; j < J; ++j) t[j] = load4<T>(yr[j] + c);
#pragma unroll
          for (int j = 0; j < J; ++j)
            if (j0 + j < a.k) v[i] += t[j];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < C; ++i) ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    ss = block_sum<kThreads / 64>(ss, red);
    const float rp = 1.f / sqrtf(ss / (float)W + a.eps);
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      if (c >= W) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[i][j] = v[i][j] * rp * g[i][j] + x0[i][j];
      if (ar != nullptr) v[i] += *reinterpret_cast<const f32x4*>(ar + c);
      if (a.xo != nullptr) *reinterpret_cast<f32x4*>(a.xo + o * W + c) = v[i];
      ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rn = 1.f / sqrtf(ss / (float)W + a.eps);
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      if (c >= W) continue;
      const f32x4 g = load4<T>(wn + c);
      f32x4 h;
#pragma unroll
      for (int j = 0; j < 4; ++j) h[j] = v[i][j] * rn * g[j];
      store4<T>(hr + c, h);
    }
  } else {
    auto ysum = [&](int c) {
      if (a.slots == nullptr) return ok ? to_f32<T>(yb[y0 * W + c]) : 0.f;
      float t = 0.f;
      for (int j = 0; j < a.k; ++j) t += to_f32<T>(yb[(int64_t)a.slots[r * a.k + j] * W + c]);
      return t;
    };
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float t = ysum(c);
      ss += t * t;
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rp = 1.f / sqrtf(ss / (float)W + a.eps);
    auto sum = [&](int c) {
      return ysum(c) * rp * to_f32<T>(wp[c]) + (xr != nullptr ? xr[c] : 0.f) + (ar != nullptr ? ar[c] : 0.f);
    };
    ss = 0.f;
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float t = sum(c);
      ss += t * t;
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rn = 1.f / sqrtf(ss / (float)W + a.eps);
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float t = sum(c);
      if (a.xo != nullptr) a.xo[o * W + c] = t;
      hr[c] = from_f32<T>(t * rn * to_f32<T>(wn[c]));
    }
  }
}

// C as above, for the columns of x
template <DT T, int C>
__global__ __launch_bounds__(kThreads) void gated_rms_norm_kernel(const typename dt_traits<T>::storage* __restrict x,
                                                                  const typename dt_traits<T>::storage* __restrict w,
                                                                  const typename dt_traits<T>::storage* __restrict gate,
                                                                  int64_t ldg, int W, float eps,
                                                                  typename dt_traits<T>::storage* __restrict out) {
  __shared__ float red[kThreads / 64];
  const int64_t t = blockIdx.x;
  const auto *xr = x + t * W, *gr = gate + t * ldg;
  float ss = 0.f;
  if constexpr (C > 0) {
    f32x4 v[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      v[i] = c < W ? load4<T>(xr + c) : f32x4{0.f, 0.f, 0.f, 0.f};
      ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rs = 1.f / sqrtf(ss / (float)W + eps);
#pragma unroll
    for (int i = 0; i < C; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      if (c >= W) continue;
      const f32x4 g = load4<T>(gr + c), q = load4<T>(w + c);
      f32x4 h;
#pragma unroll
      for (int j = 0; j < 4; ++j) h[j] = v[i][j] * rs * q[j] / (1.f + expf(-g[j]));
      store4<T>(out + t * W + c, h);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += kThreads) {
      const float v = to_f32<T>(xr[c]);
      ss += v * v;
    }
    ss = block_sum<kThreads / 64>(ss, red);
    const float rs = 1.f / sqrtf(ss / (float)W + eps);
    for (int c = threadIdx.x; c < W; c += kThreads)
      out[t * W + c] = from_f32<T>(to_f32<T>(xr[c]) * rs * to_f32<T>(w[c]) / (1.f + expf(-to_f32<T>(gr[c]))));
  }
}

struct AppendArgs {
  const void* proj;  // [T, ld]: q | k | v (| anything) columns
  int64_t ld;
  const void *qw, *kw;  // norm weights [nq * dk], [nkv * dk]
  void* q;              // [T, nq, Dq], rows zero-padded from dk
  void *kc, *vc;        // caches [blocks, nkv, bs, Dk / Dv], block strides below, rows zero-padded
  int64_t k_block, v_block;
  const int64_t* slots;
  int nq, nkv, dk, dv, Dq, Dk, Dv, bs;
  float eps;
};

// V elements per access (8 where every size is a multiple of 8, else 1)
template <DT T, int V>
__device__ __forceinline__ void ldv(const typename dt_traits<T>::storage* p, float* v) {
  if constexpr (V == 8) {
    float t[8];
    load8<T>(p, t);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = t[i];
  } else {
    v[0] = to_f32<T>(*p);
  }
}
template <DT T, int V>
__device__ __forceinline__ void stv(typename dt_traits<T>::storage* p, const float* v) {
  if constexpr (V == 8) {
    float t[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) t[i] = v[i];
    store8<T>(p, t);
  } else {
    *p = from_f32<T>(v[0]);
  }
}

template <DT T, int V>
__global__ __launch_bounds__(kThreads) void qkv_norm_append_kernel(AppendArgs a) {
  using S = typename dt_traits<T>::storage;
  __shared__ float red[2][kThreads / 64];
  const int64_t t = blockIdx.x;
  const S* row = static_cast<const S*>(a.proj) + t * a.ld;
  const int nqr = a.nq * a.dk, nkr = a.nkv * a.dk;
  float sq = 0.f, sk = 0.f, v[V];
  for (int c = threadIdx.x * V; c < nqr + nkr; c += kThreads * V) {
    ldv<T, V>(row + c, v);
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < V; ++i) s += v[i] * v[i];
    if (c < nqr) sq += s;
    else sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (lane == 0) {
    red[0][wave] = sq;
    red[1][wave] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < kThreads / 64; ++i) {
    sq += red[0][i];
    sk += red[1][i];
  }
  const float rq = 1.f / sqrtf(sq / (float)nqr + a.eps), rk = 1.f / sqrtf(sk / (float)nkr + a.eps);
  const int64_t slot = a.slots[t];
  const int64_t blk = slot / a.bs, off = slot - blk * a.bs;
  const S *qw = static_cast<const S*>(a.qw), *kw = static_cast<const S*>(a.kw);
  const int nQ = a.nq * a.Dq, nK = a.nkv * a.Dk, nV = a.nkv * a.Dv;
  S* qo = static_cast<S*>(a.q) + t * nQ;
  for (int c = threadIdx.x * V; c < nQ + nK + nV; c += kThreads * V) {
    float o[V], w[V];
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] = 0.f;
    if (c < nQ) {
      const int h = c / a.Dq, d = c - h * a.Dq;
      if (d < a.dk) {
        ldv<T, V>(row + h * a.dk + d, o);
        ldv<T, V>(qw + h * a.dk + d, w);
#pragma unroll
        for (int i = 0; i < V; ++i) o[i] = o[i] * rq * w[i];
      }
      stv<T, V>(qo + c, o);
    } else if (slot >= 0) {
      if (c < nQ + nK) {
        const int e = c - nQ, h = e / a.Dk, d = e - h * a.Dk;
        if (d < a.dk) {
          ldv<T, V>(row + nqr + h * a.dk + d, o);
          ldv<T, V>(kw + h * a.dk + d, w);
#pragma unroll
          for (int i = 0; i < V; ++i) o[i] = o[i] * rk * w[i];
        }
        stv<T, V>(static_cast<S*>(a.kc) + blk * a.k_block + ((int64_t)h * a.bs + off) * a.Dk + d, o);
      } else {
        const int e = c - nQ - nK, h = e / a.Dv, d = e - h * a.Dv;
        if (d < a.dv) ldv<T, V>(row + nqr + nkr + h * a.dv + d, o);
        stv<T, V>(static_cast<S*>(a.vc) + blk * a.v_block + ((int64_t)h * a.bs + off) * a.Dv + d, o);
      }
    }
  }
}

inline bool aligned(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

// chunks of 4 x kThreads columns held in registers, 0 for the scalar form
inline int row_chunks(int64_t W, bool vec) {
  const int64_t n = (W + 1023) / 1024;
  return !vec || n > 16 ? 0 : n <= 1 ? 1 : n <= 2 ? 2 : n <= 4 ? 4 : n <= 8 ? 8 : 16;
}

template <DT D>
void launch_sandwich(const SandwichArgs& a, int64_t rows, bool vec) {
  auto go = [&](auto kern) { hipLaunchKernelGGL(kern, dim3(rows), dim3(kThreads), 0, cur_stream(), a); };
  switch (row_chunks(a.W, vec)) {
    case 1: go(sandwich_norm_kernel<D, 1>); break;
    case 2: go(sandwich_norm_kernel<D, 2>); break;
    case 4: go(sandwich_norm_kernel<D, 4>); break;
    case 8: go(sandwich_norm_kernel<D, 8>); break;
    case 16: go(sandwich_norm_kernel<D, 16>); break;
    default: go(sandwich_norm_kernel<D, 0>); break;
  }
}

}  // namespace rn

// table [V, W], ids int64 [T], w and wn [W] like the table -> [x = rms(table[id]) w fp32, h = rms(x) wn]
std::vector<at::Tensor> embed_norm(const at::Tensor& table, const at::Tensor& ids, const at::Tensor& w, const at::Tensor& wn,
                                   double eps) {
  SXE_CHECK_CUDA(table);
  SXE_CHECK(table.dim() == 2 && table.is_contiguous(), "embed_norm: table [V, W] contiguous");
  SXE_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.is_cuda(), "embed_norm: ids int64 [T]");
  const int64_t T = ids.numel(), W = table.size(1);
  for (const auto* p : {&w, &wn})
    SXE_CHECK(p->is_cuda() && p->is_contiguous() && p->numel() == W && p->scalar_type() == table.scalar_type(),
              "embed_norm: norm weights [W] in the table's dtype");
  auto x = at::empty({T, W}, table.options().dtype(at::kFloat)), h = at::empty({T, W}, table.options());
  if (T == 0 || W == 0) return {x, h};
  c10::DeviceGuard g(table.device());
  rn::SandwichArgs a{nullptr, table.data_ptr(), w.data_ptr(), wn.data_ptr(), nullptr, nullptr, ids.data_ptr<int64_t>(),
                     nullptr, x.data_ptr<float>(), h.data_ptr(), (int)W, 1, (int)table.size(0), (float)eps};
  const bool vec = W % 4 == 0 && rn::aligned(table.data_ptr(), 16) && rn::aligned(w.data_ptr(), 16) &&
                   rn::aligned(wn.data_ptr(), 16);
  SXE_DISPATCH_DT(dtype_of(table), D, rn::launch_sandwich<D>(a, T, vec));
  SXE_LAUNCH_CHECK();
  return {x, h};
}

// x fp32 [T, W]; y [rows, W] in the weights' dtype, rows = T or, with slots int32 [T, k], any; add fp32 [T, W] or
// None; index int64 [R] or None -> [x' fp32 [R, W] (empty without need_x), h [R, W]]
std::vector<at::Tensor> sandwich_norm(const at::Tensor& x, const at::Tensor& y, const at::Tensor& wp, const at::Tensor& wn,
                                      const c10::optional<at::Tensor>& slots, const c10::optional<at::Tensor>& add,
                                      const c10::optional<at::Tensor>& index, double eps, bool need_x) {
  SXE_CHECK_CUDA(x);
  SXE_CHECK(x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "sandwich_norm: x fp32 [T, W]");
  const int64_t T = x.size(0), W = x.size(1);
  for (const auto* p : {&wp, &wn})
    SXE_CHECK(p->is_cuda() && p->is_contiguous() && p->numel() == W && p->scalar_type() == y.scalar_type(),
              "sandwich_norm: norm weights [W] in y's dtype");
  const bool has_s = slots.has_value() && slots->defined(), has_a = add.has_value() && add->defined(),
             has_i = index.has_value() && index->defined();
  SXE_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() && y.size(1) == W && (has_s || y.size(0) == T),
            "sandwich_norm: y [T, W]");
  if (has_s)
    SXE_CHECK(slots->is_cuda() && slots->scalar_type() == at::kInt && slots->is_contiguous() && slots->dim() == 2 &&
                  slots->size(0) == T && slots->size(1) * T <= y.size(0), "sandwich_norm: slots int32 [T, k] of y's rows");
  if (has_a)
    SXE_CHECK(add->is_cuda() && add->scalar_type() == at::kFloat && add->is_contiguous() && add->sizes() == x.sizes(),
              "sandwich_norm: add like x");
  if (has_i)
    SXE_CHECK(index->scalar_type() == at::kLong && index->is_contiguous() && index->is_cuda(), "sandwich_norm: index int64 [R]");
  const int64_t R = has_i ? index->numel() : T;
  auto xo = need_x ? at::empty({R, W}, x.options()) : at::empty({0}, x.options());
  auto h = at::empty({R, W}, y.options());
  if (R == 0 || W == 0) return {xo, h};
  c10::DeviceGuard g(x.device());
  rn::SandwichArgs a{x.data_ptr<float>(), y.data_ptr(), wp.data_ptr(), wn.data_ptr(), has_a ? add->data_ptr<float>() : nullptr,
                     has_s ? slots->data_ptr<int>() : nullptr, nullptr, has_i ? index->data_ptr<int64_t>() : nullptr,
                     need_x ? xo.data_ptr<float>() : nullptr, h.data_ptr(), (int)W, has_s ? (int)slots->size(1) : 1,
                     (int)y.size(0), (float)eps};
  bool vec = W % 4 == 0 && rn::aligned(a.x, 16) && rn::aligned(a.y, 16) && rn::aligned(a.wp, 16) && rn::aligned(a.wn, 16) &&
             (!has_a || rn::aligned(a.add, 16));
  SXE_DISPATCH_DT(dtype_of(y), D, rn::launch_sandwich<D>(a, R, vec));
  SXE_LAUNCH_CHECK();
  return {xo, h};
}

// x [T, N] contiguous, w [N], gate [T, N] (rows may be strided), one dtype -> rms(x) w sigmoid(gate)
at::Tensor gated_rms_norm(const at::Tensor& x, const at::Tensor& w, const at::Tensor& gate, double eps) {
  SXE_CHECK_CUDA(x);
  SXE_CHECK(x.dim() == 2 && x.is_contiguous(), "gated_rms_norm: x [T, N]");
  const int64_t T = x.size(0), W = x.size(1);
  SXE_CHECK(w.is_cuda() && w.is_contiguous() && w.numel() == W && w.scalar_type() == x.scalar_type(), "gated_rms_norm: w [N]");
  SXE_CHECK(gate.is_cuda() && gate.dim() == 2 && gate.size(0) == T && gate.size(1) == W && gate.stride(1) == 1 &&
                gate.scalar_type() == x.scalar_type(), "gated_rms_norm: gate [T, N]");
  auto out = at::empty_like(x);
  if (T == 0 || W == 0) return out;
  c10::DeviceGuard g(x.device());
  const bool vec = W % 4 == 0 && gate.stride(0) % 4 == 0 && rn::aligned(x.data_ptr(), 16) && rn::aligned(w.data_ptr(), 16) &&
                   rn::aligned(gate.data_ptr(), x.element_size() * 4);
  SXE_DISPATCH_DT(dtype_of(x), D, {
    using S = dt_traits<D>::storage;
    auto go = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T), dim3(rn::kThreads), 0, cur_stream(), static_cast<const S*>(x.data_ptr()),
                         static_cast<const S*>(w.data_ptr()), static_cast<const S*>(gate.data_ptr()), gate.stride(0), (int)W,
                         (float)eps, static_cast<S*>(out.data_ptr()));
    };
    switch (rn::row_chunks(W, vec)) {
      case 1: go(rn::gated_rms_norm_kernel<D, 1>); break;
      case 2: go(rn::gated_rms_norm_kernel<D, 2>); break;
      case 4: go(rn::gated_rms_norm_kernel<D, 4>); break;
      case 8: go(rn::gated_rms_norm_kernel<D, 8>); break;
      case 16: go(rn::gated_rms_norm_kernel<D, 16>); break;
      default: go(rn::gated_rms_norm_kernel<D, 0>); break;
    }
  });
  SXE_LAUNCH_CHECK();
  return out;
}

// table [V, W], ids int64 [T] -> [x fp32 [T, W], 16-bit copy (x itself for an fp32 table)]
std::vector<at::Tensor> embed_scale(const at::Tensor& table, const at::Tensor& ids, double scale) {
  SXE_CHECK_CUDA(table);
  SXE_CHECK(table.dim() == 2 && table.is_contiguous(), "embed_scale: table [V, W] contiguous");
  SXE_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.is_cuda(), "embed_scale: ids int64 [T]");
  const int64_t T = ids.numel(), W = table.size(1);
  auto x = at::empty({T, W}, table.options().dtype(at::kFloat));
  const DT dt = dtype_of(table);
  auto xb = dt == DT::F32 ? x : at::empty({T, W}, table.options());
  if (T == 0 || W == 0) return {x, xb};
  c10::DeviceGuard g(table.device());
  const bool vec = W % 4 == 0 && rn::aligned(table.data_ptr(), 16);
  SXE_DISPATCH_DT(dt, D, {
    using S = dt_traits<D>::storage;
    auto go = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T), dim3(rn::kThreads), 0, cur_stream(), static_cast<const S*>(table.data_ptr()),
                         ids.data_ptr<int64_t>(), (int)table.size(0), (int)W, (float)scale, x.data_ptr<float>(),
                         D == DT::F32 ? nullptr : static_cast<S*>(xb.data_ptr()));
    };
    if (vec) go(rn::embed_scale_kernel<D, true>);
    else go(rn::embed_scale_kernel<D, false>);
  });
  SXE_LAUNCH_CHECK();
  return {x, xb};
}

// x fp32 [T, W], y [T, W] in w's dtype or None, index int64 [R] or None -> [x' fp32 [R, W], x' in w's dtype]
// (need_x false: the fp32 output is not written for a 16-bit w and comes back empty)
std::vector<at::Tensor> residual_rms_norm(const at::Tensor& x, const c10::optional<at::Tensor>& y, const at::Tensor& w,
                                          const c10::optional<at::Tensor>& index, double alpha, double eps,
                                          double offset, bool need_x) {
  SXE_CHECK_CUDA(x);
  SXE_CHECK(x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "residual_rms_norm: x fp32 [T, W]");
  const int64_t W = x.size(1);
  SXE_CHECK(w.is_contiguous() && w.numel() == W && w.is_cuda(), "residual_rms_norm: w [W]");
  const bool has_y = y.has_value() && y->defined(), has_i = index.has_value() && index->defined();
  if (has_y)
    SXE_CHECK(y->is_contiguous() && y->sizes() == x.sizes() && y->scalar_type() == w.scalar_type(),
              "residual_rms_norm: y like x, in w's dtype");
  if (has_i)
    SXE_CHECK(index->scalar_type() == at::kLong && index->is_contiguous() && index->is_cuda(),
              "residual_rms_norm: index int64 [R]");
  const int64_t R = has_i ? index->numel() : x.size(0);
  const DT dt = dtype_of(w);
  const bool f32 = dt == DT::F32;
  auto xo = (need_x || f32) ? at::empty({R, W}, x.options()) : at::empty({0}, x.options());
  auto xb = f32 ? xo : at::empty({R, W}, w.options());
  if (R == 0 || W == 0) return {xo, xb};
  c10::DeviceGuard g(x.device());
  const bool vec = W % 4 == 0 && rn::aligned(x.data_ptr(), 16) && rn::aligned(w.data_ptr(), 16) &&
                   (!has_y || rn::aligned(y->data_ptr(), 16));
  const int C = rn::row_chunks(W, vec);
  SXE_DISPATCH_DT(dt, D, {
    using S = dt_traits<D>::storage;
    auto go = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(R), dim3(rn::kThreads), 0, cur_stream(), x.data_ptr<float>(),
                         has_y ? static_cast<const S*>(y->data_ptr()) : nullptr, static_cast<const S*>(w.data_ptr()),
                         has_i ? index->data_ptr<int64_t>() : nullptr, (int)W, (float)alpha, (float)eps, (float)offset,
                         xo.numel() ? xo.data_ptr<float>() : nullptr, f32 ? nullptr : static_cast<S*>(xb.data_ptr()));
    };
    switch (C) {
      case 1: go(rn::residual_rms_norm_kernel<D, 1>); break;
      case 2: go(rn::residual_rms_norm_kernel<D, 2>); break;
      case 4: go(rn::residual_rms_norm_kernel<D, 4>); break;
      case 8: go(rn::residual_rms_norm_kernel<D, 8>); break;
      case 16: go(rn::residual_rms_norm_kernel<D, 16>); break;
      default: go(rn::residual_rms_norm_kernel<D, 0>); break;
    }
  });
  SXE_LAUNCH_CHECK();
  return {xo, xb};
}

// proj [T, >= nq dk + nkv (dk + dv)] (q | k | v first), kc / vc [blocks, nkv, bs, D*] views (inner three
// dims dense), slots int64 [T] (-1 = not cached) -> q [T, nq, Dq] with Dq = the k cache's row length
at::Tensor qkv_norm_append(const at::Tensor& proj, const at::Tensor& qw, const at::Tensor& kw, at::Tensor kc,
                           at::Tensor vc, const at::Tensor& slots, int64_t nq, int64_t nkv, int64_t dk, int64_t dv,
                           double eps) {
  SXE_CHECK_CUDA(proj);
  SXE_CHECK(proj.dim() == 2 && proj.stride(1) == 1 && proj.size(1) >= nq * dk + nkv * (dk + dv), "qkv_norm_append: proj");
  SXE_CHECK(qw.is_contiguous() && qw.numel() == nq * dk && kw.is_contiguous() && kw.numel() == nkv * dk &&
                qw.scalar_type() == proj.scalar_type() && kw.scalar_type() == proj.scalar_type(),
            "qkv_norm_append: norm weights [nq dk], [nkv dk] in proj's dtype");
  for (auto* c : {&kc, &vc})
    SXE_CHECK(c->dim() == 4 && c->size(1) == nkv && c->stride(3) == 1 && c->stride(2) == c->size(3) &&
                  c->stride(1) == c->size(2) * c->size(3) && c->scalar_type() == proj.scalar_type() && c->is_cuda(),
              "qkv_norm_append: caches [blocks, nkv, bs, D]");
  SXE_CHECK(kc.size(0) == vc.size(0) && kc.size(2) == vc.size(2) && kc.size(3) >= dk && vc.size(3) >= dv,
            "qkv_norm_append: cache sizes");
  SXE_CHECK(slots.scalar_type() == at::kLong && slots.is_contiguous() && slots.numel() == proj.size(0) && slots.is_cuda(),
            "qkv_norm_append: slots int64 [T]");
  const int64_t T = proj.size(0), D = kc.size(3);
  auto q = at::empty({T, nq, D}, proj.options());
  if (T == 0) return q;
  c10::DeviceGuard g(proj.device());
  rn::AppendArgs a{proj.data_ptr(), proj.stride(0), qw.data_ptr(), kw.data_ptr(), q.data_ptr(), kc.data_ptr(),
                   vc.data_ptr(), kc.stride(0), vc.stride(0), slots.data_ptr<int64_t>(), (int)nq, (int)nkv, (int)dk,
                   (int)dv, (int)D, (int)D, (int)vc.size(3), (int)kc.size(2), (float)eps};
  bool vec = dk % 8 == 0 && dv % 8 == 0 && D % 8 == 0 && vc.size(3) % 8 == 0 && proj.stride(0) % 8 == 0 &&
             kc.stride(0) % 8 == 0 && vc.stride(0) % 8 == 0;
  for (const void* p : {(const void*)a.proj, a.qw, a.kw, (const void*)a.q, (const void*)a.kc, (const void*)a.vc})
    vec = vec && rn::aligned(p, 16);
  SXE_DISPATCH_DT(dtype_of(proj), DD, {
    if (vec) hipLaunchKernelGGL((rn::qkv_norm_append_kernel<DD, 8>), dim3(T), dim3(rn::kThreads), 0, cur_stream(), a);
    else hipLaunchKernelGGL((rn::qkv_norm_append_kernel<DD, 1>), dim3(T), dim3(rn::kThreads), 0, cur_stream(), a);
  });
  SXE_LAUNCH_CHECK();
  return q;
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("embed_scale(Tensor table, Tensor ids, float scale) -> Tensor[]");
  m.def("residual_rms_norm(Tensor x, Tensor? y, Tensor w, Tensor? index, float alpha, float eps, float offset, "
        "bool need_x) -> Tensor[]");
  m.def("embed_norm(Tensor table, Tensor ids, Tensor w, Tensor wn, float eps) -> Tensor[]");
  m.def("sandwich_norm(Tensor x, Tensor y, Tensor wp, Tensor wn, Tensor? slots, Tensor? add, Tensor? index, float eps, "
        "bool need_x) -> Tensor[]");
  m.def("gated_rms_norm(Tensor x, Tensor w, Tensor gate, float eps) -> Tensor");
  m.def("qkv_norm_append(Tensor proj, Tensor qw, Tensor kw, Tensor(a!) kc, Tensor(b!) vc, Tensor slots, int nq, int nkv, "
        "int dk, int dv, float eps) -> Tensor");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("embed_scale", &sxe::embed_scale);
  m.impl("residual_rms_norm", &sxe::residual_rms_norm);
  m.impl("embed_norm", &sxe::embed_norm);
  m.impl("sandwich_norm", &sxe::sandwich_norm);
  m.impl("gated_rms_norm", &sxe::gated_rms_norm);
  m.impl("qkv_norm_append", &sxe::qkv_norm_append);
}
