// Row kernels of decoders that keep a 32-bit residual stream (gfx950).
//
//  * embed_scale: x = table[id] * scale, fp32, plus its 16-bit copy for the next projection;
//  * residual_rms_norm: x' = rms(alpha * x + y) * (offset + w) -- the norm AFTER a scaled residual sum
//    (alpha and the weight's offset are parameters: offset 1 = a weight stored around zero, 0 = a plain
//    weight). x, x' and every intermediate are fp32, y is the sublayer's output in the compute
//    dtype; the 16-bit copy of x' the next projection reads is written in the same pass. Rows may be
//    picked by index (the last-token rows before the LM head);
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

}  // namespace rn

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
  const int64_t chunks = (W + 1023) / 1024;
  const int C = !vec || chunks > 16 ? 0 : chunks <= 1 ? 1 : chunks <= 2 ? 2 : chunks <= 4 ? 4 : chunks <= 8 ? 8 : 16;
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
  m.def("qkv_norm_append(Tensor proj, Tensor qw, Tensor kw, Tensor(a!) kc, Tensor(b!) vc, Tensor slots, int nq, int nkv, "
        "int dk, int dv, float eps) -> Tensor");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("embed_scale", &sxe::embed_scale);
  m.impl("residual_rms_norm", &sxe::residual_rms_norm);
  m.impl("qkv_norm_append", &sxe::qkv_norm_append);
}
