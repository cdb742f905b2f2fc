// Paged attention whose per-head weights are mixed across heads after the softmax (gfx950), with the
// score and mask variants such designs combine -- each one an optional argument:
//   * score_h(i, j) = scale q_h(i) . k_c(j) - r1_h ln(1 + r2_h (i - j))      (distance bias)
//   * i sees j <= i with i - j < window or j < keep_first                    (window with kept first keys)
//   * the softmax denominator also holds exp(sink_h)                         (sink: no key, no value)
//   * w_h(i, j) = sum_g talk[h, g] p_g(i, j), then head h applies w_h to the values of its own
//     key/value head c = h / (nq / nkv)                                      (talking heads)
//   * out *= sigmoid(gate) element by element                                (output gate)
// The mix couples all heads of a token BEFORE the value product and needs normalised weights, so a
// one-pass online softmax cannot carry it: every form below first finds the row's log-sum-exp, then
// forms the weights.
//
// Only visible keys are ever touched: position p has n0 = min(keep_first, lo) kept keys in front of
// its window [lo, p], lo = max(0, p + 1 - window), enumerated as one compact run of n0 + p + 1 - lo keys.
// Caches are [blocks, nkv, bs, D] views (k and v separately, block stride free).
#include "sxe_common.h"
#include <torch/library.h>

namespace sxe {
namespace ma {

constexpr float kLog2e = 1.4426950408889634f;

struct Args {
  const void* q;  // [T, nq, Dk] dense
  const void *kc, *vc;
  int64_t k_block, v_block;  // elements between blocks
  const int* block_table;
  int max_blocks;
  const int *q_start, *q_len, *kv_len;
  int S, T, nq, nkv, dk, dv, Dk, Dv, bs;  // dk / dv real sizes, Dk / Dv row lengths of the caches
  float scale;
  int window, keep_first;      // window 0: every key <= i
  const float *r1, *r2, *sink;  // [nq] or null (r1, r2 together)
  const float* talk;           // [nq, nq] or null
  const void* gate;            // [T, gate_ld] or null
  int64_t gate_ld;
  void* out;                   // [T, nq * dv]
};

struct Vis {
  int n0, lo, n;  // kept keys, window start, number of visible keys
};
__device__ __forceinline__ Vis visible(int pos, int window, int keep_first) {
  Vis v;
  v.lo = window > 0 ? max(0, pos + 1 - window) : 0;
  v.n0 = min(keep_first, v.lo);
  v.n = v.n0 + pos + 1 - v.lo;
  return v;
}
__device__ __forceinline__ int vis_key(const Vis& v, int c) { return c < v.n0 ? c : v.lo + c - v.n0; }

// ---- any type, any sizes: one workgroup per token, all heads -----------------------------------
constexpr int kGenThreads = 256, kGenKeys = 32;

template <DT T>
__global__ __launch_bounds__(kGenThreads) void mix_attn_generic_kernel(Args a, int max_q_len) {
  using S = typename dt_traits<T>::storage;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int seq = blockIdx.x / max_q_len, tok = blockIdx.x - seq * max_q_len;
  if (tok >= a.q_len[seq]) return;
  const int pos = a.kv_len[seq] - a.q_len[seq] + tok;
  const int64_t t = a.q_start[seq] + tok;
  const int G = a.nq / a.nkv, tid = threadIdx.x;
  float* ql = lds;                              // [nq * dk]
  float* ol = ql + a.nq * a.dk;                 // [nq * dv]
  float* pl = ol + a.nq * a.dv;                 // [nq][kGenKeys]
  float* wl = pl + a.nq * kGenKeys;             // [nq][kGenKeys]
  float* ml = wl + a.nq * kGenKeys;             // [nq]
  float* ll = ml + a.nq;                        // [nq]
  const S* q = static_cast<const S*>(a.q) + t * a.nq * a.Dk;
  for (int e = tid; e < a.nq * a.dk; e += kGenThreads) {
    const int h = e / a.dk;
    ql[e] = to_f32<T>(q[h * a.Dk + e - h * a.dk]);
  }
  for (int e = tid; e < a.nq * a.dv; e += kGenThreads) ol[e] = 0.f;
  for (int h = tid; h < a.nq; h += kGenThreads) {
    ml[h] = a.sink != nullptr ? a.sink[h] : -INFINITY;
    ll[h] = a.sink != nullptr ? 1.f : 0.f;
  }
  const Vis vis = visible(pos, a.window, a.keep_first);
  const int* bt = a.block_table + (int64_t)seq * a.max_blocks;
  for (int pass = 0; pass < 2; ++pass) {
    for (int c0 = 0; c0 < vis.n; c0 += kGenKeys) {
      const int nk = min(kGenKeys, vis.n - c0);
      __syncthreads();
      for (int e = tid; e < a.nq * kGenKeys; e += kGenThreads) {
        const int h = e / kGenKeys, kk = e - h * kGenKeys;
        float s = -INFINITY;
        if (kk < nk) {
          const int key = vis_key(vis, c0 + kk);
          const S* k = static_cast<const S*>(a.kc) + bt[key / a.bs] * a.k_block +
                       ((int64_t)(h / G) * a.bs + key % a.bs) * a.Dk;
          const float* qh = ql + h * a.dk;
          float d = 0.f;
          for (int i = 0; i < a.dk; ++i) d += qh[i] * to_f32<T>(k[i]);
          s = d * a.scale;
          if (a.r1 != nullptr) s -= a.r1[h] * logf(1.f + a.r2[h] * (float)(pos - key));
        }
        pl[e] = pass == 0 ? s : (kk < nk ? expf(s - ml[h]) / ll[h] : 0.f);
      }
      __syncthreads();
      if (pass == 0) {
        for (int h = tid; h < a.nq; h += kGenThreads) {
          float m = ml[h], l = ll[h];
          for (int kk = 0; kk < nk; ++kk) m = fmaxf(m, pl[h * kGenKeys + kk]);
          l *= ml[h] == -INFINITY ? 0.f : expf(ml[h] - m);
          for (int kk = 0; kk < nk; ++kk) l += expf(pl[h * kGenKeys + kk] - m);
          ml[h] = m;
          ll[h] = l;
        }
        continue;
      }
      const float* wt = pl;
      if (a.talk != nullptr) {
        for (int e = tid; e < a.nq * kGenKeys; e += kGenThreads) {
          const int h = e / kGenKeys, kk = e - h * kGenKeys;
          float w = 0.f;
          for (int g = 0; g < a.nq; ++g) w += a.talk[h * a.nq + g] * pl[g * kGenKeys + kk];
          wl[e] = w;
        }
        wt = wl;
        __syncthreads();
      }
      for (int e = tid; e < a.nq * a.dv; e += kGenThreads) {
        const int h = e / a.dv, d = e - h * a.dv;
        float o = ol[e];
        for (int kk = 0; kk < nk; ++kk) {
          const int key = vis_key(vis, c0 + kk);
          const S* v = static_cast<const S*>(a.vc) + bt[key / a.bs] * a.v_block +
                       ((int64_t)(h / G) * a.bs + key % a.bs) * a.Dv;
          o += wt[h * kGenKeys + kk] * to_f32<T>(v[d]);
        }
        ol[e] = o;
      }
    }
  }
  S* out = static_cast<S*>(a.out) + t * a.nq * a.dv;
  const S* gate = a.gate != nullptr ? static_cast<const S*>(a.gate) + t * a.gate_ld : nullptr;
  for (int e = tid; e < a.nq * a.dv; e += kGenThreads) {
    float o = ol[e];
    if (gate != nullptr) o /= 1.f + expf(-to_f32<T>(gate[e]));
    out[e] = from_f32<T>(o);
  }
}

}  // namespace ma

namespace {

const float* head_vec(const c10::optional<at::Tensor>& t, int64_t n, const char* what) {
  if (!t.has_value() || !t->defined()) return nullptr;
  SXE_CHECK(t->scalar_type() == at::kFloat && t->is_contiguous() && t->numel() == n && t->is_cuda(), "mix_attention: ",
            what, " fp32 with ", n, " elements");
  return t->data_ptr<float>();
}

}  // namespace

// q [T, nq, Dk], kc / vc [blocks, nkv, bs, Dk / Dv] -> out [T, nq * dv]; see the top of the file.
// max_q_len bounds every q_len; force_generic picks the any-size kernel (fp32 always uses it).
at::Tensor mix_attention(const at::Tensor& q, const at::Tensor& kc, const at::Tensor& vc, const at::Tensor& block_table,
                         const at::Tensor& q_start, const at::Tensor& q_len, const at::Tensor& kv_len,
                         int64_t max_q_len, int64_t max_kv_len, int64_t dk, int64_t dv, double scale, int64_t window,
                         int64_t keep_first, const c10::optional<at::Tensor>& r1, const c10::optional<at::Tensor>& r2,
                         const c10::optional<at::Tensor>& sink, const c10::optional<at::Tensor>& talk,
                         const c10::optional<at::Tensor>& gate, bool force_generic) {
  SXE_CHECK_CUDA(q);
  SXE_CHECK(q.dim() == 3 && q.is_contiguous(), "mix_attention: q [T, nq, Dk] contiguous");
  const int64_t T = q.size(0), nq = q.size(1), nkv = kc.size(1), S = block_table.size(0);
  for (auto* c : {&kc, &vc})
    SXE_CHECK(c->dim() == 4 && c->size(1) == nkv && c->stride(3) == 1 && c->stride(2) == c->size(3) &&
                  c->stride(1) == c->size(2) * c->size(3) && c->scalar_type() == q.scalar_type() && c->is_cuda(),
              "mix_attention: caches [blocks, nkv, bs, D]");
  SXE_CHECK(kc.size(0) == vc.size(0) && kc.size(2) == vc.size(2) && kc.size(3) == q.size(2) && kc.size(3) >= dk &&
                vc.size(3) >= dv && nkv > 0 && nq % nkv == 0,
            "mix_attention: head layout");
  SXE_CHECK(block_table.scalar_type() == at::kInt && block_table.is_contiguous() && block_table.dim() == 2 &&
                block_table.is_cuda() && block_table.size(1) * kc.size(2) >= max_kv_len,
            "mix_attention: block_table int32 [S, max_blocks] covering max_kv_len");
  for (auto* t : {&q_start, &q_len, &kv_len})
    SXE_CHECK(t->scalar_type() == at::kInt && t->is_contiguous() && t->numel() == S && t->is_cuda(),
              "mix_attention: q_start/q_len/kv_len int32 [S]");
  auto out = at::empty({T, nq * dv}, q.options());
  if (T == 0 || S == 0 || max_q_len == 0) return out;
  ma::Args a{};
  a.q = q.data_ptr();
  a.kc = kc.data_ptr();
  a.vc = vc.data_ptr();
  a.k_block = kc.stride(0);
  a.v_block = vc.stride(0);
  a.block_table = block_table.data_ptr<int>();
  a.max_blocks = block_table.size(1);
  a.q_start = q_start.data_ptr<int>();
  a.q_len = q_len.data_ptr<int>();
  a.kv_len = kv_len.data_ptr<int>();
  a.S = S;
  a.T = T;
  a.nq = nq;
  a.nkv = nkv;
  a.dk = dk;
  a.dv = dv;
  a.Dk = kc.size(3);
  a.Dv = vc.size(3);
  a.bs = kc.size(2);
  a.scale = (float)scale;
  a.window = (int)std::max<int64_t>(0, window);
  a.keep_first = (int)std::max<int64_t>(0, keep_first);
  a.r1 = head_vec(r1, nq, "r1");
  a.r2 = head_vec(r2, nq, "r2");
  SXE_CHECK((a.r1 == nullptr) == (a.r2 == nullptr), "mix_attention: r1 and r2 together");
  a.sink = head_vec(sink, nq, "sink");
  a.talk = head_vec(talk, nq * nq, "talk");
  if (gate.has_value() && gate->defined()) {
    SXE_CHECK(gate->dim() == 2 && gate->stride(1) == 1 && gate->size(0) == T && gate->size(1) == nq * dv &&
                  gate->scalar_type() == q.scalar_type() && gate->is_cuda(),
              "mix_attention: gate [T, nq * dv] like q");
    a.gate = gate->data_ptr();
    a.gate_ld = gate->stride(0);
  }
  a.out = out.data_ptr();
  c10::DeviceGuard g(q.device());
  const size_t lds = sizeof(float) * (nq * (dk + dv) + 2 * nq * ma::kGenKeys + 2 * nq);
  SXE_CHECK(lds <= 160 * 1024, "mix_attention: heads x sizes exceed the LDS of one compute unit");
  SXE_DISPATCH_DT(dtype_of(q), D, {
    static bool attr = false;
    if (!attr) {
      SXE_HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&ma::mix_attn_generic_kernel<D>),
                                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
      attr = true;
    }
    hipLaunchKernelGGL(ma::mix_attn_generic_kernel<D>, dim3(S * max_q_len), dim3(ma::kGenThreads), lds, cur_stream(), a,
                       (int)max_q_len);
  });
  SXE_LAUNCH_CHECK();
  return out;
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("mix_attention(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor q_start, Tensor q_len, Tensor kv_len, "
        "int max_q_len, int max_kv_len, int dk, int dv, float scale, int window, int keep_first, Tensor? r1, Tensor? r2, "
        "Tensor? sink, Tensor? talk, Tensor? gate, bool force_generic=False) -> Tensor");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) { m.impl("mix_attention", &sxe::mix_attention); }
