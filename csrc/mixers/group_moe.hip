// Feed-forward pieces without a gate product, and group-limited routing.
//
//   route_group_topk  scores s = softmax(z) over all E experts; choice = s + correction; the experts form
//                     `groups` equal runs of neighbours, a group counts as its largest choice and only the
//                     best `keep` groups' experts stand for choice; the `top` largest choices (ties: the
//                     lower index) with the weights s, not renormalised
//   activate          out = f(x) or f(x) * table[ids[row]][off + column], f one of
//                       gelu_tanh   0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))
//                       relu2       max(z, 0)^2
//                       xielu       p z^2 + z / 2 for z > 0, q (exp(z) - 1 - z) + z / 2 otherwise
//                     x a tensor of the activation type or the fp32 split-K slabs of a decode GEMM
#include "mix_common.h"

using namespace pkm;

namespace {

__device__ __forceinline__ void wave_arg_max(float& best, int& bi, int none) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(best, o, 64);
    const int oi = __shfl_xor(bi, o, 64);
    if (oi < none && (bi >= none || ov > best || (ov == best && oi < bi))) {
      best = ov;
      bi = oi;
    }
  }
}

// the largest of v[0 .. n) not yet taken (taken entries are -infinity), one wave; every lane gets its index
__device__ __forceinline__ int pick(const float* v, int n, int lane) {
  float best = -INFINITY;
  int bi = n;
  for (int e = lane; e < n; e += 64) {
    const float x = v[e];
    if (x > best) {
      best = x;
      bi = e;
    }
  }
  wave_arg_max(best, bi, n);
  return bi;
}

__global__ void __launch_bounds__(64)
route_group_topk_kernel(int* __restrict__ ids, float* __restrict__ wts, const float* __restrict__ logits, int64_t ld_logits,
                        const float* __restrict__ correction, int E, int top, int groups, int keep) {
  extern __shared__ float sm[];
  float* s = sm;            // [E] scores
  float* choice = s + E;    // [E]
  float* gmax = choice + E;  // [groups]
  float* gsel = gmax + groups;  // [groups] 1: chosen
  const int t = blockIdx.x, lane = threadIdx.x;
  float m = -INFINITY;
  for (int e = lane; e < E; e += 64) {
    const float z = logits[t * ld_logits + e];
    s[e] = z;
    m = fmaxf(m, z);
  }
  m = pk::wave_max(m);
  float sum = 0.f;
  for (int e = lane; e < E; e += 64) {
    const float p = expf(s[e] - m);
    s[e] = p;
    sum += p;
  }
  sum = pk::wave_sum(sum);
  for (int e = lane; e < E; e += 64) {
    const float p = s[e] / sum;
    s[e] = p;
    choice[e] = correction ? p + correction[e] : p;
  }
  __syncthreads();
  if (groups > 1) {
    const int n = E / groups;
    for (int g = lane; g < groups; g += 64) {
      float b = -INFINITY;
      for (int j = 0; j < n; ++j) b = fmaxf(b, choice[g * n + j]);
      gmax[g] = b;
      gsel[g] = 0.f;
    }
    __syncthreads();
    for (int k = 0; k < keep; ++k) {
      const int g = pick(gmax, groups, lane);
      __syncthreads();
      if (lane == 0 && g < groups) {
        gmax[g] = -INFINITY;
        gsel[g] = 1.f;
      }
      __syncthreads();
    }
    for (int e = lane; e < E; e += 64)
      if (gsel[e / n] == 0.f) choice[e] = -INFINITY;
    __syncthreads();
  }
  for (int k = 0; k < top; ++k) {
    int e = pick(choice, E, lane);
    __syncthreads();
    if (lane == 0) {
      const bool ok = e < E;  // always, unless a score is not a number
      ids[t * top + k] = ok ? e : 0;
      wts[t * top + k] = ok ? s[e] : 0.f;
      if (ok) choice[e] = -INFINITY;
    }
    __syncthreads();
  }
}

constexpr int kGelu = 0, kRelu2 = 1, kXielu = 2;

struct ActArgs {
  const void* x;
  int nslab;  // 0: x is of the activation type
  int64_t slab_stride;
  void* out;
  int64_t n;  // elements
  int N;      // columns
  int kind;
  float p, q;
  const void* table;
  const int* ids;
  int vocab, row_width, off;
};

__device__ __forceinline__ float act_of(float z, int kind, float p, float q) {
  if (kind == kRelu2) {
    const float r = fmaxf(z, 0.f);
    return r * r;
  }
  if (kind == kXielu) return (z > 0.f ? p * z * z : q * (expm1f(z) - z)) + 0.5f * z;
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <typename T, int VEC>
__global__ void __launch_bounds__(256) activate_kernel(ActArgs a) {
  const int64_t i0 = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * VEC;
  if (i0 >= a.n) return;
  float v[VEC];
  if (a.nslab == 0) {
    if (VEC == 8 && sizeof(T) == 2) {
      const pk::u32x4 w = *reinterpret_cast<const pk::u32x4*>(static_cast<const T*>(a.x) + i0);
#pragma unroll
      for (int j = 0; j < VEC / 2; ++j) {
        v[2 * j] = __uint_as_float(w[j] << 16);
        v[2 * j + 1] = __uint_as_float(w[j] & 0xffff0000u);
      }
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = ld<T>(static_cast<const T*>(a.x) + i0 + j);
    }
  } else {
    const float* ws = static_cast<const float*>(a.x) + i0;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = ws[j];
    for (int s = 1; s < a.nslab; ++s)
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += ws[s * a.slab_stride + j];
  }
  const T* tb = nullptr;
  if (a.table) {
    const int64_t row = i0 / a.N;
    int id = a.ids[row];
    id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
    tb = static_cast<const T*>(a.table) + static_cast<int64_t>(id) * a.row_width + a.off + (i0 - row * a.N);
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) {
    v[j] = act_of(v[j], a.kind, a.p, a.q);
    if (tb) v[j] *= ld<T>(tb + j);
  }
  T* out = static_cast<T*>(a.out) + i0;
  if (VEC == 8 && sizeof(T) == 2) {
    pk::u32x4 w;
#pragma unroll
    for (int j = 0; j < VEC / 2; ++j) w[j] = pk::pack2(v[2 * j], v[2 * j + 1]);
    *reinterpret_cast<pk::u32x4*>(out) = w;
  } else {
#pragma unroll
    for (int j = 0; j < VEC; ++j) st<T>(out + j, v[j]);
  }
}

}  // namespace

// logits [T, >= E] fp32 rows ld_logits apart, correction [E] fp32 or null
PK_EXPORT int pkm_route_group_topk(void* ids, void* wts, const void* logits, long long ld_logits, const void* correction,
                                   int T, int E, int top, int groups, int keep, hipStream_t stream) {
  if (T <= 0) return 0;
  if (E < 1 || E > 4096 || groups < 1 || E % groups || keep < 1 || keep > groups || top < 1 || top > keep * (E / groups) ||
      ld_logits < E)
    return -1;
  route_group_topk_kernel<<<T, 64, (2 * E + 2 * groups) * sizeof(float), stream>>>(
      static_cast<int*>(ids), static_cast<float*>(wts), static_cast<const float*>(logits), ld_logits,
      static_cast<const float*>(correction), E, top, groups, keep);
  return PK_CHECK_LAUNCH();
}

// out [rows, N] (dt) = f(x), optionally times table[ids[row], off + column] (table [vocab, row_width] of dt).  x: the
// same shape and type (nslab 0; out may be x), or nslab fp32 slabs [nslab, rows, N]
PK_EXPORT int pkm_activate(void* out, const void* x, int nslab, long long rows, int N, int kind, float p, float q,
                           const void* table, const void* ids, int vocab, int row_width, int off, int dt,
                           hipStream_t stream) {
  if (rows <= 0) return 0;
  if (N < 1 || nslab < 0 || kind < kGelu || kind > kXielu || (table && (!ids || vocab < 1 || off < 0 || off + N > row_width)))
    return -1;
  const int64_t n = rows * N;
  ActArgs a{x, nslab, n, out, n, N, kind, p, q, table, static_cast<const int*>(ids), vocab, row_width, off};
  if (N % 8 == 0) {
    PKM_DISPATCH(dt, E, activate_kernel<E, 8><<<static_cast<unsigned>((n / 8 + 255) / 256), 256, 0, stream>>>(a));
  } else {
    PKM_DISPATCH(dt, E, activate_kernel<E, 1><<<static_cast<unsigned>((n + 255) / 256), 256, 0, stream>>>(a));
  }
  return PK_CHECK_LAUNCH();
}
