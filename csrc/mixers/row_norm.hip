// RMS norms over a whole row or over equal parts of it, with what stands next to them.
//
//   row_norm_cache     q | k projection rows plus a bias.  The value cache takes the biased key row as it
//                      is; then all query (key) heads together are set to unit RMS times a weight, the
//                      first 2 * pairs coordinates of every head turn by the token's position, q goes to
//                      [T, QH, D] and k to the key cache [blocks, KH, block_size, D].
//   gated_group_norm   u = y silu(z); each of `parts` equal parts of the row over its own root mean
//                      square, times a weight
//
// Sums and norms are fp32 for both element types, in a fixed order, so a token's result does not depend on
// the rest of the batch.
#include "mix_common.h"

using namespace pkm;

namespace {

constexpr int kThreads = 256;

__device__ __forceinline__ void load8(const float* p, float* f) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w, f[4] = b.x, f[5] = b.y, f[6] = b.z, f[7] = b.w;
}
__device__ __forceinline__ void load8(const bf16_t* p, float* f) { pk::unpack8(*reinterpret_cast<const pk::u32x4*>(p), f); }
__device__ __forceinline__ void store8(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = float4{f[0], f[1], f[2], f[3]};
  *reinterpret_cast<float4*>(p + 4) = float4{f[4], f[5], f[6], f[7]};
}
__device__ __forceinline__ void store8(bf16_t* p, const float* f) { *reinterpret_cast<pk::u32x4*>(p) = pk::pack8(f); }

struct RowArgs {
  void* q_out;
  const void* proj;
  int64_t stride;
  const float* bias;
  const float* w[2];  // q, k norm weights
  float eps;
  const int* positions;
  const int* slot_mapping;
  const float* table;
  int pairs, table_rows, halves;
  void* k_cache;
  void* v_cache;
  int QH, KH, D, bs;
};

// blockIdx.y: 0 the query row, 1 the key row; the biased row waits in LDS for its norm and its partners.
// VEC: D, the row stride and the base addresses allow 8 elements per access.
template <typename T, bool VEC>
__global__ void __launch_bounds__(kThreads) row_norm_cache_kernel(RowArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [heads * D]
  __shared__ float red[16];
  constexpr int N = VEC ? 8 : 1;
  const int64_t t = blockIdx.x;
  const bool key = blockIdx.y == 1;
  const int slot = a.slot_mapping[t], D = a.D;
  if (key && slot < 0) return;
  const int n = (key ? a.KH : a.QH) * D, c0 = key ? a.QH * D : 0;
  const T* src = static_cast<const T*>(a.proj) + t * a.stride + c0;
  const float* bias = a.bias + c0;
  const float* w = a.w[key];
  // element (head h, coordinate d) of the token: q row or cache page
  const int64_t base = key ? (static_cast<int64_t>(slot / a.bs) * a.KH * a.bs + slot % a.bs) * D : t * n;
  const int64_t head_stride = key ? static_cast<int64_t>(a.bs) * D : D;
  T* vdst = static_cast<T*>(a.v_cache);
  T* dst = static_cast<T*>(key ? a.k_cache : a.q_out);
  float ss = 0.f;
  for (int c = N * threadIdx.x; c < n; c += N * kThreads) {
    float f[N];
    if constexpr (VEC) {
      float b[8];
      load8(src + c, f);
      load8(bias + c, b);
#pragma unroll
      for (int e = 0; e < N; ++e) f[e] += b[e];
    } else {
      f[0] = ld<T>(src + c) + bias[c];
    }
#pragma unroll
    for (int e = 0; e < N; ++e) ss += f[e] * f[e];
    if (key) {
      const int h = c / D;
      T* v = vdst + base + h * head_stride + (c - h * D);
      if constexpr (VEC) {
        store8(v, f);
      } else {
        st<T>(v, f[0]);
      }
    }
    if constexpr (VEC) {
      store8(row + c, f);
    } else {
      row[c] = f[0];
    }
  }
  const float k = 1.f / sqrtf(pk::block_sum(ss, red) / static_cast<float>(n) + a.eps);  // (its barriers publish the row)
  int pos = a.positions[t];
  pos = pos < 0 ? 0 : min(pos, a.table_rows - 1);
  const float* cs = a.table ? a.table + static_cast<int64_t>(pos) * a.pairs * 2 : nullptr;
  const int turned = cs ? 2 * a.pairs : 0;
  for (int c = N * threadIdx.x; c < n; c += N * kThreads) {
    const int h = c / D, d0 = c - h * D;
    float f[N];
#pragma unroll
    for (int e = 0; e < N; ++e) {
      const int d = d0 + e;
      float x = row[c + e] * k * w[c + e];
      if (d < turned) {
        const bool first = a.halves ? d < a.pairs : (d & 1) == 0;
        const int i = a.halves ? (first ? d : d - a.pairs) : d >> 1;
        const int o = c + e + (a.halves ? (first ? a.pairs : -a.pairs) : (first ? 1 : -1));
        const float y = row[o] * k * w[o];
        x = first ? x * cs[2 * i] - y * cs[2 * i + 1] : x * cs[2 * i] + y * cs[2 * i + 1];
      }
      f[e] = x;
    }
    T* o = dst + base + h * head_stride + d0;
    if constexpr (VEC) {
      store8(o, f);
    } else {
      st<T>(o, f[0]);
    }
  }
}

// one workgroup per (token, part).  VEC: parts of a multiple of 8 elements at 16-byte addresses.
template <typename ZT, typename OT, bool VEC>
__global__ void __launch_bounds__(kThreads)
gated_group_norm_kernel(OT* __restrict__ out, const float* __restrict__ y, const ZT* __restrict__ z, int64_t z_stride,
                        const float* __restrict__ w, int N, int parts, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [N / parts]
  __shared__ float red[16];
  constexpr int E = VEC ? 8 : 1;
  const int64_t t = blockIdx.x;
  const int n = N / parts, c0 = blockIdx.y * n;
  y += t * N + c0;
  z += t * z_stride + c0;
  out += t * N + c0;
  w += c0;
  float ss = 0.f;
  for (int c = E * threadIdx.x; c < n; c += E * kThreads) {
    float f[E], g[E];
    if constexpr (VEC) {
      load8(y + c, f);
      load8(z + c, g);
    } else {
      f[0] = y[c];
      g[0] = ld<ZT>(z + c);
    }
#pragma unroll
    for (int e = 0; e < E; ++e) {
      f[e] *= g[e] * sigmoidf(g[e]);
      ss += f[e] * f[e];
      row[c + e] = f[e];  // read back by this thread only
    }
  }
  const float k = 1.f / sqrtf(pk::block_sum(ss, red) / static_cast<float>(n) + eps);
  for (int c = E * threadIdx.x; c < n; c += E * kThreads) {
    float f[E];
#pragma unroll
    for (int e = 0; e < E; ++e) f[e] = row[c + e] * k * w[c + e];
    if constexpr (VEC) {
      store8(out + c, f);
    } else {
      st<OT>(out + c, f[0]);
    }
  }
}

constexpr size_t kMaxLds = 144 * 1024;

template <typename K>
int allow_lds(K kern, size_t lds) {
  if (lds <= 60 * 1024) return 0;
  return static_cast<int>(hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize,
                                              static_cast<int>(lds)));
}

template <typename T, bool VEC>
int launch_row(const RowArgs& a, int tokens, size_t lds, hipStream_t stream) {
  const int rc = allow_lds(row_norm_cache_kernel<T, VEC>, lds);
  if (rc) return rc;
  row_norm_cache_kernel<T, VEC><<<dim3(tokens, 2), kThreads, lds, stream>>>(a);
  return PK_CHECK_LAUNCH();
}

template <typename ZT, typename OT, bool VEC>
int launch_group(void* out, const void* y, const void* z, int64_t zs, const void* w, int T, int N, int parts, float eps,
                 hipStream_t stream) {
  const size_t lds = static_cast<size_t>(N / parts) * sizeof(float);
  const int rc = allow_lds(gated_group_norm_kernel<ZT, OT, VEC>, lds);
  if (rc) return rc;
  gated_group_norm_kernel<ZT, OT, VEC><<<dim3(T, parts), kThreads, lds, stream>>>(
      static_cast<OT*>(out), static_cast<const float*>(y), static_cast<const ZT*>(z), zs, static_cast<const float*>(w), N, parts, eps);
  return PK_CHECK_LAUNCH();
}

bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

}  // namespace

// proj [T, QH*D | KH*D] rows `stride` elements apart; bias [(QH + KH) * D], q_w [QH * D], k_w [KH * D] fp32; table
// [table_rows, pairs, 2] fp32 or null; caches [blocks, KH, bs, D]; q_out [T, QH, D]
PK_EXPORT int pkm_row_norm_cache(void* q_out, const void* proj, long long stride, const void* bias, const void* q_w,
                                 const void* k_w, float eps, const void* positions, const void* slot_mapping, const void* table,
                                 int pairs, int table_rows, int halves, void* k_cache, void* v_cache, int T, int QH, int KH,
                                 int D, int bs, int dt, hipStream_t stream) {
  if (T <= 0) return 0;
  if (D < 1 || QH < 1 || KH < 1 || bs < 1 || 2 * pairs > D || (table && table_rows < 1)) return -1;
  if (!bias || !q_w || !k_w || stride < static_cast<long long>(QH + KH) * D) return -1;
  const size_t lds = static_cast<size_t>(QH > KH ? QH : KH) * D * sizeof(float);
  if (lds > kMaxLds) return -1;
  const RowArgs a{q_out, proj, stride, static_cast<const float*>(bias), {static_cast<const float*>(q_w), static_cast<const float*>(k_w)},
                  eps, static_cast<const int*>(positions), static_cast<const int*>(slot_mapping), static_cast<const float*>(table),
                  pairs, table_rows, halves, k_cache, v_cache, QH, KH, D, bs};
  const bool vec = D % 8 == 0 && stride % 8 == 0 && aligned16(proj) && aligned16(bias) && aligned16(q_out) && aligned16(k_cache) &&
                   aligned16(v_cache);
  if (vec) {
    PKM_DISPATCH(dt, E, return (launch_row<E, true>(a, T, lds, stream)));
  }
  PKM_DISPATCH(dt, E, return (launch_row<E, false>(a, T, lds, stream)));
  return 0;
}

// out [T, N] (out_dt); y [T, N] fp32; z [T, N] rows z_stride elements apart (z_dt); w [N] fp32
PK_EXPORT int pkm_gated_group_norm(void* out, const void* y, const void* z, long long z_stride, const void* w, int T, int N,
                                   int parts, float eps, int z_dt, int out_dt, hipStream_t stream) {
  if (T <= 0) return 0;
  if (N < 1 || parts < 1 || N % parts || z_stride < N || static_cast<size_t>(N / parts) * sizeof(float) > kMaxLds) return -1;
  const bool vec = (N / parts) % 8 == 0 && z_stride % 8 == 0 && aligned16(out) && aligned16(y) && aligned16(z);
#define PKM_GG(ZT)                                                                                                     \
  if (vec) {                                                                                                           \
    PKM_DISPATCH(out_dt, O, return (launch_group<ZT, O, true>(out, y, z, z_stride, w, T, N, parts, eps, stream)));     \
  }                                                                                                                    \
  PKM_DISPATCH(out_dt, O, return (launch_group<ZT, O, false>(out, y, z, z_stride, w, T, N, parts, eps, stream)))
  if (z_dt == kF32) {
    PKM_GG(float);
  } else if (z_dt == kBF16) {
    PKM_GG(bf16_t);
  } else {
    return -2;
  }
#undef PKM_GG
  return 0;
}
