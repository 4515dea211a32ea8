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

// One workgroup per token; the biased row waits in LDS for its two norms and the partners of turned pairs.
// VEC: D, the row stride and the addresses allow 8 elements per access.  ROT8: and a pair's halves lie whole
// groups of 8 apart (halves layout, pairs a multiple of 8) or nothing turns.
template <typename T, bool VEC, bool ROT8>
__global__ void __launch_bounds__(kThreads) row_norm_cache_kernel(RowArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [(QH + KH) * D]
  __shared__ float red[16];
  constexpr int N = VEC ? 8 : 1;
  const int64_t t = blockIdx.x;
  const int slot = a.slot_mapping[t], D = a.D, nq = a.QH * D, n = nq + a.KH * D;
  const T* src = static_cast<const T*>(a.proj) + t * a.stride;
  T* q = static_cast<T*>(a.q_out) + t * nq;
  // head g, coordinate d of the token in a cache: page + g * bs * D + d
  const int64_t page = slot < 0 ? 0 : (static_cast<int64_t>(slot / a.bs) * a.KH * a.bs + slot % a.bs) * D;
  T* kc = static_cast<T*>(a.k_cache) + page;
  T* vc = static_cast<T*>(a.v_cache) + page;
  const int64_t hs = static_cast<int64_t>(a.bs) * D;
  float sq = 0.f, sk = 0.f;
  for (int c = N * threadIdx.x; c < n; c += N * kThreads) {
    float f[N], ss = 0.f;
    if constexpr (VEC) {
      float b[8];
      load8(src + c, f);
      load8(a.bias + c, b);
#pragma unroll
      for (int e = 0; e < N; ++e) f[e] += b[e];
      store8(row + c, f);
    } else {
      f[0] = ld<T>(src + c) + a.bias[c];
      row[c] = f[0];
    }
#pragma unroll
    for (int e = 0; e < N; ++e) ss += f[e] * f[e];
    if (c < nq) {
      sq += ss;
    } else {
      sk += ss;
      if (slot >= 0) {
        const int h = (c - nq) / D;
        T* v = vc + h * hs + (c - nq - h * D);
        if constexpr (VEC) {
          store8(v, f);
        } else {
          st<T>(v, f[0]);
        }
      }
    }
  }
  const float kq = 1.f / sqrtf(pk::block_sum(sq, red) / static_cast<float>(nq) + a.eps);  // (the barriers publish the row)
  const float kk = 1.f / sqrtf(pk::block_sum(sk, red) / static_cast<float>(n - nq) + a.eps);
  int pos = a.positions[t];
  pos = pos < 0 ? 0 : min(pos, a.table_rows - 1);
  const float* cs = a.table ? a.table + static_cast<int64_t>(pos) * a.pairs * 2 : nullptr;
  const int turned = cs ? 2 * a.pairs : 0;
  for (int c = N * threadIdx.x; c < n; c += N * kThreads) {
    const bool query = c < nq;
    if (!query && slot < 0) break;
    const int ck = query ? c : c - nq, h = ck / D, d0 = ck - h * D;
    const float k = query ? kq : kk;
    const float* w = query ? a.w[0] : a.w[1] - nq;  // indexed by the row's column
    float f[N];
    if constexpr (ROT8) {
      float m[8];
      load8(row + c, f);
      load8(w + c, m);
#pragma unroll
      for (int e = 0; e < N; ++e) f[e] *= k * m[e];
      if (d0 < turned) {
        const bool first = d0 < a.pairs;
        const int i = first ? d0 : d0 - a.pairs, o = first ? c + a.pairs : c - a.pairs;
        float y[8], t0[8], t1[8];
        load8(row + o, y);
        load8(w + o, m);
        load8(cs + 2 * i, t0);
        load8(cs + 2 * i + 8, t1);
#pragma unroll
        for (int e = 0; e < N; ++e) {
          const float co = e < 4 ? t0[2 * (e & 3)] : t1[2 * (e & 3)], si = e < 4 ? t0[2 * (e & 3) + 1] : t1[2 * (e & 3) + 1];
          const float p = y[e] * k * m[e];
          f[e] = first ? f[e] * co - p * si : f[e] * co + p * si;
        }
      }
    } else {
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
    }
    T* dst = query ? q + c : kc + h * hs + d0;
    if constexpr (VEC) {
      store8(dst, f);
    } else {
      st<T>(dst, f[0]);
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

template <typename T, bool VEC, bool ROT8>
int launch_row(const RowArgs& a, int tokens, size_t lds, hipStream_t stream) {
  const int rc = allow_lds(row_norm_cache_kernel<T, VEC, ROT8>, lds);
  if (rc) return rc;
  row_norm_cache_kernel<T, VEC, ROT8><<<tokens, kThreads, lds, stream>>>(a);
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
  const size_t lds = static_cast<size_t>(QH + KH) * D * sizeof(float);
  if (lds > kMaxLds) return -1;
  const RowArgs a{q_out, proj, stride, static_cast<const float*>(bias), {static_cast<const float*>(q_w), static_cast<const float*>(k_w)},
                  eps, static_cast<const int*>(positions), static_cast<const int*>(slot_mapping), static_cast<const float*>(table),
                  pairs, table_rows, halves, k_cache, v_cache, QH, KH, D, bs};
  const bool vec = D % 8 == 0 && stride % 8 == 0 && aligned16(proj) && aligned16(bias) && aligned16(q_out) && aligned16(k_cache) &&
                   aligned16(v_cache) && aligned16(q_w) && aligned16(k_w);
  if (vec && (!table || (halves && pairs % 8 == 0 && aligned16(table)))) {
    PKM_DISPATCH(dt, E, return (launch_row<E, true, true>(a, T, lds, stream)));
  }
  if (vec) {
    PKM_DISPATCH(dt, E, return (launch_row<E, true, false>(a, T, lds, stream)));
  }
  PKM_DISPATCH(dt, E, return (launch_row<E, false, false>(a, T, lds, stream)));
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
