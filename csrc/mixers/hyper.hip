// Residual streams of pre-norm layers, kept in fp32, one or several per token (hyper-connections).
//
//   spread_rows   xs[t, s] = table[ids[t]] * scale for every stream s
//   hyper_step    closes one sublayer and opens the next, per token, in one pass:
//                   y      = the sublayer's output row: a plain row, the sum of split-K slabs, or a
//                            mixture's  sum_j wts[t, j] * rows[inv[t, j]]  (+ [sigmoid(gate[t]) *] shared[t])
//                   xs'[t] = sum_s mix[s, t] xs[s] + a_out[t] y          (all streams from the old ones)
//                   u      = sum_t a_in[t] xs'[t];  z = u / sqrt(mean(u^2) + eps) * w
//                 y may first be set to unit RMS times a weight (post_w) or be scaled coordinate by
//                 coordinate (y_scale); without a norm weight the opened sum u itself is z.
//                 Either half may be absent; with `rows` only those tokens are opened (the rows whose
//                 logits are wanted).  S = 1 with unit coefficients is the plain residual.
//   pair_step     closes a sublayer of two branches on one stream: y = ca U(ya) wa + cb U(yb) wb,
//                 x <- x + U(y) post_w, act = x, U(u) = u / sqrt(mean(u^2) + eps); slabs summed on the way
//   embed_norm    x[t] = table[ids[t]] set to unit RMS times a weight, as fp32
//   tanh_cap      x <- cap * tanh(x / cap)
//
// One workgroup per token; every sum runs in a fixed order, so a token's result does not depend
// on the rest of the batch.
#include "mix_common.h"

using namespace pkm;

namespace {

constexpr int kMaxStreams = 8;

template <typename T>
__global__ void __launch_bounds__(256) spread_rows_kernel(float* __restrict__ xs, const T* __restrict__ table,
                                                          const int* __restrict__ ids, int S, int W, int vocab,
                                                          float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* src = table + static_cast<int64_t>(id) * W;
  float* dst = xs + static_cast<int64_t>(t) * S * W;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float v = ld<T>(src + i) * scale;
    for (int s = 0; s < S; ++s) dst[s * W + i] = v;
  }
}

struct HyperArgs {
  float* xs;
  int S, W;
  const void* y;
  int nslab;
  int64_t slab_stride;
  const int* inv;
  int top;
  const float* wts;
  const void* y2;
  const float* g2;
  int64_t g2_stride;
  const float* mix;
  const float* a_out;
  const float* a_in;
  const float* norm_w;
  float eps;
  void* act;
  float* z32;
  const int* rows;
  const float* y_scale;  // [W] or null
  const float* post_w;   // [W] or null: y <- y / sqrt(mean(y^2) + eps) * post_w
};

// four consecutive coordinates per thread (W % 4 == 0): 16-byte loads of the fp32 streams
template <typename E>
__device__ __forceinline__ float4 ld4(const E* p);
template <>
__device__ __forceinline__ float4 ld4<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <>
__device__ __forceinline__ float4 ld4<bf16_t>(const bf16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  return float4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                __uint_as_float(v.y & 0xffff0000u)};
}
template <typename E>
__device__ __forceinline__ void st4(E* p, float4 v);
template <>
__device__ __forceinline__ void st4<float>(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
template <>
__device__ __forceinline__ void st4<bf16_t>(bf16_t* p, float4 v) {
  uint2 w;
  w.x = pk::pack2(v.x, v.y);
  w.y = pk::pack2(v.z, v.w);
  *reinterpret_cast<uint2*>(p) = w;
}
__device__ __forceinline__ float4 mul4(float4 a, float4 b) { return float4{a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w}; }
__device__ __forceinline__ float4 fma4(float c, float4 a, float4 b) {
  return float4{c * a.x + b.x, c * a.y + b.y, c * a.z + b.z, c * a.w + b.w};
}

// the sublayer output at coordinates i .. i + 3 / at coordinate i of token src
template <typename T, typename Y>
__device__ __forceinline__ float4 sublayer_out4(const HyperArgs& a, int64_t src, int i, float gate) {
  const Y* y = static_cast<const Y*>(a.y);
  const T* y2 = static_cast<const T*>(a.y2);
  float4 yv = float4{0.f, 0.f, 0.f, 0.f};
  if (a.inv) {
    for (int j = 0; j < a.top; ++j) {
      const int row = a.inv[src * a.top + j];
      if (row >= 0) yv = fma4(a.wts[src * a.top + j], ld4<Y>(y + static_cast<int64_t>(row) * a.W + i), yv);
    }
  } else if (y) {
    yv = ld4<Y>(y + src * a.W + i);
    for (int sl = 1; sl < a.nslab; ++sl) yv = fma4(1.f, ld4<Y>(y + sl * a.slab_stride + src * a.W + i), yv);
  }
  if (y2) yv = fma4(gate, ld4<T>(y2 + src * a.W + i), yv);
  return yv;
}
template <typename T, typename Y>
__device__ __forceinline__ float sublayer_out(const HyperArgs& a, int64_t src, int i, float gate) {
  const Y* y = static_cast<const Y*>(a.y);
  const T* y2 = static_cast<const T*>(a.y2);
  float yv = 0.f;
  if (a.inv) {
    for (int j = 0; j < a.top; ++j) {
      const int row = a.inv[src * a.top + j];
      if (row >= 0) yv += a.wts[src * a.top + j] * ld<Y>(y + static_cast<int64_t>(row) * a.W + i);
    }
  } else if (y) {
    yv = ld<Y>(y + src * a.W + i);
    for (int sl = 1; sl < a.nslab; ++sl) yv += ld<Y>(y + sl * a.slab_stride + src * a.W + i);
  }
  if (y2) yv += gate * ld<T>(y2 + src * a.W + i);
  return yv;
}

// VEC >= 4 (= 4 * groups per thread): W % 4 == 0, every thread owns up to VEC / 4 groups of four
// consecutive coordinates and keeps the opened sum in registers between the two passes; VEC = 1: any
// W, one coordinate at a time, the opened sum in LDS.  POST: the sublayer output is normed first.
// NS: the most streams this form handles (1 or kMaxStreams).
template <typename T, typename Y, int VEC, bool POST, int NS>
__global__ void __launch_bounds__(1024) hyper_step_kernel(HyperArgs a) {
  constexpr int NG = VEC >= 4 ? VEC / 4 : 1;
  __shared__ float red[16];
  __shared__ float cf[kMaxStreams * kMaxStreams + 2 * kMaxStreams];
  extern __shared__ __attribute__((aligned(16))) float vbuf[];  // [W] the opened sum u, kept between the two passes
  const int r = blockIdx.x;
  const int S = NS == 1 ? 1 : a.S, W = a.W;
  const int64_t src = a.rows ? a.rows[r] : r;
  float* x = a.xs + src * S * W;
  const bool close = a.mix != nullptr, open = a.a_in != nullptr;
  float* c_mix = cf;
  float* c_out = cf + kMaxStreams * kMaxStreams;
  float* c_in = c_out + kMaxStreams;
  if (threadIdx.x < S * S && close) c_mix[threadIdx.x] = a.mix[threadIdx.x];
  if (threadIdx.x < S) {
    if (close) c_out[threadIdx.x] = a.a_out[threadIdx.x];
    if (open) c_in[threadIdx.x] = a.a_in[threadIdx.x];
  }
  __syncthreads();
  const float gate = a.y2 ? (a.g2 ? sigmoidf(a.g2[src * a.g2_stride]) : 1.f) : 0.f;
  float ss = 0.f;
  float4 ur[NG];
  float ky = 1.f;
  if (POST) {
    float sy = 0.f;
    if (VEC >= 4) {
#pragma unroll
      for (int it = 0; it < NG; ++it) {
        const int i = 4 * (threadIdx.x + it * blockDim.x);
        if (i >= W) break;
        const float4 v = sublayer_out4<T, Y>(a, src, i, gate);
        ur[it] = v;
        sy += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
      }
    } else {
      for (int i = threadIdx.x; i < W; i += blockDim.x) {
        const float v = sublayer_out<T, Y>(a, src, i, gate);
        vbuf[i] = v;
        sy += v * v;
      }
    }
    ky = 1.f / sqrtf(pk::block_sum(sy, red) / static_cast<float>(W) + a.eps);
    __syncthreads();
  }
  if (VEC >= 4) {
#pragma unroll
    for (int it = 0; it < NG; ++it) {
      const int i = 4 * (threadIdx.x + it * blockDim.x);
      if (i >= W) break;
      float4 xv[NS];
#pragma unroll
      for (int s = 0; s < NS; ++s)
        if (s < S) xv[s] = ld4<float>(x + s * W + i);
      if (close) {
        float4 yv;
        if (POST) {
          const float4 v = ur[it];
          yv = mul4(float4{v.x * ky, v.y * ky, v.z * ky, v.w * ky}, ld4<float>(a.post_w + i));
        } else {
          yv = sublayer_out4<T, Y>(a, src, i, gate);
        }
        if (a.y_scale) yv = mul4(yv, ld4<float>(a.y_scale + i));
        float4 nv[NS];
#pragma unroll
        for (int t = 0; t < NS; ++t) {
          if (t < S) {
            float4 acc = float4{0.f, 0.f, 0.f, 0.f};
            for (int s = 0; s < S; ++s) acc = fma4(c_mix[s * S + t], xv[s], acc);
            nv[t] = fma4(c_out[t], yv, acc);
            st4<float>(x + t * W + i, nv[t]);
          }
        }
#pragma unroll
        for (int t = 0; t < NS; ++t)
          if (t < S) xv[t] = nv[t];
      }
      if (open) {
        float4 u = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < NS; ++t)
          if (t < S) u = fma4(c_in[t], xv[t], u);
        ur[it] = u;
        ss += (u.x * u.x + u.y * u.y) + (u.z * u.z + u.w * u.w);
      }
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float xv[NS];
#pragma unroll
      for (int s = 0; s < NS; ++s) xv[s] = s < S ? x[s * W + i] : 0.f;
      if (close) {
        float yv = POST ? vbuf[i] * ky * a.post_w[i] : sublayer_out<T, Y>(a, src, i, gate);
        if (a.y_scale) yv *= a.y_scale[i];
        float nv[NS];
#pragma unroll
        for (int t = 0; t < NS; ++t) {
          if (t < S) {
            float acc = 0.f;
            for (int s = 0; s < S; ++s) acc += c_mix[s * S + t] * xv[s];
            nv[t] = acc + c_out[t] * yv;
            x[t * W + i] = nv[t];
          }
        }
#pragma unroll
        for (int t = 0; t < NS; ++t) xv[t] = t < S ? nv[t] : 0.f;
      }
      if (open) {
        float u = 0.f;
#pragma unroll
        for (int t = 0; t < NS; ++t)
          if (t < S) u += c_in[t] * xv[t];
        vbuf[i] = u;
        ss += u * u;
      }
    }
  }
  if (!open) return;
  float k = 1.f;
  if (a.norm_w) {
    ss = pk::block_sum(ss, red);
    k = 1.f / sqrtf(ss / static_cast<float>(W) + a.eps);
  }
  T* act = static_cast<T*>(a.act);
  if (VEC >= 4) {
#pragma unroll
    for (int it = 0; it < NG; ++it) {
      const int i = 4 * (threadIdx.x + it * blockDim.x);
      if (i >= W) break;
      const float4 u = ur[it], g = a.norm_w ? ld4<float>(a.norm_w + i) : float4{1.f, 1.f, 1.f, 1.f};
      const float4 z = float4{u.x * k * g.x, u.y * k * g.y, u.z * k * g.z, u.w * k * g.w};
      if (act) st4<T>(act + static_cast<int64_t>(r) * W + i, z);
      if (a.z32) st4<float>(a.z32 + static_cast<int64_t>(r) * W + i, z);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      const float z = a.norm_w ? vbuf[i] * k * a.norm_w[i] : vbuf[i];
      if (act) st<T>(act + static_cast<int64_t>(r) * W + i, z);
      if (a.z32) a.z32[static_cast<int64_t>(r) * W + i] = z;
    }
  }
}

struct PairArgs {
  float* x;
  int W;
  const void* y[2];
  int f32[2];    // element type of a branch: fp32 (slabs are) or bf16
  int nslab[2];
  int64_t slab_stride;
  const float* w[2];
  float c[2];
  const float* post_w;
  float eps;
  void* act;
};

// NG >= 1: W % 4 == 0, a thread owns up to NG groups of four coordinates of both branches in registers;
// NG = 0: any W, one coordinate at a time through LDS.
template <typename T, int NG>
__global__ void __launch_bounds__(1024) pair_step_kernel(PairArgs a) {
  __shared__ float red[16];
  extern __shared__ __attribute__((aligned(16))) float vbuf[];  // [2][W] (NG = 0)
  const int64_t r = blockIdx.x;
  const int W = a.W;
  float* x = a.x + r * W;
  T* act = static_cast<T*>(a.act) + r * W;
  const float inv_w = 1.f / static_cast<float>(W);
  if (NG > 0) {
    constexpr int N = NG > 0 ? NG : 1;
    float4 v[2][N];
    float ss[2] = {0.f, 0.f};
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const float* yf = static_cast<const float*>(a.y[b]) + r * W;
      const bf16_t* yh = static_cast<const bf16_t*>(a.y[b]) + r * W;
#pragma unroll
      for (int it = 0; it < N; ++it) {
        const int i = 4 * (threadIdx.x + it * blockDim.x);
        if (i >= W) break;
        float4 u = a.f32[b] ? ld4<float>(yf + i) : ld4<bf16_t>(yh + i);
        for (int sl = 1; sl < a.nslab[b]; ++sl) u = fma4(1.f, ld4<float>(yf + sl * a.slab_stride + i), u);
        v[b][it] = u;
        ss[b] += (u.x * u.x + u.y * u.y) + (u.z * u.z + u.w * u.w);
      }
    }
    const float k0 = a.c[0] / sqrtf(pk::block_sum(ss[0], red) * inv_w + a.eps);
    const float k1 = a.c[1] / sqrtf(pk::block_sum(ss[1], red) * inv_w + a.eps);
    float sy = 0.f;
#pragma unroll
    for (int it = 0; it < N; ++it) {
      const int i = 4 * (threadIdx.x + it * blockDim.x);
      if (i >= W) break;
      const float4 y0 = mul4(v[0][it], ld4<float>(a.w[0] + i)), y1 = mul4(v[1][it], ld4<float>(a.w[1] + i));
      const float4 u = fma4(k0, y0, float4{k1 * y1.x, k1 * y1.y, k1 * y1.z, k1 * y1.w});
      v[0][it] = u;
      sy += (u.x * u.x + u.y * u.y) + (u.z * u.z + u.w * u.w);
    }
    const float k = 1.f / sqrtf(pk::block_sum(sy, red) * inv_w + a.eps);
#pragma unroll
    for (int it = 0; it < N; ++it) {
      const int i = 4 * (threadIdx.x + it * blockDim.x);
      if (i >= W) break;
      const float4 z = fma4(k, mul4(v[0][it], ld4<float>(a.post_w + i)), ld4<float>(x + i));
      st4<float>(x + i, z);
      st4<T>(act + i, z);
    }
    return;
  }
  float ss[2] = {0.f, 0.f};
  for (int b = 0; b < 2; ++b) {
    const float* yf = static_cast<const float*>(a.y[b]) + r * W;
    const bf16_t* yh = static_cast<const bf16_t*>(a.y[b]) + r * W;
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float u = a.f32[b] ? yf[i] : ld<bf16_t>(yh + i);
      for (int sl = 1; sl < a.nslab[b]; ++sl) u += yf[sl * a.slab_stride + i];
      vbuf[b * W + i] = u;  // read back by this thread only
      ss[b] += u * u;
    }
  }
  const float k0 = a.c[0] / sqrtf(pk::block_sum(ss[0], red) * inv_w + a.eps);
  const float k1 = a.c[1] / sqrtf(pk::block_sum(ss[1], red) * inv_w + a.eps);
  float sy = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float u = k0 * vbuf[i] * a.w[0][i] + k1 * vbuf[W + i] * a.w[1][i];
    vbuf[i] = u;
    sy += u * u;
  }
  const float k = 1.f / sqrtf(pk::block_sum(sy, red) * inv_w + a.eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float z = x[i] + k * vbuf[i] * a.post_w[i];
    x[i] = z;
    st<T>(act + i, z);
  }
}

template <typename T>
__global__ void __launch_bounds__(256) embed_norm_kernel(float* __restrict__ x, const T* __restrict__ table,
                                                         const int* __restrict__ ids, const float* __restrict__ w, int W,
                                                         int vocab, float eps) {
  __shared__ float red[16];
  const int t = blockIdx.x;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* src = table + static_cast<int64_t>(id) * W;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float v = ld<T>(src + i);
    ss += v * v;
  }
  ss = pk::block_sum(ss, red);
  const float k = 1.f / sqrtf(ss / static_cast<float>(W) + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) x[static_cast<int64_t>(t) * W + i] = ld<T>(src + i) * k * w[i];
}

__global__ void __launch_bounds__(256) tanh_cap_kernel(float* __restrict__ x, int64_t n, float cap) {
  const int64_t i = static_cast<int64_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] / cap);
}

}  // namespace

PK_EXPORT int pkm_spread_rows(void* xs, const void* table, const void* ids, int T, int S, int W, int vocab, int dt,
                              float scale, hipStream_t stream) {
  if (T <= 0) return 0;
  if (S < 1 || S > kMaxStreams) return -1;
  PKM_DISPATCH(dt, E, spread_rows_kernel<E><<<T, 256, 0, stream>>>(static_cast<float*>(xs), static_cast<const E*>(table),
                                                                    static_cast<const int*>(ids), S, W, vocab, scale));
  return PK_CHECK_LAUNCH();
}

// x [T, W] fp32 <- unit-RMS rows of the table times w [W]
PK_EXPORT int pkm_embed_norm(void* x, const void* table, const void* ids, const void* w, int T, int W, int vocab, float eps,
                             int dt, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W < 1 || vocab < 1) return -1;
  PKM_DISPATCH(dt, E, embed_norm_kernel<E><<<T, 256, 0, stream>>>(static_cast<float*>(x), static_cast<const E*>(table),
                                                                   static_cast<const int*>(ids), static_cast<const float*>(w),
                                                                   W, vocab, eps));
  return PK_CHECK_LAUNCH();
}

// xs [tokens, S, W] fp32, updated in place when mix / a_out are given (then y, or inv / wts / y rows,
// is the sublayer output; y_dt its element type, -1: none).  y2 / g2: a second row per token in the
// activation type and its pre-sigmoid gate (fp32, element stride g2_stride; null: the row is added as it is).  a_in / norm_w: open.
// norm_w null with a_in: the opened sum as it is.  y_scale, post_w [W] fp32 or null: y scaled per coordinate /
// set to unit RMS times post_w (S = 1 only) before it is folded in.  rows: R token indices to open (no close).  act (element type act_dt) and z32 may each be null.
PK_EXPORT int pkm_hyper_step(void* xs, int R, int S, int W, const void* y, int y_dt, int nslab, const void* inv, int top,
                             const void* wts, const void* y2, int y2_dt, const void* g2, long long g2_stride,
                             const void* mix, const void* a_out, const void* a_in, const void* norm_w, float eps,
                             void* act, int act_dt, void* z32, const void* rows, const void* y_scale,
                             const void* post_w, hipStream_t stream) {
  if (R <= 0) return 0;
  if (S < 1 || S > kMaxStreams || W > 16384 || nslab < 1) return -1;
  if ((mix == nullptr) != (a_out == nullptr) || (norm_w != nullptr && a_in == nullptr)) return -1;
  if ((y_scale || post_w) && (!mix || !y)) return -1;
  if (post_w && S != 1) return -1;
  if (rows && mix) return -1;
  if (inv && (!y || !wts || top < 1 || nslab > 1)) return -1;
  if (y2 && y2_dt != act_dt) return -1;
  HyperArgs a{static_cast<float*>(xs), S, W, y, nslab, static_cast<int64_t>(R) * W, static_cast<const int*>(inv), top,
              static_cast<const float*>(wts), y2, static_cast<const float*>(g2), g2_stride,
              static_cast<const float*>(mix), static_cast<const float*>(a_out), static_cast<const float*>(a_in),
              static_cast<const float*>(norm_w), eps, act, static_cast<float*>(z32), static_cast<const int*>(rows),
              static_cast<const float*>(y_scale), static_cast<const float*>(post_w)};
  const size_t lds = (a_in || post_w) ? static_cast<size_t>(W) * sizeof(float) : 0;
  if (y_dt != kF32 && y_dt != kBF16 && y != nullptr) return -2;
  const bool y32 = y == nullptr || y_dt == kF32;
  if (W % 4 == 0) {  // up to 256 threads, each with 1, 2, 4 or 8 groups of four coordinates
    // prompt-sized launches: eight groups per thread (one wave per token up to 2048 coordinates: no
    // barrier partner to wait for, many tokens and many loads in flight per CU); decode-sized ones:
    // one group per thread, the shortest chain for the few workgroups there are
    const int groups = W / 4;
    const int want = R > 1024 ? (groups + 7) / 8 : groups;
    int threads = (want + 63) / 64 * 64;
    threads = threads > 1024 ? 1024 : threads;
    const int per = (groups + threads - 1) / threads;
#define PKM_HS(YT, VEC)                                                                             \
  if (post_w) {                                                                                                \
    PKM_DISPATCH(act_dt, E, hyper_step_kernel<E, YT, VEC, true, 1><<<R, threads, 0, stream>>>(a));             \
  } else if (S == 1) {                                                                                         \
    PKM_DISPATCH(act_dt, E, hyper_step_kernel<E, YT, VEC, false, 1><<<R, threads, 0, stream>>>(a));            \
  } else {                                                                                                     \
    PKM_DISPATCH(act_dt, E, hyper_step_kernel<E, YT, VEC, false, kMaxStreams><<<R, threads, 0, stream>>>(a));  \
  }
#define PKM_HS_Y(VEC)   \
  if (y32) {            \
    PKM_HS(float, VEC); \
  } else {              \
    PKM_HS(bf16_t, VEC); \
  }
    if (per <= 1) {
      PKM_HS_Y(4)
    } else if (per <= 2) {
      PKM_HS_Y(8)
    } else if (per <= 4) {
      PKM_HS_Y(16)
    } else if (per <= 8) {
      PKM_HS_Y(32)
    } else {
      PKM_HS_Y(64)
    }
#undef PKM_HS_Y
#undef PKM_HS
  } else {
#define PKM_HS1(YT)                                                                               \
  if (post_w) {                                                                                             \
    PKM_DISPATCH(act_dt, E, hyper_step_kernel<E, YT, 1, true, 1><<<R, threads, lds, stream>>>(a));            \
  } else {                                                                                                  \
    PKM_DISPATCH(act_dt, E, hyper_step_kernel<E, YT, 1, false, kMaxStreams><<<R, threads, lds, stream>>>(a)); \
  }
    const int threads = W >= 4096 ? 1024 : (W >= 1024 ? 512 : 256);
    if (y32) {
      PKM_HS1(float)
    } else {
      PKM_HS1(bf16_t)
    }
#undef PKM_HS1
  }
  return PK_CHECK_LAUNCH();
}

// x [R, W] fp32, updated in place; ya / yb: [R, W] rows (na, nb > 1: fp32 slabs [n][R][W]), each of its own element type; wa, wb,
// post_w [W] fp32; act [R, W] of type act_dt takes the new rows
PK_EXPORT int pkm_pair_step(void* x, int R, int W, const void* ya, int na, int ya_dt, const void* yb, int nb, int yb_dt,
                            const void* wa, const void* wb, float ca, float cb, const void* post_w, float eps, void* act,
                            int act_dt, hipStream_t stream) {
  if (R <= 0) return 0;
  if (W < 1 || W > 16384 || na < 1 || nb < 1 || !ya || !yb || !wa || !wb || !post_w || !act) return -1;
  if ((ya_dt != kF32 && (ya_dt != kBF16 || na > 1)) || (yb_dt != kF32 && (yb_dt != kBF16 || nb > 1))) return -2;
  const PairArgs a{static_cast<float*>(x), W, {ya, yb}, {ya_dt == kF32, yb_dt == kF32}, {na, nb}, static_cast<int64_t>(R) * W,
                   {static_cast<const float*>(wa), static_cast<const float*>(wb)}, {ca, cb}, static_cast<const float*>(post_w), eps, act};
#define PKM_PS(NG, THREADS, LDS) PKM_DISPATCH(act_dt, E, pair_step_kernel<E, NG><<<R, THREADS, LDS, stream>>>(a))
  if (W % 4) {
    const size_t lds = 2 * static_cast<size_t>(W) * sizeof(float);
    const int threads = W >= 4096 ? 1024 : 256;
    if (lds > 60 * 1024) {
      const void* kern = act_dt == kF32 ? reinterpret_cast<const void*>(pair_step_kernel<float, 0>)
                                        : reinterpret_cast<const void*>(pair_step_kernel<bf16_t, 0>);
      const hipError_t e = hipFuncSetAttribute(kern, hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds));
      if (e != hipSuccess) return static_cast<int>(e);
    }
    PKM_PS(0, threads, lds);
    return PK_CHECK_LAUNCH();
  }
  // prompt-sized launches: up to four groups per thread (few waves per token, many tokens per CU); decode-sized
  // ones: one group per thread
  const int groups = W / 4;
  int threads = ((R > 1024 ? (groups + 3) / 4 : groups) + 63) / 64 * 64;
  threads = threads > 1024 ? 1024 : threads;
  const int per = (groups + threads - 1) / threads;
  if (per <= 1) {
    PKM_PS(1, threads, 0);
  } else if (per <= 2) {
    PKM_PS(2, threads, 0);
  } else {
    PKM_PS(4, threads, 0);
  }
#undef PKM_PS
  return PK_CHECK_LAUNCH();
}

PK_EXPORT int pkm_tanh_cap(void* x, long long n, float cap, hipStream_t stream) {
  if (n <= 0) return 0;
  tanh_cap_kernel<<<static_cast<unsigned>((n + 255) / 256), 256, 0, stream>>>(static_cast<float*>(x), n, cap);
  return PK_CHECK_LAUNCH();
}
