// Short causal filter over time on each channel, with the sequence's last inputs in its state slot.
//
//   causal_conv   y_t = sum_j taps[c, j] x_(t - K + 1 + j) (+ bias), optional SiLU, optional + x_t.
//                 Inputs before the portion come from the slot's [K - 1, C] fp32 rows (oldest first),
//                 zeros when the portion starts at position 0 or the sequence has no slot.  An input
//                 bias is added to every row of x on the way in (the slot keeps biased rows).
//   conv_state    the slot takes the last K - 1 inputs after the portion.
//
// One thread per (token, channel), or (bf16 rows of many tokens, K <= 4) one per 8 channels of a run of
// tokens with the last K inputs in registers; the sum runs in tap order in fp32 whether an input comes from the
// portion or from the slot, so a position's result does not depend on how its prompt was cut.
#include "mix_common.h"

using namespace pkm;

namespace {

constexpr int kActNone = 0, kActSilu = 1;

template <typename TI, typename TO>
__global__ void __launch_bounds__(256)
causal_conv_kernel(TO* __restrict__ out, const TI* __restrict__ x, int64_t xs, const float* __restrict__ in_bias,
                   const float* __restrict__ taps, int K, const float* __restrict__ bias, const float* __restrict__ state,
                   const int* __restrict__ cu_q, const int* __restrict__ positions, const int* __restrict__ slots,
                   const int* __restrict__ token_seq, int C, int act, int residual) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int s = token_seq[t];
  const int q0 = cu_q[s];
  const int i = t - q0;
  const int slot = slots[s];
  const bool carry = state != nullptr && slot >= 0 && positions[q0] > 0;
  const float ib = in_bias ? in_bias[c] : 0.f;
  const float* w = taps + static_cast<int64_t>(c) * K;
  float acc = 0.f;
  for (int j = 0; j < K; ++j) {
    const int src = i - (K - 1) + j;
    float v = 0.f;
    if (src >= 0) {
      v = ld<TI>(x + static_cast<int64_t>(q0 + src) * xs + c) + ib;
    } else if (carry) {
      v = state[(static_cast<int64_t>(slot) * (K - 1) + (K - 1 + src)) * C + c];
    }
    acc += w[j] * v;
  }
  if (bias) acc += bias[c];
  if (act == kActSilu) acc = acc * sigmoidf(acc);
  if (residual) acc += ld<TI>(x + static_cast<int64_t>(t) * xs + c) + ib;
  st<TO>(out + static_cast<int64_t>(t) * C + c, acc);
}

// one thread per (sequence, channel): row i of the new state is entry n + i of (old rows, portion rows);
// n >= 1, so every read of an old row lies at or ahead of the row being written
template <typename TI>
__global__ void __launch_bounds__(256)
conv_state_kernel(float* __restrict__ state, const TI* __restrict__ x, int64_t xs, const float* __restrict__ in_bias,
                  const int* __restrict__ cu_q, const int* __restrict__ positions, const int* __restrict__ slots, int K,
                  int C) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int q0 = cu_q[s], n = cu_q[s + 1] - q0, slot = slots[s];
  if (n <= 0 || slot < 0) return;
  const bool carry = positions[q0] > 0;
  const float ib = in_bias ? in_bias[c] : 0.f;
  float* rows = state + static_cast<int64_t>(slot) * (K - 1) * C + c;
  for (int i = 0; i < K - 1; ++i) {
    const int idx = n + i - (K - 1);
    float v = 0.f;
    if (idx >= 0) {
      v = ld<TI>(x + static_cast<int64_t>(q0 + idx) * xs + c) + ib;
    } else if (carry) {
      v = rows[static_cast<int64_t>(n + i) * C];
    }
    rows[static_cast<int64_t>(i) * C] = v;
  }
}

// bf16 rows, C and the row stride multiples of 8: a thread owns 8 channels (16-byte accesses) of kRunT
// consecutive tokens of the step; win[j] is the input of K - 1 - j tokens ago, refilled from the portion
// or the slot where the run or a sequence starts.
constexpr int kRunT = 8;

template <int K>
__global__ void __launch_bounds__(256)
causal_conv_run_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ x, int64_t xs, const float* __restrict__ in_bias,
                       const float* __restrict__ taps, const float* __restrict__ bias, const float* __restrict__ state,
                       const int* __restrict__ cu_q, const int* __restrict__ positions, const int* __restrict__ slots,
                       const int* __restrict__ token_seq, int T, int C, int act, int residual) {
  const int c = 8 * (blockIdx.y * 256 + threadIdx.x);
  if (c >= C) return;
  const int t0 = blockIdx.x * kRunT, t1 = min(T, t0 + kRunT);
  float w[8][K], ib[8], ob[8], win[K][8];
#pragma unroll
  for (int e = 0; e < 8; ++e) {
#pragma unroll
    for (int j = 0; j < K; ++j) w[e][j] = taps[static_cast<int64_t>(c + e) * K + j];
    ib[e] = in_bias ? in_bias[c + e] : 0.f;
    ob[e] = bias ? bias[c + e] : 0.f;
  }
  auto row = [&](float* v, int64_t t) {
    const pk::u32x4 r = *reinterpret_cast<const pk::u32x4*>(x + t * xs + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[2 * e] = __uint_as_float(r[e] << 16) + ib[2 * e];
      v[2 * e + 1] = __uint_as_float(r[e] & 0xffff0000u) + ib[2 * e + 1];
    }
  };
  for (int t = t0; t < t1; ++t) {
    const int s = token_seq[t], q0 = cu_q[s], i = t - q0;
    if (t == t0 || i == 0) {
      const int slot = slots[s];
      const bool carry = K > 1 && slot >= 0 && positions[q0] > 0;
#pragma unroll
      for (int j = 0; j < K - 1; ++j) {  // win[j + 1] moves to win[j] below
        const int src = i - (K - 1) + j;
        if (src >= 0) {
          row(win[j + 1], q0 + src);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            win[j + 1][e] = carry ? state[(static_cast<int64_t>(slot) * (K - 1) + (K - 1 + src)) * C + c + e] : 0.f;
        }
      }
    }
#pragma unroll
    for (int j = 0; j < K - 1; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) win[j][e] = win[j + 1][e];
    row(win[K - 1], t);
    float y[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < K; ++j) acc += w[e][j] * win[j][e];
      if (bias) acc += ob[e];
      if (act == kActSilu) acc = acc * sigmoidf(acc);
      if (residual) acc += win[K - 1][e];
      y[e] = acc;
    }
    pk::u32x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = pk::pack2(y[2 * e], y[2 * e + 1]);
    *reinterpret_cast<pk::u32x4*>(out + static_cast<int64_t>(t) * C + c) = o;
  }
}

// Steps in which every sequence holds one token: one thread per (sequence, channel) filters and moves
// the slot's rows (row j is read before row j - 1 takes it).  The same sums in the same order.
template <typename TI, typename TO>
__global__ void __launch_bounds__(256)
conv_step_kernel(TO* __restrict__ out, const TI* __restrict__ x, int64_t xs, const float* __restrict__ in_bias,
                 const float* __restrict__ taps, int K, const float* __restrict__ bias, float* __restrict__ state,
                 const int* __restrict__ positions, const int* __restrict__ slots, int C, int act, int residual) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int slot = slots[t];
  const bool carry = slot >= 0 && positions[t] > 0;
  float* rows = slot >= 0 ? state + static_cast<int64_t>(slot) * (K - 1) * C + c : nullptr;
  const float* w = taps + static_cast<int64_t>(c) * K;
  const float xv = ld<TI>(x + static_cast<int64_t>(t) * xs + c) + (in_bias ? in_bias[c] : 0.f);
  float acc = 0.f;
  for (int j = 0; j < K - 1; ++j) {
    const float v = carry ? rows[static_cast<int64_t>(j) * C] : 0.f;
    acc += w[j] * v;
    if (rows && j > 0) rows[static_cast<int64_t>(j - 1) * C] = v;
  }
  if (rows) rows[static_cast<int64_t>(K - 2) * C] = xv;
  acc += w[K - 1] * xv;
  if (bias) acc += bias[c];
  if (act == kActSilu) acc = acc * sigmoidf(acc);
  if (residual) acc += xv;
  st<TO>(out + static_cast<int64_t>(t) * C + c, acc);
}

}  // namespace

// single: every sequence holds one token (n_seqs == T).
// x [T, C] rows x_stride elements apart (x_dt); out [T, C] contiguous (out_dt); taps [C, K] fp32; in_bias, bias [C]
// fp32 or null; state [slots, K - 1, C] fp32 (null with K = 1), brought up to date after the outputs
PK_EXPORT int pkm_causal_conv(void* out, int out_dt, const void* x, int x_dt, long long x_stride, const void* in_bias,
                              const void* taps, int K, const void* bias, void* state, const void* cu_q,
                              const void* positions, const void* slots, const void* token_seq, int n_seqs, int T, int C,
                              int act, int residual, int single, hipStream_t stream) {
  if (T <= 0) return 0;
  if (K < 1 || C < 1 || (K > 1 && state == nullptr) || x_stride < C) return -1;
  if (single && n_seqs != T) return -1;
  const dim3 grid(T, (C + 255) / 256);
  const bool runs = !single && T >= 64 && K >= 2 && K <= 4 && x_dt == kBF16 && out_dt == kBF16 && C % 8 == 0 &&
                    x_stride % 8 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0;
  if (single && K > 1) {
#define PKM_CS(TI)                                                                                                     \
  PKM_DISPATCH(out_dt, O, conv_step_kernel<TI, O><<<grid, 256, 0, stream>>>(                                             \
                              static_cast<O*>(out), static_cast<const TI*>(x), x_stride, static_cast<const float*>(in_bias), \
                              static_cast<const float*>(taps), K, static_cast<const float*>(bias),                         \
                              static_cast<float*>(state), static_cast<const int*>(positions),                              \
                              static_cast<const int*>(slots), C, act, residual))
    if (x_dt == kF32) {
      PKM_CS(float);
    } else if (x_dt == kBF16) {
      PKM_CS(bf16_t);
    } else {
      return -2;
    }
#undef PKM_CS
    return PK_CHECK_LAUNCH();
  }
#define PKM_CC(TI)                                                                                                       \
  PKM_DISPATCH(out_dt, O, causal_conv_kernel<TI, O><<<grid, 256, 0, stream>>>(                                             \
                              static_cast<O*>(out), static_cast<const TI*>(x), x_stride, static_cast<const float*>(in_bias), \
                              static_cast<const float*>(taps), K, static_cast<const float*>(bias),                         \
                              static_cast<const float*>(state), static_cast<const int*>(cu_q),                             \
                              static_cast<const int*>(positions), static_cast<const int*>(slots),                          \
                              static_cast<const int*>(token_seq), C, act, residual))
  if (runs) {
    const dim3 rgrid((T + kRunT - 1) / kRunT, (C / 8 + 255) / 256);
#define PKM_CR(KK)                                                                                                    \
  causal_conv_run_kernel<KK><<<rgrid, 256, 0, stream>>>(                                                               \
      static_cast<bf16_t*>(out), static_cast<const bf16_t*>(x), x_stride, static_cast<const float*>(in_bias),          \
      static_cast<const float*>(taps), static_cast<const float*>(bias), static_cast<const float*>(state),              \
      static_cast<const int*>(cu_q), static_cast<const int*>(positions), static_cast<const int*>(slots),               \
      static_cast<const int*>(token_seq), T, C, act, residual)
    if (K == 2) {
      PKM_CR(2);
    } else if (K == 3) {
      PKM_CR(3);
    } else {
      PKM_CR(4);
    }
#undef PKM_CR
  } else if (x_dt == kF32) {
    PKM_CC(float);
  } else if (x_dt == kBF16) {
    PKM_CC(bf16_t);
  } else {
    return -2;
  }
#undef PKM_CC
  int rc = PK_CHECK_LAUNCH();
  if (rc != 0 || K == 1) return rc;
  const dim3 sgrid(n_seqs, (C + 255) / 256);
  PKM_DISPATCH(x_dt, E, conv_state_kernel<E><<<sgrid, 256, 0, stream>>>(
                            static_cast<float*>(state), static_cast<const E*>(x), x_stride, static_cast<const float*>(in_bias),
                            static_cast<const int*>(cu_q), static_cast<const int*>(positions), static_cast<const int*>(slots),
                            K, C));
  return PK_CHECK_LAUNCH();
}
