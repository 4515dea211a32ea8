// Real-gated linear recurrence (one fp32 number of state per channel) between block-diagonal gates
// and a GELU branch.
//
//   r = sigmoid(R_b u_b + rb),  i = sigmoid(I_b u_b + ib)      u in `blocks` equal parts u_b
//   a = exp(lam * r),  b = sqrt(1 - a^2) i u                   lam [C] fp32, negative
//   S <- a S + b;   out = S * gelu_tanh(y + yb)
//
// The gate products accumulate in fp32 and never leave it; a, b and S are fp32.  bf16 models with parts
// that are multiples of 64 wide take the matrix cores, everything else FMA tiles.  A step in which
// every sequence holds one token does gates, recurrence and output in one kernel.  Otherwise the gates
// write (a, b) per token and channel and the recurrence runs in three kernels over runs of 32 tokens of
// a sequence: each run's product of a and its end value from zero, the state in front of each run
// (a walk over the runs, which also moves the slot's state), and the outputs from those states.
// State [slots, C] fp32: read by a portion's first token unless it is position 0, written after its
// last token; sequences without a slot start from zeros and leave nothing.
#include "mix_common.h"

using namespace pkm;

namespace {

constexpr int kRun = 32;  // tokens per run of the prompt scan

struct LruArgs {
  const void* u;
  int64_t us;
  const void* y;
  int64_t ys;
  const float* yb;
  const void* ra;
  const void* ri;
  const float* rb;
  const float* ib;
  const float* lam;
  float* state;
  void* out;
  int64_t os;
  float post;
  const int* positions;
  const int* slots;
  float2* ab;  // [T, C] or null: every sequence holds one token and the recurrence happens here
  int T, C, wb;
};

__device__ __forceinline__ float gelu_tanhf(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// the gates' pre-activations of (token t, channel c) -> (a, b), or the step itself
template <typename T>
__device__ __forceinline__ void finish(const LruArgs& g, int t, int c, float rz, float iz) {
  const float u = ld<T>(static_cast<const T*>(g.u) + static_cast<int64_t>(t) * g.us + c);
  const float r = sigmoidf(rz + g.rb[c]), i = sigmoidf(iz + g.ib[c]);
  const float la = g.lam[c] * r;
  const float a = expf(la), b = sqrtf(-expm1f(2.f * la)) * i * u;
  if (g.ab) {
    g.ab[static_cast<int64_t>(t) * g.C + c] = make_float2(a, b);
    return;
  }
  const int slot = g.slots[t];
  float* sp = slot >= 0 ? g.state + static_cast<int64_t>(slot) * g.C + c : nullptr;
  float S = (sp && g.positions[t] > 0) ? *sp : 0.f;
  S = a * S + b;
  if (sp) *sp = S;
  const float y = ld<T>(static_cast<const T*>(g.y) + static_cast<int64_t>(t) * g.ys + c) + g.yb[c];
  st<T>(static_cast<T*>(g.out) + static_cast<int64_t>(t) * g.os + c, S * gelu_tanhf(y) * g.post);
}

// any part width, both element types: 32 tokens x 32 channels of one part per workgroup
template <typename T>
__global__ void __launch_bounds__(256) lru_gates_fma_kernel(LruArgs g) {
  constexpr int B = 32;
  __shared__ float us[B][B + 1], rs[B][B + 1], is[B][B + 1];
  const int ct = (g.wb + B - 1) / B;
  const int part = blockIdx.y / ct, n0 = (blockIdx.y - part * ct) * B, t0 = blockIdx.x * B;
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const T* u = static_cast<const T*>(g.u) + part * g.wb;
  const T* ra = static_cast<const T*>(g.ra) + static_cast<int64_t>(part) * g.wb * g.wb;
  const T* ri = static_cast<const T*>(g.ri) + static_cast<int64_t>(part) * g.wb * g.wb;
  float ar[2][2] = {{0.f, 0.f}, {0.f, 0.f}}, ai[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
  for (int k0 = 0; k0 < g.wb; k0 += B) {
    for (int e = tid; e < B * B; e += 256) {
      const int r = e / B, c = e - r * B;
      const bool kc = k0 + c < g.wb, nr = n0 + r < g.wb;
      us[r][c] = (kc && t0 + r < g.T) ? ld<T>(u + static_cast<int64_t>(t0 + r) * g.us + k0 + c) : 0.f;
      rs[r][c] = (kc && nr) ? ld<T>(ra + static_cast<int64_t>(n0 + r) * g.wb + k0 + c) : 0.f;
      is[r][c] = (kc && nr) ? ld<T>(ri + static_cast<int64_t>(n0 + r) * g.wb + k0 + c) : 0.f;
    }
    __syncthreads();
#pragma unroll 8
    for (int c = 0; c < B; ++c) {
      const float u0 = us[ty][c], u1 = us[ty + 16][c];
      const float r0 = rs[tx][c], r1 = rs[tx + 16][c], i0 = is[tx][c], i1 = is[tx + 16][c];
      ar[0][0] += u0 * r0;
      ar[0][1] += u0 * r1;
      ar[1][0] += u1 * r0;
      ar[1][1] += u1 * r1;
      ai[0][0] += u0 * i0;
      ai[0][1] += u0 * i1;
      ai[1][0] += u1 * i0;
      ai[1][1] += u1 * i1;
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = t0 + ty + 16 * i;
    if (t >= g.T) continue;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + tx + 16 * j;
      if (n < g.wb) finish<T>(g, t, part * g.wb + n, ar[i][j], ai[i][j]);
    }
  }
}

// bf16, wb % 64 == 0: products transposed on mfma_f32_16x16x32_bf16 (A = gate rows, B = token rows), so a
// lane ends with four neighbouring channels of one token.  A wave owns RT 16-channel tiles x NT 16-token
// tiles; the four waves of a workgroup lie along the tokens (TOK) or along the channels.
template <int RT, int NT, bool TOK>
__global__ void __launch_bounds__(256) lru_gates_mfma_kernel(LruArgs g) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = lane & 15, q = lane >> 4;
  const int c0 = blockIdx.y * (TOK ? 16 * RT : 64 * RT) + (TOK ? 0 : wave * 16 * RT);
  const int t0 = blockIdx.x * (TOK ? 64 * NT : 16 * NT) + (TOK ? wave * 16 * NT : 0);
  const int part = c0 / g.wb, row0 = c0 - part * g.wb;
  const bf16_t* u = static_cast<const bf16_t*>(g.u) + part * g.wb + 8 * q;
  const int64_t wo = (static_cast<int64_t>(part) * g.wb + row0 + n) * g.wb + 8 * q;
  const bf16_t* ra = static_cast<const bf16_t*>(g.ra) + wo;
  const bf16_t* ri = static_cast<const bf16_t*>(g.ri) + wo;
  pk::f32x4 ar[RT][NT], ai[RT][NT];
#pragma unroll
  for (int r = 0; r < RT; ++r)
#pragma unroll
    for (int j = 0; j < NT; ++j) ar[r][j] = ai[r][j] = pk::f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16_t* ur[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) ur[j] = u + static_cast<int64_t>(min(t0 + 16 * j + n, g.T - 1)) * g.us;
  for (int k = 0; k < g.wb; k += 32) {
    pk::bf16x8_t ub[NT], wr[RT], wi[RT];
#pragma unroll
    for (int j = 0; j < NT; ++j) ub[j] = pk::ld8(ur[j] + k);
#pragma unroll
    for (int r = 0; r < RT; ++r) {
      wr[r] = pk::ld8(ra + static_cast<int64_t>(16 * r) * g.wb + k);
      wi[r] = pk::ld8(ri + static_cast<int64_t>(16 * r) * g.wb + k);
    }
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        ar[r][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wr[r], ub[j], ar[r][j], 0, 0, 0);
        ai[r][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wi[r], ub[j], ai[r][j], 0, 0, 0);
      }
  }
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    const int t = t0 + 16 * j + n;
    if (t >= g.T) continue;
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int e = 0; e < 4; ++e) finish<bf16_t>(g, t, c0 + 16 * r + 4 * q + e, ar[r][j][e], ai[r][j][e]);
  }
}

// which run of which sequence is number `tile`; false: past the last
__device__ __forceinline__ bool find_run(const int* cu_q, int n_seqs, int tile, int& s, int& t0, int& t1) {
  for (s = 0; s < n_seqs; ++s) {
    const int a = cu_q[s], b = cu_q[s + 1];
    const int n = (b - a + kRun - 1) / kRun;
    if (tile < n) {
      t0 = a + tile * kRun;
      t1 = min(b, t0 + kRun);
      return true;
    }
    tile -= n;
  }
  return false;
}

__global__ void __launch_bounds__(256) lru_run_ends_kernel(float2* __restrict__ ends, const float2* __restrict__ ab,
                                                           const int* __restrict__ cu_q, int n_seqs, int C) {
  int s, t0, t1;
  if (!find_run(cu_q, n_seqs, blockIdx.x, s, t0, t1)) return;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  float P = 1.f, B = 0.f;
#pragma unroll 8
  for (int t = t0; t < t1; ++t) {
    const float2 v = ab[static_cast<int64_t>(t) * C + c];
    P *= v.x;
    B = v.x * B + v.y;
  }
  ends[static_cast<int64_t>(blockIdx.x) * C + c] = make_float2(P, B);
}

// starts[run] = the state in front of it; the slot takes the state behind the last run
__global__ void __launch_bounds__(64) lru_run_starts_kernel(float* __restrict__ starts, const float2* __restrict__ ends,
                                                            float* __restrict__ state, const int* __restrict__ cu_q,
                                                            const int* __restrict__ positions,
                                                            const int* __restrict__ slots, int C) {
  const int s = blockIdx.y, c = blockIdx.x * 64 + threadIdx.x;
  const int a = cu_q[s], b = cu_q[s + 1];
  if (b <= a || c >= C) return;
  int64_t tile = 0;
  for (int i = 0; i < s; ++i) tile += (cu_q[i + 1] - cu_q[i] + kRun - 1) / kRun;
  const int n = (b - a + kRun - 1) / kRun;
  const int slot = slots[s];
  float* sp = slot >= 0 ? state + static_cast<int64_t>(slot) * C + c : nullptr;
  float S = (sp && positions[a] > 0) ? *sp : 0.f;
#pragma unroll 8
  for (int j = 0; j < n; ++j) {
    const float2 v = ends[(tile + j) * C + c];
    starts[(tile + j) * C + c] = S;
    S = v.x * S + v.y;
  }
  if (sp) *sp = S;
}

template <typename T>
__global__ void __launch_bounds__(256) lru_run_out_kernel(LruArgs g, const float* __restrict__ starts,
                                                          const float2* __restrict__ ab, const int* __restrict__ cu_q,
                                                          int n_seqs) {
  int s, t0, t1;
  if (!find_run(cu_q, n_seqs, blockIdx.x, s, t0, t1)) return;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= g.C) return;
  float S = starts[static_cast<int64_t>(blockIdx.x) * g.C + c];
  const T* y = static_cast<const T*>(g.y) + c;
  T* out = static_cast<T*>(g.out) + c;
  const float yb = g.yb[c];
#pragma unroll 8
  for (int t = t0; t < t1; ++t) {
    const float2 v = ab[static_cast<int64_t>(t) * g.C + c];
    S = v.x * S + v.y;
    st<T>(out + static_cast<int64_t>(t) * g.os, S * gelu_tanhf(ld<T>(y + static_cast<int64_t>(t) * g.ys) + yb) * g.post);
  }
}

int g_lru_mfma = 1;  // 0: every launch takes the FMA gates (tests compare the two)

}  // namespace

PK_EXPORT int pkm_set_lru_mfma(int on) {
  g_lru_mfma = on;
  return 0;
}

// u, y [T, C] (element type dt, own row strides), ra / ri [blocks, C / blocks, C / blocks] of dt, rb / ib / lam / yb [C]
// fp32, state [slots, C] fp32, out rows os elements apart, times post.  single: every sequence holds one token
// (n_seqs == T); otherwise ab [T, C, 2], ends [T / 32 + n_seqs, C, 2] and starts [T / 32 + n_seqs, C] fp32 are scratch.
PK_EXPORT int pkm_gated_lru(void* out, long long os, const void* u, long long us, const void* y, long long ys, const void* yb,
                            const void* ra, const void* ri, const void* rb, const void* ib, const void* lam, void* state,
                            const void* cu_q, const void* positions, const void* slots, int n_seqs, int T, int C, int blocks,
                            float post, int single, void* ab, void* ends, void* starts, int dt, hipStream_t stream) {
  if (T <= 0 || n_seqs <= 0) return 0;
  if (C < 1 || blocks < 1 || C % blocks || us < C || ys < C || os < C) return -1;
  if (single ? n_seqs != T : (!ab || !ends || !starts)) return -1;
  LruArgs g{u, us, y, ys, static_cast<const float*>(yb), ra, ri, static_cast<const float*>(rb), static_cast<const float*>(ib),
            static_cast<const float*>(lam), static_cast<float*>(state), out, os, post, static_cast<const int*>(positions),
            static_cast<const int*>(slots), single ? nullptr : static_cast<float2*>(ab), T, C, C / blocks};
  if (g_lru_mfma && dt == kBF16 && g.wb % 64 == 0 && us % 8 == 0) {
    if (T > 256) {
      lru_gates_mfma_kernel<4, 2, true><<<dim3((T + 127) / 128, C / 64), 256, 0, stream>>>(g);
    } else {
      lru_gates_mfma_kernel<1, 1, false><<<dim3((T + 15) / 16, C / 64), 256, 0, stream>>>(g);
    }
  } else {
    const dim3 grid((T + 31) / 32, blocks * ((g.wb + 31) / 32));
    PKM_DISPATCH(dt, E, lru_gates_fma_kernel<E><<<grid, 256, 0, stream>>>(g));
  }
  int rc = PK_CHECK_LAUNCH();
  if (rc != 0 || single) return rc;
  const int runs = T / kRun + n_seqs;
  const int* cq = static_cast<const int*>(cu_q);
  const dim3 rgrid(runs, (C + 255) / 256);
  lru_run_ends_kernel<<<rgrid, 256, 0, stream>>>(static_cast<float2*>(ends), g.ab, cq, n_seqs, C);
  rc = PK_CHECK_LAUNCH();
  if (rc != 0) return rc;
  lru_run_starts_kernel<<<dim3((C + 63) / 64, n_seqs), 64, 0, stream>>>(static_cast<float*>(starts),
                                                                         static_cast<const float2*>(ends), g.state, cq,
                                                                         g.positions, g.slots, C);
  rc = PK_CHECK_LAUNCH();
  if (rc != 0) return rc;
  PKM_DISPATCH(dt, E, lru_run_out_kernel<E><<<rgrid, 256, 0, stream>>>(g, static_cast<const float*>(starts), g.ab, cq, n_seqs));
  return PK_CHECK_LAUNCH();
}
