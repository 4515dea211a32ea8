// Lightning attention: linear attention with one constant decay per head.
//
//     S_t = decay_h * S_{t-1} + k_t v_t^T        o_t = S_t^T q_t        q, k, v = silu(projections)
//
// Retention is the same recurrence on plain projections (no SiLU): q and k turn by the token's
// position in fp32 (pair (i, i + pairs), (cos, sin) table rows) and k is multiplied by k_scale.
// The step form (state-space duality) has a step size d = softplus(dt + bias) per (token, head): decay
// exp(-exp(a_log_h) d), v scaled by d on its way in, k / q shared by groups of heads, skip_h v added to o.
// The state S [D, V] of a (sequence, head) is fp32 and lives in the sequence's state slot between
// steps.  One workgroup owns 16 value columns of one (sequence, head): thread (dg, vc) keeps rows
// dg, dg + 16, ... of column vc in registers and walks the portion's tokens in order; q, k, v of up to
// 32 tokens at a time are staged in LDS with the SiLU applied.  A token's sums run in the same order
// whether it arrives in a long prompt portion or alone, so results do not depend on the cut.
// The first token of a portion reads the slot unless it is position 0 (a new sequence starts from
// zeros whatever an earlier owner left); the state after the portion's last token is written back.
#include "mix_common.h"

using namespace pkm;

namespace {

constexpr int kMaxChunk = 32;  // tokens staged per group (fewer when a head is wide)
constexpr int kCols = 16;   // value columns per workgroup

// what happens to a projection on its way into the recurrence
struct HeadIn {
  const float* table;    // [rows, pairs, 2] fp32 (cos, sin) or null
  int pairs, rows;
  const int* positions;
  float k_scale;
  // step form: rows of the input are [H*V v | G*D k | G*D q]
  const void* dt;        // [T, H] pre-activations, rows dt_stride apart
  int64_t dt_stride;
  int groups;
  const float* dt_bias;  // [H] each
  const float* a_log;
  const float* skip;
};

enum Form { kSilu, kTurned, kStep };

struct HeadAt {
  int64_t q, k, v;  // first columns of a head in the input row
};

template <Form F>
__device__ __forceinline__ HeadAt head_at(const HeadIn& in, int h, int H, int D, int V) {
  if (F == kStep) {
    const int64_t g = h / (H / in.groups), k0 = static_cast<int64_t>(H) * V;
    return HeadAt{k0 + (in.groups + g) * D, k0 + g * D, static_cast<int64_t>(h) * V};
  }
  const int64_t q = static_cast<int64_t>(h) * D, hd = static_cast<int64_t>(H) * D;
  return HeadAt{q, hd + q, 2 * hd + static_cast<int64_t>(h) * V};
}

__device__ __forceinline__ float softplusf(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// step size and decay of (token t, head h)
template <typename T>
__device__ __forceinline__ void step_at(const HeadIn& in, int64_t t, int h, float& d, float& dec) {
  d = softplusf(ld<T>(static_cast<const T*>(in.dt) + t * in.dt_stride + h) + in.dt_bias[h]);
  dec = expf(-expf(in.a_log[h]) * d);
}

__device__ __forceinline__ float siluf(float z) { return z / (1.f + expf(-z)); }

// coordinate d of a head's projection row `src`, turned by token t's position
template <typename T>
__device__ __forceinline__ float turned(const T* src, int d, int64_t t, const HeadIn& in) {
  const float x = ld<T>(src + d);
  if (in.table == nullptr || d >= 2 * in.pairs) return x;
  const bool first = d < in.pairs;
  const int i = first ? d : d - in.pairs;
  const float y = ld<T>(src + (first ? d + in.pairs : i));
  const int pos = in.positions[t];
  const float* cs = in.table + (static_cast<int64_t>(pos < 0 ? 0 : min(pos, in.rows - 1)) * in.pairs + i) * 2;
  return first ? x * cs[0] - y * cs[1] : x * cs[0] + y * cs[1];
}

template <typename T, int ND, Form F>
__global__ void __launch_bounds__(256)
lightning_kernel(float* __restrict__ out, const T* __restrict__ qkv, int64_t stride, float* __restrict__ state,
                 const float* __restrict__ decay, const int* __restrict__ cu_q, const int* __restrict__ positions,
                 const int* __restrict__ slots, int H, int D, int V, int kChunk, HeadIn in) {
  extern __shared__ float smem[];
  float* qs = smem;                 // [kChunk][D]
  float* ks = qs + kChunk * D;      // [kChunk][D]
  float* vs = ks + kChunk * D;      // [kChunk][kCols]
  float* ds = vs + kChunk * kCols;  // [kChunk][2] step size, decay (kStep)
  const int s = blockIdx.x / H, h = blockIdx.x - s * H;
  const int v0 = blockIdx.y * kCols;
  const int a = cu_q[s], b = cu_q[s + 1];
  if (b <= a) return;
  const int tid = threadIdx.x, dg = tid & 15, vc = tid >> 4;
  const int col = v0 + vc;
  const int slot = slots[s];
  const float dec_h = F == kStep ? 0.f : decay[h], skip = F == kStep ? in.skip[h] : 0.f;
  float S[ND];
  float* sp = slot >= 0 ? state + ((static_cast<int64_t>(slot) * H + h) * D) * V : nullptr;
  const bool carry = sp != nullptr && positions[a] > 0;
#pragma unroll
  for (int i = 0; i < ND; ++i) {
    const int d = dg + 16 * i;
    S[i] = (carry && d < D && col < V) ? sp[static_cast<int64_t>(d) * V + col] : 0.f;
  }
  const HeadAt at = head_at<F>(in, h, H, D, V);
  const int64_t qo = at.q, ko = at.k, vo = at.v + v0;
  for (int t0 = a; t0 < b; t0 += kChunk) {
    const int nt = min(kChunk, b - t0);
    __syncthreads();
    for (int e = tid; e < nt * D; e += 256) {
      const int t = e / D, d = e - t * D;
      const T* row = qkv + static_cast<int64_t>(t0 + t) * stride;
      if (F == kTurned) {
        qs[e] = turned(row + qo, d, t0 + t, in);
        ks[e] = turned(row + ko, d, t0 + t, in) * in.k_scale;
      } else {
        const float q = ld<T>(row + qo + d), k = ld<T>(row + ko + d);
        qs[e] = F == kSilu ? siluf(q) : q;
        ks[e] = F == kSilu ? siluf(k) : k;
      }
    }
    for (int e = tid; e < nt * kCols; e += 256) {
      const int t = e / kCols, c = e - t * kCols;
      const float v = v0 + c < V ? ld<T>(qkv + static_cast<int64_t>(t0 + t) * stride + vo + c) : 0.f;
      vs[e] = F == kSilu ? siluf(v) : v;
    }
    if (F == kStep && tid < nt) step_at<T>(in, t0 + tid, h, ds[2 * tid], ds[2 * tid + 1]);
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float dec = F == kStep ? ds[2 * t + 1] : dec_h;
      const float vv = F == kStep ? ds[2 * t] * vs[t * kCols + vc] : vs[t * kCols + vc];
      const float* kr = ks + t * D;
      const float* qr = qs + t * D;
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < ND; ++i) {
        const int d = dg + 16 * i;
        if (d < D) {
          S[i] = dec * S[i] + kr[d] * vv;
          o += S[i] * qr[d];
        }
      }
      o += __shfl_xor(o, 8, 64);
      o += __shfl_xor(o, 4, 64);
      o += __shfl_xor(o, 2, 64);
      o += __shfl_xor(o, 1, 64);
      if (F == kStep) o += skip * vs[t * kCols + vc];
      if (dg == 0 && col < V) out[(static_cast<int64_t>(t0 + t) * H + h) * V + col] = o;
    }
  }
  if (sp != nullptr && col < V) {
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int d = dg + 16 * i;
      if (d < D) sp[static_cast<int64_t>(d) * V + col] = S[i];
    }
  }
}

// The wider form for heads of up to 256 key coordinates: a workgroup owns 64 value columns of one
// (sequence, head), lane = column; wave w of NW keeps key rows w * NR .. w * NR + NR - 1 of its
// columns in registers, so a token costs each wave NR broadcast reads of k and q for 2 * NR * 64
// multiply-adds and no cross-lane traffic; the waves' partial outputs of a 16-token group are
// summed in wave order through LDS (coalesced stores).  The next group's q, k, v are fetched into
// registers before the current group is computed.  Same order of sums for any cut of the prompt.
constexpr int kWideChunk = 16;
constexpr int kWideCols = 64;

template <typename T, int NR, int NW, Form F>
__global__ void __launch_bounds__(64 * NW)
lightning_wide_kernel(float* __restrict__ out, const T* __restrict__ qkv, int64_t stride, float* __restrict__ state,
                      const float* __restrict__ decay, const int* __restrict__ cu_q, const int* __restrict__ positions,
                      const int* __restrict__ slots, int H, int D, int V, HeadIn in) {
  constexpr int DP = NW * NR;  // padded key width: rows past D hold zeros
  constexpr int NT = 64 * NW;
  constexpr int QK_IT = (kWideChunk * DP + NT - 1) / NT, V_IT = (kWideChunk * kWideCols + NT - 1) / NT;
  __shared__ __attribute__((aligned(16))) float qs[kWideChunk][DP];
  __shared__ __attribute__((aligned(16))) float ks[kWideChunk][DP];
  __shared__ float vs[kWideChunk][kWideCols];
  __shared__ float po[NW][kWideChunk][kWideCols];
  __shared__ float ds[F == kStep ? kWideChunk : 1][2];  // step size, decay
  const int s = blockIdx.x / H, h = blockIdx.x - s * H;
  const int v0 = blockIdx.y * kWideCols;
  const int a = cu_q[s], b = cu_q[s + 1];
  if (b <= a) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int col = v0 + lane;
  const int slot = slots[s];
  const float dec_h = F == kStep ? 0.f : decay[h], skip = F == kStep ? in.skip[h] : 0.f;
  float* sp = slot >= 0 ? state + ((static_cast<int64_t>(slot) * H + h) * D) * V : nullptr;
  const bool carry = sp != nullptr && positions[a] > 0;
  float S[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = w * NR + i;
    S[i] = (carry && d < D && col < V) ? sp[static_cast<int64_t>(d) * V + col] : 0.f;
  }
  const HeadAt at = head_at<F>(in, h, H, D, V);
  const int64_t qo = at.q, ko = at.k, vo = at.v + v0;
  float rq[QK_IT], rk[QK_IT], rv[V_IT];
  auto fetch = [&](int t0) {  // raw projections of the group starting at token t0 (zeros outside)
    const int nt = min(kWideChunk, b - t0);
#pragma unroll
    for (int i = 0; i < QK_IT; ++i) {
      const int e = tid + NT * i, t = e / DP, d = e - t * DP;
      const bool ok = t < nt && d < D;
      const T* row = qkv + static_cast<int64_t>(t0 + (ok ? t : 0)) * stride;
      if (F == kTurned) {
        rq[i] = ok ? turned(row + qo, d, t0 + t, in) : 0.f;
        rk[i] = ok ? turned(row + ko, d, t0 + t, in) * in.k_scale : 0.f;
      } else {
        rq[i] = ok ? ld<T>(row + qo + d) : (F == kSilu ? -INFINITY : 0.f);
        rk[i] = ok ? ld<T>(row + ko + d) : (F == kSilu ? -INFINITY : 0.f);
      }
    }
#pragma unroll
    for (int i = 0; i < V_IT; ++i) {
      const int e = tid + NT * i, t = e / kWideCols, c = e - t * kWideCols;
      const bool ok = t < nt && v0 + c < V;
      rv[i] = ok ? ld<T>(qkv + static_cast<int64_t>(t0 + (ok ? t : 0)) * stride + vo + c) : (F == kSilu ? -INFINITY : 0.f);
    }
  };
  fetch(a);
  for (int t0 = a; t0 < b; t0 += kWideChunk) {
    const int nt = min(kWideChunk, b - t0);
#pragma unroll
    for (int i = 0; i < QK_IT; ++i) {
      const int e = tid + NT * i;
      if (e < kWideChunk * DP) {
        (&qs[0][0])[e] = F != kSilu ? rq[i] : (rq[i] == -INFINITY ? 0.f : siluf(rq[i]));
        (&ks[0][0])[e] = F != kSilu ? rk[i] : (rk[i] == -INFINITY ? 0.f : siluf(rk[i]));
      }
    }
#pragma unroll
    for (int i = 0; i < V_IT; ++i) {
      const int e = tid + NT * i;
      if (e < kWideChunk * kWideCols) (&vs[0][0])[e] = F != kSilu ? rv[i] : (rv[i] == -INFINITY ? 0.f : siluf(rv[i]));
    }
    if (F == kStep && tid < nt) step_at<T>(in, t0 + tid, h, ds[tid][0], ds[tid][1]);
    __syncthreads();
    if (t0 + kWideChunk < b) fetch(t0 + kWideChunk);  // in flight while this group is computed
#pragma unroll 4
    for (int t = 0; t < nt; ++t) {
      const float dec = F == kStep ? ds[t][1] : dec_h;
      const float vv = F == kStep ? ds[t][0] * vs[t][lane] : vs[t][lane];
      const float* kr = &ks[t][w * NR];
      const float* qr = &qs[t][w * NR];
      float o0 = (F == kStep && w == 0) ? skip * vs[t][lane] : 0.f, o1 = 0.f;
      if (NR % 4 == 0) {
#pragma unroll
        for (int i = 0; i < NR; i += 4) {
          const float4 k4 = *reinterpret_cast<const float4*>(kr + i), q4 = *reinterpret_cast<const float4*>(qr + i);
          S[i] = dec * S[i] + k4.x * vv;
          o0 += S[i] * q4.x;
          S[i + 1] = dec * S[i + 1] + k4.y * vv;
          o1 += S[i + 1] * q4.y;
          S[i + 2] = dec * S[i + 2] + k4.z * vv;
          o0 += S[i + 2] * q4.z;
          S[i + 3] = dec * S[i + 3] + k4.w * vv;
          o1 += S[i + 3] * q4.w;
        }
      } else {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          S[i] = dec * S[i] + kr[i] * vv;
          if (i & 1) {
            o1 += S[i] * qr[i];
          } else {
            o0 += S[i] * qr[i];
          }
        }
      }
      po[w][t][lane] = o0 + o1;
    }
    __syncthreads();
    for (int e = tid; e < nt * kWideCols; e += NT) {
      const int t = e / kWideCols, c = e - t * kWideCols;
      if (v0 + c < V) {
        float o = po[0][t][c];
#pragma unroll
        for (int ww = 1; ww < NW; ++ww) o += po[ww][t][c];
        out[(static_cast<int64_t>(t0 + t) * H + h) * V + v0 + c] = o;
      }
    }
    // the next group's staging writes qs / ks / vs / ds only; po is rewritten after its barrier
  }
  if (sp != nullptr && col < V) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = w * NR + i;
      if (d < D) sp[static_cast<int64_t>(d) * V + col] = S[i];
    }
  }
}

}  // namespace

namespace {

template <Form F>
int launch_linear(void* out, const void* qkv, long long stride, void* state, const void* decay, const void* cu_q,
                  const void* positions, const void* slots, int n_seqs, int H, int D, int V, int dt, const HeadIn& in,
                  hipStream_t stream) {
  if (D <= 256) {
    const dim3 wgrid(n_seqs * H, (V + kWideCols - 1) / kWideCols);
    const int nw = D > 64 ? 8 : 4;
    const int nr = (D + nw - 1) / nw;
#define PKM_LIGHTW(NR, NW)                                                                                          \
  PKM_DISPATCH(dt, E, lightning_wide_kernel<E, NR, NW, F><<<wgrid, 64 * NW, 0, stream>>>(                          \
                          static_cast<float*>(out), static_cast<const E*>(qkv), stride, static_cast<float*>(state), \
                          static_cast<const float*>(decay), static_cast<const int*>(cu_q),                          \
                          static_cast<const int*>(positions), static_cast<const int*>(slots), H, D, V, in))
    if (nw == 4) {
      if (nr <= 2) {
        PKM_LIGHTW(2, 4);
      } else if (nr <= 4) {
        PKM_LIGHTW(4, 4);
      } else if (nr <= 8) {
        PKM_LIGHTW(8, 4);
      } else {
        PKM_LIGHTW(16, 4);
      }
    } else if (nr <= 12) {
      PKM_LIGHTW(12, 8);
    } else if (nr <= 16) {
      PKM_LIGHTW(16, 8);
    } else if (nr <= 24) {
      PKM_LIGHTW(24, 8);
    } else {
      PKM_LIGHTW(32, 8);
    }
#undef PKM_LIGHTW
    return PK_CHECK_LAUNCH();
  }
  const dim3 grid(n_seqs * H, (V + kCols - 1) / kCols);
  const int chunk = max(1, min(kMaxChunk, 15360 / (2 * D + kCols + 2)));  // at most 60 KiB of LDS
  const size_t lds = static_cast<size_t>(chunk) * (2 * D + kCols + 2) * sizeof(float);
  // heads of more than 256 key coordinates (narrower ones took the wider form)
  PKM_DISPATCH(dt, E, lightning_kernel<E, 32, F><<<grid, 256, lds, stream>>>(
                          static_cast<float*>(out), static_cast<const E*>(qkv), stride, static_cast<float*>(state),
                          static_cast<const float*>(decay), static_cast<const int*>(cu_q),
                          static_cast<const int*>(positions), static_cast<const int*>(slots), H, D, V, chunk, in));
  return PK_CHECK_LAUNCH();
}

}  // namespace

// out [T, H, V] fp32; qkv [T, H*D | H*D | H*V] projections (row stride `stride` elements);
// state [slots, H, D, V] fp32; sequences 0..n_seqs-1 own tokens cu_q[s]..cu_q[s+1]-1.
PK_EXPORT int pkm_lightning_attention(void* out, const void* qkv, long long stride, void* state, const void* decay,
                                      const void* cu_q, const void* positions, const void* slots, int n_seqs, int T,
                                      int H, int D, int V, int num_decode, int dt, hipStream_t stream) {
  if (n_seqs <= 0 || T <= 0) return 0;
  if (D < 1 || D > 512 || V < 1) return -1;
  return launch_linear<kSilu>(out, qkv, stride, state, decay, cu_q, positions, slots, n_seqs, H, D, V, dt,
                              HeadIn{nullptr, 0, 0, nullptr, 1.f, nullptr, 0, 1, nullptr, nullptr, nullptr}, stream);
}

// the recurrence on plain projections: q and k turned by the position (table [rows, pairs, 2] fp32 or null), k
// times k_scale
PK_EXPORT int pkm_retention(void* out, const void* qkv, long long stride, void* state, const void* decay,
                            const void* table, int pairs, int rows, float k_scale, const void* cu_q,
                            const void* positions, const void* slots, int n_seqs, int T, int H, int D, int V, int dt,
                            hipStream_t stream) {
  if (n_seqs <= 0 || T <= 0) return 0;
  if (D < 1 || D > 512 || V < 1 || 2 * pairs > D || (table && (rows < 1 || pairs < 1))) return -1;
  return launch_linear<kTurned>(out, qkv, stride, state, decay, cu_q, positions, slots, n_seqs, H, D, V, dt,
                             HeadIn{static_cast<const float*>(table), pairs, rows, static_cast<const int*>(positions), k_scale,
                                    nullptr, 0, 1, nullptr, nullptr, nullptr},
                             stream);
}

// the step form: out [T, H, V] fp32; xbc [T, H*V | G*N | G*N] rows `stride` elements apart; dt [T, H] of the same element
// type, rows dt_stride apart; dt_bias, a_log, skip [H] fp32; state [slots, H, N, V] fp32
PK_EXPORT int pkm_step_scan(void* out, const void* xbc, long long stride, const void* dt, long long dt_stride, int G,
                            const void* dt_bias, const void* a_log, const void* skip, void* state, const void* cu_q,
                            const void* positions, const void* slots, int n_seqs, int T, int H, int N, int V, int dtype,
                            hipStream_t stream) {
  if (n_seqs <= 0 || T <= 0) return 0;
  if (N < 1 || N > 512 || V < 1 || G < 1 || H < 1 || H % G || !dt || !dt_bias || !a_log || !skip) return -1;
  if (stride < static_cast<long long>(H) * V + 2ll * G * N || dt_stride < H) return -1;
  return launch_linear<kStep>(out, xbc, stride, state, nullptr, cu_q, positions, slots, n_seqs, H, N, V, dtype,
                              HeadIn{nullptr, 0, 0, nullptr, 1.f, dt, dt_stride, G, static_cast<const float*>(dt_bias),
                                     static_cast<const float*>(a_log), static_cast<const float*>(skip)},
                              stream);
}
