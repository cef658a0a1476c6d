// Kernels of the stacks with one tanh norm per layer and gated matrix states (models/mixers.py: SingleNormLayer, DeltaRule,
// MatrixMemory, StateSpace; ops/seqmix.py): the residual update fused with the tanh norm, the plain GELU of a feed-forward,
// exponential gates with a running maximum, and the recurrence itself — S ← a S + k uᵀ, o = Sᵀ q with a decay a and a weight per
// head and token — or a decay per key channel, acting on the rows of S — u = weight · v or, for the delta rule, weight · (v - Sᵀ k).  (The convolutions in front of it, rotation and
// cache write of the attention beside it and the norm / gate behind it are extensions of recurmix.hip and seqmix.hip.)
//
// Arithmetic: the stream, norms, gates, decays, the state and every product with it are fp32 (prefill blocks on the fp32 matrix
// cores); sums of log decays are double, so that differences of long sums keep their digits.  Activations between GEMMs are the
// template type A = float or bf16 (uint16_t bit pattern).
//
// Step metadata (int32, static device buffers): positions[T], query_start_loc[B+1], state_slots[B] (< 0: none), tile_seq / tile_q0
// (64-token prefill tiles), counts[2] / counts[3] = number of valid tiles / batch rows.
#include <algorithm>
#include <type_traits>
#include <utility>

#include "common.h"
#include "kernels.h"

namespace dli {

namespace {

constexpr int NT = 256;
constexpr int BT = 64;            // tokens per block of the recurrence (= the step's prefill tiles)
constexpr int BS = BT + 4;        // LDS row stride of [·][64] arrays: 16-byte reads of consecutive rows fall on different banks
constexpr int GM_STEP_MAX_D = 512;
constexpr int GM_BLOCK_MAX_D = 256;

template <typename A> __device__ __forceinline__ float ldf(const A* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf2f(*p); }
template <typename A> __device__ __forceinline__ void stf(A* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<uint16_t>(uint16_t* p, float v) { *p = f2bf(v); }

template <typename A> __device__ __forceinline__ f32x4 ld4(const A* p);
template <> __device__ __forceinline__ f32x4 ld4<float>(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
template <> __device__ __forceinline__ f32x4 ld4<uint16_t>(const uint16_t* p) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{bf2f((uint16_t)v[0]), bf2f((uint16_t)v[1]), bf2f((uint16_t)v[2]), bf2f((uint16_t)v[3])};
}
template <typename A> __device__ __forceinline__ void st4(A* p, f32x4 v);
template <> __device__ __forceinline__ void st4<float>(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
template <> __device__ __forceinline__ void st4<uint16_t>(uint16_t* p, f32x4 v) {
  bf16x4 o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = (short)f2bf(v[j]);
  *reinterpret_cast<bf16x4*>(p) = o;
}

// V = 4: one wide access, V = 1: one element
template <int V, typename A> __device__ __forceinline__ void ldv(const A* p, float* d) {
  if constexpr (V == 4) {
    const f32x4 v = ld4<A>(p);
    d[0] = v[0]; d[1] = v[1]; d[2] = v[2]; d[3] = v[3];
  } else {
    d[0] = ldf<A>(p);
  }
}
template <int V, typename A> __device__ __forceinline__ void stv(A* p, const float* d) {
  if constexpr (V == 4) st4<A>(p, f32x4{d[0], d[1], d[2], d[3]});
  else stf<A>(p, d[0]);
}

// D(16x16) += A(16x4) · B(4x16), fp32.  Lane l holds A[row l&15][k l>>4], B[k l>>4][col l&15], D[row 4(l>>4)+r][col l&15].
__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
// four of them over 16 consecutive k: lane group l>>4 supplies k = 4(l>>4)+j in step j on both sides
__device__ __forceinline__ f32x4 mfma_k16(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 4; ++j) c = mfma_f32(a[j], b[j], c);
  return c;
}

// ------------------------------------------------------------------------------------------------ residual update + tanh norm
// x += mult · (y + ½ (rms(l) · wl + rms(r) · wr)), out = tanh(alpha · x) · w + b; one workgroup per token when there is a pair
// (two row statistics), else a grid over elements
template <typename Y, typename O, int V, bool PAIR>
__global__ __launch_bounds__(NT) void residual_tanh_kernel(float* __restrict__ x, const Y* __restrict__ y, const Y* __restrict__ l,
                                                           const Y* __restrict__ r, const float* __restrict__ wl,
                                                           const float* __restrict__ wr, float mult, const float* __restrict__ alpha,
                                                           const float* __restrict__ w, const float* __restrict__ b, float eps, int rows,
                                                           int W, O* __restrict__ out) {
  __shared__ float red[NT / 64];
  const float al = alpha[0];
  auto one = [&](int64_t t, int c, float il, float ir) {
    float xv[V], u[V], v[V];
    ldv<V>(x + t * W + c, xv);
    if (PAIR || y != nullptr) {
      float add[V];
#pragma unroll
      for (int j = 0; j < V; ++j) add[j] = 0.f;
      if constexpr (PAIR) {
        float pl[V], pr[V];
        ldv<V>(l + t * W + c, pl);
        ldv<V>(r + t * W + c, pr);
        ldv<V>(wl + c, u);
        ldv<V>(wr + c, v);
#pragma unroll
        for (int j = 0; j < V; ++j) add[j] = 0.5f * (pl[j] * il * u[j] + pr[j] * ir * v[j]);
      }
      if (y != nullptr) {
        ldv<V>(y + t * W + c, u);
#pragma unroll
        for (int j = 0; j < V; ++j) add[j] += u[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) xv[j] += mult * add[j];
      stv<V>(x + t * W + c, xv);
    }
    ldv<V>(w + c, u);
    ldv<V>(b + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) xv[j] = tanhf(al * xv[j]) * u[j] + v[j];
    stv<V>(out + t * W + c, xv);
  };
  if constexpr (PAIR) {
    const int64_t t = blockIdx.x;
    float sl = 0.f, sr = 0.f;
    for (int c = threadIdx.x * V; c < W; c += NT * V) {
      float u[V];
      ldv<V>(l + t * W + c, u);
#pragma unroll
      for (int j = 0; j < V; ++j) sl += u[j] * u[j];
      ldv<V>(r + t * W + c, u);
#pragma unroll
      for (int j = 0; j < V; ++j) sr += u[j] * u[j];
    }
    const float il = 1.f / sqrtf(block_sum<NT>(sl, red) / (float)W + eps);
    const float ir = 1.f / sqrtf(block_sum<NT>(sr, red) / (float)W + eps);
    for (int c = threadIdx.x * V; c < W; c += NT * V) one(t, c, il, ir);
  } else {
    const int64_t n = (int64_t)rows * W / V;
    const int per = W / V;
    for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < n; i += (int64_t)gridDim.x * NT) {
      const int64_t t = i / per;
      one(t, (int)(i - t * per) * V, 0.f, 0.f);
    }
  }
}

// 0.5 z (1 + tanh(√(2/π) (z + 0.044715 z³))) = z · sigmoid(2 · …)
template <typename A, int V>
__global__ __launch_bounds__(NT) void gelu_rows_kernel(const A* __restrict__ x, int64_t x_stride, int rows, int F, A* __restrict__ out,
                                                       int64_t o_stride) {
  const int per = F / V;
  const int64_t n = (int64_t)rows * per;
  for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < n; i += (int64_t)gridDim.x * NT) {
    const int64_t t = i / per;
    const int c = (int)(i - t * per) * V;
    float v[V];
    ldv<V>(x + t * x_stride + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float z = v[j];
      v[j] = z * fast_rcp(1.f + fast_exp2(-1.4426950408889634f * 1.5957691216057308f * (z + 0.044715f * z * z * z)));
    }
    stv<V>(out + t * o_stride + c, v);
  }
}

// ------------------------------------------------------------------------------------------------ gates with a running maximum
// Per (sequence, head): i = cap · tanh((g_i + b_i) / cap), f = logsigmoid(cap · tanh((g_f + b_f) / cap)), m ← max(f + m, i); out:
// f + m_before - m, exp(i - m), exp(-m).  A workgroup takes NTH tokens at a time: max-plus prefix of (Σ f, max_j (i_j + Σ f after j))
// over lanes, waves and trips.
template <typename A, int NTH>
__global__ __launch_bounds__(NTH) void max_gates_kernel(const A* __restrict__ g, int64_t g_stride, const float* __restrict__ bias, float cap,
                                                        float* __restrict__ state, const int* __restrict__ positions,
                                                        const int* __restrict__ qsl, const int* __restrict__ state_slots,
                                                        const int* __restrict__ counts, int H, float* __restrict__ keep,
                                                        float* __restrict__ write, float* __restrict__ floor_) {
  __shared__ float wF[NTH / 64], wM[NTH / 64];
  const int seq = blockIdx.x, h = blockIdx.y;
  if (seq >= counts[3]) return;
  const int t0 = qsl[seq], t1 = qsl[seq + 1];
  const int slot = state_slots[seq];
  if (slot < 0 || t1 <= t0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const float bi = bias[h], bf = bias[H + h];
  float m0 = positions[t0] > 0 ? state[(int64_t)slot * H + h] : 0.f;
  for (int tb = t0; tb < t1; tb += NTH) {
    const int t = tb + threadIdx.x;
    const bool live = t < t1;
    float i = -INFINITY, f = 0.f;
    if (live) {
      i = cap * tanhf((ldf<A>(g + (int64_t)t * g_stride + h) + bi) / cap);
      const float z = cap * tanhf((ldf<A>(g + (int64_t)t * g_stride + H + h) + bf) / cap);
      f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
    }
    float F = f, M = i;                                    // inclusive prefix over the wave: m = max(F + m_start, M)
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float pF = __shfl_up(F, o, 64), pM = __shfl_up(M, o, 64);
      if (lane >= o) {
        M = fmaxf(pM + F, M);
        F += pF;
      }
    }
    if (lane == 63) {
      wF[wave] = F;
      wM[wave] = M;
    }
    __syncthreads();
    float ms = m0;                                         // maximum before this wave's first token
    for (int v = 0; v < wave; ++v) ms = fmaxf(wF[v] + ms, wM[v]);
    const float m = fmaxf(F + ms, M);
    float mp = __shfl_up(m, 1, 64);
    if (lane == 0) mp = ms;
    if (live) {
      const int64_t o = (int64_t)t * H + h;
      keep[o] = f + mp - m;
      write[o] = expf(i - m);
      floor_[o] = expf(-m);
    }
    for (int v = 0; v < NTH / 64; ++v) m0 = fmaxf(wF[v] + m0, wM[v]);      // dead lanes: (0, -inf) changes nothing
    __syncthreads();
  }
  if (threadIdx.x == 0) state[(int64_t)slot * H + h] = m0;
}

// ------------------------------------------------------------------------------------------------ recurrence
// state [slots][H][D · Dv (+ D)]: the [D][Dv] matrix of a head, then (normaliser) its vector n.

// Token by token: one workgroup per (sequence, head, 64 state columns); wave v keeps rows v·DR … of its lane's column in registers,
// the workgroup of the first columns also the normaliser.  Serves single tokens (and, with single_only = 0, whole chunks: sizes
// the block path does not take).
//
// Channel decays (Z, the type of z, not void; delta rule): g[d] = exp(-rate[h] · softplus(z[t, h, d] + bias[h, d])) instead of exp(decay).
template <typename Z> struct ChannelArgs {
  const Z* z;
  int64_t stride;
  const float *rate, *bias;
};
template <> struct ChannelArgs<void> {};
template <typename Z> __device__ __forceinline__ float channel_decay(float z, float rate);
template <> __device__ __forceinline__ float channel_decay<float>(float z, float rate) {
  return expf(-rate * (fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)))));
}
// bf16 projections: the hardware's exp2 / log2, the series of log1p where 1 + e would lose digits
template <> __device__ __forceinline__ float channel_decay<uint16_t>(float z, float rate) {
  const float e = fast_exp2(-1.4426950408889634f * fabsf(z));
  const float l = e < 0.0625f ? e * (1.f - e * (0.5f - e * (0.33333333f - e * (0.25f - e * 0.2f)))) : 0.6931471805599453f * __builtin_amdgcn_logf(1.f + e);
  return fast_exp2(-1.4426950408889634f * rate * (fmaxf(z, 0.f) + l));
}

template <typename A, int DRMAX, bool DELTA, typename Z>
__global__ __launch_bounds__(NT) void scan_step_kernel(const A* __restrict__ q, int64_t q_stride, const A* __restrict__ k, int64_t k_stride,
                                                       const A* __restrict__ v, int64_t v_stride, const float* __restrict__ decay,
                                                       const float* __restrict__ weight, float* __restrict__ state,
                                                       const int* __restrict__ positions, const int* __restrict__ qsl,
                                                       const int* __restrict__ state_slots, const int* __restrict__ counts, int H, int G,
                                                       int D, int Dv, float q_scale, float* __restrict__ out, float* __restrict__ nq,
                                                       int single_only, ChannelArgs<Z> ch) {
  constexpr bool CHAN = !std::is_void_v<Z>;
  __shared__ float qs[DRMAX * 4], ks[DRMAX * 4], gs[CHAN ? DRMAX * 4 : 1], red[4][64], red2[4][64], sred[NT / 64];
  const int h = blockIdx.x, seq = blockIdx.z;
  if (seq >= counts[3]) return;
  const int t0 = qsl[seq], t1 = qsl[seq + 1];
  const int slot = state_slots[seq];
  if (slot < 0 || t1 <= t0 || (single_only && t1 - t0 != 1)) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int e = blockIdx.y * 64 + lane;
  const bool active = e < Dv, norm = nq != nullptr && blockIdx.y == 0;
  const int g = h / (H / G);
  const int DR = (D + 3) >> 2, d0 = wave * DR, dn = min(DR, D - d0);
  float* head = state + ((int64_t)slot * H + h) * D * (Dv + (nq != nullptr ? 1 : 0));
  const bool carry = positions[t0] > 0;
  float S[DRMAX];
#pragma unroll
  for (int i = 0; i < DRMAX; ++i) S[i] = (carry && active && i < dn) ? head[(int64_t)(d0 + i) * Dv + e] : 0.f;
  constexpr int NN = (DRMAX * 4 + NT - 1) / NT;
  float nv[NN];
#pragma unroll
  for (int i = 0; i < NN; ++i) {
    const int d = threadIdx.x + NT * i;
    nv[i] = (norm && carry && d < D) ? head[(int64_t)D * Dv + d] : 0.f;
  }
  for (int t = t0; t < t1; ++t) {
    for (int d = threadIdx.x; d < D; d += NT) {
      qs[d] = ldf<A>(q + (int64_t)t * q_stride + g * D + d);
      ks[d] = ldf<A>(k + (int64_t)t * k_stride + g * D + d);
      if constexpr (CHAN) gs[d] = channel_decay<Z>(ldf<Z>(ch.z + (int64_t)t * ch.stride + (int64_t)h * D + d) + ch.bias[(int64_t)h * D + d], ch.rate[h]);
    }
    const float a = CHAN ? 1.f : expf(decay[(int64_t)t * H + h]), wt = weight[(int64_t)t * H + h];
    float ve = active ? ldf<A>(v + (int64_t)t * v_stride + (int64_t)h * Dv + e) : 0.f;
    __syncthreads();
    float seen = 0.f;
#pragma unroll
    for (int i = 0; i < DRMAX; ++i)
      if (i < dn) {
        S[i] *= CHAN ? gs[d0 + i] : a;
        if (DELTA) seen += S[i] * ks[d0 + i];
      }
    if (DELTA) {
      red[wave][lane] = seen;
      __syncthreads();
      ve -= (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]);
    }
    const float u = wt * ve;
    float o = 0.f;
#pragma unroll
    for (int i = 0; i < DRMAX; ++i)
      if (i < dn) {
        S[i] += ks[d0 + i] * u;
        o += S[i] * qs[d0 + i];
      }
    red2[wave][lane] = o;
    if (norm) {
      float p = 0.f;
#pragma unroll
      for (int i = 0; i < NN; ++i) {
        const int d = threadIdx.x + NT * i;
        if (d < D) {
          nv[i] = a * nv[i] + wt * ks[d];
          p += nv[i] * qs[d];
        }
      }
      p = block_sum<NT>(p, sred) * q_scale;
      if (threadIdx.x == 0) nq[(int64_t)t * H + h] = p;
    }
    __syncthreads();
    if (wave == 0 && active)
      out[((int64_t)t * H + h) * Dv + e] = ((red2[0][lane] + red2[1][lane]) + (red2[2][lane] + red2[3][lane])) * q_scale;
  }
#pragma unroll
  for (int i = 0; i < DRMAX; ++i)
    if (active && i < dn) head[(int64_t)(d0 + i) * Dv + e] = S[i];
#pragma unroll
  for (int i = 0; i < NN; ++i) {
    const int d = threadIdx.x + NT * i;
    if (norm && d < D) head[(int64_t)D * Dv + d] = nv[i];
  }
}

// Chunks of two tokens or more, in blocks of 64 tokens.  With P_t = Σ_{s ≤ t} decay_s inside the block and S0 the state at its start,
//   o_t = q_t · (exp(P_t) S0 + Σ_{j ≤ t} exp(P_t - P_j) k_j u_jᵀ),   S = exp(P_end) S0 + Σ_j exp(P_end - P_j) k_j u_jᵀ
// and u = w ⊙ v, or for the delta rule the solution of u_t = w_t (v_t - exp(P_t) S0ᵀ k_t - Σ_{j < t} exp(P_t - P_j) (k_t · k_j) u_j), i.e.
// U = (I + M)⁻¹ diag(w) (V - diag(exp P) K S0) with M strictly lower triangular.
//   scan_block_kernel: per (block, head), all blocks side by side: A = tril(exp(P_t - P_j) q_t · k_j), (I + M)⁻¹ and the vectors
//     exp(P), exp(P_end - P), w → workspace
//   scan_walk_kernel: per (sequence, head, 16·CT state columns) over its blocks in order, the state on the matrix cores' accumulators;
//     everything a block reads from memory is fetched while the block before it is computed (one register set: a fragment is
//     refilled as soon as it has been used).  The normaliser n = exp(P_end) n0 + Σ_j exp(P_end - P_j) w_j k_j and its product with q
//     ride on the fragments of the first columns' workgroup.
// Workspace row of a block = (first token >> 6) + batch row (unique: rows of later sequences start at later tokens): per head
// [64][64] A | delta: [64][64] (I + M)⁻¹ | [3][64] vectors.
template <bool DELTA> __host__ __device__ constexpr int64_t block_floats() { return (DELTA ? 2 : 1) * BT * BT + 3 * BT; }

// 4 consecutive entries of a row of D (zero past its end)
template <typename A> __device__ __forceinline__ f32x4 row4(const A* row, int d, int D, bool wide) {
  if (wide) return d < D ? ld4<A>(row + d) : f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 r;
#pragma unroll
  for (int j = 0; j < 4; ++j) r[j] = d + j < D ? ldf<A>(row + d + j) : 0.f;
  return r;
}

// one wave: column `lane` of (I + M)⁻¹ by forward substitution, rows of M [64][BS] (strictly lower part) broadcast from LDS
__device__ __forceinline__ void unit_lower_inverse(const float* M, float* __restrict__ wi, int lane) {
  float x[BT];
#pragma unroll
  for (int t = 0; t < BT; ++t) {
    float a0 = t == lane ? 1.f : 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
    for (int s = 0; s < t; s += 4) {
      const f32x4 m = *reinterpret_cast<const f32x4*>(M + t * BS + s);
      a0 -= m[0] * x[s];
      if (s + 1 < t) a1 -= m[1] * x[s + 1];
      if (s + 2 < t) a2 -= m[2] * x[s + 2];
      if (s + 3 < t) a3 -= m[3] * x[s + 3];
    }
    x[t] = (a0 + a1) + (a2 + a3);
    wi[t * BT + lane] = x[t];
  }
}
// sum over the four lane groups l>>4 (every lane gets it)
__device__ __forceinline__ float group_sum(float v) {
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}

template <typename A, bool DELTA>
__global__ __launch_bounds__(NT) void scan_block_kernel(const A* __restrict__ q, int64_t q_stride, const A* __restrict__ k, int64_t k_stride,
                                                        const float* __restrict__ decay, const float* __restrict__ weight,
                                                        const int* __restrict__ qsl, const int* __restrict__ state_slots,
                                                        const int* __restrict__ counts, const int* __restrict__ tile_seq,
                                                        const int* __restrict__ tile_q0, int num_tiles, int H, int G, int D, int wide,
                                                        float q_scale, float* __restrict__ ws) {
  __shared__ double P[BT];
  __shared__ float wt[BT];
  __shared__ __align__(16) float M[DELTA ? BT * BS : 4];
  const int tile = blockIdx.x, h = blockIdx.y;
  if (tile >= min(counts[2], num_tiles)) return;
  const int seq = tile_seq[tile];
  const int s0 = qsl[seq], s1 = qsl[seq + 1];
  if (s1 - s0 < 2 || state_slots[seq] < 0) return;        // single tokens belong to the step kernel
  const int t0 = s0 + tile_q0[tile];
  const int n = min(BT, s1 - t0);
  if (n <= 0) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g4 = lane >> 4, c = lane & 15;
  const int g = h / (H / G);
  float* wa = ws + ((int64_t)((t0 >> 6) + seq) * H + h) * block_floats<DELTA>();
  float* wi = wa + BT * BT;                               // delta: (I + M)⁻¹
  float* wv = wa + (DELTA ? 2 : 1) * BT * BT;             // exp(P) | exp(P_end - P) | w
  if (wave == 0) {
    double p = lane < n ? (double)decay[(int64_t)(t0 + lane) * H + h] : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double x = __shfl_up(p, o, 64);
      if (lane >= o) p += x;
    }
    const double end = __shfl(p, 63, 64);
    const float wl = lane < n ? weight[(int64_t)(t0 + lane) * H + h] : 0.f;
    P[lane] = p;
    wt[lane] = wl;
    wv[lane] = expf((float)p);
    wv[BT + lane] = expf((float)(end - p));
    wv[2 * BT + lane] = wl;
  }
  // rows 16·wave … of Q Kᵀ (and K Kᵀ) against the column tiles up to the diagonal; rows past the block repeat its last token
  auto row_of = [&](int i) { return (int64_t)(t0 + min(i, n - 1)); };
  f32x4 qk[4], kk[4];
#pragma unroll
  for (int s = 0; s < 4; ++s) qk[s] = kk[s] = f32x4{0.f, 0.f, 0.f, 0.f};
  const A* qr = q + row_of(16 * wave + c) * q_stride + g * D;
  const A* kr = k + row_of(16 * wave + c) * k_stride + g * D;
  const A* kc[4];
#pragma unroll
  for (int s = 0; s < 4; ++s) kc[s] = k + row_of(16 * s + c) * k_stride + g * D;
#pragma unroll 2
  for (int d0 = 0; d0 < D; d0 += 16) {
    const int d = d0 + 4 * g4;
    const f32x4 qa = row4(qr, d, D, wide);
    f32x4 ka;
    if (DELTA) ka = row4(kr, d, D, wide);
#pragma unroll
    for (int s = 0; s < 4; ++s)
      if (s <= wave) {
        const f32x4 kb = row4(kc[s], d, D, wide);
        qk[s] = mfma_k16(qa, kb, qk[s]);
        if (DELTA) kk[s] = mfma_k16(ka, kb, kk[s]);
      }
  }
  __syncthreads();
#pragma unroll
  for (int s = 0; s < 4; ++s)
    if (s <= wave) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * wave + 4 * g4 + r, col = 16 * s + c;
        const float f = col <= row ? expf((float)(P[row] - P[col])) : 0.f;
        wa[row * BT + col] = f * q_scale * qk[s][r];
        if (DELTA) M[row * BS + col] = col < row ? f * wt[row] * kk[s][r] : 0.f;
      }
    }
  if (!DELTA) return;
  __syncthreads();
  if (wave != 0) return;
  unit_lower_inverse(M, wi, lane);
}

// Channel decays.  With P_t[d] the log decays summed to token t inside the block, the same block form reads
//   o_t = (q_t ⊙ e^{P_t}) S0 + Σ_{j ≤ t} (Σ_d q_t[d] k_j[d] e^{P_t[d] - P_j[d]}) u_j,  S = e^{P_end} ⊙ S0 + Σ_j (k_j ⊙ e^{P_end - P_j}) u_jᵀ,
// and likewise with k_t for the system that u solves.  Every exponential here is a product of decays ≤ 1, never a quotient:
// wave w holds rows 16w … of the block as A fragments (lane c = token, 4 channels); L = product from the sub-block's first token
// through the lane's own, R = product from the next token to the sub-block's end, both prefix products over 16 lanes.  A sub-block
// of rows meets an earlier sub-block of columns as (q ⊙ L) · (k ⊙ R ⊙ totals of the sub-blocks between)ᵀ on the fp32 matrix cores;
// inside a sub-block, pairs at distance s use the running product of the s decays between them (lane rotations, no exponential).
// Workspace per (block, head): A [64][64] | (I + M)⁻¹ [64][64] | weights [64] | e^{P_end} [DP] | q ⊙ e^{P} [64][DP] |
// k ⊙ e^{P} [64][DP] | (k ⊙ e^{P_end - P})ᵀ [DP][64], DP = D rounded up to 16.
__host__ __device__ constexpr int64_t channel_block_floats(int DP) { return 2 * BT * BT + BT + DP + 3 * (int64_t)BT * DP; }

// value of the lane N below (ror: rotated within 16 lanes; shr / shl: `fill` where there is none)
template <int N> __device__ __forceinline__ float row_ror(float v) {
  if constexpr (N == 0) return v;
  else return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x120 + N, 0xf, 0xf, false));
}
template <int N> __device__ __forceinline__ float row_shr(float v, float fill) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(fill), __float_as_int(v), 0x110 + N, 0xf, 0xf, false));
}
template <int N> __device__ __forceinline__ float row_shl(float v, float fill) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(fill), __float_as_int(v), 0x100 + N, 0xf, 0xf, false));
}

// pairs (row c, column c - S) of a 16-token sub-block, S = 1 … 15: `e` holds the product of the S decays between them
template <int S>
__device__ __forceinline__ void near_pairs(const f32x4& q, const f32x4& k, const f32x4& g, f32x4& e, float* aq, float* ak) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    e[j] *= row_ror<S - 1>(g[j]);
    const float x = e[j] * row_ror<S>(k[j]);
    aq[S] += q[j] * x;
    ak[S] += k[j] * x;
  }
}
template <int... S>
__device__ __forceinline__ void all_near_pairs(std::integer_sequence<int, S...>, const f32x4& q, const f32x4& k, const f32x4& g, float* aq,
                                               float* ak) {
  f32x4 e = {1.f, 1.f, 1.f, 1.f};
  (near_pairs<S + 1>(q, k, g, e, aq, ak), ...);
}

template <typename Z>
__global__ __launch_bounds__(NT) void channel_block_kernel(const float* __restrict__ q, int64_t q_stride, const float* __restrict__ k,
                                                           int64_t k_stride, ChannelArgs<Z> ch, const float* __restrict__ weight,
                                                           const int* __restrict__ qsl, const int* __restrict__ state_slots,
                                                           const int* __restrict__ counts, const int* __restrict__ tile_seq,
                                                           const int* __restrict__ tile_q0, int num_tiles, int H, int G, int D, int wide,
                                                           float* __restrict__ ws) {
  __shared__ float wt[BT];
  __shared__ __align__(16) float M[BT * BS];
  __shared__ __align__(16) float KR[2][BT][20], EM[2][4][16];
  const int tile = blockIdx.x, h = blockIdx.y;
  if (tile >= min(counts[2], num_tiles)) return;
  const int seq = tile_seq[tile];
  const int s0 = qsl[seq], s1 = qsl[seq + 1];
  if (s1 - s0 < 2 || state_slots[seq] < 0) return;        // single tokens belong to the step kernel
  const int t0 = s0 + tile_q0[tile];
  const int n = min(BT, s1 - t0);
  if (n <= 0) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g4 = lane >> 4, c = lane & 15;
  const int g = h / (H / G), DP = (D + 15) & ~15;
  float* wa = ws + ((int64_t)((t0 >> 6) + seq) * H + h) * channel_block_floats(DP);
  float* wi = wa + BT * BT;
  float* we = wi + BT * BT + BT;                          // e^{P_end}
  float* wq = we + DP;
  float* wk = wq + BT * DP;
  float* wkt = wk + BT * DP;
  if (wave == 0) wt[lane] = wi[BT * BT + lane] = lane < n ? weight[(int64_t)(t0 + lane) * H + h] : 0.f;
  const int row = 16 * wave + c;
  const bool live = row < n;
  const int64_t tok = t0 + min(row, n - 1);               // rows past the block repeat its last token, with decay 1
  const float* qr = q + tok * q_stride + g * D;
  const float* kr = k + tok * k_stride + g * D;
  const Z* zr = ch.z + tok * ch.stride + (int64_t)h * D;
  const float* br = ch.bias + (int64_t)h * D;
  const float rate = ch.rate[h];
  f32x4 qk[3], kk[3];
#pragma unroll
  for (int s = 0; s < 3; ++s) qk[s] = kk[s] = f32x4{0.f, 0.f, 0.f, 0.f};
  float aq[16], ak[16];
#pragma unroll
  for (int s = 0; s < 16; ++s) aq[s] = ak[s] = 0.f;
  f32x4 qn = row4(qr, 4 * g4, D, wide), kn = row4(kr, 4 * g4, D, wide), zn = row4(zr, 4 * g4, D, wide), bn = row4(br, 4 * g4, D, wide);
  for (int d0 = 0, it = 0; d0 < D; d0 += 16, ++it) {
    const int d = d0 + 4 * g4, buf = it & 1;
    const f32x4 qc = qn, kc = kn, zc = zn, bc = bn;
    if (d0 + 16 < D) {                                    // the next channels are fetched while these are computed
      qn = row4(qr, d + 16, D, wide);
      kn = row4(kr, d + 16, D, wide);
      zn = row4(zr, d + 16, D, wide);
      bn = row4(br, d + 16, D, wide);
    }
    f32x4 gd, L, R, ql, kl, kR;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      gd[j] = live && d + j < D ? channel_decay<Z>(zc[j] + bc[j], rate) : 1.f;
      float p = gd[j];
      p *= row_shr<1>(p, 1.f);
      p *= row_shr<2>(p, 1.f);
      p *= row_shr<4>(p, 1.f);
      p *= row_shr<8>(p, 1.f);
      L[j] = p;
      float r = row_shl<1>(gd[j], 1.f);
      r *= row_shl<1>(r, 1.f);
      r *= row_shl<2>(r, 1.f);
      r *= row_shl<4>(r, 1.f);
      r *= row_shl<8>(r, 1.f);
      R[j] = r;
      ql[j] = qc[j] * p;
      kl[j] = kc[j] * p;
      kR[j] = kc[j] * r;
    }
    *reinterpret_cast<f32x4*>(&KR[buf][row][4 * g4]) = kR;
    if (c == 15) *reinterpret_cast<f32x4*>(&EM[buf][wave][4 * g4]) = L;
    __syncthreads();                                      // (the other buffer's readers are past the barrier before this one)
    f32x4 before = {1.f, 1.f, 1.f, 1.f}, behind = before;
#pragma unroll
    for (int b = 2; b >= 0; --b)
      if (b < wave) {                                     // `before`: totals of the sub-blocks between b and this one
        const f32x4 kb = *reinterpret_cast<const f32x4*>(&KR[buf][16 * b + c][4 * g4]);
        const f32x4 f = {kb[0] * before[0], kb[1] * before[1], kb[2] * before[2], kb[3] * before[3]};
        qk[b] = mfma_k16(ql, f, qk[b]);
        kk[b] = mfma_k16(kl, f, kk[b]);
        const f32x4 m = *reinterpret_cast<const f32x4*>(&EM[buf][b][4 * g4]);
#pragma unroll
        for (int j = 0; j < 4; ++j) before[j] *= m[j];
      }
#pragma unroll
    for (int b = 1; b < 4; ++b)
      if (b > wave) {
        const f32x4 m = *reinterpret_cast<const f32x4*>(&EM[buf][b][4 * g4]);
#pragma unroll
        for (int j = 0; j < 4; ++j) behind[j] *= m[j];
      }
    f32x4 oq, ok;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      oq[j] = ql[j] * before[j];
      ok[j] = kl[j] * before[j];
      wkt[(int64_t)(d + j) * BT + row] = kR[j] * behind[j];
      aq[0] += qc[j] * kc[j];
    }
    *reinterpret_cast<f32x4*>(wq + (int64_t)row * DP + d) = oq;
    *reinterpret_cast<f32x4*>(wk + (int64_t)row * DP + d) = ok;
    if (wave == 3 && c == 15)
      *reinterpret_cast<f32x4*>(we + d) = f32x4{L[0] * before[0], L[1] * before[1], L[2] * before[2], L[3] * before[3]};
    all_near_pairs(std::make_integer_sequence<int, 15>{}, qc, kc, gd, aq, ak);
  }
  // off-diagonal tiles
#pragma unroll
  for (int b = 0; b < 3; ++b)
    if (b < wave) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * wave + 4 * g4 + r, col = 16 * b + c;
        wa[i * BT + col] = qk[b][r];
        M[i * BS + col] = wt[i] * kk[b][r];
      }
    }
  // the diagonal tile: lane c's entry at distance s; the lanes that wrapped around hold nothing and clear the upper triangle
  const float wr = wt[row];
#pragma unroll
  for (int s = 0; s < 16; ++s) {
    const float x = group_sum(aq[s]), y = group_sum(ak[s]);
    if (g4 == (s & 3)) {
      const int col = 16 * wave + ((c - s) & 15);
      wa[row * BT + col] = c >= s ? x : 0.f;
      M[row * BS + col] = s > 0 && c >= s ? wr * y : 0.f;
    }
  }
  __syncthreads();
  if (wave == 0) unit_lower_inverse(M, wi, lane);
}

// fragments as they come from memory (converted where they are used, so that a fetch ahead does not wait for its data)
template <typename A> struct Raw;
template <> struct Raw<float> {
  using v4 = f32x4;
  static __device__ __forceinline__ f32x4 cvt(v4 v) { return v; }
};
template <> struct Raw<uint16_t> {
  using v4 = bf16x4;
  static __device__ __forceinline__ f32x4 cvt(v4 v) {
    return f32x4{bf2f((uint16_t)v[0]), bf2f((uint16_t)v[1]), bf2f((uint16_t)v[2]), bf2f((uint16_t)v[3])};
  }
};
template <typename A> __device__ __forceinline__ typename Raw<A>::v4 raw4(const A* row, int d, int D, bool wide) {
  typename Raw<A>::v4 r;
  if (wide) {
    if (d < D) return *reinterpret_cast<const typename Raw<A>::v4*>(row + d);
#pragma unroll
    for (int j = 0; j < 4; ++j) r[j] = 0;
    return r;
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) r[j] = d + j < D ? row[d + j] : A(0);
  return r;
}
// CHAN (delta rule, A = float): q, k and kᵀ come from the workspace with their channel decays in them (channel_block_kernel).
template <typename A, bool DELTA, int DTMAX, int CT, bool CHAN>
__global__ __launch_bounds__(NT) void scan_walk_kernel(const A* __restrict__ q, int64_t q_stride, const A* __restrict__ k, int64_t k_stride,
                                                       const A* __restrict__ v, int64_t v_stride, float* __restrict__ state,
                                                       const int* __restrict__ positions, const int* __restrict__ qsl,
                                                       const int* __restrict__ state_slots, const int* __restrict__ counts, int H, int G,
                                                       int D, int Dv, int wide, float q_scale, const float* __restrict__ ws,
                                                       float* __restrict__ out, float* __restrict__ nq) {
  extern __shared__ __align__(16) float sh[];
  __shared__ float wts[2][BT], ews[2][BT], ns[GM_BLOCK_MAX_D];       // (normaliser) w, exp(P_end - P) w, n at the block's start
  const int h = blockIdx.x, seq = blockIdx.z;                        // a head's column slices share an XCD (its q / k stay in one L2)
  if (seq >= counts[3]) return;
  const int s0 = qsl[seq], n = qsl[seq + 1] - s0;
  const int slot = state_slots[seq];
  if (slot < 0 || n < 2) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g4 = lane >> 4, c = lane & 15;
  const int g = h / (H / G);
  const int DT = (D + 15) >> 4, DS = DT * 16 + 4;
  constexpr int DW = (DTMAX + 3) / 4;                     // state row tiles per wave: wave, wave + 4, …
  float* St = sh;                                         // [16·CT columns][DS]: the state at the block's start
  float* Rt = St + 16 * CT * DS;                          // [columns][BS]: right-hand sides of the delta rule
  float* Ut = Rt + (DELTA ? 16 * CT * BS : 0);            // [columns][BS]: u
  float* Us = CHAN ? Ut : Ut + 16 * CT * BS;              // [columns][BS]: exp(P_end - P) u
  const int e0 = blockIdx.y * 16 * CT;
  const bool norm = !DELTA && nq != nullptr && blockIdx.y == 0;
  float* head = state + ((int64_t)slot * H + h) * D * (Dv + (nq != nullptr ? 1 : 0));
  const bool carry = positions[s0] > 0;
  const int blocks = (n + BT - 1) / BT;

  using R4 = typename Raw<A>::v4;
  R4 qf[DTMAX], kf[DELTA ? DTMAX : 1], kt[DW][4];
  A vf[CT][4];
  f32x4 ia[DELTA ? 4 : 1], aa[4], ep, er, wt;
  f32x4 pe4[CHAN ? DW : 1];                               // decay of this wave's state rows over the block
  float pend = 0.f, wl = 0.f, el = 0.f, epc = 0.f;
  const int DP = DT * 16;
  const int64_t bf = CHAN ? channel_block_floats(DP) : block_floats<DELTA>();
  auto base_of = [&](int b) { return ws + ((int64_t)(((s0 + BT * b) >> 6) + seq) * H + h) * bf; };
  auto fetch_rows = [&](int b) {                          // q (and k) rows 16·wave + c; rows past the chunk repeat its last token
    if constexpr (CHAN) {
      const float* wq = base_of(b) + 2 * BT * BT + BT + DP + (int64_t)(16 * wave + c) * DP + 4 * g4;
#pragma unroll
      for (int i = 0; i < DTMAX; ++i)
        if (i < DT) {
          qf[i] = ld4<float>(wq + 16 * i);
          kf[i] = ld4<float>(wq + (int64_t)BT * DP + 16 * i);
        }
      return;
    }
    const int64_t tr = s0 + min(BT * b + 16 * wave + c, n - 1);
    const A* qr = q + tr * q_stride + g * D;
    const A* kr = k + tr * k_stride + g * D;
#pragma unroll
    for (int i = 0; i < DTMAX; ++i)
      if (i < DT) {
        qf[i] = raw4<A>(qr, 16 * i + 4 * g4, D, wide);
        if (DELTA) kf[i] = raw4<A>(kr, 16 * i + 4 * g4, D, wide);
      }
  };
  auto fetch_values = [&](int b) {
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
      const int e = min(e0 + 16 * ct + c, Dv - 1);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        vf[ct][r] = v[(int64_t)(s0 + min(BT * b + 16 * wave + 4 * g4 + r, n - 1)) * v_stride + (int64_t)h * Dv + e];
    }
  };
  auto fetch_vectors = [&](int b) {
    if constexpr (CHAN) {
      const float* wv = base_of(b) + 2 * BT * BT;
      wt = ld4<float>(wv + 16 * wave + 4 * g4);
#pragma unroll
      for (int i = 0; i < DW; ++i)
        if (wave + 4 * i < DT) pe4[i] = ld4<float>(wv + BT + 16 * (wave + 4 * i) + 4 * g4);
      return;
    }
    const float* wv = base_of(b) + (DELTA ? 2 : 1) * BT * BT;
    ep = ld4<float>(wv + 16 * wave + 4 * g4);
    er = ld4<float>(wv + BT + 16 * wave + 4 * g4);
    wt = ld4<float>(wv + 2 * BT + 16 * wave + 4 * g4);
    pend = wv[BT - 1];
    if (norm) {
      wl = wv[2 * BT + lane];
      el = wv[BT + lane];
      epc = wv[16 * wave + c];
    }
  };
  auto fetch_inverse = [&](int b) {
    const float* wi = base_of(b) + BT * BT;
#pragma unroll
    for (int s = 0; s < 4; ++s)
      if (DELTA && s <= wave) ia[s] = ld4<float>(wi + (16 * wave + c) * BT + 16 * s + 4 * g4);
  };
  auto fetch_scores = [&](int b) {
    const float* wa = base_of(b);
#pragma unroll
    for (int s = 0; s < 4; ++s)
      if (s <= wave) aa[s] = ld4<float>(wa + (16 * wave + c) * BT + 16 * s + 4 * g4);
  };
  auto fetch_columns = [&](int b) {                       // kᵀ of this wave's state row tiles
    if constexpr (CHAN) {
      const float* wkt = base_of(b) + 2 * BT * BT + BT + DP + 2 * (int64_t)BT * DP + (int64_t)c * BT + 4 * g4;
#pragma unroll
      for (int i = 0; i < DW; ++i)
        if (wave + 4 * i < DT) {
#pragma unroll
          for (int s = 0; s < 4; ++s) kt[i][s] = ld4<float>(wkt + (int64_t)16 * (wave + 4 * i) * BT + 16 * s);
        }
      return;
    }
#pragma unroll
    for (int i = 0; i < DW; ++i)
      if (wave + 4 * i < DT) {
        const int d = min(16 * (wave + 4 * i) + c, D - 1);
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
          for (int j = 0; j < 4; ++j) kt[i][s][j] = k[(int64_t)(s0 + min(BT * b + 16 * s + 4 * g4 + j, n - 1)) * k_stride + g * D + d];
      }
  };
  fetch_rows(0);
  fetch_vectors(0);
  fetch_values(0);
  fetch_inverse(0);
  fetch_scores(0);
  fetch_columns(0);

  f32x4 S[DW][CT];
#pragma unroll
  for (int i = 0; i < DW; ++i)
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * (wave + 4 * i) + 4 * g4 + r, e = e0 + 16 * ct + c;
        S[i][ct][r] = (carry && d < D && e < Dv) ? head[(int64_t)d * Dv + e] : 0.f;
      }
  if (norm)
    for (int d = threadIdx.x; d < DT * 16; d += NT) ns[d] = (carry && d < D) ? head[(int64_t)D * Dv + d] : 0.f;

  for (int b = 0; b < blocks; ++b) {
    const int t0 = s0 + BT * b, nn = min(BT, n - BT * b);
    const bool more = b + 1 < blocks;
#pragma unroll
    for (int i = 0; i < DW; ++i)
      if (wave + 4 * i < DT)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) *reinterpret_cast<f32x4*>(St + (16 * ct + c) * DS + 16 * (wave + 4 * i) + 4 * g4) = S[i][ct];
    if (norm && wave == 0) {
      wts[b & 1][lane] = wl;
      ews[b & 1][lane] = wl * el;
    }
    lds_barrier();
    // rows 16·wave … of K S0 and Q S0
    f32x4 ks[CT], o[CT];
    float pn = 0.f;
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) ks[ct] = o[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < DTMAX; ++i)
      if (i < DT) {
        const int d = 16 * i + 4 * g4;
        const f32x4 qa = Raw<A>::cvt(qf[i]);
        f32x4 ka;
        if (DELTA) ka = Raw<A>::cvt(kf[i]);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          const f32x4 sb = *reinterpret_cast<const f32x4*>(St + (16 * ct + c) * DS + d);
          o[ct] = mfma_k16(qa, sb, o[ct]);
          if (DELTA) ks[ct] = mfma_k16(ka, sb, ks[ct]);
        }
        if (norm) pn += (qa[0] * ns[d] + qa[1] * ns[d + 1]) + (qa[2] * ns[d + 2] + qa[3] * ns[d + 3]);
      }
    if (more) fetch_rows(b + 1);
    f32x4 u[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float x = ldf<A>(&vf[ct][r]);
        if (CHAN) x -= ks[ct][r];
        else if (DELTA) x -= ep[r] * ks[ct][r];
        u[ct][r] = 16 * wave + 4 * g4 + r < nn ? wt[r] * x : 0.f;
        if (!CHAN) o[ct][r] *= ep[r] * q_scale;
      }
    }
    if (more) fetch_values(b + 1);
    if (DELTA) {
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        *reinterpret_cast<f32x4*>(Rt + (16 * ct + c) * BS + 16 * wave + 4 * g4) = u[ct];
        u[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
      }
      lds_barrier();
#pragma unroll
      for (int s = 0; s < 4; ++s)
        if (s <= wave) {
#pragma unroll
          for (int ct = 0; ct < CT; ++ct)
            u[ct] = mfma_k16(ia[s], *reinterpret_cast<const f32x4*>(Rt + (16 * ct + c) * BS + 16 * s + 4 * g4), u[ct]);
        }
      if (more) fetch_inverse(b + 1);
    }
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
      float* p = Ut + (16 * ct + c) * BS + 16 * wave + 4 * g4;
      *reinterpret_cast<f32x4*>(p) = u[ct];
      if (!CHAN) *reinterpret_cast<f32x4*>(p + (Us - Ut)) = f32x4{u[ct][0] * er[0], u[ct][1] * er[1], u[ct][2] * er[2], u[ct][3] * er[3]};
    }
    lds_barrier();
    float rs = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s)
      if (s <= wave) {
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
          o[ct] = mfma_k16(aa[s], *reinterpret_cast<const f32x4*>(Ut + (16 * ct + c) * BS + 16 * s + 4 * g4), o[ct]);
        if (norm) {
          const float* w4 = wts[b & 1] + 16 * s + 4 * g4;
          rs += (aa[s][0] * w4[0] + aa[s][1] * w4[1]) + (aa[s][2] * w4[2] + aa[s][3] * w4[3]);
        }
      }
    if (norm) {
      const float x = group_sum(epc * q_scale * pn + rs);
      if (g4 == 0 && 16 * wave + c < nn) nq[(int64_t)(t0 + 16 * wave + c) * H + h] = x;
    }
    const float pe = pend;
    if (CHAN)                                             // (before the next block's decays arrive)
#pragma unroll
      for (int i = 0; i < DW; ++i)
        if (wave + 4 * i < DT)
#pragma unroll
          for (int ct = 0; ct < CT; ++ct)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[i][ct][r] *= pe4[CHAN ? i : 0][r];
    if (more) {
      fetch_scores(b + 1);
      fetch_vectors(b + 1);
    }
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
      const int e = e0 + 16 * ct + c;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * wave + 4 * g4 + r;
        if (i < nn && e < Dv) out[((int64_t)(t0 + i) * H + h) * Dv + e] = o[ct][r];
      }
    }
    // S ← exp(P_end) S + Kᵀ (exp(P_end - P) u): this wave's row tiles, k running over the block's tokens
#pragma unroll
    for (int i = 0; i < DW; ++i)
      if (wave + 4 * i < DT) {
        const int d = 16 * (wave + 4 * i) + c;
        float kn = 0.f;
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (!CHAN) S[i][ct][r] *= pe;
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          f32x4 ka = Raw<A>::cvt(kt[i][s]);
          if (d >= D) ka = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ct = 0; ct < CT; ++ct)
            S[i][ct] = mfma_k16(ka, *reinterpret_cast<const f32x4*>(Us + (16 * ct + c) * BS + 16 * s + 4 * g4), S[i][ct]);
          if (norm) {
            const float* w4 = ews[b & 1] + 16 * s + 4 * g4;
            kn += (ka[0] * w4[0] + ka[1] * w4[1]) + (ka[2] * w4[2] + ka[3] * w4[3]);
          }
        }
        if (norm) {
          kn = group_sum(kn);
          if (g4 == 0) ns[d] = pe * ns[d] + kn;
        }
      }
    if (more) fetch_columns(b + 1);
  }
#pragma unroll
  for (int i = 0; i < DW; ++i) {
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * (wave + 4 * i) + 4 * g4 + r, e = e0 + 16 * ct + c;
        if (d < D && e < Dv) head[(int64_t)d * Dv + e] = S[i][ct][r];
      }
    const int d = 16 * (wave + 4 * i) + c;
    if (norm && g4 == 0 && d < D) head[(int64_t)D * Dv + d] = ns[d];
  }
}

}  // namespace

// ================================================================================================ launchers
#define GM_BF16(flag, T, ...) \
  do {                        \
    if (flag) {               \
      using T = uint16_t;     \
      __VA_ARGS__;            \
    } else {                  \
      using T = float;        \
      __VA_ARGS__;            \
    }                         \
  } while (0)

static bool al16(const void* p) { return p == nullptr || reinterpret_cast<uintptr_t>(p) % 16 == 0; }

void launch_gm_residual_tanh_norm(float* x, const void* y, const void* l, const void* r, bool bf16, const float* wl, const float* wr,
                                  float mult, const float* alpha, const float* w, const float* b, float eps, int rows, int W, void* out,
                                  bool out_bf16, hipStream_t stream) {
  if (rows == 0) return;
  const bool v4 = W % 4 == 0 && al16(x) && al16(y) && al16(l) && al16(r) && al16(wl) && al16(wr) && al16(w) && al16(b) && al16(out);
  const int64_t items = (int64_t)rows * W / (v4 ? 4 : 1);
  const dim3 flat((unsigned)std::min<int64_t>((items + NT - 1) / NT, 16384));
#define GM_RT(VV, PAIR, GRID)                                                                                                         \
  GM_BF16(bf16, Y, GM_BF16(out_bf16, O, hipLaunchKernelGGL((residual_tanh_kernel<Y, O, VV, PAIR>), GRID, dim3(NT), 0, stream, x,       \
                                                           (const Y*)y, (const Y*)l, (const Y*)r, wl, wr, mult, alpha, w, b, eps, rows, \
                                                           W, (O*)out)))
  if (l != nullptr) {
    if (v4) GM_RT(4, true, dim3(rows));
    else GM_RT(1, true, dim3(rows));
  } else {
    if (v4) GM_RT(4, false, flat);
    else GM_RT(1, false, flat);
  }
#undef GM_RT
}

void launch_gm_gelu_rows(const void* x, bool bf16, int64_t x_stride, int rows, int F, void* out, int64_t o_stride, hipStream_t stream) {
  if (rows == 0 || F == 0) return;
  const bool v4 = F % 4 == 0 && x_stride % 4 == 0 && o_stride % 4 == 0 && al16(x) && al16(out);
  const int64_t items = (int64_t)rows * F / (v4 ? 4 : 1);
  const dim3 grid((unsigned)std::min<int64_t>((items + NT - 1) / NT, 16384));
  if (v4) GM_BF16(bf16, A, hipLaunchKernelGGL((gelu_rows_kernel<A, 4>), grid, dim3(NT), 0, stream, (const A*)x, x_stride, rows, F, (A*)out, o_stride));
  else GM_BF16(bf16, A, hipLaunchKernelGGL((gelu_rows_kernel<A, 1>), grid, dim3(NT), 0, stream, (const A*)x, x_stride, rows, F, (A*)out, o_stride));
}

void launch_gm_max_gates(const void* g, bool bf16, int64_t g_stride, const float* bias, float cap, float* state, const int* positions,
                         const int* qsl, const int* state_slots, const int* counts, int seqs, int H, float* keep, float* write,
                         float* floor_, bool chunks, hipStream_t stream) {
  if (seqs == 0) return;
#define GM_MG(N)                                                                                                                   \
  GM_BF16(bf16, A, hipLaunchKernelGGL((max_gates_kernel<A, N>), dim3(seqs, H), dim3(N), 0, stream, (const A*)g, g_stride, bias, cap, \
                                      state, positions, qsl, state_slots, counts, H, keep, write, floor_))
  if (chunks) GM_MG(512);
  else GM_MG(64);
#undef GM_MG
}

int gm_step_max_dim() { return GM_STEP_MAX_D; }
int gm_block_max_dim() { return GM_BLOCK_MAX_D; }
int64_t gm_scan_ws_floats(int rows, int seqs, int H, bool delta) {
  return (int64_t)((rows >> 6) + seqs + 1) * H * (delta ? block_floats<true>() : block_floats<false>());
}

template <typename A, bool DELTA>
static void gated_scan(const A* q, int64_t q_stride, const A* k, int64_t k_stride, const A* v, int64_t v_stride, const float* decay,
                       const float* weight, float* state, const int* positions, const int* qsl, const int* state_slots,
                       const int* counts, int seqs, int H, int G, int D, int Dv, float q_scale, float* out, float* nq,
                       const int* tile_seq, const int* tile_q0, int num_tiles, float* ws, hipStream_t stream) {
  const bool blocks = num_tiles > 0 && ws != nullptr && D <= GM_BLOCK_MAX_D;
#define GM_STEP(DR)                                                                                                                   \
  hipLaunchKernelGGL((scan_step_kernel<A, DR, DELTA, void>), dim3(H, (Dv + 63) / 64, seqs), dim3(NT), 0, stream, q, q_stride, k, k_stride, \
                     v, v_stride, decay, weight, state, positions, qsl, state_slots, counts, H, G, D, Dv, q_scale, out, nq,           \
                     blocks ? 1 : 0, ChannelArgs<void>{})
  const int dr = (D + 3) / 4;
  if (dr <= 8) GM_STEP(8);
  else if (dr <= 16) GM_STEP(16);
  else if (dr <= 32) GM_STEP(32);
  else if (dr <= 64) GM_STEP(64);
  else GM_STEP(128);
#undef GM_STEP
  if (!blocks) return;
  const int wide = D % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && al16(q) && al16(k);     // 4 entries at a time
  hipLaunchKernelGGL((scan_block_kernel<A, DELTA>), dim3(num_tiles, H), dim3(NT), 0, stream, q, q_stride, k, k_stride, decay, weight, qsl,
                     state_slots, counts, tile_seq, tile_q0, num_tiles, H, G, D, wide, q_scale, ws);
  const int ct = H * ((Dv + 31) / 32) >= 128 ? 2 : 1;   // 32 state columns per workgroup where that still leaves enough of them
  const int DS = ((D + 15) / 16) * 16 + 4;
  const size_t lds = (size_t)16 * ct * (DS + (DELTA ? 3 : 2) * BS) * sizeof(float);
  const dim3 grid(H, (Dv + 16 * ct - 1) / (16 * ct), seqs);
#define GM_WALK(DT, CTV)                                                                                                               \
  hipLaunchKernelGGL((scan_walk_kernel<A, DELTA, DT, CTV, false>), grid, dim3(NT), lds, stream, q, q_stride, k, k_stride, v, v_stride, state,  \
                     positions, qsl, state_slots, counts, H, G, D, Dv, wide, q_scale, ws, out, nq)
#define GM_WALK_D(DT)          \
  do {                         \
    if (ct == 2) GM_WALK(DT, 2); \
    else GM_WALK(DT, 1);       \
  } while (0)
  if (D <= 64) GM_WALK_D(4);
  else if (D <= 128) GM_WALK_D(8);
  else GM_WALK_D(16);
#undef GM_WALK_D
#undef GM_WALK
}

void launch_gm_gated_scan(const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v, int64_t v_stride, bool bf16,
                          const float* decay, const float* weight, float* state, const int* positions, const int* qsl,
                          const int* state_slots, const int* counts, int seqs, int H, int G, int D, int Dv, bool delta, float q_scale,
                          bool normaliser, float* out, float* nq, const int* tile_seq, const int* tile_q0, int num_tiles, float* ws,
                          hipStream_t stream) {
  if (seqs == 0) return;
  if (!normaliser) nq = nullptr;
#define GM_SCAN(DELTA)                                                                                                                 \
  GM_BF16(bf16, A, (gated_scan<A, DELTA>((const A*)q, q_stride, (const A*)k, k_stride, (const A*)v, v_stride, decay, weight, state,     \
                                         positions, qsl, state_slots, counts, seqs, H, G, D, Dv, q_scale, out, nq, tile_seq,           \
                                         tile_q0, num_tiles, ws, stream)))
  if (delta) GM_SCAN(true);
  else GM_SCAN(false);
#undef GM_SCAN
}

int64_t gm_channel_ws_floats(int rows, int seqs, int H, int D) {
  return (int64_t)((rows >> 6) + seqs + 1) * H * channel_block_floats((D + 15) & ~15);
}

void launch_gm_channel_scan(const float* q, int64_t q_stride, const float* k, int64_t k_stride, const float* v, int64_t v_stride,
                            const void* z, bool z_bf16, int64_t z_stride, const float* rate, const float* bias, const float* weight,
                            float* state, const int* positions, const int* qsl, const int* state_slots, const int* counts, int seqs,
                            int H, int G, int D, int Dv, float* out, const int* tile_seq, const int* tile_q0, int num_tiles, float* ws,
                            hipStream_t stream) {
  if (seqs == 0) return;
  const bool blocks = num_tiles > 0 && ws != nullptr && D <= GM_BLOCK_MAX_D;
#define GM_STEP(DR)                                                                                                                    \
  GM_BF16(z_bf16, Z, hipLaunchKernelGGL((scan_step_kernel<float, DR, true, Z>), dim3(H, (Dv + 63) / 64, seqs), dim3(NT), 0, stream, q, q_stride, \
                                        k, k_stride, v, v_stride, (const float*)nullptr, weight, state, positions, qsl, state_slots,   \
                                        counts, H, G, D, Dv, 1.f, out, (float*)nullptr, blocks ? 1 : 0,                                \
                                        (ChannelArgs<Z>{(const Z*)z, z_stride, rate, bias})))
  const int dr = (D + 3) / 4;
  if (dr <= 8) GM_STEP(8);
  else if (dr <= 16) GM_STEP(16);
  else if (dr <= 32) GM_STEP(32);
  else if (dr <= 64) GM_STEP(64);
  else GM_STEP(128);
#undef GM_STEP
  if (!blocks) return;
  const int wide = D % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && z_stride % 4 == 0 && al16(q) && al16(k) && al16(z) && al16(bias);
  GM_BF16(z_bf16, Z, hipLaunchKernelGGL(channel_block_kernel<Z>, dim3(num_tiles, H), dim3(NT), 0, stream, q, q_stride, k, k_stride,
                                        (ChannelArgs<Z>{(const Z*)z, z_stride, rate, bias}), weight, qsl, state_slots, counts, tile_seq,
                                        tile_q0, num_tiles, H, G, D, wide, ws));
  const int ct = H * ((Dv + 31) / 32) >= 128 ? 2 : 1;   // 32 state columns per workgroup where that still leaves enough of them
  const int DS = ((D + 15) / 16) * 16 + 4;
  const size_t lds = (size_t)16 * ct * (DS + 2 * BS) * sizeof(float);
  const dim3 grid(H, (Dv + 16 * ct - 1) / (16 * ct), seqs);
#define GM_WALK(DT, CTV)                                                                                                                \
  hipLaunchKernelGGL((scan_walk_kernel<float, true, DT, CTV, true>), grid, dim3(NT), lds, stream, q, q_stride, k, k_stride, v, v_stride, state, \
                     positions, qsl, state_slots, counts, H, G, D, Dv, wide, 1.f, ws, out, (float*)nullptr)
#define GM_WALK_D(DT)          \
  do {                         \
    if (ct == 2) GM_WALK(DT, 2); \
    else GM_WALK(DT, 1);       \
  } while (0)
  if (D <= 64) GM_WALK_D(4);
  else if (D <= 128) GM_WALK_D(8);
  else GM_WALK_D(16);
#undef GM_WALK_D
#undef GM_WALK
}

}  // namespace dli
