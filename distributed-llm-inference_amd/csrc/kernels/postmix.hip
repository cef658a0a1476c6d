// Kernels of the post-norm stacks (models/mixers.py: PostNormLayer, MaskedAttention; ops/seqmix.py): embedding rows, the residual
// update with a norm of the sublayer's output, per-head q / k norm with half-split rotation and cache write, and the difference of
// two attention maps with its per-head norm.  (Chunk / window masks, kept tokens, soft cap and the fused two-map tiles are options of
// the attention kernels in seqmix.hip; the clamped activation of hypermix.hip's act_mul; the delta rule with channel decays is in
// gatemix.hip.)
//
// Arithmetic: the stream, norm statistics, rotation angles (double until reduced) and the maps' difference are fp32; activations
// between GEMMs are the template type A = float or bf16 (uint16_t bit pattern).
#include <algorithm>

#include "common.h"
#include "kernels.h"

namespace dli {

namespace {

constexpr int NT = 256;

template <typename A> __device__ __forceinline__ float ldf(const A* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf2f(*p); }
template <typename A> __device__ __forceinline__ void stf(A* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<uint16_t>(uint16_t* p, float v) { *p = f2bf(v); }

// V consecutive elements ↔ fp32: V = 4 one wide access (the launchers check alignment), V = 1 one element
template <int V, typename A> __device__ __forceinline__ void ldv(const A* p, float* d) {
  if constexpr (V == 1) {
    d[0] = ldf<A>(p);
  } else if constexpr (sizeof(A) == 4) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) d[j] = v[j];
  } else {
    const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) d[j] = bf2f((uint16_t)v[j]);
  }
}
template <int V, typename A> __device__ __forceinline__ void stv(A* p, const float* d) {
  if constexpr (V == 1) {
    stf<A>(p, d[0]);
  } else if constexpr (sizeof(A) == 4) {
    *reinterpret_cast<f32x4*>(p) = f32x4{d[0], d[1], d[2], d[3]};
  } else {
    bf16x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (short)f2bf(d[j]);
    *reinterpret_cast<bf16x4*>(p) = o;
  }
}

// x = scale · table[id] (fp32) and the same rounded to the table's type
template <typename A, int V>
__global__ __launch_bounds__(NT) void embed_rows_kernel(const int* __restrict__ ids, const A* __restrict__ table, int vocab, float scale,
                                                        int W, float* __restrict__ x, A* __restrict__ h) {
  const int64_t t = blockIdx.x;
  const int64_t id = min(max(ids[t], 0), vocab - 1);
  for (int c = threadIdx.x * V; c < W; c += NT * V) {
    float v[V];
    ldv<V>(table + id * W + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] *= scale;
    stv<V>(x + t * W + c, v);
    stv<V>(h + t * W + c, v);
  }
}

// x += y / rms(y) · (1 + w); out = x, or x / rms(x) · (1 + w2).  One workgroup per row; a thread re-reads only what it wrote itself.
template <typename Y, typename O, int V>
__global__ __launch_bounds__(NT) void post_norm_add_kernel(float* __restrict__ x, const Y* __restrict__ y, const float* __restrict__ w,
                                                           float eps, const float* __restrict__ w2, int W, O* __restrict__ out) {
  __shared__ float red[NT / 64];
  const int64_t t = blockIdx.x;
  const Y* yr = y + t * W;
  float* xr = x + t * W;
  float s = 0.f;
  for (int c = threadIdx.x * V; c < W; c += NT * V) {
    float v[V];
    ldv<V>(yr + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) s += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(block_sum<NT>(s, red) / (float)W + eps);
  s = 0.f;
  for (int c = threadIdx.x * V; c < W; c += NT * V) {
    float v[V], u[V], ww[V];
    ldv<V>(yr + c, v);
    ldv<V>(xr + c, u);
    ldv<V>(w + c, ww);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      u[j] += v[j] * inv * (1.f + ww[j]);
      s += u[j] * u[j];
    }
    stv<V>(xr + c, u);
    if (w2 == nullptr) stv<V>(out + t * W + c, u);
  }
  if (w2 == nullptr) return;
  const float inv2 = 1.f / sqrtf(block_sum<NT>(s, red) / (float)W + eps);
  for (int c = threadIdx.x * V; c < W; c += NT * V) {
    float u[V], ww[V];
    ldv<V>(xr + c, u);
    ldv<V>(w2 + c, ww);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] *= inv2 * (1.f + ww[j]);
    stv<V>(out + t * W + c, u);
  }
}

// One workgroup per token; groups of LP lanes (a power of two ≤ 64) take one query / key vector each: unit RMS, weight, rotation.  A
// lane's item is V pairs (i, i + half) or V entries past the rotated ones.  Queries leave ordered (key head, map, head of its group).
template <typename A, int V>
__global__ __launch_bounds__(NT) void head_norm_rope_cache_kernel(const A* __restrict__ proj, int64_t p_stride, const float* __restrict__ qw,
                                                                  const float* __restrict__ kw, float eps,
                                                                  const int* __restrict__ positions, const double* __restrict__ freq,
                                                                  int rot_dims, const int* __restrict__ slot_mapping,
                                                                  A* __restrict__ k_cache, A* __restrict__ v_cache, int H, int G, int D,
                                                                  int Dv, int maps, int LP, A* __restrict__ q) {
  extern __shared__ float sh[];                            // cos [half] | sin [half]
  const int64_t t = blockIdx.x;
  const int half = rot_dims >> 1, nq = H * maps, nv = (H + G) * maps;
  float* cs = sh;
  float* sn = sh + half;
  for (int i = threadIdx.x; i < half; i += NT) {
    const double two_pi = 6.283185307179586476925286766559;
    double a = (double)positions[t] * freq[i];
    a -= floor(a / two_pi) * two_pi;
    cs[i] = cosf((float)a);
    sn[i] = sinf((float)a);
  }
  __syncthreads();
  const int slot = slot_mapping[t];
  const A* row = proj + t * p_stride;
  const int lane = threadIdx.x & (LP - 1), first = threadIdx.x / LP, step = NT / LP;
  const int pairs = half / V, items = pairs + (D - rot_dims) / V;
  const int trips = (nv + step - 1) / step;                // every lane takes part in the reductions of every trip
  for (int r = 0; r < trips; ++r) {
    const int u = first + r * step;
    const bool live = u < nv;
    const A* p = row + (int64_t)min(u, nv - 1) * D;
    float ss = 0.f;
    for (int i = lane; i < items; i += LP) {
      float a[V], b[V];
      const int c = i < pairs ? i * V : rot_dims + (i - pairs) * V;
      ldv<V>(p + c, a);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += a[j] * a[j];
      if (i < pairs) {
        ldv<V>(p + c + half, b);
#pragma unroll
        for (int j = 0; j < V; ++j) ss += b[j] * b[j];
      }
    }
    for (int o = LP >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float inv = 1.f / sqrtf(ss / (float)D + eps);
    if (!live || (u >= nq && slot < 0)) continue;
    A* dst;
    const float* w;
    if (u < nq) {
      const int per = H / G, h = u / maps, m = u - h * maps, g = h / per;
      dst = q + (t * nq + (g * maps + m) * per + (h - g * per)) * D;
      w = qw;
    } else {
      dst = k_cache + ((int64_t)slot * (G * maps) + (u - nq)) * D;
      w = kw;
    }
    for (int i = lane; i < items; i += LP) {
      float a[V], b[V], ww[V];
      const int c = i < pairs ? i * V : rot_dims + (i - pairs) * V;
      ldv<V>(p + c, a);
      if (w != nullptr) ldv<V>(w + c, ww);
#pragma unroll
      for (int j = 0; j < V; ++j) a[j] *= w != nullptr ? inv * ww[j] : inv;
      if (i < pairs) {
        ldv<V>(p + c + half, b);
        if (w != nullptr) ldv<V>(w + c + half, ww);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const float y = w != nullptr ? b[j] * inv * ww[j] : b[j] * inv;
          b[j] = y * cs[c + j] + a[j] * sn[c + j];
          a[j] = a[j] * cs[c + j] - y * sn[c + j];
        }
        stv<V>(dst + c + half, b);
      }
      stv<V>(dst + c, a);
    }
  }
  if (slot < 0) return;
  const A* v = row + (int64_t)nv * D;
  for (int i = threadIdx.x * V; i < G * Dv; i += NT * V) {
    float a[V];
    ldv<V>(v + i, a);
    stv<V>(v_cache + (int64_t)slot * G * Dv + i, a);
  }
}

// a wave per (token, head): out = scale · d / rms(d), d = map 1 - lam · map 2; o [T][2H][Dv] ordered (key head, map, head of its group)
template <typename O, int V>
__global__ __launch_bounds__(NT) void map_combine_kernel(const float* __restrict__ o, const float* __restrict__ lam, float eps, float scale,
                                                         int rows, int H, int G, int Dv, const int* __restrict__ token_seq,
                                                         O* __restrict__ out, int64_t out_stride) {
  const int lane = threadIdx.x & 63;
  const int64_t i = (int64_t)blockIdx.x * (NT / 64) + (threadIdx.x >> 6);
  if (i >= (int64_t)rows * H) return;                      // whole waves
  const int64_t t = i / H;
  const int h = (int)(i - t * H), per = H / G, g = h / per;
  O* dst = out + t * out_stride + (int64_t)h * Dv;
  if (token_seq != nullptr && token_seq[t] < 0) {
    for (int e = lane; e < Dv; e += 64) stf<O>(dst + e, 0.f);
    return;
  }
  const float* a = o + (t * 2 * H + (int64_t)g * 2 * per + (h - g * per)) * Dv;
  const float* b = a + (int64_t)per * Dv;
  const float l = lam[0];
  float ss = 0.f;
  for (int e = lane * V; e < Dv; e += 64 * V) {
    float x[V], y[V];
    ldv<V>(a + e, x);
    ldv<V>(b + e, y);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += (x[j] - l * y[j]) * (x[j] - l * y[j]);
  }
  const float inv = scale / sqrtf(wave_sum(ss) / (float)Dv + eps);
  for (int e = lane * V; e < Dv; e += 64 * V) {
    float x[V], y[V];
    ldv<V>(a + e, x);
    ldv<V>(b + e, y);
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] = (x[j] - l * y[j]) * inv;
    stv<V>(dst + e, x);
  }
}

}  // namespace

// ================================================================================================ launchers
#define PM_BF16(flag, T, ...) \
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

void launch_pm_embed_rows(const int* ids, const void* table, bool bf16, int vocab, float scale, int rows, int W, float* x, void* h,
                          hipStream_t stream) {
  if (rows == 0) return;
#define PM_ER(V) \
  PM_BF16(bf16, A, hipLaunchKernelGGL((embed_rows_kernel<A, V>), dim3(rows), dim3(NT), 0, stream, ids, (const A*)table, vocab, scale, W, x, (A*)h))
  if (W % 4 == 0 && al16(table) && al16(x) && al16(h)) PM_ER(4);
  else PM_ER(1);
#undef PM_ER
}

void launch_pm_post_norm_add(float* x, const void* y, bool bf16, const float* w, float eps, const float* w2, int rows, int W, void* out,
                             bool out_bf16, hipStream_t stream) {
  if (rows == 0) return;
#define PM_PN(V)                                                                                                                      \
  PM_BF16(bf16, Y, PM_BF16(out_bf16, O, hipLaunchKernelGGL((post_norm_add_kernel<Y, O, V>), dim3(rows), dim3(NT), 0, stream, x, (const Y*)y, \
                                                           w, eps, w2, W, (O*)out)))
  if (W % 4 == 0 && al16(x) && al16(y) && al16(w) && al16(w2) && al16(out)) PM_PN(4);
  else PM_PN(1);
#undef PM_PN
}

void launch_pm_head_norm_rope_cache(const void* proj, bool bf16, int64_t p_stride, const float* qw, const float* kw, float eps,
                                    const int* positions, const double* freq, int rot_dims, const int* slot_mapping, void* k_cache,
                                    void* v_cache, int rows, int H, int G, int D, int Dv, int maps, void* q, hipStream_t stream) {
  if (rows == 0) return;
  const bool wide = D % 4 == 0 && rot_dims % 8 == 0 && (G * Dv) % 4 == 0 && p_stride % 4 == 0 && al16(proj) && al16(qw) && al16(kw) &&
                    al16(k_cache) && al16(v_cache) && al16(q);
  const int items = wide ? (D - rot_dims / 2) / 4 : D - rot_dims / 2;
  int LP = 1;
  while (LP < 64 && LP < items) LP <<= 1;
#define PM_HN(V)                                                                                                                        \
  PM_BF16(bf16, A, hipLaunchKernelGGL((head_norm_rope_cache_kernel<A, V>), dim3(rows), dim3(NT), std::max(rot_dims, 2) * sizeof(float), \
                                      stream, (const A*)proj, p_stride, qw, kw, eps, positions, freq, rot_dims, slot_mapping,           \
                                      (A*)k_cache, (A*)v_cache, H, G, D, Dv, maps, LP, (A*)q))
  if (wide) PM_HN(4);
  else PM_HN(1);
#undef PM_HN
}

void launch_pm_map_combine(const float* o, const float* lam, float eps, float scale, int rows, int H, int G, int Dv, const int* token_seq,
                           void* out, bool out_bf16, int64_t out_stride, hipStream_t stream) {
  if (rows == 0) return;
  const dim3 grid((unsigned)(((int64_t)rows * H + NT / 64 - 1) / (NT / 64)));
#define PM_MC(V)                                                                                                                        \
  PM_BF16(out_bf16, O, hipLaunchKernelGGL((map_combine_kernel<O, V>), grid, dim3(NT), 0, stream, o, lam, eps, scale, rows, H, G, Dv, token_seq, \
                                          (O*)out, out_stride))
  if (Dv % 4 == 0 && out_stride % 4 == 0 && al16(o) && al16(out)) PM_MC(4);
  else PM_MC(1);
#undef PM_MC
}

}  // namespace dli
