// Kernels of the layer-spec layers whose mixer and feed-forward run side by side on their own norms of one
// stream (ops/seqmix.py): embedding with a learned row per position; the residual sum of both sublayers (scale
// vectors, a shared expert's weight, the chosen experts' weighted sum) with the next layer's Dynamic Tanh norms
// in the same pass; and the gelu-gated unit.
//
// Storage is fp32 or bf16 (template T); the stream, norms and scales are fp32 in both.
#include "common.h"
#include "seqmix/seqmix_common.h"

namespace {

// 4 consecutive elements (16 or 8 bytes)
template <typename T> __device__ __forceinline__ void load4(const T* p, float* f);
template <> __device__ __forceinline__ void load4<float>(const float* p, float* f) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
}
template <> __device__ __forceinline__ void load4<bf16_t>(const bf16_t* p, float* f) {
  const uint2 a = *reinterpret_cast<const uint2*>(p);
  f[0] = __uint_as_float(a.x << 16); f[1] = __uint_as_float(a.x & 0xffff0000u);
  f[2] = __uint_as_float(a.y << 16); f[3] = __uint_as_float(a.y & 0xffff0000u);
}
template <typename T> __device__ __forceinline__ void store4(T* p, const float* f);
template <> __device__ __forceinline__ void store4<float>(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
}
template <> __device__ __forceinline__ void store4<bf16_t>(bf16_t* p, const float* f) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(f[0], f[1]), pack_bf2(f[2], f[3]));
}
// C elements: 4 with wide accesses or 1
template <typename T, int C> __device__ __forceinline__ void loadc(const T* p, float* f) {
  if constexpr (C == 4) load4<T>(p, f);
  else f[0] = ldf<T>(p);
}
template <typename T, int C> __device__ __forceinline__ void storec(T* p, const float* f) {
  if constexpr (C == 4) store4<T>(p, f);
  else stf<T>(p, f[0]);
}

// ---------------------------------------------------------------------------------- embedding
template <typename T>
__global__ void __launch_bounds__(NT) embed_learned_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                           const T* __restrict__ pos_table, const int* __restrict__ tok_pos,
                                                           float* __restrict__ out, int W, int V, int positions) {
  const size_t t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);
  const int p = min(max(tok_pos[t], 0), positions - 1);
  for (int c = threadIdx.x; c < W; c += NT)
    out[t * W + c] = ldf<T>(table + (size_t)id * W + c) + ldf<T>(pos_table + (size_t)p * W + c);
}

// ---------------------------------------------------------------------------------- residual sum + next norms
struct UpdateArgs {
  const void* m;             // [rows, W] the mixer's output, or null
  const float* m_scale;      // [W], null: 1
  const void* y;             // [rows, W], or null
  const float* y_w;          // [rows], null: 1
  const void* parts;         // [rows * K, W], or null (K = 0)
  const float* part_w;       // [rows, K]
  const int* part_rows;      // [rows, K], null: row t K + k
  const float* f_scale;      // [W], null: 1
  const float* w[2];         // Dynamic Tanh norms of the new stream
  const float* b[2];
  const float* alpha[2];
  void* h[2];
  int K, part_total;         // part_total: rows of parts
};

// x += m_scale m + f_scale (y_w y + sum_k part_w[k] parts[k]);  h_i = tanh(alpha_i x) w_i + b_i, i < NN
template <typename T, int C, int NN>
__global__ void __launch_bounds__(NT) parallel_update_kernel(float* __restrict__ x, UpdateArgs a, int W) {
  const size_t t = blockIdx.x;
  const int c = (blockIdx.y * NT + threadIdx.x) * C;
  if (c >= W) return;
  float v[C], f[C];
  loadc<float, C>(x + t * W + c, v);
  const bool ff = a.y || a.K > 0;
  if (a.m) {
    loadc<T, C>((const T*)a.m + t * W + c, f);
    if (a.m_scale) {
      float s[C];
      loadc<float, C>(a.m_scale + c, s);
#pragma unroll
      for (int i = 0; i < C; ++i) f[i] *= s[i];
    }
#pragma unroll
    for (int i = 0; i < C; ++i) v[i] += f[i];
  }
  if (ff) {
#pragma unroll
    for (int i = 0; i < C; ++i) f[i] = 0.f;
    if (a.y) {
      loadc<T, C>((const T*)a.y + t * W + c, f);
      const float g = a.y_w ? a.y_w[t] : 1.f;
#pragma unroll
      for (int i = 0; i < C; ++i) f[i] *= g;
    }
#pragma unroll 4
    for (int k = 0; k < a.K; ++k) {
      const size_t r = a.part_rows ? (size_t)min(max(a.part_rows[t * a.K + k], 0), a.part_total - 1) : t * a.K + k;
      const float g = a.part_w[t * a.K + k];
      float p[C];
      loadc<T, C>((const T*)a.parts + r * W + c, p);
#pragma unroll
      for (int i = 0; i < C; ++i) f[i] += g * p[i];
    }
    if (a.f_scale) {
      float s[C];
      loadc<float, C>(a.f_scale + c, s);
#pragma unroll
      for (int i = 0; i < C; ++i) f[i] *= s[i];
    }
#pragma unroll
    for (int i = 0; i < C; ++i) v[i] += f[i];
  }
  if (a.m || ff) storec<float, C>(x + t * W + c, v);
#pragma unroll
  for (int n = 0; n < NN; ++n) {
    float w[C], b[C], h[C];
    const float al = a.alpha[n][0];
    loadc<float, C>(a.w[n] + c, w);
    loadc<float, C>(a.b[n] + c, b);
#pragma unroll
    for (int i = 0; i < C; ++i) h[i] = tanhf(al * v[i]) * w[i] + b[i];
    storec<T, C>((T*)a.h[n] + t * W + c, h);
  }
}

// ---------------------------------------------------------------------------------- gelu-gated unit
// gelu(g) = g / (1 + e^{-2 s}), s = sqrt(2 / pi) (g + 0.044715 g^3): the tanh form, 0.5 (1 + tanh s) = 1 / (1 + e^{-2 s})
__device__ __forceinline__ float gelu_tanh_f(float g) {
  const float s = 0.7978845608028654f * (g + 0.044715f * g * g * g);
  return g * sigmoidf_(2.f * s);
}

template <typename T, bool VEC>
__global__ void __launch_bounds__(NT) glu_gelu_kernel(const T* __restrict__ u, int ld, T* __restrict__ y, int ff) {
  const size_t t = blockIdx.x;
  if constexpr (VEC) {
    const int c = (blockIdx.y * NT + threadIdx.x) * 8;
    if (c >= ff) return;
    float g[8], p[8];
    load8<T>(u + t * ld + c, g);
    load8<T>(u + t * ld + ff + c, p);
#pragma unroll
    for (int i = 0; i < 8; ++i) g[i] = gelu_tanh_f(g[i]) * p[i];
    store8<T>(y + t * ff + c, g);
  } else {
    for (int c = blockIdx.y * NT + threadIdx.x; c < ff; c += NT * gridDim.y)
      stf<T>(y + t * ff + c, gelu_tanh_f(ldf<T>(u + t * ld + c)) * ldf<T>(u + t * ld + ff + c));
  }
}

}  // namespace

#define SM_T(f32, ...)                                  \
  do {                                                  \
    if (f32) { using T = float; __VA_ARGS__; }          \
    else { using T = bf16_t; __VA_ARGS__; }             \
  } while (0)

extern "C" {

int edge_sm_embed_learned(const int64_t* ids, const void* table, const void* pos_table, const int* tok_pos, float* out, int rows,
                          int W, int V, int positions, int f32, hipStream_t st) {
  if (rows == 0) return 0;
  if (V < 1 || positions < 1) return -2;
  SM_T(f32, hipLaunchKernelGGL(embed_learned_kernel<T>, dim3(rows), dim3(NT), 0, st, ids, (const T*)table, (const T*)pos_table,
                               tok_pos, out, W, V, positions));
  return (int)hipGetLastError();
}

// norms: nn <= 2 Dynamic Tanh norms as (w, b, alpha) pointers; h: their outputs
int edge_sm_parallel_update(float* x, const void* m, const float* m_scale, const void* y, const float* y_w, const void* parts,
                            const float* part_w, const int* part_rows, int K, int part_total, const float* f_scale,
                            const float* const* norms, void* const* h, int nn, int rows, int W, int f32, hipStream_t st) {
  if (rows == 0 || W == 0) return 0;
  if (nn < 0 || nn > 2 || (K > 0 && (!parts || !part_w || part_total < 1))) return -2;
  UpdateArgs a{m, m_scale, y, y_w, parts, part_w, part_rows, f_scale, {}, {}, {}, {}, parts ? K : 0, part_total};
  uintptr_t al = (uintptr_t)x | (uintptr_t)m | (uintptr_t)m_scale | (uintptr_t)y | (uintptr_t)parts | (uintptr_t)f_scale;
  for (int i = 0; i < nn; ++i) {
    a.w[i] = norms[3 * i]; a.b[i] = norms[3 * i + 1]; a.alpha[i] = norms[3 * i + 2]; a.h[i] = h[i];
    al |= (uintptr_t)a.w[i] | (uintptr_t)a.b[i] | (uintptr_t)a.h[i];
  }
  const bool vec = W % 4 == 0 && (al & 15) == 0;
  const int per = NT * (vec ? 4 : 1);
  const dim3 grid(rows, (W + per - 1) / per);
#define SM_PU(C, NN) SM_T(f32, hipLaunchKernelGGL((parallel_update_kernel<T, C, NN>), grid, dim3(NT), 0, st, x, a, W))
  if (vec) { if (nn == 0) SM_PU(4, 0); else if (nn == 1) SM_PU(4, 1); else SM_PU(4, 2); }
  else { if (nn == 0) SM_PU(1, 0); else if (nn == 1) SM_PU(1, 1); else SM_PU(1, 2); }
#undef SM_PU
  return (int)hipGetLastError();
}

int edge_sm_glu_gelu(const void* u, int ld, void* y, int rows, int ff, int f32, hipStream_t st) {
  if (rows == 0 || ff == 0) return 0;
  if (ff % 8 == 0 && ld % 8 == 0 && (((uintptr_t)u | (uintptr_t)y) & 31) == 0)
    SM_T(f32, hipLaunchKernelGGL((glu_gelu_kernel<T, true>), dim3(rows, (ff / 8 + NT - 1) / NT), dim3(NT), 0, st, (const T*)u,
                                 ld, (T*)y, ff));
  else
    SM_T(f32, hipLaunchKernelGGL((glu_gelu_kernel<T, false>), dim3(rows, (ff + NT * 4 - 1) / (NT * 4)), dim3(NT), 0, st,
                                 (const T*)u, ld, (T*)y, ff));
  return (int)hipGetLastError();
}

}  // extern "C"
