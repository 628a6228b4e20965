// Kernels of the layer-spec layers whose mixer and feed-forward run side by side on their own norms of one
// stream (ops/seqmix.py): embedding with a learned row per position; the residual sum of both sublayers (scale
// vectors, a shared expert's weight, the chosen experts' weighted sum) with the next layer's Dynamic Tanh norms
// in the same pass; the gelu-gated unit; the router whose choice is corrected and limited to groups of experts;
// squared-ReLU experts with the shared expert of decode-sized steps; and the two ends of latent attention on
// decode-sized steps (queries through the key expansion + cache write, heads through the value expansion + gate).
//
// Storage is fp32 or bf16 (template T); the stream, norms, scales, router and rotation are fp32 in both.
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

// ---------------------------------------------------------------------------------- router
// Logits: one wave per (token, row of the router); the router may carry one row more than there are experts (a
// shared expert's gate).
template <typename T>
__global__ void __launch_bounds__(NT) route_logits_kernel(const T* __restrict__ h, int W, const float* __restrict__ router,
                                                          int E, float* __restrict__ z) {
  const size_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, e = blockIdx.y * (NT / 64) + (threadIdx.x >> 6);
  if (e >= E) return;
  const T* hr = h + t * W;
  const float* rr = router + (size_t)e * W;
  float acc = 0.f;
  if (W % 8 == 0) {
    for (int c = lane * 8; c < W; c += 64 * 8) {
      float a[8], r[8];
      load8<T>(hr + c, a);
      load8<float>(rr + c, r);
#pragma unroll
      for (int k = 0; k < 8; ++k) acc += a[k] * r[k];
    }
  } else {
    for (int c = lane; c < W; c += 64) acc += ldf<T>(hr + c) * rr[c];
  }
  acc = wave_sum(acc);
  if (lane == 0) z[t * E + e] = acc;
}

// One wave per token over its logits z [E + gate]: s = softmax over the experts, c = s + corr; a group (E / groups
// neighbours) is as good as its best c, experts outside the `keep` best groups (the lower group on a tie) leave
// the choice; the `top` largest c (the lower id on a tie) are chosen, weights s / (their sum + 1e-20) * scale.
// gate_w: sigmoid of the last logit.  LDS: s [E] | c [E] | group scores [groups].
__global__ void __launch_bounds__(64) route_grouped_kernel(const float* __restrict__ z, int E, int gate,
                                                           const float* __restrict__ corr, int groups, int keep, int top,
                                                           float scale, int* __restrict__ idx, float* __restrict__ wts,
                                                           float* __restrict__ gate_w) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float *s_s = smem, *c_s = smem + E, *g_s = smem + 2 * E;
  const size_t t = blockIdx.x;
  const int lane = threadIdx.x, size = E / groups;
  const float* zr = z + t * (E + gate);
  float mx = -INFINITY, sum = 0.f;
  for (int e = lane; e < E; e += 64) { s_s[e] = zr[e]; mx = fmaxf(mx, s_s[e]); }
  mx = wave_max(mx);
  for (int e = lane; e < E; e += 64) sum += expf(s_s[e] - mx);
  sum = wave_sum(sum);
  for (int e = lane; e < E; e += 64) {
    const float s = expf(s_s[e] - mx) / sum;
    s_s[e] = s;
    c_s[e] = s + (corr ? corr[e] : 0.f);
  }
  __syncthreads();
  if (groups > 1) {
    for (int g = lane; g < groups; g += 64) {
      float b = -INFINITY;
      for (int e = g * size; e < (g + 1) * size; ++e) b = fmaxf(b, c_s[e]);
      g_s[g] = b;
    }
    __syncthreads();
    for (int g = lane; g < groups; g += 64) {
      int better = 0;
      for (int o = 0; o < groups; ++o) better += g_s[o] > g_s[g] || (g_s[o] == g_s[g] && o < g);
      if (better >= keep)
        for (int e = g * size; e < (g + 1) * size; ++e) c_s[e] = -INFINITY;
    }
    __syncthreads();
  }
  float tot = 0.f, my_w = 0.f;
  int my_i = 0;                                              // lane k keeps the k-th choice
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int bi = E;
    for (int e = lane; e < E; e += 64)
      if (c_s[e] > best) { best = c_s[e]; bi = e; }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
    }
    if (bi >= E) bi = k;                                     // scores that compare with nothing (NaN): keep the ids in range
    const float s = s_s[bi];
    if (lane == k) { my_w = s; my_i = bi; }
    tot += s;
    __syncthreads();
    if (lane == 0) c_s[bi] = -INFINITY;
    __syncthreads();
  }
  if (lane < top) {
    idx[t * top + lane] = my_i;
    wts[t * top + lane] = my_w / (tot + 1e-20f) * scale;
  }
  if (gate && lane == 0) gate_w[t] = sigmoidf_(zr[E]);
}

// ---------------------------------------------------------------------------------- squared-ReLU experts
// dot product of a weight row with a vector in LDS by one wave (every lane gets the sum)
template <typename T>
__device__ __forceinline__ float wave_dot(const T* __restrict__ w, const float* v_s, int n, int lane) {
  float acc = 0.f;
  if (n % 8 == 0) {
#pragma unroll 2
    for (int c = lane * 8; c < n; c += 64 * 8) {
      float a[8];
      load8<T>(w + c, a);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc += a[e] * v_s[c + e];
    }
  } else {
    for (int c = lane; c < n; c += 64) acc += ldf<T>(w + c) * v_s[c];
  }
  return wave_sum(acc);
}

// Pairs p < rows * top are (token, choice) of the routed experts, pairs after them one per token of the shared
// expert (own weights and width).  UP: y = max(W_up h, 0)^2;  else out = W_down y.
template <typename T, bool UP>
__global__ void __launch_bounds__(NT) relu2_experts_kernel(const T* __restrict__ in, const T* __restrict__ in_sh,
                                                           const int* __restrict__ idx, int routed, int top,
                                                           const T* __restrict__ w, const T* __restrict__ w_sh, int W, int ff,
                                                           int sff, T* __restrict__ out, T* __restrict__ out_sh,
                                                           int rows_per_wg, int E) {
  extern __shared__ __attribute__((aligned(16))) float v_s[];
  const int pair = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const bool sh = pair >= routed;
  const int t = sh ? pair - routed : pair / top, f = sh ? sff : ff, K = UP ? W : f, R = UP ? f : W;
  const int r0 = blockIdx.y * rows_per_wg, r1 = min(R, r0 + rows_per_wg);
  if (r0 >= R) return;
  const T* src = UP ? in + (size_t)t * W : sh ? in_sh + (size_t)t * sff : in + (size_t)pair * ff;
  for (int c = tid; c < K; c += NT) v_s[c] = ldf<T>(src + c);
  __syncthreads();
  const T* wm = sh ? w_sh : w + (size_t)min(max(idx[pair], 0), E - 1) * ff * W;
  T* dst = sh ? out_sh + (size_t)t * R : out + (size_t)pair * R;
  for (int r = r0 + wave; r < r1; r += NT / 64) {
    float v = wave_dot<T>(wm + (size_t)r * K, v_s, K, lane);
    if constexpr (UP) { v = fmaxf(v, 0.f); v *= v; }
    if (lane == 0) stf<T>(dst + r, v);
  }
}

// ---------------------------------------------------------------------------------- latent attention, few tokens
// out_s[n] = sum_k x_s[k] M[k][n] (M row-major [K, N]) by the whole workgroup; red_s: 8 NT floats.  With N a
// multiple of 8 a thread takes 8 columns of every (NT / (N / 8))-th row and the shares are added up in order.
template <typename T>
__device__ __forceinline__ void vec_mat(const float* x_s, const T* __restrict__ M, int K, int N, float* out_s, float* red_s) {
  const int tid = threadIdx.x, cpr = N / 8;
  if (N % 8 == 0 && cpr <= NT) {
    const int ng = NT / cpr, g = tid / cpr, c = (tid % cpr) * 8;
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = 0.f;
    if (g < ng) {
#pragma unroll 4
      for (int k = g; k < K; k += ng) {
        float m[8];
        load8<T>(M + (size_t)k * N + c, m);
        const float xv = x_s[k];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += xv * m[e];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) red_s[g * N + c + e] = acc[e];
    }
    __syncthreads();
    for (int n = tid; n < N; n += NT) {
      float s = 0.f;
      for (int q = 0; q < ng; ++q) s += red_s[q * N + n];
      out_s[n] = s;
    }
  } else {
    for (int n = tid; n < N; n += NT) {
      float s = 0.f;
      for (int k = 0; k < K; ++k) s += x_s[k] * ldf<T>(M + (size_t)k * N + n);
      out_s[n] = s;
    }
  }
  __syncthreads();
}

// Workgroup (t, h < H): qc[t, h] = (sum_d q[t, h, d] uk[h, d, :]) | rotate(q[t, h, D : D + R]).  Workgroup (t, H): the
// cached row rms(u[c0 : c0 + kvr]) w | rotate(u[c0 + kvr : ..]).  LDS: x [max(D, 1)] | out [kvr] | shares [8 NT].
template <typename T>
__global__ void __launch_bounds__(NT) latent_expand_write_kernel(
    const T* __restrict__ u, int ld, int c0, const float* __restrict__ w, float eps, const T* __restrict__ q,
    const T* __restrict__ uk, const int* __restrict__ tok_seq, const int* __restrict__ tok_pos, const int* __restrict__ seq_slot,
    const int* __restrict__ ptab, int ptab_ld, const float* __restrict__ cs, T* __restrict__ pages, T* __restrict__ qc, int H,
    int D, int R, int kvr, int rot, int page) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  __shared__ float red[NT / 64];
  const int t = blockIdx.x, h = blockIdx.y, pos = tok_pos[t], tid = threadIdx.x;
  const float* c = cs ? cs + (size_t)pos * rot : nullptr;    // rot / 2 pairs of (cos, sin)
  auto turned = [&](const T* v, int d) {                     // coordinate d of the rotated R-vector v
    const float a = ldf<T>(v + d);
    if (d >= rot || !c) return a;
    const float o = ldf<T>(v + (d ^ 1)), co = c[d & ~1], si = c[(d & ~1) + 1];
    return (d & 1) ? a * co + o * si : a * co - o * si;
  };
  if (h == H) {
    const T* ur = u + (size_t)t * ld + c0;
    float ss = 0.f;
    for (int e = tid; e < kvr; e += NT) { const float v = ldf<T>(ur + e); ss += v * v; }
    const float r = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)kvr + eps);
    const int slot = seq_slot[tok_seq[t]];
    T* row = pages + ((size_t)ptab[(size_t)slot * ptab_ld + pos / page] * page + pos % page) * (kvr + R);
    for (int e = tid; e < kvr; e += NT) stf<T>(row + e, ldf<T>(ur + e) * r * w[e]);
    for (int e = tid; e < R; e += NT) stf<T>(row + kvr + e, turned(ur + kvr, e));
    return;
  }
  float *x_s = smem, *out_s = smem + D, *red_s = smem + D + kvr;
  const T* qr = q + ((size_t)t * H + h) * (D + R);
  T* dst = qc + ((size_t)t * H + h) * (kvr + R);
  for (int d = tid; d < D; d += NT) x_s[d] = ldf<T>(qr + d);
  __syncthreads();
  vec_mat<T>(x_s, uk + (size_t)h * D * kvr, D, kvr, out_s, red_s);
  for (int e = tid; e < kvr; e += NT) stf<T>(dst + e, out_s[e]);
  for (int e = tid; e < R; e += NT) stf<T>(dst + kvr + e, turned(qr + D, e));
}

// out[t, h] = (a[t, h] uv[h]) * sigmoid(gate[t, h])  (gate null: 1).  LDS: a [R] | out [Dv] | shares [8 NT]
template <typename T>
__global__ void __launch_bounds__(NT) head_expand_gate_kernel(const T* __restrict__ a, const T* __restrict__ uv,
                                                              const T* __restrict__ gate, int gate_ld, T* __restrict__ out,
                                                              int H, int R, int Dv) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float *x_s = smem, *out_s = smem + R, *red_s = smem + R + Dv;
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  for (int r = tid; r < R; r += NT) x_s[r] = ldf<T>(a + ((size_t)t * H + h) * R + r);
  __syncthreads();
  vec_mat<T>(x_s, uv + (size_t)h * R * Dv, R, Dv, out_s, red_s);
  for (int d = tid; d < Dv; d += NT) {
    float v = out_s[d];
    if (gate) v *= sigmoidf_(ldf<T>(gate + (size_t)t * gate_ld + h * Dv + d));
    stf<T>(out + ((size_t)t * H + h) * Dv + d, v);
  }
}

// out[t, h, d] = v[h, t, d] * sigmoid(gate[t, h Dv + d]): the batched product's layout back to rows, with the gate.
// C = 8 (Dv, gate_ld multiples of 8, aligned) or 1 columns per thread.
template <typename T, int C>
__global__ void __launch_bounds__(NT) heads_gate_kernel(const T* __restrict__ v, const T* __restrict__ gate, int gate_ld,
                                                        T* __restrict__ out, int rows, int H, int Dv) {
  const size_t t = blockIdx.x;
  const int HD = H * Dv;
  for (int e = (blockIdx.y * NT + threadIdx.x) * C; e < HD; e += gridDim.y * NT * C) {
    const int h = e / Dv, d = e % Dv;
    const T* src = v + ((size_t)h * rows + t) * Dv + d;
    if constexpr (C == 8) {
      float a[8], g[8];
      load8<T>(src, a);
      load8<T>(gate + t * gate_ld + e, g);
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] *= sigmoidf_(g[i]);
      store8<T>(out + t * HD + e, a);
    } else {
      stf<T>(out + t * HD + e, ldf<T>(src) * sigmoidf_(ldf<T>(gate + t * gate_ld + e)));
    }
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

// router: fp32 [E + gate, W]; z: fp32 scratch [rows, E + gate]
int edge_sm_moe_route_grouped(const void* h, int W, const float* router, int E, int gate, const float* corr, int groups,
                              int keep, int top, float scale, float* z, int* idx, float* wts, float* gate_w, int rows, int f32,
                              hipStream_t st) {
  if (rows == 0) return 0;
  if (E < 1 || groups < 1 || E % groups || keep < 1 || keep > groups || top < 1 || top > 64 || top > E / groups * keep ||
      E > 4096 || (gate && !gate_w))
    return -2;
  SM_T(f32, hipLaunchKernelGGL(route_logits_kernel<T>, dim3(rows, (E + gate + NT / 64 - 1) / (NT / 64)), dim3(NT), 0, st,
                               (const T*)h, W, router, E + gate, z));
  hipLaunchKernelGGL(route_grouped_kernel, dim3(rows), dim3(64), (size_t)(2 * E + groups) * 4, st, (const float*)z, E, gate,
                     corr, groups, keep, top, scale, idx, wts, gate_w);
  return (int)hipGetLastError();
}

// w_up [E, ff, W], w_down [E, W, ff]; sff > 0: the shared expert su [sff, W], sd [W, sff].  Scratch y [rows * top, ff]
// and ys [rows, sff]; out [rows * top, W], out_sh [rows, W]
int edge_sm_moe_experts_relu2(const void* h, int W, const int* idx, int top, const void* w_up, const void* w_down, int ff,
                              const void* su, const void* sd, int sff, void* y, void* ys, void* out, void* out_sh, int rows,
                              int E, int f32, hipStream_t st) {
  if (rows == 0) return 0;
  if (ff < 1 || W < 1 || (sff > 0 && (!su || !sd || !ys || !out_sh))) return -2;
  const int big = sff > ff ? sff : ff;
  if ((size_t)W * 4 > 60 * 1024 || (size_t)big * 4 > 60 * 1024) return -3;
  const int rpw = 16, routed = rows * top, pairs = routed + (sff > 0 ? rows : 0);
  SM_T(f32, hipLaunchKernelGGL((relu2_experts_kernel<T, true>), dim3(pairs, (big + rpw - 1) / rpw), dim3(NT), (size_t)W * 4, st,
                               (const T*)h, (const T*)h, idx, routed, top, (const T*)w_up, (const T*)su, W, ff, sff, (T*)y,
                               (T*)ys, rpw, E));
  SM_T(f32, hipLaunchKernelGGL((relu2_experts_kernel<T, false>), dim3(pairs, (W + rpw - 1) / rpw), dim3(NT), (size_t)big * 4,
                               st, (const T*)y, (const T*)ys, idx, routed, top, (const T*)w_down, (const T*)sd, W, ff, sff,
                               (T*)out, (T*)out_sh, rpw, E));
  return (int)hipGetLastError();
}

int edge_sm_latent_expand_write(const void* u, int ld, int c0, const float* w, float eps, const void* q, const void* uk,
                                const int* tok_seq, const int* tok_pos, const int* seq_slot, const int* ptab, int ptab_ld,
                                const float* cs, void* pages, void* qc, int rows, int H, int D, int R, int kvr, int rot, int page,
                                int f32, hipStream_t st) {
  if (rows == 0) return 0;
  if (rot % 2 || rot > R || (rot > 0 && !cs) || !u || !w) return -2;
  const size_t lds = sizeof(float) * ((size_t)D + kvr + 8 * NT);
  if (lds > 60 * 1024) return -3;
  SM_T(f32, hipLaunchKernelGGL(latent_expand_write_kernel<T>, dim3(rows, H + 1), dim3(NT), lds, st, (const T*)u, ld, c0, w, eps,
                               (const T*)q, (const T*)uk, tok_seq, tok_pos, seq_slot, ptab, ptab_ld, cs, (T*)pages, (T*)qc, H,
                               D, R, kvr, rot, page));
  return (int)hipGetLastError();
}

int edge_sm_head_expand_gate(const void* a, const void* uv, const void* gate, int gate_ld, void* out, int rows, int H, int R,
                             int Dv, int f32, hipStream_t st) {
  if (rows == 0) return 0;
  const size_t lds = sizeof(float) * ((size_t)R + Dv + 8 * NT);
  if (lds > 60 * 1024) return -3;
  SM_T(f32, hipLaunchKernelGGL(head_expand_gate_kernel<T>, dim3(rows, H), dim3(NT), lds, st, (const T*)a, (const T*)uv,
                               (const T*)gate, gate_ld, (T*)out, H, R, Dv));
  return (int)hipGetLastError();
}

int edge_sm_heads_gate(const void* v, const void* gate, int gate_ld, void* out, int rows, int H, int Dv, int f32,
                       hipStream_t st) {
  if (rows == 0 || H * Dv == 0) return 0;
  const bool vec = Dv % 8 == 0 && gate_ld % 8 == 0 && (((uintptr_t)v | (uintptr_t)gate | (uintptr_t)out) & 15) == 0;
  const int per = NT * (vec ? 8 : 1), gy = (H * Dv + per - 1) / per < 8 ? (H * Dv + per - 1) / per : 8;
  if (vec)
    SM_T(f32, hipLaunchKernelGGL((heads_gate_kernel<T, 8>), dim3(rows, gy), dim3(NT), 0, st, (const T*)v, (const T*)gate,
                                 gate_ld, (T*)out, rows, H, Dv));
  else
    SM_T(f32, hipLaunchKernelGGL((heads_gate_kernel<T, 1>), dim3(rows, gy), dim3(NT), 0, st, (const T*)v, (const T*)gate,
                                 gate_ld, (T*)out, rows, H, Dv));
  return (int)hipGetLastError();
}

}  // extern "C"
