// Linear attention with one fixed decay d per head over a ragged step (ops/seqmix.py::decay_linear_attention):
//   S_t = d S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t,
// u row (from the mixer's first column) = q [H, N] | k [H, N] | v [H, P] | g [H, P]; q, k, v optionally through silu, the
// first coordinates of q and k optionally turned by their position (coordinate i with i + rot / 2), k times a constant;
// o over its root mean square per head or over all heads together, times a weight, times silu(g) or sigmoid(g).
//
// Two forms.  Short portions (decode): one workgroup per (sequence, head, value columns) steps token by token.  Long
// portions: chunks of 64 tokens in parallel, a chunk's first token being number 1:
//   S_t = d^t S_in + sum_{s<=t} d^(t-s) k_s v_s^T
//   o_t = d^t S_in^T q_t + sum_{s<=t} d^(t-s) (q_t . k_s) v_s
// (1) every chunk's own contribution to its end state, (2) the states at the chunk borders, (3) the outputs.  No power is
// negative, so strong decays only underflow.  The norm over a head and the gate are part of the output kernels while a
// workgroup holds the whole head (P <= 128); wider heads and the norm over all heads follow in row_norm_gate_kernel.
//
// Storage of u / out is fp32 or bf16 (template T); everything between them is fp32 (the tile products run on
// v_mfma_f32_16x16x4_f32).  State rows live per slot and are taken as zero by a portion that starts at position 0.
#include "common.h"
#include "seqmix/seqmix_common.h"

namespace {

struct DecayIn {
  const float* dec;          // [2, H]: decays, their log2
  const float* cs;           // [positions, rot / 2, 2] (cos, sin), null: nothing is turned
  int ld, H, N, P, rot, silu;
  float k_scale;
};

struct DecayOut {
  const float* norm_w;       // [P] (one head) or [H P] (all heads), null: 1
  int ld, gate_silu;         // row stride of out
  float eps, scale;
};

// coordinate n of a head's q or k row
template <typename T>
__device__ __forceinline__ float qk_elem(const T* __restrict__ row, int n, const DecayIn& a, const float* __restrict__ cs) {
  float v = ldf<T>(row + n);
  if (a.silu) v = siluf_(v);
  if (n < a.rot) {
    const int half = a.rot >> 1, i = n < half ? n : n - half;
    float o = ldf<T>(row + (n < half ? n + half : n - half));
    if (a.silu) o = siluf_(o);
    v = n < half ? v * cs[2 * i] - o * cs[2 * i + 1] : v * cs[2 * i] + o * cs[2 * i + 1];
  }
  return v;
}

// eight coordinates (n, rot / 2 and the row's alignment: multiples of 8)
template <typename T>
__device__ __forceinline__ void qk_elem8(const T* __restrict__ row, int n, const DecayIn& a, const float* __restrict__ cs, float* v) {
  load8<T>(row + n, v);
  if (a.silu) {
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = siluf_(v[k]);
  }
  if (n < a.rot) {
    const int half = a.rot >> 1, i = n < half ? n : n - half;
    float o[8], tab[16];
    load8<T>(row + (n < half ? n + half : n - half), o);
    load8<float>(cs + 2 * i, tab);
    load8<float>(cs + 2 * i + 8, tab + 8);
    if (a.silu) {
#pragma unroll
      for (int k = 0; k < 8; ++k) o[k] = siluf_(o[k]);
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = n < half ? v[k] * tab[2 * k] - o[k] * tab[2 * k + 1] : v[k] * tab[2 * k] + o[k] * tab[2 * k + 1];
  }
}

__device__ __forceinline__ float gate_f(float g, int silu) { return silu ? siluf_(g) : sigmoidf_(g); }

// ---------------------------------------------------------------------------------- token by token
// One workgroup of NW waves per (sequence, head, 64 CG value columns): lane = column, wave w keeps the state rows
// n = w, w + NW, .. (NRW of them) of its columns in registers; TC tokens are staged at a time, the waves' partial
// sums of o are added up per staged group.  FUSE: all columns of the head are here, so the norm and the gate follow.
template <typename T, int NW, int NRW, int CG, bool FUSE>
__global__ void __launch_bounds__(64 * NW) decay_step_kernel(
    const T* __restrict__ u, DecayIn a, float* __restrict__ state, const int* __restrict__ seq_slot,
    const int* __restrict__ seq_start, const int* __restrict__ seq_len, const int* __restrict__ seq_off, DecayOut po,
    T* __restrict__ out, float* __restrict__ y) {
  constexpr int TH = 64 * NW, TC = 8, CW = 64 * CG, NMAX = NW * NRW;
  __shared__ float q_s[TC][NMAX], k_s[TC][NMAX], part_s[TC][NW][CW];
  const int s = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * CW, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int N = a.N, P = a.P, HN = a.H * N, HP = a.H * P, v0 = 2 * HN, g0 = v0 + HP;
  const int start = seq_start[s], len = seq_len[s], off = seq_off[s];
  const float d = a.dec[h];
  float* st = state + ((size_t)seq_slot[s] * a.H + h) * N * P;
  float S[NRW][CG];
#pragma unroll
  for (int i = 0; i < NRW; ++i)
#pragma unroll
    for (int j = 0; j < CG; ++j) {
      const int n = wave + NW * i, p = p0 + lane + 64 * j;
      S[i][j] = (start > 0 && n < N && p < P) ? st[(size_t)n * P + p] : 0.f;
    }
  for (int t0 = 0; t0 < len; t0 += TC) {
    const int tc = min(TC, len - t0);
    for (int e = tid; e < tc * N; e += TH) {
      const int tt = e / N, n = e % N;
      const T* row = u + (size_t)(off + t0 + tt) * a.ld + h * N;
      const float* cs = a.cs ? a.cs + (size_t)(start + t0 + tt) * a.rot : nullptr;
      q_s[tt][n] = qk_elem<T>(row, n, a, cs);
      k_s[tt][n] = qk_elem<T>(row + HN, n, a, cs) * a.k_scale;
    }
    __syncthreads();
    for (int tt = 0; tt < tc; ++tt) {
      const T* row = u + (size_t)(off + t0 + tt) * a.ld + v0 + h * P;
      float v[CG], o[CG];
#pragma unroll
      for (int j = 0; j < CG; ++j) {
        const int p = p0 + lane + 64 * j;
        v[j] = p < P ? ldf<T>(row + p) : 0.f;
        if (a.silu) v[j] = siluf_(v[j]);
        o[j] = 0.f;
      }
#pragma unroll
      for (int i = 0; i < NRW; ++i) {
        const int n = wave + NW * i;
        if (n < N) {
          const float kv = k_s[tt][n], qv = q_s[tt][n];
#pragma unroll
          for (int j = 0; j < CG; ++j) {
            S[i][j] = d * S[i][j] + kv * v[j];
            o[j] += S[i][j] * qv;
          }
        }
      }
#pragma unroll
      for (int j = 0; j < CG; ++j) part_s[tt][wave][lane + 64 * j] = o[j];
    }
    __syncthreads();
    for (int tt = wave; tt < tc; tt += NW) {                 // a wave finishes a token: sum of the waves' shares, norm, gate
      const size_t t = (size_t)(off + t0 + tt);
      float o[CG], ss = 0.f;
#pragma unroll
      for (int j = 0; j < CG; ++j) {
        o[j] = 0.f;
        for (int w = 0; w < NW; ++w) o[j] += part_s[tt][w][lane + 64 * j];
        ss += o[j] * o[j];                                   // columns past P are zero
      }
      const float r = FUSE ? 1.f / sqrtf(wave_sum(ss) / (float)P + po.eps) * po.scale : 1.f;
#pragma unroll
      for (int j = 0; j < CG; ++j) {
        const int p = p0 + lane + 64 * j;
        if (p < P) {
          if constexpr (FUSE)
            stf<T>(out + t * po.ld + h * P + p,
                   o[j] * r * (po.norm_w ? po.norm_w[p] : 1.f) * gate_f(ldf<T>(u + t * a.ld + g0 + h * P + p), po.gate_silu));
          else y[t * HP + h * P + p] = o[j];
        }
      }
    }
    __syncthreads();                                         // the staged rows and shares are written again
  }
#pragma unroll
  for (int i = 0; i < NRW; ++i)
#pragma unroll
    for (int j = 0; j < CG; ++j) {
      const int n = wave + NW * i, p = p0 + lane + 64 * j;
      if (n < N && p < P) st[(size_t)n * P + p] = S[i][j];
    }
}

// ---------------------------------------------------------------------------------- chunks
// q or k rows of a chunk, COLS coordinates from n0, to LDS rows of LDT floats, row r times m2^(e0 - r) (log2 m; e0 < 0: 1),
// zeros past (rl, N).  SWZ: the 16-column groups of row r are stored in the order g ^ (r mod 4).
template <typename T, int COLS, int LDT, bool VEC, bool SWZ>
__device__ __forceinline__ void stage_qk(float (*dst)[LDT], const T* __restrict__ src, const DecayIn& a, int pos0, int rl, int n0,
                                         float mul, float l2, int e0) {
  if constexpr (VEC) {
#pragma unroll
    for (int i = 0; i < (CL * COLS / 8 + NT - 1) / NT; ++i) {
      const int e = threadIdx.x + i * NT, r = e / (COLS / 8), c = (e % (COLS / 8)) * 8;
      float f[8];
      if (r < rl && n0 + c < a.N) {
        qk_elem8<T>(src + (size_t)r * a.ld, n0 + c, a, a.cs ? a.cs + (size_t)(pos0 + r) * a.rot : nullptr, f);
        const float m = e0 < 0 ? mul : mul * ex2(l2 * (float)(e0 - r));
#pragma unroll
        for (int k = 0; k < 8; ++k) f[k] *= m;
      } else {
#pragma unroll
        for (int k = 0; k < 8; ++k) f[k] = 0.f;
      }
      store8<float>(&dst[r][SWZ ? c ^ ((r & 3) << 4) : c], f);
    }
  } else {
    for (int e = threadIdx.x; e < CL * COLS; e += NT) {
      const int r = e / COLS, c = e % COLS;
      float v = 0.f;
      if (r < rl && n0 + c < a.N)
        v = qk_elem<T>(src + (size_t)r * a.ld, n0 + c, a, a.cs ? a.cs + (size_t)(pos0 + r) * a.rot : nullptr) *
            (e0 < 0 ? mul : mul * ex2(l2 * (float)(e0 - r)));
      dst[r][SWZ ? c ^ ((r & 3) << 4) : c] = v;
    }
  }
}

// ROWS x COLS of a plain tile (values, states), optionally through silu
template <typename T, int ROWS, int COLS, int LDT, bool VEC, bool SWZ>
__device__ __forceinline__ void stage_plain(float (*dst)[LDT], const T* __restrict__ src, size_t ld, int rl, int cl, int silu) {
  if constexpr (VEC) {
#pragma unroll
    for (int i = 0; i < (ROWS * COLS / 8 + NT - 1) / NT; ++i) {
      const int e = threadIdx.x + i * NT, r = e / (COLS / 8), c = (e % (COLS / 8)) * 8;
      if (ROWS * COLS / 8 % NT && r >= ROWS) break;
      float f[8];
      if (r < rl && c < cl) load8<T>(src + r * ld + c, f);
      else {
#pragma unroll
        for (int k = 0; k < 8; ++k) f[k] = 0.f;
      }
      if (silu) {
#pragma unroll
        for (int k = 0; k < 8; ++k) f[k] = siluf_(f[k]);
      }
      store8<float>(&dst[r][SWZ ? c ^ ((r & 3) << 4) : c], f);
    }
  } else {
    for (int e = threadIdx.x; e < ROWS * COLS; e += NT) {
      const int r = e / COLS, c = e % COLS;
      float v = r < rl && c < cl ? ldf<T>(src + r * ld + c) : 0.f;
      if (silu) v = siluf_(v);
      dst[r][SWZ ? c ^ ((r & 3) << 4) : c] = v;
    }
  }
}

// (1) Sloc[n][p] = sum_s d^(last - s) k_s[n] v_s[p] for one 64 x 64 tile of (n, p).  Wave w: rows 16 w .. of the tile.
template <typename T, bool VEC>
__global__ void __launch_bounds__(NT) decay_chunk_state_kernel(const T* __restrict__ u, DecayIn a, const int* __restrict__ seq_start,
                                                               const int* __restrict__ seq_len, const int* __restrict__ seq_off,
                                                               float* __restrict__ sloc, int ntn, int ntp) {
  __shared__ __attribute__((aligned(16))) float K_s[CL][CL], V_s[CL][CL];
  const int tile = blockIdx.x % (ntn * ntp), c = blockIdx.x / (ntn * ntp), s = blockIdx.y, h = blockIdx.z;
  const int len = seq_len[s];
  if (c * CL >= len) return;
  const int N = a.N, P = a.P, HN = a.H * N;
  const int tc = min(CL, len - c * CL), n0 = (tile / ntp) * CL, p0 = (tile % ntp) * CL;
  const T* base = u + ((size_t)seq_off[s] + (size_t)c * CL) * a.ld;
  stage_qk<T, CL, CL, VEC, true>(K_s, base + HN + h * N, a, seq_start[s] + c * CL, tc, n0, a.k_scale, a.dec[a.H + h], tc - 1);
  stage_plain<T, CL, CL, CL, VEC, true>(V_s, base + 2 * HN + h * P + p0, a.ld, tc, P - p0, a.silu);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, g4 = lane >> 4;
  v4f acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kk = 0; kk < CL / 4; ++kk) {
    const float k = K_s[4 * kk + g4][16 * (wave ^ g4) + l16];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = mfma4(k, V_s[4 * kk + g4][16 * (j ^ g4) + l16], acc[j]);
  }
  float* dst = sloc + (((size_t)chunk_base(seq_len, s) + c) * a.H + h) * (size_t)N * P;
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = n0 + 16 * wave + 4 * g4 + i, p = p0 + 16 * j + l16;
      if (r < N && p < P) dst[(size_t)r * P + p] = acc[j][i];
    }
}

// (2) the state entering every chunk (written over that chunk's own contribution) and the final state; eight
// chunks' rows are in flight at a time
__global__ void __launch_bounds__(NT) decay_chunk_scan_kernel(float* __restrict__ sloc, const float* __restrict__ dec,
                                                              float* __restrict__ state, const int* __restrict__ seq_slot,
                                                              const int* __restrict__ seq_start, const int* __restrict__ seq_len,
                                                              int H, int NP) {
  constexpr int UN = 8;
  const int s = blockIdx.x, h = blockIdx.y, e = blockIdx.z * NT + threadIdx.x;
  if (e >= NP) return;
  const int len = seq_len[s], nc = (len + CL - 1) / CL;
  const float l2 = dec[H + h], full = ex2(l2 * (float)CL);
  float* q = sloc + ((size_t)chunk_base(seq_len, s) * H + h) * (size_t)NP + e;
  const size_t step = (size_t)H * NP;
  float* st = state + ((size_t)seq_slot[s] * H + h) * NP + e;
  float S = seq_start[s] > 0 ? *st : 0.f;
  for (int c0 = 0; c0 < nc; c0 += UN) {
    float own[UN];
#pragma unroll
    for (int i = 0; i < UN; ++i) own[i] = c0 + i < nc ? q[(c0 + i) * step] : 0.f;
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (c0 + i < nc) {
        q[(c0 + i) * step] = S;
        S = (c0 + i + 1 < nc ? full : ex2(l2 * (float)(len - (nc - 1) * CL))) * S + own[i];
      }
    }
  }
  *st = S;
}

// (3) the outputs of one chunk and 16 PT value columns.  Wave w owns the token rows 16 w .. .  A product over 16 steps
// takes them in the order 4 g4 + r (r the instruction, g4 the lane's quarter), so a lane's operands along a row are one
// 16-byte read.  FUSE: all columns of the head are here, so the norm and the gate follow.
template <typename T, int PT, bool FUSE, bool VEC>
__global__ void __launch_bounds__(NT) decay_chunk_out_kernel(const T* __restrict__ u, DecayIn a, const int* __restrict__ seq_start,
                                                             const int* __restrict__ seq_len, const int* __restrict__ seq_off,
                                                             const float* __restrict__ sin_, DecayOut po, T* __restrict__ out,
                                                             float* __restrict__ y, int ntp) {
  constexpr int NK = 32, LQ = NK + 4, CW = 16 * PT, LS = CW + 4, LA = CL + 4;
  constexpr int STAGE = 2 * CL * LQ + NK * LS, TAIL = CL * LA + CL * LS;
  __shared__ __attribute__((aligned(16))) float buf[STAGE > TAIL ? STAGE : TAIL];
  float(*Q_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf);
  float(*K_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf + CL * LQ);
  float(*S_s)[LS] = reinterpret_cast<float(*)[LS]>(buf + 2 * CL * LQ);
  float(*A_s)[LA] = reinterpret_cast<float(*)[LA]>(buf);     // after the key channels: scores and values
  float(*V_s)[LS] = reinterpret_cast<float(*)[LS]>(buf + CL * LA);
  const int pt = blockIdx.x % ntp, c = blockIdx.x / ntp, s = blockIdx.y, h = blockIdx.z;
  const int len = seq_len[s];
  if (c * CL >= len) return;
  const int N = a.N, P = a.P, HN = a.H * N, HP = a.H * P;
  const int tc = min(CL, len - c * CL), p0 = pt * CW, pos0 = seq_start[s] + c * CL;
  const size_t row0 = (size_t)seq_off[s] + (size_t)c * CL;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, g4 = lane >> 4;
  const float* sin_c = sin_ + (((size_t)chunk_base(seq_len, s) + c) * a.H + h) * (size_t)N * P + p0;
  const T* base = u + row0 * a.ld;
  const float l2 = a.dec[a.H + h];
  const bool carry = pos0 > 0;                               // a sequence's first chunk enters with a state of zero
  v4f o[PT], sc[4];
#pragma unroll
  for (int j = 0; j < PT; ++j) o[j] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < 4; ++j) sc[j] = v4f{0.f, 0.f, 0.f, 0.f};
  for (int n0 = 0; n0 < N; n0 += NK) {
    __syncthreads();                                         // the last channels' tiles are done with
    stage_qk<T, NK, LQ, VEC, false>(Q_s, base + h * N, a, pos0, tc, n0, 1.f, 0.f, -1);
    stage_qk<T, NK, LQ, VEC, false>(K_s, base + HN + h * N, a, pos0, tc, n0, a.k_scale, 0.f, -1);
    if (carry) stage_plain<float, NK, CW, LS, VEC, false>(S_s, sin_c + (size_t)n0 * P, P, N - n0, P - p0, 0);
    __syncthreads();
#pragma unroll
    for (int kg = 0; kg < NK / 16; ++kg) {
      const float4 q = *reinterpret_cast<const float4*>(&Q_s[16 * wave + l16][16 * kg + 4 * g4]);
      const float qv[4] = {q.x, q.y, q.z, q.w};
      if (carry) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int j = 0; j < PT; ++j) o[j] = mfma4(qv[r], S_s[16 * kg + 4 * g4 + r][16 * j + l16], o[j]);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j <= wave) {
          const float4 k = *reinterpret_cast<const float4*>(&K_s[16 * j + l16][16 * kg + 4 * g4]);
          sc[j] = mfma4(qv[0], k.x, sc[j]);
          sc[j] = mfma4(qv[1], k.y, sc[j]);
          sc[j] = mfma4(qv[2], k.z, sc[j]);
          sc[j] = mfma4(qv[3], k.w, sc[j]);
        }
    }
  }
  __syncthreads();
  // lane holds scores (row 4 g4 + i of its wave, column l16 of block j)
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = 16 * wave + 4 * g4 + i;
    const float f = ex2(l2 * (float)(t + 1));
#pragma unroll
    for (int j = 0; j < PT; ++j) o[j][i] *= f;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) {
        const int sp = 16 * j + l16;
        A_s[t][sp] = sp <= t ? sc[j][i] * ex2(l2 * (float)(t - sp)) : 0.f;
      }
  }
  stage_plain<T, CL, CW, LS, VEC, false>(V_s, base + 2 * HN + h * P + p0, a.ld, tc, P - p0, a.silu);
  __syncthreads();
  for (int kg = 0; kg <= wave; ++kg) {
    const float4 w = *reinterpret_cast<const float4*>(&A_s[16 * wave + l16][16 * kg + 4 * g4]);
    const float wv[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int j = 0; j < PT; ++j) o[j] = mfma4(wv[r], V_s[16 * kg + 4 * g4 + r][16 * j + l16], o[j]);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int to = 16 * wave + 4 * g4 + i;
    float r = 1.f;
    if constexpr (FUSE) {
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < PT; ++j) ss += o[j][i] * o[j][i];  // columns past P are zero
      r = 1.f / sqrtf(row16_sum(ss) / (float)P + po.eps) * po.scale;
    }
    if (to < tc) {
      const size_t row = row0 + to;
#pragma unroll
      for (int j = 0; j < PT; ++j) {
        const int p = p0 + 16 * j + l16;
        if (p < P) {
          if constexpr (FUSE)
            stf<T>(out + row * po.ld + h * P + p, o[j][i] * r * (po.norm_w ? po.norm_w[p] : 1.f) *
                                                      gate_f(ldf<T>(u + row * a.ld + 2 * HN + HP + h * P + p), po.gate_silu));
          else
            y[row * HP + h * P + p] = o[j][i];
        }
      }
    }
  }
}

// ---------------------------------------------------------------------------------- norm over a row part, gate
// y fp32 [rows, parts C] -> out = y / rms(part) * w * gate(g) * scale; one workgroup per (row, part).  VEC: 8 per access
template <typename T, bool VEC>
__global__ void __launch_bounds__(NT) row_norm_gate_kernel(const float* __restrict__ y, const T* __restrict__ g, int g_ld, int C,
                                                           DecayOut po, T* __restrict__ out) {
  __shared__ float red[NT / 64];
  const size_t t = blockIdx.x, c0 = (size_t)blockIdx.y * C;
  const float* yr = y + t * (size_t)(gridDim.y * C) + c0;
  const T* gr = g + t * g_ld + c0;
  T* o = out + t * po.ld + c0;
  float ss = 0.f;
  if constexpr (VEC) {
    float f[8];                                              // rows of up to 2048 stay in registers
    const int c1 = threadIdx.x * 8;
    if (c1 < C) {
      load8<float>(yr + c1, f);
#pragma unroll
      for (int k = 0; k < 8; ++k) ss += f[k] * f[k];
    }
    for (int c = c1 + NT * 8; c < C; c += NT * 8) {
      float v[8];
      load8<float>(yr + c, v);
#pragma unroll
      for (int k = 0; k < 8; ++k) ss += v[k] * v[k];
    }
    const float r = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)C + po.eps) * po.scale;
    for (int c = c1; c < C; c += NT * 8) {
      float gv[8];
      load8<T>(gr + c, gv);
      if (c != c1) load8<float>(yr + c, f);
#pragma unroll
      for (int k = 0; k < 8; ++k) f[k] *= r * gate_f(gv[k], po.gate_silu);
      if (po.norm_w) {
        float w[8];
        load8<float>(po.norm_w + c, w);
#pragma unroll
        for (int k = 0; k < 8; ++k) f[k] *= w[k];
      }
      store8<T>(o + c, f);
    }
  } else {
    for (int c = threadIdx.x; c < C; c += NT) ss += yr[c] * yr[c];
    const float r = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)C + po.eps) * po.scale;
    for (int c = threadIdx.x; c < C; c += NT)
      stf<T>(o + c, yr[c] * r * (po.norm_w ? po.norm_w[c] : 1.f) * gate_f(ldf<T>(gr + c), po.gate_silu));
  }
}

// cap tanh(z / cap) as fp32
template <typename T>
__global__ void __launch_bounds__(NT) softcap_kernel(const T* __restrict__ z, float* __restrict__ out, long n, float cap) {
  for (long i = (long)blockIdx.x * NT + threadIdx.x; i < n; i += (long)gridDim.x * NT) out[i] = cap * tanhf(ldf<T>(z + i) / cap);
}

}  // namespace

#define SM_T(f32, ...)                                  \
  do {                                                  \
    if (f32) { using T = float; __VA_ARGS__; }          \
    else { using T = bf16_t; __VA_ARGS__; }             \
  } while (0)

extern "C" {

// value columns of a head that one workgroup of either form can hold; key channels that the token-by-token form can hold
int edge_sm_decay_fused(int P) { return P <= 128; }
int edge_sm_decay_step_ok(int N) { return N <= 256; }

// u: the mixer's first column (rows ld apart); all_heads: the norm runs over the heads together (scratch y fp32 [rows,
// H P], as for heads wider than the fused form); chunked: sloc fp32 [chunks, H, N, P] scratch, max_chunks = the most
// 64-token chunks any sequence brings (0: token by token)
int edge_sm_decay_attn(const void* u, int ld, const float* dec, const float* cs, int rot, float k_scale, int silu,
                       const float* norm_w, int all_heads, int gate_silu, float* state, const int* seq_slot,
                       const int* seq_start, const int* seq_len, const int* seq_off, void* out, int out_ld, float out_scale,
                       float* y, float* sloc, int rows, int n, int max_chunks, int H, int N, int P, float eps, int f32,
                       hipStream_t st) {
  if (n == 0 || rows == 0) return 0;
  if (N < 1 || P < 1 || H < 1 || rot < 0 || rot % 2 || rot > N || (rot > 0 && !cs) || out_ld < H * P) return -2;
  if (max_chunks <= 0 && !edge_sm_decay_step_ok(N)) return -2;
  const bool fuse = !all_heads && edge_sm_decay_fused(P);
  if ((!fuse && !y) || (max_chunks > 0 && !sloc)) return -2;
  const DecayIn a{dec, rot > 0 ? cs : nullptr, ld, H, N, P, rot, silu, k_scale};
  const DecayOut po{norm_w, out_ld, gate_silu, eps, out_scale};
  if (max_chunks <= 0) {
#define SM_DS(NW, NRW, CG, FUSE)                                                                                              \
  SM_T(f32, hipLaunchKernelGGL((decay_step_kernel<T, NW, NRW, CG, FUSE>), dim3(n, H, (P + 64 * CG - 1) / (64 * CG)),           \
                               dim3(64 * NW), 0, st, (const T*)u, a, state, seq_slot, seq_start, seq_len, seq_off, po,         \
                               (T*)out, y))
#define SM_DSC(NW, NRW)                       \
  do {                                        \
    if (!fuse) SM_DS(NW, NRW, 1, false);      \
    else if (P <= 64) SM_DS(NW, NRW, 1, true);\
    else SM_DS(NW, NRW, 2, true);             \
  } while (0)
    if (N <= 64) SM_DSC(4, 16);
    else if (N <= 128) SM_DSC(8, 16);
    else SM_DSC(8, 32);
#undef SM_DSC
#undef SM_DS
  } else {
    const int ntn = (N + CL - 1) / CL, ntp = (P + CL - 1) / CL;
    const bool vec = N % 8 == 0 && P % 8 == 0 && ld % 8 == 0 && rot % 16 == 0 &&
                     (((uintptr_t)u | (uintptr_t)sloc | (uintptr_t)cs) & 15) == 0;
#define SM_DC(V)                                                                                                              \
  SM_T(f32, hipLaunchKernelGGL((decay_chunk_state_kernel<T, V>), dim3(max_chunks * ntn * ntp, n, H), dim3(NT), 0, st,          \
                               (const T*)u, a, seq_start, seq_len, seq_off, sloc, ntn, ntp))
    if (vec) SM_DC(true);
    else SM_DC(false);
#undef SM_DC
    hipLaunchKernelGGL(decay_chunk_scan_kernel, dim3(n, H, (N * P + NT - 1) / NT), dim3(NT), 0, st, sloc, dec, state, seq_slot,
                       seq_start, seq_len, H, N * P);
#define SM_DOV(PT, FUSE, V)                                                                                                   \
  SM_T(f32, hipLaunchKernelGGL((decay_chunk_out_kernel<T, PT, FUSE, V>), dim3(max_chunks * ((P + 16 * PT - 1) / (16 * PT)), n, \
                               H), dim3(NT), 0, st, (const T*)u, a, seq_start, seq_len, seq_off, sloc, po, (T*)out, y,         \
                               (P + 16 * PT - 1) / (16 * PT)))
#define SM_DO(PT, FUSE)              \
  do {                               \
    if (vec) SM_DOV(PT, FUSE, true); \
    else SM_DOV(PT, FUSE, false);    \
  } while (0)
    if (fuse) {
      if (P <= 64) SM_DO(4, true);
      else SM_DO(8, true);
    } else {
      if (P <= 64) SM_DO(4, false);
      else SM_DO(8, false);
    }
#undef SM_DO
#undef SM_DOV
  }
  if (!fuse) {
    const int parts = all_heads ? 1 : H, C = all_heads ? H * P : P;
    const size_t col = 2 * (size_t)H * N + (size_t)H * P;
    const void* g = f32 ? (const void*)((const float*)u + col) : (const void*)((const bf16_t*)u + col);
    if (C % 8 == 0 && ld % 8 == 0 && out_ld % 8 == 0 && (((uintptr_t)y | (uintptr_t)g | (uintptr_t)out | (uintptr_t)norm_w) & 15) == 0)
      SM_T(f32, hipLaunchKernelGGL((row_norm_gate_kernel<T, true>), dim3(rows, parts), dim3(NT), 0, st, y, (const T*)g, ld, C, po,
                                   (T*)out));
    else
      SM_T(f32, hipLaunchKernelGGL((row_norm_gate_kernel<T, false>), dim3(rows, parts), dim3(NT), 0, st, y, (const T*)g, ld, C, po,
                                   (T*)out));
  }
  return (int)hipGetLastError();
}

int edge_sm_softcap(const void* z, float* out, long n, float cap, int f32, hipStream_t st) {
  if (n == 0) return 0;
  if (!(cap > 0.f)) return -2;
  const long wg = (n + NT * 4 - 1) / (NT * 4);
  SM_T(f32, hipLaunchKernelGGL(softcap_kernel<T>, dim3((unsigned)(wg < 4096 ? wg : 4096)), dim3(NT), 0, st, (const T*)z, out, n, cap));
  return (int)hipGetLastError();
}

}  // extern "C"
