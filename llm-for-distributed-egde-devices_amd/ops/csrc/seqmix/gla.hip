// Gated linear attention over a ragged step (ops/seqmix.py::gated_linear_attention): per head
//   log a_t = log sigmoid(A2 d_t + b) / tau per key channel,  S_t = diag(a_t) S_{t-1} + k_t v_t^T,
//   o_t = S_t^T q_t N^-1/2,  out_t = o_t / rms(o_t) * w * silu(g_t).
// u row = q [H, N] | k [H, N] | v [H, P] | g [H, P] | d [rank].
//
// Two forms.  Short portions (decode): one workgroup per (sequence, head) steps token by token, decays, norm and
// gate included.  Long portions: chunks of 64 tokens in parallel.  With B_t the sum of log a inside the chunk,
//   S_t = e^{B_t} S_in + sum_{s<=t} e^{B_t - B_s} k_s v_s^T
//   o_t = (q_t e^{B_t})^T S_in + sum_{s<=t} [sum_n q_t k_s e^{B_t - B_s}]_n v_s
// (1) every chunk's own contribution to its end state, (2) the states at the chunk borders, (3) the outputs.
// A decay ratio is never formed as a quotient and no exponent is positive, so strong decays only underflow.  From a
// token s to a later 16-token block it is e^{what s's block decays after s + the blocks between} e^{t's block up to
// t}: sums of terms of one sign, so a weak decay behind strong ones loses nothing to cancellation.  Inside a block it
// is e^{B_t - B_s} with B counted from the block's start.
//
// Storage of u / out is fp32 or bf16 (template T); decays, products, sums and the state are fp32 (the tile
// products run on v_mfma_f32_16x16x4_f32).  State rows live per slot and are taken as zero by a portion that
// starts at position 0.
#include "common.h"
#include "seqmix/seqmix_common.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float log_sigmoid(float z) {
  return z >= 0.f ? -log1pf(expf(-z)) : z - log1pf(expf(z));
}
// log2 sigmoid(z) = -(max(-z, 0) log2 e + log2(1 + 2^{-|z| log2 e}))
__device__ __forceinline__ float log2_sigmoid(float z) {
  return -(fmaxf(-z, 0.f) * LOG2E + __builtin_amdgcn_logf(1.f + ex2(-fabsf(z) * LOG2E)));
}

// ---------------------------------------------------------------------------------- token by token
// One workgroup of NW waves per (sequence, head, 64 CG value columns): lane = column, wave w keeps the state rows
// n = w, w + NW, .. (NRW of them) of its columns in registers; TC tokens are staged at a time, the waves' partial
// sums of o are added up per staged group.  FUSE: all columns of the head are here, so the norm and the gate follow.
template <typename T, int NW, int NRW, int CG, bool FUSE>
__global__ void __launch_bounds__(64 * NW) gla_step_kernel(
    const T* __restrict__ u, int ld, const float* __restrict__ a2, const float* __restrict__ b, int rank,
    const float* __restrict__ norm_w, float* __restrict__ state, const int* __restrict__ seq_slot,
    const int* __restrict__ seq_start, const int* __restrict__ seq_len, const int* __restrict__ seq_off, T* __restrict__ out,
    float* __restrict__ y, int H, int N, int P, float inv_tau, float eps) {
  constexpr int TH = 64 * NW, TC = 8, CW = 64 * CG, NMAX = NW * NRW;
  __shared__ float q_s[TC][NMAX], k_s[TC][NMAX], a_s[TC][NMAX], part_s[TC][NW][CW];
  const int s = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * CW, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int start = seq_start[s], len = seq_len[s], off = seq_off[s];
  const int HN = H * N, HP = H * P, v0 = 2 * HN, g0 = v0 + HP, d0 = g0 + HP;
  const float qs = 1.f / sqrtf((float)N);
  float* st = state + ((size_t)seq_slot[s] * H + h) * N * P;
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
      const T* row = u + (size_t)(off + t0 + tt) * ld;
      const float* wr = a2 + (size_t)(h * N + n) * rank;
      float z = b[h * N + n];
      for (int r = 0; r < rank; ++r) z += wr[r] * ldf<T>(row + d0 + r);
      q_s[tt][n] = ldf<T>(row + h * N + n) * qs;
      k_s[tt][n] = ldf<T>(row + HN + h * N + n);
      a_s[tt][n] = expf(log_sigmoid(z) * inv_tau);
    }
    __syncthreads();
    for (int tt = 0; tt < tc; ++tt) {
      const T* row = u + (size_t)(off + t0 + tt) * ld + v0 + h * P;
      float v[CG], o[CG];
#pragma unroll
      for (int j = 0; j < CG; ++j) {
        const int p = p0 + lane + 64 * j;
        v[j] = p < P ? ldf<T>(row + p) : 0.f;
        o[j] = 0.f;
      }
#pragma unroll
      for (int i = 0; i < NRW; ++i) {
        const int n = wave + NW * i;
        if (n < N) {
          const float av = a_s[tt][n], kv = k_s[tt][n], qv = q_s[tt][n];
#pragma unroll
          for (int j = 0; j < CG; ++j) {
            S[i][j] = av * S[i][j] + kv * v[j];
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
      const float r = FUSE ? 1.f / sqrtf(wave_sum(ss) / (float)P + eps) : 1.f;
#pragma unroll
      for (int j = 0; j < CG; ++j) {
        const int p = p0 + lane + 64 * j;
        if (p < P) {
          if constexpr (FUSE) stf<T>(out + t * HP + h * P + p, o[j] * r * norm_w[p] * siluf_(ldf<T>(u + t * ld + g0 + h * P + p)));
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
// rows x cols of a tile to LDS rows of LDT floats, zeros past (rl, cl); VEC: 8 elements per access (cols, cl, the
// source's stride and alignment allow it)
// SWZ: the 16-column groups of row r are stored in the order g ^ (r mod 4), so four token rows of an operand hit
// different banks without padding
template <typename T, int ROWS, int COLS, int LDT, bool VEC, bool SWZ = false>
__device__ __forceinline__ void stage_tile(float (*dst)[LDT], const T* __restrict__ src, size_t ld, int rl, int cl, float mul) {
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
#pragma unroll
      for (int k = 0; k < 8; ++k) f[k] *= mul;
      store8<float>(&dst[r][SWZ ? c ^ ((r & 3) << 4) : c], f);
    }
  } else {
    for (int e = threadIdx.x; e < ROWS * COLS; e += NT) {
      const int r = e / COLS, c = e % COLS;
      dst[r][SWZ ? c ^ ((r & 3) << 4) : c] = r < rl && c < cl ? ldf<T>(src + r * ld + c) * mul : 0.f;
    }
  }
}

// (1) Sloc[n][p] = sum_s k_s[n] e^{B_end - B_s}[n] v_s[p] for one 64 x 64 tile of (n, p).  A thread computes the log2
// decays of one key channel over a 16-token block; they go to la [rows, H N] for the outputs, the chunk's whole decay
// e^{B_end} per key channel to cdec.  Wave w: rows 16 w .. of the tile.  The decay projection's inner rows are staged
// RS at a time.
template <typename T, bool VEC>
__global__ void __launch_bounds__(NT) gla_chunk_state_kernel(const T* __restrict__ u, int ld, const float* __restrict__ a2,
                                                             const float* __restrict__ b, int rank, float scale,
                                                             const int* __restrict__ seq_len, const int* __restrict__ seq_off,
                                                             float* __restrict__ sloc, float* __restrict__ cdec,
                                                             float* __restrict__ la, int H, int N, int P, int ntn, int ntp) {
  constexpr int LDT = CL;
  constexpr int RS = 16;
  __shared__ __attribute__((aligned(16))) float d_s[RS][CL];
  __shared__ __attribute__((aligned(16))) float K_s[CL][LDT], V_s[CL][LDT];
  __shared__ float seg_s[4][CL];
  const int tile = blockIdx.x % (ntn * ntp), c = blockIdx.x / (ntn * ntp), s = blockIdx.y, h = blockIdx.z;
  const int len = seq_len[s];
  if (c * CL >= len) return;
  const int tc = min(CL, len - c * CL), n0 = (tile / ntp) * CL, p0 = (tile % ntp) * CL;
  const size_t row0 = (size_t)seq_off[s] + (size_t)c * CL;
  const int HN = H * N, HP = H * P, tid = threadIdx.x, nn = tid & 63, seg = tid >> 6, n = n0 + nn;
  const T* base = u + row0 * ld;
  stage_tile<T, CL, CL, LDT, VEC, true>(K_s, base + HN + h * N + n0, ld, tc, N - n0, 1.f);
  stage_tile<T, CL, CL, LDT, VEC, true>(V_s, base + 2 * HN + h * P + p0, ld, tc, P - p0, 1.f);
  float bl[16];
  {
    const int nc = min(n, N - 1);
    const float* wr = a2 + (size_t)(h * N + nc) * rank;
    const float bias = b[h * N + nc];
#pragma unroll
    for (int i = 0; i < 16; ++i) bl[i] = bias;
    for (int r0 = 0; r0 < rank; r0 += RS) {
      if (r0) __syncthreads();                               // the last slice is read
      for (int e = tid; e < CL * RS; e += NT) {
        const int t = e / RS, r = e % RS;
        d_s[r][t] = t < tc && r0 + r < rank ? ldf<T>(base + (size_t)t * ld + 2 * HN + 2 * HP + r0 + r) : 0.f;
      }
      __syncthreads();
      float w[RS];
#pragma unroll
      for (int r = 0; r < RS; ++r) w[r] = r0 + r < rank ? wr[r0 + r] : 0.f;
#pragma unroll
      for (int r = 0; r < RS; ++r) {
        const float4* dq = reinterpret_cast<const float4*>(&d_s[r][seg * 16]);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float4 d = dq[i];
          bl[4 * i] += w[r] * d.x; bl[4 * i + 1] += w[r] * d.y; bl[4 * i + 2] += w[r] * d.z; bl[4 * i + 3] += w[r] * d.w;
        }
      }
    }
    float run = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = seg * 16 + i;
      bl[i] = (t < tc && n < N) ? log2_sigmoid(bl[i]) * scale : 0.f;
      run += bl[i];
      if (p0 == 0 && t < tc && n < N) la[(row0 + t) * HN + h * N + n] = bl[i];
    }
    seg_s[seg][nn] = run;
  }
  __syncthreads();
  float after = 0.f, end = 0.f;                              // the later blocks' decay, the chunk's
#pragma unroll
  for (int g = 0; g < 4; ++g) { const float v = seg_s[g][nn]; if (g > seg) after += v; end += v; }
#pragma unroll
  for (int i = 15; i >= 0; --i) {
    K_s[seg * 16 + i][nn ^ ((i & 3) << 4)] *= ex2(after);
    after += bl[i];
  }
  const size_t cb = (size_t)chunk_base(seq_len, s) + c;
  if (p0 == 0 && seg == 0 && n < N) cdec[(cb * H + h) * N + n] = ex2(end);
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g4 = lane >> 4;
  v4f acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kk = 0; kk < CL / 4; ++kk) {
    const float a = K_s[4 * kk + g4][16 * (wave ^ g4) + l16];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = mfma4(a, V_s[4 * kk + g4][16 * (j ^ g4) + l16], acc[j]);
  }
  float* dst = sloc + (cb * H + h) * (size_t)N * P;
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
__global__ void __launch_bounds__(NT) gla_chunk_scan_kernel(float* __restrict__ sloc, const float* __restrict__ cdec,
                                                            float* __restrict__ state, const int* __restrict__ seq_slot,
                                                            const int* __restrict__ seq_start, const int* __restrict__ seq_len,
                                                            int H, int N, int P) {
  constexpr int UN = 8;
  const int s = blockIdx.x, h = blockIdx.y, e = blockIdx.z * NT + threadIdx.x, NP = N * P;
  if (e >= NP) return;
  const int nc = (seq_len[s] + CL - 1) / CL, n = e / P;
  const size_t cb = chunk_base(seq_len, s);
  float* st = state + ((size_t)seq_slot[s] * H + h) * NP + e;
  float S = seq_start[s] > 0 ? *st : 0.f;
  for (int c0 = 0; c0 < nc; c0 += UN) {
    float own[UN], dec[UN];
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      const bool ok = c0 + i < nc;
      own[i] = ok ? sloc[((cb + c0 + i) * H + h) * (size_t)NP + e] : 0.f;
      dec[i] = ok ? cdec[((cb + c0 + i) * H + h) * N + n] : 1.f;
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (c0 + i < nc) {
        sloc[((cb + c0 + i) * H + h) * (size_t)NP + e] = S;
        S = dec[i] * S + own[i];
      }
    }
  }
  *st = S;
}

// (3) the outputs of one chunk and 16 PT value columns.  Wave i owns the token rows of block i (16 tokens).
// FUSE: all columns of the head are here, so the norm and the gate follow.
template <typename T, int PT, bool FUSE, bool VEC>
__global__ void __launch_bounds__(NT) gla_chunk_out_kernel(const T* __restrict__ u, int ld, const float* __restrict__ la,
                                                           const int* __restrict__ seq_len, const int* __restrict__ seq_off,
                                                           const float* __restrict__ sin_, const float* __restrict__ norm_w,
                                                           T* __restrict__ out, float* __restrict__ y, int H, int N, int P,
                                                           int ntp, float eps) {
  constexpr int NK = 32, LQ = NK + 4, CW = 16 * PT, LS = CW + 16, LA = CL + 4;
  constexpr int STAGE = 4 * CL * LQ + NK * LS, TAIL = CL * LA + CL * LS;
  __shared__ __attribute__((aligned(16))) float buf[STAGE > TAIL ? STAGE : TAIL];
  float(*Q_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf);
  float(*K_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf + CL * LQ);
  float(*B_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf + 2 * CL * LQ);
  float(*E_s)[LQ] = reinterpret_cast<float(*)[LQ]>(buf + 3 * CL * LQ);
  float(*S_s)[LS] = reinterpret_cast<float(*)[LS]>(buf + 4 * CL * LQ);
  float(*A_s)[LA] = reinterpret_cast<float(*)[LA]>(buf);     // after the key channels: scores and values
  float(*V_s)[LS] = reinterpret_cast<float(*)[LS]>(buf + CL * LA);
  const int pt = blockIdx.x % ntp, c = blockIdx.x / ntp, s = blockIdx.y, h = blockIdx.z;
  const int len = seq_len[s];
  if (c * CL >= len) return;
  const int tc = min(CL, len - c * CL), p0 = pt * CW;
  const size_t row0 = (size_t)seq_off[s] + (size_t)c * CL;
  const int HN = H * N, HP = H * P, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g4 = lane >> 4;
  const float* sin_c = sin_ + (((size_t)chunk_base(seq_len, s) + c) * H + h) * (size_t)N * P + p0;
  const T* base = u + row0 * ld;
  const float qs = 1.f / sqrtf((float)N);
  const int t = 16 * wave + l16;                             // this lane's token row as a product operand
  v4f o[PT], off_[3], dg = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < PT; ++j) o[j] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < 3; ++j) off_[j] = v4f{0.f, 0.f, 0.f, 0.f};
  for (int n0 = 0; n0 < N; n0 += NK) {
    __syncthreads();                                         // the last channels' tiles are done with
    stage_tile<T, CL, NK, LQ, VEC>(Q_s, base + h * N + n0, ld, tc, N - n0, qs);
    stage_tile<T, CL, NK, LQ, VEC>(K_s, base + HN + h * N + n0, ld, tc, N - n0, 1.f);
    stage_tile<float, CL, NK, LQ, VEC>(B_s, la + row0 * HN + h * N + n0, HN, tc, N - n0, 1.f);
    stage_tile<float, NK, CW, LS, VEC>(S_s, sin_c + (size_t)n0 * P, P, N - n0, P - p0, 1.f);
    __syncthreads();
    {
      // per 16-token block and channel: B = the log decays up to and with each token, E = those after it; half a wave
      // holds a block's first eight tokens, the other half its last eight
      const int nn = tid % NK, seg = tid / NK;
      float a[8], sum = 0.f, back = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) { a[i] = B_s[seg * 8 + i][nn]; sum += a[i]; }
      const float other = __shfl_xor(sum, 32, 64);
      float fwd = seg & 1 ? other : 0.f;
      back = seg & 1 ? 0.f : other;
#pragma unroll
      for (int i = 0; i < 8; ++i) { fwd += a[i]; B_s[seg * 8 + i][nn] = fwd; }
#pragma unroll
      for (int i = 7; i >= 0; --i) { E_s[seg * 8 + i][nn] = back; back += a[i]; }
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < NK / 4; ++kk) {
      const int n = 4 * kk + g4;
      const float q = Q_s[t][n], bt = B_s[t][n];
      float tot[3], pre = 0.f;                               // whole-block decays before this wave's block
#pragma unroll
      for (int j = 0; j < 3; ++j) { tot[j] = j < wave ? B_s[16 * j + 15][n] : 0.f; pre += tot[j]; }
      const float qr = q * ex2(bt), qa = q * ex2(bt + pre);
#pragma unroll
      for (int j = 0; j < PT; ++j) o[j] = mfma4(qa, S_s[n][16 * j + l16], o[j]);
      float mid = 0.f;                                       // the blocks between j and this wave's
#pragma unroll
      for (int j = 2; j >= 0; --j)
        if (j < wave) {
          off_[j] = mfma4(qr, K_s[16 * j + l16][n] * ex2(E_s[16 * j + l16][n] + mid), off_[j]);
          mid += tot[j];
        }
    }
    // the block against itself: lane holds (row 4 g4 + i, column l16), as the products' results lie
#pragma unroll 2
    for (int n = 0; n < NK; n += 4) {
      const float4 kv = *reinterpret_cast<const float4*>(&K_s[t][n]), bs = *reinterpret_cast<const float4*>(&B_s[t][n]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * wave + 4 * g4 + i;
        const float4 q = *reinterpret_cast<const float4*>(&Q_s[r][n]), br = *reinterpret_cast<const float4*>(&B_s[r][n]);
        dg[i] += q.x * kv.x * ex2(fminf(br.x - bs.x, 0.f)) + q.y * kv.y * ex2(fminf(br.y - bs.y, 0.f)) +
                 q.z * kv.z * ex2(fminf(br.z - bs.z, 0.f)) + q.w * kv.w * ex2(fminf(br.w - bs.w, 0.f));
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 4 * g4 + i;
#pragma unroll
    for (int j = 0; j < 3; ++j)
      if (j < wave) A_s[16 * wave + r][16 * j + l16] = off_[j][i];
    A_s[16 * wave + r][16 * wave + l16] = l16 <= r ? dg[i] : 0.f;
  }
  stage_tile<T, CL, CW, LS, VEC>(V_s, base + 2 * HN + h * P + p0, ld, tc, P - p0, 1.f);
  __syncthreads();
  for (int kk = 0; kk < 4 * (wave + 1); ++kk) {
    const float a = A_s[16 * wave + l16][4 * kk + g4];
#pragma unroll
    for (int j = 0; j < PT; ++j) o[j] = mfma4(a, V_s[4 * kk + g4][16 * j + l16], o[j]);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int to = 16 * wave + 4 * g4 + i;
    float r = 1.f;
    if constexpr (FUSE) {
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < PT; ++j) ss += o[j][i] * o[j][i];  // columns past P are zero
      r = 1.f / sqrtf(row16_sum(ss) / (float)P + eps);
    }
    if (to < tc) {
#pragma unroll
      for (int j = 0; j < PT; ++j) {
        const int p = p0 + 16 * j + l16;
        if (p < P) {
          const size_t row = row0 + to;
          if constexpr (FUSE)
            stf<T>(out + row * HP + h * P + p, o[j][i] * r * norm_w[p] * siluf_(ldf<T>(u + row * ld + 2 * HN + HP + h * P + p)));
          else
            y[row * HP + h * P + p] = o[j][i];
        }
      }
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

int edge_sm_head_norm_gate(const float* y, const void* z, int z_ld, const float* w, void* out, int rows, int H, int P,
                           float eps, int silu, int f32, hipStream_t st);

// value columns of a head that one workgroup of either form can hold (wider heads: norm and gate in a kernel of
// their own over y fp32 [rows, H P])
int edge_sm_gla_fused(int P) { return P <= 128; }
// key channels per head that the token-by-token form can hold
int edge_sm_gla_step_ok(int N) { return N <= 256; }

static int gla_norm(const void* u, int ld, const float* norm_w, void* out, const float* y, int rows, int H, int N, int P,
                    float eps, int f32, hipStream_t st) {
  const size_t col = 2 * (size_t)H * N + (size_t)H * P;
  const void* z = f32 ? (const void*)((const float*)u + col) : (const void*)((const bf16_t*)u + col);
  return edge_sm_head_norm_gate(y, z, ld, norm_w, out, rows, H, P, eps, 1, f32, st);
}

int edge_sm_gla_step(const void* u, int ld, const float* a2, const float* b, int rank, const float* norm_w, float* state,
                     const int* seq_slot, const int* seq_start, const int* seq_len, const int* seq_off, void* out, float* y,
                     int rows, int n, int H, int N, int P, float inv_tau, float eps, int f32, hipStream_t st) {
  if (n == 0 || rows == 0) return 0;
  if (N < 1 || N > 256 || P < 1 || rank < 1) return -2;
  const bool fuse = edge_sm_gla_fused(P);
  if (!fuse && !y) return -2;
#define SM_GS(NW, NRW, CG, FUSE)                                                                                             \
  SM_T(f32, hipLaunchKernelGGL((gla_step_kernel<T, NW, NRW, CG, FUSE>), dim3(n, H, (P + 64 * CG - 1) / (64 * CG)),            \
                               dim3(64 * NW), 0, st, (const T*)u, ld, a2, b, rank, norm_w, state, seq_slot, seq_start,        \
                               seq_len, seq_off, (T*)out, y, H, N, P, inv_tau, eps))
#define SM_GSC(NW, NRW)                                  \
  do {                                                   \
    if (P <= 64) SM_GS(NW, NRW, 1, true);                \
    else if (fuse) SM_GS(NW, NRW, 2, true);              \
    else SM_GS(NW, NRW, 2, false);                       \
  } while (0)
  if (N <= 64) SM_GSC(4, 16);
  else if (N <= 128) SM_GSC(8, 16);
  else SM_GSC(8, 32);
#undef SM_GSC
#undef SM_GS
  if (!fuse) {
    const int rc = gla_norm(u, ld, norm_w, out, y, rows, H, N, P, eps, f32, st);
    if (rc) return rc;
  }
  return (int)hipGetLastError();
}

// scratch: la [rows, H N], sloc [chunks, H, N, P], cdec [chunks, H, N], y [rows, H P] (heads wider than the fused
// form), all fp32; max_chunks = the most 64-token chunks any sequence brings
int edge_sm_gla_chunked(const void* u, int ld, const float* a2, const float* b, int rank, const float* norm_w, float* state,
                        const int* seq_slot, const int* seq_start, const int* seq_len, const int* seq_off, void* out,
                        float* la, float* sloc, float* cdec, float* y, int rows, int n, int max_chunks, int H, int N, int P,
                        float inv_tau, float eps, int f32, hipStream_t st) {
  if (n == 0 || rows == 0 || max_chunks <= 0) return 0;
  if (N < 1 || P < 1 || rank < 1) return -2;
  const bool fuse = edge_sm_gla_fused(P);
  if (!fuse && !y) return -2;
  const int ntn = (N + CL - 1) / CL, ntp = (P + CL - 1) / CL;
  const bool vec = N % 8 == 0 && P % 8 == 0 && ld % 8 == 0 && (((uintptr_t)u | (uintptr_t)la | (uintptr_t)sloc) & 31) == 0;
#define SM_GC(V)                                                                                                             \
  SM_T(f32, hipLaunchKernelGGL((gla_chunk_state_kernel<T, V>), dim3(max_chunks * ntn * ntp, n, H), dim3(NT),                  \
                               0, st, (const T*)u, ld, a2, b, rank, inv_tau, seq_len, seq_off,    \
                               sloc, cdec, la, H, N, P, ntn, ntp))
  if (vec) SM_GC(true);
  else SM_GC(false);
#undef SM_GC
  hipLaunchKernelGGL(gla_chunk_scan_kernel, dim3(n, H, (N * P + NT - 1) / NT), dim3(NT), 0, st, sloc, cdec, state, seq_slot,
                     seq_start, seq_len, H, N, P);
#define SM_GOV(PT, FUSE, V)                                                                                                  \
  SM_T(f32, hipLaunchKernelGGL((gla_chunk_out_kernel<T, PT, FUSE, V>), dim3(max_chunks * ((P + 16 * PT - 1) / (16 * PT)), n, \
                               H), dim3(NT), 0, st, (const T*)u, ld, la, seq_len, seq_off, sloc, norm_w, (T*)out, y, H, N, P, \
                               (P + 16 * PT - 1) / (16 * PT), eps))
#define SM_GO(PT, FUSE)              \
  do {                               \
    if (vec) SM_GOV(PT, FUSE, true); \
    else SM_GOV(PT, FUSE, false);    \
  } while (0)
  if (P <= 64) SM_GO(4, true);
  else if (fuse) SM_GO(8, true);
  else SM_GO(8, false);
#undef SM_GO
#undef SM_GOV
  if (!fuse) {
    const int rc = gla_norm(u, ld, norm_w, out, y, rows, H, N, P, eps, f32, st);
    if (rc) return rc;
  }
  return (int)hipGetLastError();
}

}  // extern "C"
