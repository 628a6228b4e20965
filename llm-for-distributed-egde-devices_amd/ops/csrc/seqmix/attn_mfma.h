// The bf16 prompt attention over a paged cache on the matrix cores, shared by the kernel files that instantiate it.
#pragma once
#include "common.h"
#include "seqmix/seqmix_common.h"

namespace {

// ---------------------------------------------------------------------------------- attention, bf16 MFMA
// Prompt portions in bf16: 64 query rows of one (sequence, head) per workgroup, 16 per wave, on
// v_mfma_f32_16x16x32_bf16.  A key tile is one page of the sequence (64 tokens, rows G * D apart) or
// 64 pooled blocks (fp32 rows rounded to bf16 while staging); per tile S = Q K^T from a padded-row
// LDS image of K, the mask (window / block-complete rule) and the online softmax in fp32 in the
// log2 domain, P to per-wave LDS as bf16, O += P V with V fragments read transposed from the
// row-major V tile.  Tiles wholly outside a workgroup's window are never visited.
constexpr int MQ = 64, MK = 64;

// RH query heads of one kv head per workgroup: a staged key / value tile serves all of them
// (second launch bound: workgroups per CU the register budget must allow - four for 64-wide heads, so the
// 1024 workgroups of a 4096-token, 16-head prompt are resident at once)
// KVS: the value of a cached row is its first Dv numbers (a latent cache, or values that are the keys): the
// staged key tile serves as the value tile, nothing is loaded twice
// EXT: scores are capped (cap tanh(s / cap), cap > 0) and lose slopes[head] * distance; chunked: `window` is a
// chunk size (a query sees its own chunk's start .. itself), else a sliding window beside the sequence's first
// keep_first tokens; sink[head] joins the softmax denominator; the gate is [T, H * Dv], one per output coordinate
// REL (with EXT, no cap, slopes or chunks): a score gains rel[head, min(distance, rel_n - 1)].  A tile all of whose keys
// lie rel_n - 1 or further behind takes one number; for a nearer one the 127 numbers of its distances travel with its
// rows.  Head sizes are dim <= 32 DK and vdim <= 16 DV (multiples of 8, the rest is zero).  The softmax weights enter
// the value product as two bf16 numbers (their rounding and what it left), so they keep more than 16 bits.
struct AttnExt {
  float scale, cap;
  const float* slopes;
  const float* sink;
  int chunked, keep_first;
  const float* rel;
  int rel_n, dim, vdim;
};

template <int DK, int DV, int RH, bool KVS, bool EXT = false, bool REL = false>
__global__ void __launch_bounds__(NT, (DV * RH <= 4 ? (REL && DK > 2 ? 2 : 4) : (DV * RH <= 8 ? 2 : 1))) attn_mfma_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ gate, int gate_ld, const bf16_t* __restrict__ kp,
    const bf16_t* __restrict__ vp, const float* __restrict__ kb, const float* __restrict__ vb,
    const int* __restrict__ seq_slot, const int* __restrict__ seq_start, const int* __restrict__ seq_len,
    const int* __restrict__ seq_off, const int* __restrict__ ptab, int ptab_ld, bf16_t* __restrict__ out, int n, int H,
    int G, int PB, float scale_log2, int window, int pool, int kld, int vld, int out_ld, float out_scale,
    AttnExt ext = AttnExt{}) {
  static_assert(!REL || (EXT && !KVS), "the distance bias extends the EXT form over separate key and value pages");
  constexpr int DP = 32 * DK, DvP = 16 * DV;                 // what the tiles hold
  const int D = REL ? ext.dim : DP, Dv = REL ? ext.vdim : DvP;
  constexpr float LOG2E = 1.4426950408889634f;
  constexpr int KS = DP * 2 + 16, VS = KVS ? KS : DvP * 2 + 16, PS = MK * 2 + 16;    // LDS row strides in bytes
  static_assert(!KVS || DvP <= DP, "a value slice lies inside the key row");
  __shared__ __attribute__((aligned(16))) char k_lds[MK * KS];
  __shared__ __attribute__((aligned(16))) char v_own[KVS ? 16 : MK * VS];
  char* const v_lds = KVS ? k_lds : v_own;
  __shared__ __attribute__((aligned(16))) char p_all[4 * 16 * PS * (REL ? 2 : 1)];
  __shared__ float b_s[REL ? RH : 1][REL ? 2 * MQ : 1];      // this tile's biases: query row - key row + 63
  constexpr int NPID = REL ? 512 : 1024;
  __shared__ int pid_s[NPID];                                // the sequence's first page ids (one global hop per tile less)
  typedef __attribute__((address_space(3))) v4s lds_v4s;
  int qt = blockIdx.x, s = 0;
  for (; s < n; ++s) {
    const int nq = (seq_len[s] + MQ - 1) / MQ;
    if (qt < nq) break;
    qt -= nq;
  }
  if (s == n) return;
  const int h0 = blockIdx.y * RH, g = h0 / (H / G);
  const int start = seq_start[s], len = seq_len[s], off = seq_off[s];
  const int* pt = ptab + (size_t)seq_slot[s] * ptab_ld;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, c16 = lane & 15;
  char* p_lds = p_all + wave * 16 * PS * (REL ? 2 : 1);
  const int wq0 = qt * MQ + wave * 16;                       // this wave's first row inside the portion
  v8s qf[RH][DK];
  {
    const int t = wq0 + c16;
#pragma unroll
    for (int r = 0; r < RH; ++r)
#pragma unroll
      for (int kk = 0; kk < DK; ++kk)
        qf[r][kk] = t < len && (!REL || kk * 32 + 8 * g4 < D) ? *reinterpret_cast<const v8s*>(q + ((size_t)(off + t) * H + h0 + r) * D + kk * 32 + 8 * g4)
                            : v8s{0, 0, 0, 0, 0, 0, 0, 0};
  }
  v4f o[RH][DV];
  float m_i[RH][4], l_i[RH][4];
#pragma unroll
  for (int r = 0; r < RH; ++r) {
#pragma unroll
    for (int i = 0; i < DV; ++i) o[r][i] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) { m_i[r][i] = -INFINITY; l_i[r][i] = 0.f; }
  }
  // EXT: a score in the log2 domain is c1 - c2 / (2^(xs s) + 1) - sl2 (i - j)  (cap tanh(x / cap) written with one
  // exp2 and one rcp; no cap: s scale_log2 - sl2 (i - j)); clo = first position of each row's chunk
  float sl2[RH];
  int clo[4];
  const float c1 = ext.cap * LOG2E, c2 = 2.f * ext.cap * LOG2E, xs = ext.cap > 0.f ? ext.scale * 2.f * LOG2E / ext.cap : 0.f;
#pragma unroll
  for (int r = 0; r < RH; ++r) sl2[r] = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) clo[i] = 0;
  if constexpr (EXT) {
    if (window > 0) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int qpos = start + wq0 + 4 * g4 + i;
        clo[i] = ext.chunked ? (qpos / window) * window : max(0, qpos - window + 1);
      }
    }
#pragma unroll
    for (int r = 0; r < RH; ++r) {
      if (ext.slopes) sl2[r] = ext.slopes[h0 + r] * LOG2E;
      if (ext.sink) {                                        // the sink: a starting maximum with sum 1 and no value
#pragma unroll
        for (int i = 0; i < 4; ++i) { m_i[r][i] = ext.sink[h0 + r] * LOG2E; l_i[r][i] = 1.f; }
      }
    }
  }
  const int imin = start + qt * MQ, imax = start + min(len, qt * MQ + MQ) - 1;
  const int jlo = window > 0 ? ((EXT && ext.chunked) ? (imin / window) * window : max(0, imin - window + 1)) : 0;
  const int nbmax = (window > 0 && pool > 0 && imax - window + 1 > 0) ? (imax - window + 1) / pool : 0;
  // the tiles that hold kept first tokens and lie wholly before the window's first tile come first
  const int nfirst = (EXT && window > 0 && !ext.chunked) ? min((ext.keep_first + MK - 1) / MK, jlo / MK) : 0;
  const int tok_tiles = nfirst + imax / MK - jlo / MK + 1, ntiles = tok_tiles + (nbmax + MK - 1) / MK;
  auto tile_base = [&](int tile) {                           // first position (token tiles) / block (pooled tiles) of a tile
    return tile < nfirst ? tile * MK : tile < tok_tiles ? (jlo / MK + tile - nfirst) * MK : (tile - tok_tiles) * MK;
  };
  auto rel_far = [&](int base) { return imin - (base + MK - 1) >= ext.rel_n - 1; };
  float breg[REL ? RH : 1] = {}, bfar[REL ? RH : 1];
  if constexpr (REL) {
#pragma unroll
    for (int r = 0; r < RH; ++r) bfar[r] = ext.rel[(size_t)(h0 + r + 1) * ext.rel_n - 1] * LOG2E;
  }
  for (int i = tid; i < min(imax / MK + 1, NPID); i += NT) pid_s[i] = pt[i];
  __syncthreads();
  auto page_of = [&](int idx) { return idx < NPID ? pid_s[idx] : pt[idx]; };

  // a tile's rows travel global -> registers while the tile before it computes, registers -> LDS
  // between the two barriers
  static_assert(DV % 2 == 0, "value chunks per thread");
  constexpr int KL = DK, VL = KVS ? 0 : DV / 2;              // 16-byte chunks per thread per tile
  uint4 kreg[KL], vreg[VL > 0 ? VL : 1];
  auto load_tile = [&](int tile) {
    const bool tok = tile < tok_tiles;
    const int base = tile_base(tile);
    const size_t prow = tok ? (size_t)page_of(base / MK) * MK : 0;
#pragma unroll
    for (int i = 0; i < KL + VL; ++i) {
      const bool isk = i < KL;
      const int e = tid + (isk ? i : i - KL) * NT, cpr = isk ? DP / 8 : DvP / 8;
      const int r = e / cpr, c = e % cpr;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (REL && c * 8 >= (isk ? D : Dv)) {
      } else if (tok) {
        v = isk ? *reinterpret_cast<const uint4*>(kp + (prow + r) * kld + g * D + c * 8)
                : *reinterpret_cast<const uint4*>(vp + (prow + r) * vld + g * Dv + c * 8);
      } else if (base + r < nbmax) {
        const int p0 = (base + r) * pool;
        const size_t row = ((size_t)page_of(p0 / MK) * PB + (p0 % MK) / pool) * G + g;
        float f[8];
        load8<float>(isk ? kb + row * D + c * 8 : vb + row * Dv + c * 8, f);
        v = pack8(f);
      }
      if (isk) kreg[i] = v;
      else vreg[VL > 0 ? i - KL : 0] = v;
    }
    if constexpr (REL) {
      if (tid < 2 * MQ && !rel_far(base)) {
        const int dist = min(max(imin - base + tid - (MK - 1), 0), ext.rel_n - 1);
#pragma unroll
        for (int r = 0; r < RH; ++r) breg[r] = ext.rel[(size_t)(h0 + r) * ext.rel_n + dist] * LOG2E;
      }
    }
  };
  auto store_tile = [&]() {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int e = tid + i * NT;
      *reinterpret_cast<uint4*>(k_lds + (e / (DP / 8)) * KS + (e % (DP / 8)) * 16) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int e = tid + i * NT;
      *reinterpret_cast<uint4*>(v_lds + (e / (DvP / 8)) * VS + (e % (DvP / 8)) * 16) = vreg[i];
    }
    if constexpr (REL) {
      if (tid < 2 * MQ) {
#pragma unroll
        for (int r = 0; r < RH; ++r) b_s[r][tid] = breg[r];  // a far tile's are not read
      }
    }
  };
  if (ntiles > 0) load_tile(0);
  for (int tile = 0; tile < ntiles; ++tile) {
    const bool tok = tile < tok_tiles;
    const int base = tile_base(tile);
    __syncthreads();                                         // every wave is done with the previous tile
    store_tile();
    __syncthreads();
    if (tile + 1 < ntiles) load_tile(tile + 1);
    const bool far = REL && rel_far(base);
#pragma unroll
    for (int r = 0; r < RH; ++r) {
    v4f sc[4];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) {
      sc[nt] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < DK; ++kk) {
        const v8s kf = *reinterpret_cast<const v8s*>(k_lds + (nt * 16 + c16) * KS + (kk * 32 + 8 * g4) * 2);
        sc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[r][kk], kf, sc[nt], 0, 0, 0);
      }
    }
    // lane holds S[row = 4 g4 + i][key = 16 nt + c16]
    float alpha[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int qpos = start + wq0 + 4 * g4 + i;
      const int seen = (window > 0 && pool > 0 && qpos - window + 1 > 0) ? (qpos - window + 1) / pool : 0;
      float mx = -INFINITY;
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        const int key = base + nt * 16 + c16;
        bool vis;
        float v;
        if constexpr (EXT) {
          vis = key <= qpos && (key >= clo[i] || key < ext.keep_first);
          const float bias = REL ? 0.f : sl2[r] * (float)(qpos - key);
          if constexpr (REL)
            v = sc[nt][i] * scale_log2 + (far ? bfar[r] : b_s[r][wave * 16 + 4 * g4 + i + MK - 1 - nt * 16 - c16]);
          else if (ext.cap > 0.f)                                 // 2^(xs s) = inf gives the cap itself, 0 gives -cap
            v = c1 - c2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(sc[nt][i] * xs) + 1.f) - bias;
          else
            v = sc[nt][i] * scale_log2 - bias;
          v = vis ? v : -INFINITY;
        } else {
          vis = tok ? (key <= qpos && (window <= 0 || qpos - key < window)) : key < seen;
          v = vis ? sc[nt][i] * scale_log2 : -INFINITY;
        }
        sc[nt][i] = v;
        mx = fmaxf(mx, v);
      }
#pragma unroll
      for (int o_ = 1; o_ < 16; o_ <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o_, 64));
      const float mnew = fmaxf(m_i[r][i], mx);
      const float msafe = (mnew == -INFINITY) ? 0.f : mnew;
      alpha[i] = __builtin_amdgcn_exp2f(m_i[r][i] - msafe);
      float rs = 0.f;
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        const float p = __builtin_amdgcn_exp2f(sc[nt][i] - msafe);
        sc[nt][i] = p;
        rs += p;
      }
#pragma unroll
      for (int o_ = 1; o_ < 16; o_ <<= 1) rs += __shfl_xor(rs, o_, 64);
      l_i[r][i] = l_i[r][i] * alpha[i] + rs;
      m_i[r][i] = mnew;
    }
#pragma unroll
    for (int dt = 0; dt < DV; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[r][dt][i] *= alpha[i];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i)
      {
        const bf16_t hi = f2bf(sc[nt][i]);
        *reinterpret_cast<bf16_t*>(p_lds + (4 * g4 + i) * PS + (nt * 16 + c16) * 2) = hi;
        if constexpr (REL)
          *reinterpret_cast<bf16_t*>(p_lds + (16 + 4 * g4 + i) * PS + (nt * 16 + c16) * 2) = f2bf(sc[nt][i] - bf2f(hi));
      }
    __builtin_amdgcn_s_waitcnt(0xC07F);                      // lgkmcnt(0): this wave's P rows are in LDS
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const v8s pf = *reinterpret_cast<const v8s*>(p_lds + c16 * PS + (ks * 32 + 8 * g4) * 2);
      v8s pl = pf;
      if constexpr (REL) pl = *reinterpret_cast<const v8s*>(p_lds + (16 + c16) * PS + (ks * 32 + 8 * g4) * 2);
      const int key0 = ks * 32 + 8 * g4, qq = c16 >> 2, pp = c16 & 3;
#pragma unroll
      for (int dt = 0; dt < DV; ++dt) {
        const char* a0 = v_lds + (key0 + qq) * VS + (dt * 16 + 4 * pp) * 2;
        const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)(a0));
        const v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)(a0 + 4 * VS));
        const v8s vf = v8s{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
        o[r][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf, vf, o[r][dt], 0, 0, 0);
        if constexpr (REL) o[r][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, vf, o[r][dt], 0, 0, 0);
      }
    }
      __builtin_amdgcn_wave_barrier();                     // this wave's P reads precede the next head's P writes
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = wq0 + 4 * g4 + i;
    if (t < len) {
#pragma unroll
      for (int r = 0; r < RH; ++r) {
        float inv = l_i[r][i] > 0.f ? 1.f / l_i[r][i] : 0.f;
        if constexpr (!EXT) {
          if (gate) inv *= sigmoidf_(bf2f(gate[(size_t)(off + t) * gate_ld + h0 + r]));
        }
#pragma unroll
        for (int dt = 0; dt < DV; ++dt) {
          float ov = o[r][dt][i] * inv;
          if (REL && dt * 16 + c16 >= Dv) continue;
          if constexpr (EXT) {
            if (gate) ov *= sigmoidf_(bf2f(gate[(size_t)(off + t) * gate_ld + (h0 + r) * Dv + dt * 16 + c16]));
          }
          out[(size_t)(off + t) * out_ld + (h0 + r) * Dv + dt * 16 + c16] = f2bf(ov * out_scale);
        }
      }
    }
  }
}

}  // namespace
