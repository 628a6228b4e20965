// Prompt attention with a learned bias by distance: the instantiations of attn_mfma_kernel that edge_sm_attention_mfma
// picks when a bias table is given (bf16, separate key and value pages).
#include "common.h"
#include "seqmix/attn_mfma.h"

extern "C" {

// returns 1 when no instantiation takes (D, Dv)
int edge_sm_attention_mfma_rel(const void* q, const void* gate, int gate_ld, const void* kp, const void* vp, const int* seq_slot,
                               const int* seq_start, const int* seq_len, const int* seq_off, const int* ptab, int ptab_ld,
                               void* out, int n, int qtiles, int H, int G, int D, int Dv, float scale, int window, int kld, int vld,
                               const float* sink, int keep_first, const float* rel, int rel_n, int out_ld, float out_scale, int rh,
                               hipStream_t st) {
  if (D % 8 || Dv % 8 || D > 128 || Dv > 128 || rel_n < 1) return 1;
  AttnExt ext{};
  ext.scale = scale; ext.sink = sink; ext.keep_first = keep_first; ext.rel = rel; ext.rel_n = rel_n; ext.dim = D; ext.vdim = Dv;
  const float sl2 = scale * 1.4426950408889634f;
#define SM_REL(DK, DV, RH)                                                                                                   \
  hipLaunchKernelGGL((attn_mfma_kernel<DK, DV, RH, false, true, true>), dim3(qtiles, H / RH), dim3(NT), 0, st,                \
                     (const bf16_t*)q, (const bf16_t*)gate, gate_ld, (const bf16_t*)kp, (const bf16_t*)vp,                    \
                     (const float*)nullptr, (const float*)nullptr, seq_slot, seq_start, seq_len, seq_off, ptab, ptab_ld,      \
                     (bf16_t*)out, n, H, G, 0, sl2, window, 0, kld, vld, out_ld, out_scale, ext)
#define SM_REL_R(DK, DV)                 \
  do {                                   \
    if (rh == 4) SM_REL(DK, DV, 4);      \
    else if (rh == 2) SM_REL(DK, DV, 2); \
    else SM_REL(DK, DV, 1);              \
  } while (0)
  if (D <= 64) {
    if (Dv <= 64) SM_REL_R(2, 4);
    else if (Dv <= 96) SM_REL_R(2, 6);
    else SM_REL_R(2, 8);
  } else {
    if (Dv <= 64) SM_REL_R(4, 4);
    else if (Dv <= 96) SM_REL_R(4, 6);
    else SM_REL_R(4, 8);
  }
#undef SM_REL_R
#undef SM_REL
  return (int)hipGetLastError();
}

}  // extern "C"
