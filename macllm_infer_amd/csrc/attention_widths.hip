// Prompt attention on the matrix cores for heads of other widths than 64 or 128, and for keys and values of different
// widths with every term of a softmax.
#include "attn_prefill.h"

// The kernel of attn_prefill.h for keys of any width up to 128 in steps of 8 beside values of any width up to 128 in steps of 4, with every
// term of a softmax but the logarithmic bias: a bias by distance (slopes), sinks, kept first keys behind a window, a gate
// on the outputs.  The products run at the next width of 64, 96 or 128.
// Returns ERR_UNSUPPORTED_SIZE for shapes it does not cover (the caller uses mi_paged_attention).
extern "C" int mi_prefill_attention_padded(const void* q, long q_ld, int Hq, int Hkv, int dh, int dv, const void* k_base,
                                           const void* v_base, long page_stride, int page_size,
                                           const int* block_tables, int max_pages, const int* tiles, int n_tiles,
                                           const int* cu_seqlens, const int* start_pos, float scale, int window,
                                           int max_seq_len, void* out, long out_ld, const float* sinks,
                                           int kept, const float* slopes, const void* gate,
                                           long gate_ld, hipStream_t stream) {
  if (n_tiles <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || page_size <= 0 || max_pages <= 0 || dh <= 0 || dv <= 0)
    return ERR_BAD_ARGUMENT;
  if (kept < 0 || (kept > 0 && window <= 0)) return ERR_BAD_ARGUMENT;
  if (gate && (gate_ld < (long)Hq * dv || gate_ld % 4 != 0 || (uintptr_t)gate % 8 != 0)) return ERR_BAD_ARGUMENT;
  const int G = Hq / Hkv;
  if (dh % 8 != 0 || dh > 128 || dv % 4 != 0 || dv > 128 || page_size % 4 != 0 || q_ld % 8 != 0 || out_ld % 4 != 0 ||
      Hkv > 65535 || G > 64 || n_tiles > (1 << 28))
    return ERR_UNSUPPORTED_SIZE;
  const int key_width = dh <= 64 ? 64 : dh <= 96 ? 96 : 128;
  const int width = dv <= 64 ? 64 : dv <= 96 ? 96 : 128;
  int most = key_width == 64 && width == 64 ? 4 : 2;
  if (most > 2 && max_seq_len <= 2048 && 4L * n_tiles * Hkv * ((G + most - 1) / most) < PREFILL_FILL_BLOCKS) most = 2;
  const int passes = (G + most - 1) / most;
  const int nset = (G + passes - 1) / passes;
  const dim3 grid(4 * n_tiles, Hkv, passes);
#define WIDTH_LAUNCH(DH_, DV_, NSET_, BIAS_)                                                                    \
  prefill_attention_kernel<DH_, NSET_, BIAS_, DV_, false, true, true><<<grid, PREFILL_WAVES * WAVE, 0, stream>>>( \
      (const bf16_t*)q, q_ld, Hq, Hkv, (const bf16_t*)k_base, (const bf16_t*)v_base, page_stride, page_size,    \
      block_tables, max_pages, tiles, cu_seqlens, start_pos, scale, window, (bf16_t*)out, out_ld, nullptr, sinks, \
      dv, nullptr, nullptr, kept, slopes, (const bf16_t*)gate, gate_ld, dh)
#define WIDTH_CASE(DH_, DV_, NSET_)                                                                             \
  if (key_width == DH_ && width == DV_ && nset == NSET_) {                                                      \
    if (slopes) WIDTH_LAUNCH(DH_, DV_, NSET_, BIAS_LINEAR);                                                     \
    else WIDTH_LAUNCH(DH_, DV_, NSET_, BIAS_NONE);                                                              \
  }
  WIDTH_CASE(64, 64, 1) WIDTH_CASE(64, 64, 2) WIDTH_CASE(64, 64, 3) WIDTH_CASE(64, 64, 4)
  WIDTH_CASE(64, 96, 1) WIDTH_CASE(64, 96, 2) WIDTH_CASE(64, 128, 1) WIDTH_CASE(64, 128, 2)
  WIDTH_CASE(96, 64, 1) WIDTH_CASE(96, 64, 2) WIDTH_CASE(96, 96, 1) WIDTH_CASE(96, 96, 2)
  WIDTH_CASE(96, 128, 1) WIDTH_CASE(96, 128, 2) WIDTH_CASE(128, 64, 1) WIDTH_CASE(128, 64, 2)
  WIDTH_CASE(128, 96, 1) WIDTH_CASE(128, 96, 2) WIDTH_CASE(128, 128, 1) WIDTH_CASE(128, 128, 2)
#undef WIDTH_CASE
#undef WIDTH_LAUNCH
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}
