// Prompt attention: the entry point, and the forms whose values are as wide as their keys (the kernel is in
// attention_prefill_kernel.h; the forms with other value widths are compiled in a file of their own).
#include "attention_prefill_kernel.h"

// the head sizes the kernel is compiled for with values of the same width
#define SHARPI_PREFILL_HEAD_SIZES(X) X(32) X(64) X(96) X(128) X(160) X(192)

// defined beside the kernels with other value widths
int prefill_other_values(int hd, int vd, const PrefillArgs& a, hipStream_t stream);
int prefill_takes_other_values(int hd, int vd);

// q [T, nh, hd] bf16; caches K [pages, nkv, page_size, hd], V [pages, nkv, vd, page_size] bf16;
// tiles int32 [n_tiles, 3] = (entry, first token, rows <= tile_tokens), tokens of a tile consecutive
// in one entry; tile_tokens 128 or 64 (what the caller cut the tiles to: no tile may hold more);
// out [T, nh, vd] bf16 (rows of the listed tiles).  softcap > 0: scores become softcap * tanh(score /
// softcap); sink: the denominator holds one more term exp(0), or, with sink_vals (float [nh]),
// exp(sink_vals[head]): a learned score per head that is not scaled.  keep > 0: keys at positions below it
// are seen beside the window's.  gate (or null): bf16 rows of gate_stride elements, row t's element h gates
// head h of token t (the output times its sigmoid).
SHARPI_EXPORT int sharpi_attention_prefill(const void* q, const void* k_cache, const void* v_cache,
                                           const int* block_table, const int* positions, const int* tiles,
                                           void* out, int n_tiles, int tile_tokens, int window_kind, int window,
                                           float scale, int nh, int nkv, int hd, int vd, int page_size, int max_blocks,
                                           int num_pages, float softcap, int sink, const float* sink_vals, int keep,
                                           const void* gate, int gate_stride, hipStream_t stream) {
  if (n_tiles <= 0) return SHARPI_OK;
  if (nh <= 0 || nkv <= 0 || nh % nkv != 0 || n_tiles > 65535) return SHARPI_ERR_ARG;
  if (tile_tokens != kTileTokens && tile_tokens != kTileTokens / 2) return SHARPI_ERR_ARG;
  if (page_size <= 0 || page_size % 16 != 0 || max_blocks <= 0 || num_pages <= 0) return SHARPI_ERR_ARG;
  if (window_kind < 0 || window_kind > 2 || (window_kind != 0 && window <= 0) || !(softcap >= 0.f)) return SHARPI_ERR_ARG;
  if (keep < 0 || (gate && gate_stride < nh)) return SHARPI_ERR_ARG;
  if (window_kind == 0) keep = 0;             // (every earlier key is seen as it is)
  const PrefillArgs a{q, k_cache, v_cache, block_table, positions, tiles, out, n_tiles, tile_tokens, window_kind, window, scale, nh,
                      nkv, page_size, max_blocks, num_pages, softcap, sink, sink_vals, keep, gate, gate_stride};
  if (vd != hd) return prefill_other_values(hd, vd, a, stream);
#define PRE(HDV) if (hd == HDV) return launch_prefill<HDV, HDV>(a, stream);
  SHARPI_PREFILL_HEAD_SIZES(PRE)
#undef PRE
  return SHARPI_ERR_ARG;  // other head sizes go to the generic kernel
}

// 1 if the kernel is compiled for keys of width hd and values of width vd (the caller's choice of kernel asks here).
SHARPI_EXPORT int sharpi_attention_prefill_takes(int hd, int vd) {
  if (vd != hd) return prefill_takes_other_values(hd, vd);
#define PRE(HDV) if (hd == HDV) return 1;
  SHARPI_PREFILL_HEAD_SIZES(PRE)
#undef PRE
  return 0;
}

SHARPI_EXPORT int sharpi_attention_prefill_tile_tokens() { return kTileTokens; }
