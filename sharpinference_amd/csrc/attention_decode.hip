// Attention for single tokens: the entry points, and the forms whose values are as wide as their keys (the kernel
// is in attention_decode_kernel.h; the forms with other value widths are compiled in a file of their own).
#include "attention_decode_kernel.h"
#include "sharpi_noalloc.h"
#include <mutex>

// the head sizes the kernel is compiled for with values of the same width
#define SHARPI_DECODE_HEAD_SIZES(X) X(32) X(64) X(96) X(128) X(160) X(192) X(224) X(256)

// defined beside the kernels with other value widths
int decode_other_values(int hd, int vd, const DecodeArgs& a, hipStream_t stream);
int decode_takes_other_values(int hd, int vd);

// q [T, nh, hd] bf16; caches K [pages, nkv, page_size, hd], V [pages, nkv, vd, page_size] bf16;
// token_list [n_list] (or null: tokens 0..n_list-1); part_o float [n_list, nh, max_splits, vd];
// part_ml float [n_list, nh, max_splits, 2]; out [T, nh, vd] bf16 (rows of the listed tokens).
// max_splits must cover every listed token: a token walks the 16-key blocks from its window's first key to its own
// (and, with keep > 0, those that hold the sequence's first `keep` keys), 16 of them a run;
// ((context - 1) >> 4) / 16 + 1 runs cover every window of a
// context.  A token whose runs exceed max_splits gets a row of NaN.  softcap > 0: scores become
// softcap * tanh(score / softcap); sink: the denominator holds one more term exp(0), or, with sink_vals
// (float [nh]), exp(sink_vals[head]): a learned score per head that is not scaled.  gate (or null): bf16 rows of
// gate_stride elements, row t's element h gates head h of token t (the output times its sigmoid).
SHARPI_EXPORT int sharpi_attention_decode_values(const void* q, const void* k_cache, const void* v_cache,
                                                 const int* block_table, const int* entry_of_token, const int* positions,
                                                 const int* token_list, float* part_o, float* part_ml, void* out,
                                                 int window_kind, int window, float scale, int n_list, int nh, int nkv,
                                                 int hd, int vd, int page_size, int max_blocks, int num_pages, int max_splits,
                                                 float softcap, int sink, const float* sink_vals, int keep, const void* gate,
                                                 int gate_stride, hipStream_t stream) {
  if (n_list <= 0) return SHARPI_OK;
  if (nh <= 0 || nkv <= 0 || nh % nkv != 0 || nh > 65535 || n_list > 65535) return SHARPI_ERR_ARG;
  if (page_size <= 0 || page_size % 16 != 0 || max_blocks <= 0 || num_pages <= 0 || max_splits <= 0 || max_splits > 65535) return SHARPI_ERR_ARG;
  if (window_kind < 0 || window_kind > 2 || (window_kind != 0 && window <= 0) || !(softcap >= 0.f)) return SHARPI_ERR_ARG;
  if (nkv * ((nh / nkv + 15) / 16) > 65535) return SHARPI_ERR_ARG;
  if (keep < 0 || (gate && gate_stride < nh)) return SHARPI_ERR_ARG;
  if (window_kind == 0) keep = 0;             // (every earlier key is seen as it is)
  const DecodeArgs a{q, k_cache, v_cache, block_table, entry_of_token, positions, token_list, part_o, part_ml, out, window_kind,
                     window, scale, n_list, nh, nkv, page_size, max_blocks, num_pages, max_splits, softcap, sink, sink_vals, keep,
                     gate, gate_stride};
  if (vd != hd) return decode_other_values(hd, vd, a, stream);
#define DEC(HDV) if (hd == HDV) return launch_decode<HDV, HDV>(a, stream);
  SHARPI_DECODE_HEAD_SIZES(DEC)
#undef DEC
  return SHARPI_ERR_ARG;  // other head sizes go to the generic kernel
}

// The same for values as wide as the keys, without kept tokens and without a gate.
SHARPI_EXPORT int sharpi_attention_decode(const void* q, const void* k_cache, const void* v_cache,
                                          const int* block_table, const int* entry_of_token, const int* positions,
                                          const int* token_list, float* part_o, float* part_ml, void* out,
                                          int window_kind, int window, float scale, int n_list, int nh, int nkv,
                                          int hd, int page_size, int max_blocks, int num_pages, int max_splits,
                                          float softcap, int sink, const float* sink_vals, hipStream_t stream) {
  return sharpi_attention_decode_values(q, k_cache, v_cache, block_table, entry_of_token, positions, token_list, part_o, part_ml,
                                        out, window_kind, window, scale, n_list, nh, nkv, hd, hd, page_size, max_blocks,
                                        num_pages, max_splits, softcap, sink, sink_vals, 0, nullptr, 0, stream);
}

// 1 if the kernel is compiled for keys of width hd and values of width vd (the caller's choice of kernel asks here).
SHARPI_EXPORT int sharpi_attention_decode_takes(int hd, int vd) {
  if (vd != hd) return decode_takes_other_values(hd, vd);
#define DEC(HDV) if (hd == HDV) return 1;
  SHARPI_DECODE_HEAD_SIZES(DEC)
#undef DEC
  return 0;
}

SHARPI_EXPORT int sharpi_attention_decode_split_keys() { return kSplitBlocks * 16; }

// ---------------------------------------------------------------------------------------------
// The same without workspace arguments, for callers that cannot allocate: the partial results go
// to a file-scope device array.  In host code the array's name is only a stand-in for the symbol,
// not a device address; each device's address is looked up once, with that device current, and
// that pointer is what the kernels get.
static __device__ __align__(256) float scratch[SHARPI_NOALLOC_SCRATCH_FLOATS];

constexpr int kMaxDevices = 64;
static float* scratch_of_device[kMaxDevices];   // per device: where its copy of `scratch` lies
static std::mutex scratch_lock;

static int scratch_here(float** out) {
  int dev = -1;
  hipError_t e = hipGetDevice(&dev);
  if (e != hipSuccess) return (int)e;
  if (dev < 0 || dev >= kMaxDevices) return SHARPI_ERR_ARG;
  std::lock_guard<std::mutex> guard(scratch_lock);
  if (!scratch_of_device[dev]) {
    float* p = nullptr;
    e = hipGetSymbolAddress((void**)&p, HIP_SYMBOL(scratch));
    if (e != hipSuccess) return (int)e;
    if (!p) return SHARPI_ERR_LAUNCH;
    scratch_of_device[dev] = p;
  }
  *out = scratch_of_device[dev];
  return SHARPI_OK;
}

int sharpi_attention_decode_noalloc(const void* q, const void* k_cache, const void* v_cache, const int* block_table,
                                    const int* entry_of_token, const int* positions, const int* token_list, void* out,
                                    int window_kind, int window, float scale, int n_list, int nh, int nkv, int hd,
                                    int page_size, int max_blocks, int num_pages, int max_splits, hipStream_t stream) {
  if (n_list <= 0) return SHARPI_OK;
  if (nh <= 0 || hd <= 0 || max_splits <= 0) return SHARPI_ERR_ARG;
  // part_o [n_list, nh, max_splits, hd] then part_ml [n_list, nh, max_splits, 2]
  const unsigned long long runs = (unsigned long long)n_list * (unsigned long long)nh * (unsigned long long)max_splits;
  if (runs * (unsigned long long)(hd + 2) > (unsigned long long)SHARPI_NOALLOC_SCRATCH_FLOATS) return SHARPI_ERR_ARG;
  float* ws = nullptr;
  const int rc = scratch_here(&ws);
  if (rc != SHARPI_OK) return rc;
  float* part_o = ws;
  float* part_ml = ws + runs * (unsigned long long)hd;   // hd is a multiple of 32: stays 16-byte aligned
  return sharpi_attention_decode(q, k_cache, v_cache, block_table, entry_of_token, positions, token_list, part_o,
                                 part_ml, out, window_kind, window, scale, n_list, nh, nkv, hd, page_size, max_blocks,
                                 num_pages, max_splits, 0.f, 0, nullptr, stream);
}
