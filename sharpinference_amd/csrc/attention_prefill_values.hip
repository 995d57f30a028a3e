// Prompt attention whose values have another width than its keys (the kernel is in attention_prefill_kernel.h).
#include "attention_prefill_kernel.h"

// (key width, value width) pairs the kernel is compiled for
#define SHARPI_PREFILL_VALUE_SIZES(X)                            \
  X(32, 64) X(32, 96) X(32, 128)                                 \
  X(64, 32) X(64, 48) X(64, 96) X(64, 128)                       \
  X(96, 32) X(96, 48) X(96, 64) X(96, 128)                       \
  X(128, 32) X(128, 48) X(128, 64) X(128, 96) X(128, 192)        \
  X(160, 64) X(160, 96) X(160, 128)                              \
  X(192, 64) X(192, 96) X(192, 128)

int prefill_other_values(int hd, int vd, const PrefillArgs& a, hipStream_t stream) {
#define PRE(HDV, VDV) if (hd == HDV && vd == VDV) return launch_prefill<HDV, VDV>(a, stream);
  SHARPI_PREFILL_VALUE_SIZES(PRE)
#undef PRE
  return SHARPI_ERR_ARG;
}

int prefill_takes_other_values(int hd, int vd) {
#define PRE(HDV, VDV) if (hd == HDV && vd == VDV) return 1;
  SHARPI_PREFILL_VALUE_SIZES(PRE)
#undef PRE
  return 0;
}
