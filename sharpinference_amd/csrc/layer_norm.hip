// Layers whose branches end in a layer norm and begin with a short convolution over the residual sum; layers with a
// layer norm of the whole sum behind each branch; the embedding with a second table indexed by a pair of tokens, and
// the embedding with a norm.
//
// layer_norm:      x = h[r] (+ LN(delta[r]) w + b); the new x back into h; and, by what is asked for, x itself, LN of
//                  x (a model's last norm), or x + conv(x) (what the next branch reads; steps of single
//                  tokens) in the activations' storage type.  delta is a tensor or an expert sum still to be formed.
// residual_conv:   out[t] = h[t] + sum_j w[:, j] h[t - taps + 1 + j], for steps that bring longer entries.
// sum_norm:        x = LN(alpha h + delta) w + b, the new x back into h, and x in the activations' storage type.
// embed_norm:      out[t] = LN(table[id] * scale) w + b, likewise with a copy in the activations' storage type.
// embed_bigram:    out[t] = table[id] * scale + pairs[(previous id * a + id * b) mod buckets].
//
// A convolution's last inputs lie in a ring [slots, taps, channels] of floats, position p at p mod taps; what lies
// before position 0 is never read.  Statistics, sums and the residual sum are float.
#include "common.h"

constexpr int kLnMaxTaps = 8;

struct LnDelta {
  const void* y;                 // [T, hidden], or the experts' rows
  const int* pos;                // [T, k]: places of a token's rows (null: y is a tensor)
  const float* w;                // [T, k] or null
  const void* shared;            // [T, hidden] or null (expert sums only)
  int k;
  const int* ids = nullptr;      // [T, k]: picks of n_experts and above are identity experts (sum_norm)
  int n_experts = 0;
  const void* ident = nullptr;   // [T, hidden]: their outputs (null: the row of h itself, in float)
};

template <typename TD, int V>
__device__ __forceinline__ void ln_load(const TD* p, float* v) {
  if constexpr (V == 8) load8(p, v);
  else v[0] = to_f32<TD>(*p);
}
template <typename TO, int V>
__device__ __forceinline__ void ln_store(TO* p, const float* v) {
  if constexpr (V == 8) store8(p, v);
  else *p = from_f32<TO>(v[0]);
}

template <typename TD, int V>
__device__ __forceinline__ void ln_delta(const LnDelta& d, size_t r, int hidden, int c, float* v) {
  if (!d.pos) {
    ln_load<TD, V>((const TD*)d.y + r * hidden + c, v);
    return;
  }
#pragma unroll
  for (int i = 0; i < V; ++i) v[i] = 0.f;
  for (int q0 = 0; q0 < d.k; q0 += 4) {    // (four rows are requested before the first is added)
    float x[4][V], wq[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int q = min(q0 + j, d.k - 1);
      ln_load<TD, V>((const TD*)d.y + (size_t)d.pos[r * d.k + q] * hidden + c, x[j]);
      wq[j] = d.w ? d.w[r * d.k + q] : 1.0f;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (q0 + j < d.k) {
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] = fmaf(wq[j], x[j][i], v[i]);
      }
  }
  if (d.shared) {
    float x[V];
    ln_load<TD, V>((const TD*)d.shared + r * hidden + c, x);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] += x[i];
  }
}

enum : int { LN_COPY = 0, LN_NORM = 1, LN_CONV = 2 };    // what `out` is

struct LnConv {
  const float* w;                // [hidden, taps]
  float* ring;                   // [slots, taps, hidden] (null with one tap)
  int taps;
  const int *positions, *state_slots, *entry_of_token;
};

template <typename TD, typename TO, int V>
__global__ __launch_bounds__(1024) void layer_norm_kernel(float* __restrict__ h, LnDelta delta, const float* __restrict__ w,
                                                          const float* __restrict__ b, float eps, const int* __restrict__ rows,
                                                          int write_back, TO* __restrict__ out, int mode,
                                                          const float* __restrict__ w2, const float* __restrict__ b2, float eps2,
                                                          LnConv cv, int hidden) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[16];
  const size_t i = blockIdx.x, r = rows ? rows[i] : i;
  float* hr = h + r * hidden;
  const int step = blockDim.x * V, c_first = threadIdx.x * V;
  float x[V], y[V], wv[V], bv[V];
  if (delta.y) {
    float s = 0.f;
    for (int c = c_first; c < hidden; c += step) {
      ln_delta<TD, V>(delta, r, hidden, c, y);
      ln_store<float, V>(row + c, y);
#pragma unroll
      for (int k = 0; k < V; ++k) s += y[k];
    }
    const float mean = block_sum(s, red) / (float)hidden;
    s = 0.f;
    for (int c = c_first; c < hidden; c += step) {     // (a thread reads what it wrote)
      ln_load<float, V>(row + c, y);
#pragma unroll
      for (int k = 0; k < V; ++k) s = fmaf(y[k] - mean, y[k] - mean, s);
    }
    const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, y);
      ln_load<float, V>(hr + c, x);
      ln_load<float, V>(w + c, wv);
      ln_load<float, V>(b + c, bv);
#pragma unroll
      for (int k = 0; k < V; ++k) x[k] += fmaf((y[k] - mean) * inv, wv[k], bv[k]);
      if (write_back) ln_store<float, V>(hr + c, x);
      if (out) ln_store<float, V>(row + c, x);
    }
  } else {
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(hr + c, x);
      ln_store<float, V>(row + c, x);
    }
  }
  if (!out) return;
  TO* o = out + i * hidden;
  if (mode == LN_COPY) {
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, x);
      ln_store<TO, V>(o + c, x);
    }
  } else if (mode == LN_NORM) {
    float s = 0.f;
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, x);
#pragma unroll
      for (int k = 0; k < V; ++k) s += x[k];
    }
    const float mean = block_sum(s, red) / (float)hidden;
    s = 0.f;
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, x);
#pragma unroll
      for (int k = 0; k < V; ++k) s = fmaf(x[k] - mean, x[k] - mean, s);
    }
    const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps2);
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, x);
      ln_load<float, V>(w2 + c, wv);
      ln_load<float, V>(b2 + c, bv);
#pragma unroll
      for (int k = 0; k < V; ++k) x[k] = fmaf((x[k] - mean) * inv, wv[k], bv[k]);
      ln_store<TO, V>(o + c, x);
    }
  } else {
    const int p = cv.positions[r];
    float* ring = cv.ring ? cv.ring + (size_t)cv.state_slots[cv.entry_of_token[r]] * cv.taps * hidden : nullptr;
    for (int c = c_first; c < hidden; c += step) {
      ln_load<float, V>(row + c, x);
#pragma unroll
      for (int k = 0; k < V; ++k) y[k] = 0.f;
      for (int back = cv.taps - 1; back > 0; --back)
        if (p >= back) {
          float u[V];
          ln_load<float, V>(ring + (size_t)((p - back) % cv.taps) * hidden + c, u);
#pragma unroll
          for (int k = 0; k < V; ++k) y[k] = fmaf(cv.w[(size_t)(c + k) * cv.taps + cv.taps - 1 - back], u[k], y[k]);
        }
      if (ring) ln_store<float, V>(ring + (size_t)(p % cv.taps) * hidden + c, x);
#pragma unroll
      for (int k = 0; k < V; ++k) x[k] += fmaf(cv.w[(size_t)(c + k) * cv.taps + cv.taps - 1], x[k], y[k]);
      ln_store<TO, V>(o + c, x);
    }
  }
}

// The same where a thread has one run of eight elements of the row (hidden a multiple of 8 up to 8,192): everything stays in
// registers, and what is needed behind the two reductions (h, weights, the earlier inputs of the convolution) is
// requested before them: with a handful of rows (decode) the kernel is nothing but the latency of its loads.
template <typename TD, typename TO, int TAPS>      // TAPS: the convolution's (LN_CONV), else 0
__global__ __launch_bounds__(1024) void layer_norm_run_kernel(float* __restrict__ h, LnDelta delta, const float* __restrict__ w,
                                                              const float* __restrict__ b, float eps, const int* __restrict__ rows,
                                                              int write_back, TO* __restrict__ out, int mode,
                                                              const float* __restrict__ w2, const float* __restrict__ b2, float eps2,
                                                              LnConv cv, int hidden) {
  __shared__ float red[16];
  constexpr int N = TAPS > 1 ? TAPS : 1;
  const size_t i = blockIdx.x, r = rows ? rows[i] : i;
  const int c = threadIdx.x * 8;
  const bool in = c < hidden;
  float* hr = h + r * hidden;
  float x[8], y[8], wv[8], bv[8], past[N][8], cw[N * 8];
  float* ring = nullptr;
  int p = 0;
  if (in) {
    load8(hr + c, x);
    if (delta.y) {
      ln_delta<TD, 8>(delta, r, hidden, c, y);
      load8(w + c, wv);
      load8(b + c, bv);
    }
    if constexpr (TAPS > 0) {
      p = cv.positions[r];
#pragma unroll
      for (int k = 0; k < TAPS; ++k) load8(cv.w + (size_t)c * TAPS + k * 8, cw + k * 8);      // channel c + k's taps at k TAPS
      if constexpr (TAPS > 1) {
        ring = cv.ring + (size_t)cv.state_slots[cv.entry_of_token[r]] * TAPS * hidden + c;
#pragma unroll
        for (int back = 1; back < TAPS; ++back)          // (before position 0: some row of the ring, not used)
          load8(ring + (size_t)((p + TAPS - back) % TAPS) * hidden, past[back]);
      }
    }
  }
  if (delta.y) {
    float s = 0.f;
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) s += y[k];
    }
    const float mean = block_sum(s, red) / (float)hidden;
    s = 0.f;
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) s = fmaf(y[k] - mean, y[k] - mean, s);
    }
    const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) x[k] += fmaf((y[k] - mean) * inv, wv[k], bv[k]);
      if (write_back) store8(hr + c, x);
    }
  }
  if (!out) return;
  TO* o = out + i * hidden + c;
  if (mode == LN_COPY) {
    if (in) store8(o, x);
  } else if (mode == LN_NORM) {
    float s = 0.f;
    if (in) {
      load8(w2 + c, wv);
      load8(b2 + c, bv);
#pragma unroll
      for (int k = 0; k < 8; ++k) s += x[k];
    }
    const float mean = block_sum(s, red) / (float)hidden;
    s = 0.f;
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) s = fmaf(x[k] - mean, x[k] - mean, s);
    }
    const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps2);
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) x[k] = fmaf((x[k] - mean) * inv, wv[k], bv[k]);
      store8(o, x);
    }
  } else if constexpr (TAPS > 0) {
    if (in) {
#pragma unroll
      for (int k = 0; k < 8; ++k) y[k] = 0.f;
#pragma unroll
      for (int back = TAPS - 1; back > 0; --back)
#pragma unroll
        for (int k = 0; k < 8; ++k) y[k] = p >= back ? fmaf(cw[k * TAPS + TAPS - 1 - back], past[back][k], y[k]) : y[k];
      if constexpr (TAPS > 1) store8(ring + (size_t)(p % TAPS) * hidden, x);
#pragma unroll
      for (int k = 0; k < 8; ++k) x[k] += fmaf(cw[k * TAPS + TAPS - 1], x[k], y[k]);
      store8(o, x);
    }
  }
}

// h [T, hidden] float.  With delta (y of d_dtype; pos/sum_w/k/shared describe an expert sum): x = h + LN(delta) w + b,
// back into h unless `rows` (int32 [n_rows]: only those rows, h unchanged) is given.  out (o_dtype, or null), mode 0:
// x; 1: LN(x) w2 + b2; 2: x + conv(x) with conv_w float [hidden, taps] and the entries' rings (every entry of
// the step one token: row = token).
SHARPI_EXPORT int sharpi_layer_norm(float* h, const void* delta, int d_dtype, const int* pos, const float* sum_w, int k,
                                    const void* shared, const float* w, const float* b, float eps, const int* rows, int n_rows,
                                    int hidden, void* out, int o_dtype, int mode, const float* w2, const float* b2, float eps2,
                                    const float* conv_w, float* ring, int taps, const int* positions, const int* state_slots,
                                    const int* entry_of_token, hipStream_t stream) {
  if (n_rows <= 0) return SHARPI_OK;
  if (hidden <= 0 || (size_t)hidden * sizeof(float) > 60 * 1024) return SHARPI_ERR_ARG;
  if (delta && (!w || !b || !(eps > 0.f) || (pos && k <= 0))) return SHARPI_ERR_ARG;
  if (!delta && !out) return SHARPI_OK;
  if (mode < 0 || mode > 2 || (mode == LN_NORM && (!w2 || !b2 || !(eps2 > 0.f)))) return SHARPI_ERR_ARG;
  if (mode == LN_CONV && out && (!conv_w || taps < 1 || taps > kLnMaxTaps || (taps > 1 && !ring) || !positions || !state_slots || !entry_of_token || rows))
    return SHARPI_ERR_ARG;
  if ((d_dtype != DT_F32 && d_dtype != DT_BF16) || (out && o_dtype != DT_F32 && o_dtype != DT_BF16)) return SHARPI_ERR_ARG;
  auto aligned = [](const void* p) { return ((uintptr_t)p & 31) == 0; };
  const bool wide = hidden % 8 == 0 && aligned(h) && aligned(delta) && aligned(shared) && aligned(w) && aligned(b) && aligned(out) &&
                    aligned(w2) && aligned(b2) && aligned(ring);
  const LnDelta d{delta, pos, sum_w, shared, k};
  const LnConv cv{conv_w, taps > 1 ? ring : nullptr, taps, positions, state_slots, entry_of_token};
  const int runs = wide ? hidden / 8 : hidden;
  int threads = ceil_div(runs, kWave) * kWave;
  if (threads > (wide ? 1024 : 256)) threads = wide ? 1024 : 256;
  const size_t lds = (size_t)hidden * sizeof(float);
  const int wb = rows ? 0 : 1;
  // (with more taps the registers do not reach)
  if (wide && hidden <= 8192 && (mode != LN_CONV || !out || (aligned(conv_w) && taps <= 5))) {
    const int t = mode == LN_CONV && out ? taps : 0;
#define LNR(TD, TO, TAPS)                                                                                                             \
  case TAPS:                                                                                                                          \
    layer_norm_run_kernel<TD, TO, TAPS><<<n_rows, threads, 0, stream>>>(h, d, w, b, eps, rows, wb, (TO*)out, mode, w2, b2, eps2, cv, hidden); \
    break
#define LNR_BY(TD, TO)                                                                                                                \
  switch (t) {                                                                                                                        \
    LNR(TD, TO, 0); LNR(TD, TO, 1); LNR(TD, TO, 2); LNR(TD, TO, 3); LNR(TD, TO, 4); LNR(TD, TO, 5); \
    default: return SHARPI_ERR_ARG;                                                                                                   \
  }
    const bool to_f = !out || o_dtype == DT_F32;
    if (d_dtype == DT_F32) {
      if (to_f) { LNR_BY(float, float) }
      else { LNR_BY(float, bf16_t) }
    } else {
      if (to_f) { LNR_BY(bf16_t, float) }
      else { LNR_BY(bf16_t, bf16_t) }
    }
#undef LNR_BY
#undef LNR
    SHARPI_CHECK_LAUNCH();
    return SHARPI_OK;
  }
#define LN(TD, TO)                                                                                                                    \
  do {                                                                                                                                \
    if (wide) layer_norm_kernel<TD, TO, 8><<<n_rows, threads, lds, stream>>>(h, d, w, b, eps, rows, wb, (TO*)out, mode, w2, b2, eps2, cv, hidden); \
    else layer_norm_kernel<TD, TO, 1><<<n_rows, threads, lds, stream>>>(h, d, w, b, eps, rows, wb, (TO*)out, mode, w2, b2, eps2, cv, hidden);      \
  } while (0)
  const bool of = !out || o_dtype == DT_F32;
  if (d_dtype == DT_F32) {
    if (of) LN(float, float);
    else LN(float, bf16_t);
  } else {
    if (of) LN(bf16_t, float);
    else LN(bf16_t, bf16_t);
  }
#undef LN
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// ---------------------------------------------------------------------------
// The norm of the sum: x = LN(alpha h[t] + delta[t]) w + b back into h, and, with out, x in the activations' storage
// type.  delta: a tensor or an expert sum still to be formed, whose identity picks add weight * (the layer's input row):
// a row of `ident`, or h itself in float (then they only change the coefficient of h).
// ---------------------------------------------------------------------------
template <typename TD, int V>
__device__ __forceinline__ void sum_of_row(const LnDelta& d, size_t r, int hidden, int c, float alpha, const float* x, float* v) {
  if (!d.ids) {
    ln_delta<TD, V>(d, r, hidden, c, v);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = 0.f;
    for (int q0 = 0; q0 < d.k; q0 += 4) {    // (four rows are requested before the first is added)
      float y[4][V], wq[4];
      bool own[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const size_t q = r * d.k + min(q0 + j, d.k - 1);
        own[j] = d.ids[q] >= d.n_experts;
        const TD* row = own[j] ? (d.ident ? (const TD*)d.ident + r * hidden : nullptr) : (const TD*)d.y + (size_t)d.pos[q] * hidden;
        if (row) ln_load<TD, V>(row + c, y[j]);
        else {
#pragma unroll
          for (int i = 0; i < V; ++i) y[j][i] = x[i];
        }
        wq[j] = d.w ? d.w[q] : 1.0f;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (q0 + j < d.k) {
#pragma unroll
          for (int i = 0; i < V; ++i) v[i] = fmaf(wq[j], y[j][i], v[i]);
        }
    }
    if (d.shared) {
      float y[V];
      ln_load<TD, V>((const TD*)d.shared + r * hidden + c, y);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += y[i];
    }
  }
#pragma unroll
  for (int i = 0; i < V; ++i) v[i] = fmaf(alpha, x[i], v[i]);
}

// A thread has one run of eight elements (hidden a multiple of 8 up to 8,192): everything in registers, all loads ahead of the
// reductions.
template <typename TD, typename TO>
__global__ __launch_bounds__(1024) void sum_norm_run_kernel(float* __restrict__ h, LnDelta delta, float alpha,
                                                            const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                            TO* __restrict__ out, int hidden) {
  __shared__ float red[16];
  const size_t r = blockIdx.x;
  const int c = threadIdx.x * 8;
  const bool in = c < hidden;
  float x[8], y[8], wv[8], bv[8];
  float s = 0.f;
  if (in) {
    load8(h + r * hidden + c, x);
    load8(w + c, wv);
    load8(b + c, bv);
    sum_of_row<TD, 8>(delta, r, hidden, c, alpha, x, y);
#pragma unroll
    for (int k = 0; k < 8; ++k) s += y[k];
  }
  const float mean = block_sum(s, red) / (float)hidden;
  s = 0.f;
  if (in) {
#pragma unroll
    for (int k = 0; k < 8; ++k) s = fmaf(y[k] - mean, y[k] - mean, s);
  }
  const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
  if (in) {
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] = fmaf((y[k] - mean) * inv, wv[k], bv[k]);
    store8(h + r * hidden + c, x);
    if (out) store8(out + r * hidden + c, x);
  }
}

template <typename TD, typename TO>
__global__ __launch_bounds__(256) void sum_norm_kernel(float* __restrict__ h, LnDelta delta, float alpha, const float* __restrict__ w,
                                                       const float* __restrict__ b, float eps, TO* __restrict__ out, int hidden) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[16];
  const size_t r = blockIdx.x;
  float* hr = h + r * hidden;
  float s = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {     // (a thread reads what it wrote)
    float y;
    sum_of_row<TD, 1>(delta, r, hidden, c, alpha, hr + c, &y);
    row[c] = y;
    s += y;
  }
  const float mean = block_sum(s, red) / (float)hidden;
  s = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) s = fmaf(row[c] - mean, row[c] - mean, s);
  const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    const float x = fmaf((row[c] - mean) * inv, w[c], b[c]);
    hr[c] = x;
    if (out) out[r * hidden + c] = from_f32<TO>(x);
  }
}

// h float [T, hidden]; delta [T, hidden] of d_dtype, or (pos) the experts' rows with pos int32 [T, k], sum_w float [T, k] or
// null, shared [T, hidden] or null, and (ids int32 [T, k]) identity picks from n_experts on, whose output is row t of
// ident [T, hidden] of d_dtype or, with ident null, of h.  out [T, hidden] of o_dtype, or null.
SHARPI_EXPORT int sharpi_sum_norm(float* h, const void* delta, int d_dtype, const int* pos, const float* sum_w, int k, const void* shared,
                                  const int* ids, int n_experts, const void* ident, float alpha, const float* w, const float* b,
                                  float eps, int n_rows, int hidden, void* out, int o_dtype, hipStream_t stream) {
  if (n_rows <= 0) return SHARPI_OK;
  if (hidden <= 0 || (size_t)hidden * sizeof(float) > 60 * 1024 || !delta || !w || !b || !(eps > 0.f)) return SHARPI_ERR_ARG;
  if ((pos && k <= 0) || (ids && !pos)) return SHARPI_ERR_ARG;
  if ((d_dtype != DT_F32 && d_dtype != DT_BF16) || (out && o_dtype != DT_F32 && o_dtype != DT_BF16)) return SHARPI_ERR_ARG;
  auto aligned = [](const void* p) { return ((uintptr_t)p & 31) == 0; };
  const bool wide = hidden % 8 == 0 && hidden <= 8192 && aligned(h) && aligned(delta) && aligned(shared) && aligned(ident) && aligned(w) &&
                    aligned(b) && aligned(out);
  LnDelta d{delta, pos, sum_w, shared, k, ids, n_experts, ident};
  const int runs = wide ? hidden / 8 : hidden;
  int threads = ceil_div(runs, kWave) * kWave;
  if (threads > (wide ? 1024 : 256)) threads = wide ? 1024 : 256;
  const size_t lds = (size_t)hidden * sizeof(float);
#define SN(TD, TO)                                                                                                \
  do {                                                                                                            \
    if (wide) sum_norm_run_kernel<TD, TO><<<n_rows, threads, 0, stream>>>(h, d, alpha, w, b, eps, (TO*)out, hidden); \
    else sum_norm_kernel<TD, TO><<<n_rows, threads, lds, stream>>>(h, d, alpha, w, b, eps, (TO*)out, hidden);      \
  } while (0)
  const bool of = !out || o_dtype == DT_F32;
  if (d_dtype == DT_F32) {
    if (of) SN(float, float);
    else SN(float, bf16_t);
  } else {
    if (of) SN(bf16_t, float);
    else SN(bf16_t, bf16_t);
  }
#undef SN
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// ---------------------------------------------------------------------------
// The embedding with a norm: out[t] = LN(table[ids[t]] * scale) w + b in float, and a copy in the activations' storage
// type (copy null: none).
// ---------------------------------------------------------------------------
template <typename T, typename TO>
__global__ __launch_bounds__(256) void embed_norm_kernel(const int* __restrict__ ids, const T* __restrict__ table, float scale,
                                                         const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                         float* __restrict__ out, TO* __restrict__ copy, int hidden) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[16];
  const size_t t = blockIdx.x;
  const T* src = table + (size_t)ids[t] * hidden;
  float s = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {     // (a thread reads what it wrote)
    const float v = to_f32<T>(src[c]) * scale;
    row[c] = v;
    s += v;
  }
  const float mean = block_sum(s, red) / (float)hidden;
  s = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) s = fmaf(row[c] - mean, row[c] - mean, s);
  const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    const float x = fmaf((row[c] - mean) * inv, w[c], b[c]);
    out[t * hidden + c] = x;
    if (copy) copy[t * hidden + c] = from_f32<TO>(x);
  }
}

// A thread has one run of eight elements (hidden a multiple of 8 up to 8,192).
template <typename T, typename TO>
__global__ __launch_bounds__(1024) void embed_norm_run_kernel(const int* __restrict__ ids, const T* __restrict__ table, float scale,
                                                              const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                              float* __restrict__ out, TO* __restrict__ copy, int hidden) {
  __shared__ float red[16];
  const size_t t = blockIdx.x;
  const int c = threadIdx.x * 8;
  const bool in = c < hidden;
  float x[8], wv[8], bv[8];
  float s = 0.f;
  if (in) {
    load8(table + (size_t)ids[t] * hidden + c, x);
    load8(w + c, wv);
    load8(b + c, bv);
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      x[k] *= scale;
      s += x[k];
    }
  }
  const float mean = block_sum(s, red) / (float)hidden;
  s = 0.f;
  if (in) {
#pragma unroll
    for (int k = 0; k < 8; ++k) s = fmaf(x[k] - mean, x[k] - mean, s);
  }
  const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)hidden + eps);
  if (!in) return;
#pragma unroll
  for (int k = 0; k < 8; ++k) x[k] = fmaf((x[k] - mean) * inv, wv[k], bv[k]);
  store8(out + t * hidden + c, x);
  if (copy) store8(copy + t * hidden + c, x);
}

SHARPI_EXPORT int sharpi_embed_norm(const int* ids, const void* table, int t_dtype, float scale, const float* w, const float* b,
                                    float eps, float* out, void* copy, int c_dtype, int n_tokens, int hidden, hipStream_t stream) {
  if (n_tokens <= 0) return SHARPI_OK;
  if (hidden <= 0 || (size_t)hidden * sizeof(float) > 60 * 1024 || !w || !b || !(eps > 0.f)) return SHARPI_ERR_ARG;
  if ((t_dtype != DT_F32 && t_dtype != DT_BF16) || (copy && c_dtype != DT_F32 && c_dtype != DT_BF16)) return SHARPI_ERR_ARG;
  const size_t lds = (size_t)hidden * sizeof(float);
  auto aligned = [](const void* p) { return ((uintptr_t)p & 31) == 0; };
  const bool wide = hidden % 8 == 0 && hidden <= 8192 && aligned(table) && aligned(w) && aligned(b) && aligned(out) && aligned(copy);
  const int threads = ceil_div(hidden / 8, kWave) * kWave;
#define EN(T, TO)                                                                                                                        \
  do {                                                                                                                                   \
    if (wide) embed_norm_run_kernel<T, TO><<<n_tokens, threads, 0, stream>>>(ids, (const T*)table, scale, w, b, eps, out, (TO*)copy, hidden); \
    else embed_norm_kernel<T, TO><<<n_tokens, 256, lds, stream>>>(ids, (const T*)table, scale, w, b, eps, out, (TO*)copy, hidden);          \
  } while (0)
  const bool cf = !copy || c_dtype == DT_F32;
  if (t_dtype == DT_F32) {
    if (cf) EN(float, float);
    else EN(float, bf16_t);
  } else {
    if (cf) EN(bf16_t, float);
    else EN(bf16_t, bf16_t);
  }
#undef EN
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// ---------------------------------------------------------------------------
// The convolution over the residual sum in steps of longer entries.  A block: `tok` tokens x 256 V channels, a thread
// V channels with the last TAPS - 1 inputs in registers.  Only an entry's first TAPS - 1 tokens reach back
// beyond the step, into the ring; all of them are taken by the block in which the entry begins (also where they
// run past its tokens), whose threads then bring the ring up to date: no other block reads it.
// ---------------------------------------------------------------------------
template <typename TO, int TAPS, int V>
__global__ __launch_bounds__(256) void residual_conv_kernel(const float* __restrict__ h, const float* __restrict__ w,
                                                            float* __restrict__ ring_all, const int* __restrict__ positions,
                                                            const int* __restrict__ state_slots, const int* __restrict__ entry_of_token,
                                                            const int* __restrict__ cu_tokens, TO* __restrict__ out, int n_tokens,
                                                            int hidden, int tok) {
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
  if (c >= hidden) return;
  const int t0 = blockIdx.x * tok, t1 = min(t0 + tok, n_tokens);
  float wt[TAPS][V];
#pragma unroll
  for (int back = 0; back < TAPS; ++back)
#pragma unroll
    for (int k = 0; k < V; ++k) wt[back][k] = w[(size_t)(c + k) * TAPS + TAPS - 1 - back];
  int t = t0;
  {
    const int first = cu_tokens[entry_of_token[t0]];
    if (first < t0 && t0 - first < TAPS - 1) t = min(first + TAPS - 1, cu_tokens[entry_of_token[t0] + 1]);   // taken by an earlier block
  }
  float past[TAPS][V];                     // past[b]: the input b tokens back (b >= 1)
  bool fresh = true;                       // the window has to be read anew
  int e = -1, first = 0, end = 0;
  for (; t < n_tokens; ++t) {
    if (e < 0 || t >= end) {
      e = entry_of_token[t];
      first = cu_tokens[e];
      end = cu_tokens[e + 1];
      fresh = true;
    }
    const int local = t - first;
    if (t >= t1 && !(local < TAPS - 1 && first >= t0 && first < t1)) break;
    if (fresh) {
      fresh = false;
      const int p = positions[t];
      float* ring = TAPS > 1 ? ring_all + (size_t)state_slots[e] * TAPS * hidden + c : nullptr;
#pragma unroll
      for (int back = 1; back < TAPS; ++back) {
#pragma unroll
        for (int k = 0; k < V; ++k) past[back][k] = 0.f;
        if (back <= local) ln_load<float, V>(h + (size_t)(t - back) * hidden + c, past[back]);
        else if (back <= p) ln_load<float, V>(ring + (size_t)((p - back) % TAPS) * hidden, past[back]);
      }
      if (local == 0) {                    // the entry begins here: its last inputs into the ring (read above, by this thread)
        const int len = end - first;
#pragma unroll
        for (int back = 0; back < TAPS - 1; ++back)
          if (back < len) {
            float u[V];
            ln_load<float, V>(h + (size_t)(end - 1 - back) * hidden + c, u);
            ln_store<float, V>(ring + (size_t)((p + len - 1 - back) % TAPS) * hidden, u);
          }
      }
    }
    float x[V], y[V];
    ln_load<float, V>(h + (size_t)t * hidden + c, x);
#pragma unroll
    for (int k = 0; k < V; ++k) y[k] = 0.f;
#pragma unroll
    for (int back = TAPS - 1; back >= 1; --back)
#pragma unroll
      for (int k = 0; k < V; ++k) y[k] = fmaf(wt[back][k], past[back][k], y[k]);
#pragma unroll
    for (int k = 0; k < V; ++k) y[k] = x[k] + fmaf(wt[0][k], x[k], y[k]);
    ln_store<TO, V>(out + (size_t)t * hidden + c, y);
#pragma unroll
    for (int back = TAPS - 1; back >= 2; --back)
#pragma unroll
      for (int k = 0; k < V; ++k) past[back][k] = past[back - 1][k];
    if (TAPS > 1) {
#pragma unroll
      for (int k = 0; k < V; ++k) past[TAPS > 1 ? 1 : 0][k] = x[k];
    }
  }
}

template <typename TO, int V>
static int launch_residual_conv(const float* h, const float* w, int taps, float* ring, const int* positions, const int* state_slots,
                                const int* entry_of_token, const int* cu_tokens, void* out, int n_tokens, int hidden, int tok, hipStream_t stream) {
  const int threads = hidden / V >= 256 ? 256 : ceil_div(ceil_div(hidden, V), kWave) * kWave;
  dim3 grid(ceil_div(n_tokens, tok), ceil_div(ceil_div(hidden, V), threads));
#define RC(N)                                                                                                                        \
  case N:                                                                                                                            \
    residual_conv_kernel<TO, N, V><<<grid, threads, 0, stream>>>(h, w, ring, positions, state_slots, entry_of_token, cu_tokens, (TO*)out, \
                                                                 n_tokens, hidden, tok);                                             \
    break
  switch (taps) {
    RC(1); RC(2); RC(3); RC(4); RC(5); RC(6); RC(7); RC(8);
    default: return SHARPI_ERR_ARG;
  }
#undef RC
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// h float [T, hidden]; w float [hidden, taps]; ring float [slots, taps, hidden] (null with one tap); out [T, hidden] of o_dtype.
SHARPI_EXPORT int sharpi_residual_conv(const float* h, const float* w, int taps, float* ring, const int* positions,
                                       const int* state_slots, const int* entry_of_token, const int* cu_tokens, void* out, int o_dtype,
                                       int n_tokens, int hidden, hipStream_t stream) {
  if (n_tokens <= 0) return SHARPI_OK;
  if (hidden <= 0 || taps < 1 || taps > kLnMaxTaps || (taps > 1 && !ring) || !out) return SHARPI_ERR_ARG;
  if (o_dtype != DT_F32 && o_dtype != DT_BF16) return SHARPI_ERR_ARG;
  const int tok = n_tokens >= 1024 ? 8 : n_tokens >= 128 ? 4 : 1;
  const bool by8 = hidden % 8 == 0 && ((uintptr_t)h & 31) == 0 && ((uintptr_t)out & 31) == 0 && ((uintptr_t)ring & 31) == 0;
  if (o_dtype == DT_F32) {
    if (by8) return launch_residual_conv<float, 8>(h, w, taps, ring, positions, state_slots, entry_of_token, cu_tokens, out, n_tokens, hidden, tok, stream);
    return launch_residual_conv<float, 1>(h, w, taps, ring, positions, state_slots, entry_of_token, cu_tokens, out, n_tokens, hidden, tok, stream);
  }
  if (by8) return launch_residual_conv<bf16_t, 8>(h, w, taps, ring, positions, state_slots, entry_of_token, cu_tokens, out, n_tokens, hidden, tok, stream);
  return launch_residual_conv<bf16_t, 1>(h, w, taps, ring, positions, state_slots, entry_of_token, cu_tokens, out, n_tokens, hidden, tok, stream);
}

// ---------------------------------------------------------------------------
// out[t] = table[id] * scale + pairs[row], row = (previous id * mul_prev + id * mul_cur) mod buckets, or `buckets` at
// position 0.  The previous id of an entry's first token lies in its request's slot, [slots, 2] int32, position p at
// p mod 2; the block of that token reads it and then leaves there the id of the entry's last token.
// ---------------------------------------------------------------------------
template <typename T, typename TP>
__global__ __launch_bounds__(256) void embed_bigram_kernel(const int* __restrict__ ids, const T* __restrict__ table, float scale,
                                                           const TP* __restrict__ pairs, long long mul_prev, long long mul_cur,
                                                           long long buckets, int* __restrict__ before, const int* __restrict__ positions,
                                                           const int* __restrict__ state_slots, const int* __restrict__ entry_of_token,
                                                           const int* __restrict__ cu_tokens, float* __restrict__ out, int hidden) {
  __shared__ long long row_s;
  const int t = blockIdx.x;
  if (threadIdx.x == 0) {
    const int e = entry_of_token[t], first = cu_tokens[e], p = positions[t];
    int* mine = before + 2 * state_slots[e];
    long long row = buckets;
    if (p > 0) row = ((long long)(t > first ? ids[t - 1] : mine[(p - 1) & 1]) * mul_prev + (long long)ids[t] * mul_cur) % buckets;
    row_s = row < 0 ? row + buckets : row;
    if (t == first) {
      const int last = cu_tokens[e + 1] - 1;
      mine[positions[last] & 1] = ids[last];
    }
  }
  __syncthreads();
  const T* a = table + (size_t)ids[t] * hidden;
  const TP* b = pairs + (size_t)row_s * hidden;
  float* o = out + (size_t)t * hidden;
  if (hidden % 8 == 0) {           // (the tables begin on 32-byte borders: whole tensors)
    for (int i = threadIdx.x * 8; i < hidden; i += blockDim.x * 8) {
      float x[8], y[8];
      load8(a + i, x);
      load8(b + i, y);
#pragma unroll
      for (int k = 0; k < 8; ++k) x[k] = fmaf(x[k], scale, y[k]);
      store8(o + i, x);
    }
    return;
  }
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) o[i] = fmaf(to_f32<T>(a[i]), scale, to_f32<TP>(b[i]));
}

SHARPI_EXPORT int sharpi_embed_bigram(const int* ids, const void* table, int t_dtype, float scale, const void* pairs, int p_dtype,
                                      long long mul_prev, long long mul_cur, int buckets, int* before, const int* positions,
                                      const int* state_slots, const int* entry_of_token, const int* cu_tokens, float* out, int n_tokens,
                                      int hidden, hipStream_t stream) {
  if (n_tokens <= 0) return SHARPI_OK;
  if (hidden <= 0 || buckets <= 0 || !before || !pairs) return SHARPI_ERR_ARG;
  if (((uintptr_t)table | (uintptr_t)pairs | (uintptr_t)out) & 31) return SHARPI_ERR_ARG;
#define EB(T, TP)                                                                                                                  \
  embed_bigram_kernel<T, TP><<<n_tokens, 256, 0, stream>>>(ids, (const T*)table, scale, (const TP*)pairs, mul_prev, mul_cur, buckets, \
                                                           before, positions, state_slots, entry_of_token, cu_tokens, out, hidden)
  if (t_dtype == DT_F32 && p_dtype == DT_F32) EB(float, float);
  else if (t_dtype == DT_BF16 && p_dtype == DT_BF16) EB(bf16_t, bf16_t);
  else if (t_dtype == DT_BF16 && p_dtype == DT_F32) EB(bf16_t, float);
  else if (t_dtype == DT_F32 && p_dtype == DT_BF16) EB(float, bf16_t);
  else return SHARPI_ERR_ARG;
#undef EB
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}
