// The gated delta rule with a decay per key channel.  Per head a state S [dk, dv] (float), token by token
//   S <- diag(exp(l_t)) S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t,
// with l_t <= 0 the logarithms of the decays, beta_t = sigmoid of one number per head, q, k and v behind a short
// causal convolution and SiLU, q and k unit vectors (q times dk^-1/2 besides).
//
// From the projections on everything is float: the convolution's sums, unit norms, decays and their
// exponentials, the state, every sum over it (the matrix products of the chunked form run on the float
// matrix instruction v_mfma_f32_16x16x4_f32: float operands, float sums).
//
// lowrank:      out[t, n] = f(sum_r x[t, r] w[n, r]) for the two projections through a narrow middle, as plain
//               sums (the output gate) or as the decays' logarithms -exp(A_h) softplus(sum + bias_n).
// delta_step:   steps of single tokens.  A block takes one (entry, head): convolution, norms and decays into LDS
//               (once for all value columns), then a wave a 16-column strip of S: both products with the decayed
//               state in one pass (o = (aS)^T q + u (k.q)), the write, the norm over dv and the output gate.
// delta_chunk_prep, delta_chunk_walk: steps with longer entries, 16 tokens (a chunk) at a time.  With b_t the
//               running sum of l within the chunk and S_0 the state before it,
//                 u_t = beta_t (v_t - S_0^T (e^(b_t) k_t) - sum_(s<t) L_ts u_s),  L_ts = sum_i k_ti k_si e^(b_ti - b_si),
//                 o_t = S_0^T (e^(b_t) q_t) + sum_(s<=t) A_ts u_s,                A_ts = sum_i q_ti k_si e^(b_ti - b_si),
//                 S_C = e^(b_C) S_0 + sum_s (e^(b_C - b_s) k_s) u_s^T,
//               where every exponent is <= 0, so nothing overflows and what underflows is nothing.  The first kernel
//               makes, for all chunks at once, what does not depend on S_0: the triangular system is solved by forward
//               substitution for the right sides v (U0) and e^b k (W), so that u = U0 - W S_0.  The second walks the
//               chunks of an entry: three small matrix products a chunk, a block a (entry, head, 16 columns), its
//               waves each holding some 16-row tiles of the state in the registers of the matrix instruction's
//               result, which are at once the layout of its B operand: the state never moves between lanes.
//
// A request's state lies in its slot as [heads, ceil(dv / 16), ceil(dk / 16), 64, 4] floats: lane 16 g + j of a tile
// keeps rows 4 g .. 4 g + 3 of column j.  The convolution's last inputs lie in a ring [slots, taps, channels],
// position p at p mod taps: the rows a step reads (p - 1 .. p - taps + 1) are never the one a single token
// writes (p), so a step of single tokens reads and writes in one kernel.  What lies before position 0 is
// never read.
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;

constexpr int kDcTokens = 16;            // tokens of a chunk
constexpr int kDrMaxTaps = 8;
constexpr int kDies = 8;                 // dies that blocks are dealt to, round robin
constexpr float kUnitFloor = 1e-6f;      // added to a sum of squares under the unit vectors' root
constexpr float kLog2e = 1.4426950408889634f;

SHARPI_EXPORT int sharpi_delta_chunk_tokens() { return kDcTokens; }

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f32(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float exp2_f32(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// ---------------------------------------------------------------------------
// Products through a narrow middle, on the float matrix instruction.  A wave: 16 outputs x 16 kTT tokens.
// ---------------------------------------------------------------------------
enum : int { LOWRANK_PLAIN = 0, LOWRANK_LOG_DECAY = 1 };
constexpr int kLrTiles = 4;       // 16-token tiles a wave
struct LowRankJob {
  int x_off, rank, N, mode, per;  // columns of x, their number, outputs, and (log decays) outputs a head
  const void* w;                  // [N, rank]
  const float *bias, *a_log;      // LOWRANK_LOG_DECAY: [N], [N / per]
  void* out;                      // [T, N]: floats (log decays) or the activations' type (plain)
  int blocks;                     // blocks of 64 outputs
};
struct LowRankJobs { LowRankJob j[2]; };

// n of four elements as floats, the rest zero (VEC: all four there, 8 or 16 bytes at once)
template <typename T, bool VEC>
__device__ __forceinline__ void load4(const T* p, int n, float* v) {
  if constexpr (VEC && sizeof(T) == 4) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  } else if constexpr (VEC) {
    const uint2 x = *reinterpret_cast<const uint2*>(p);
    v[0] = bf16_bits_to_f32(x.x & 0xffffu); v[1] = bf16_bits_to_f32(x.x >> 16);
    v[2] = bf16_bits_to_f32(x.y & 0xffffu); v[3] = bf16_bits_to_f32(x.y >> 16);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = i < n ? to_f32<T>(p[i]) : 0.f;
  }
}

template <typename T, bool VEC, int TT>      // VEC: ranks multiples of 16, rows and columns of x and w on 16-byte borders
__global__ __launch_bounds__(256) void lowrank_kernel(const float* __restrict__ x, int stride, LowRankJobs jobs, int n_tokens) {
  const LowRankJob& jb = (int)blockIdx.y < jobs.j[0].blocks ? jobs.j[0] : jobs.j[1];
  const int nb = (int)blockIdx.y < jobs.j[0].blocks ? blockIdx.y : blockIdx.y - jobs.j[0].blocks;
  const int lane = threadIdx.x & 63, m = lane & 15, g = lane >> 4;
  const int n0 = (nb * 4 + (threadIdx.x >> 6)) * 16;
  const int rank = jb.rank, N = jb.N;
  if (n0 >= N) return;
  const T* wr = (const T*)jb.w + (size_t)min(n0 + m, N - 1) * rank;
  const float* xr[TT];
#pragma unroll
  for (int a = 0; a < TT; ++a)
    xr[a] = x + (size_t)min((int)(blockIdx.x * TT + a) * 16 + m, n_tokens - 1) * stride + jb.x_off;
  f32x4 acc[TT];
#pragma unroll
  for (int a = 0; a < TT; ++a) acc[a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int k0 = 0; k0 < rank; k0 += 16) {
    const int k = k0 + 4 * g, left = rank - k;
    float wv[4], xv[TT][4];
    load4<T, VEC>(wr + k, left, wv);
#pragma unroll
    for (int a = 0; a < TT; ++a) load4<float, VEC>(xr[a] + k, left, xv[a]);
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int a = 0; a < TT; ++a) acc[a] = mfma4(wv[i], xv[a][i], acc[a]);
  }
  const bool decay = jb.mode == LOWRANK_LOG_DECAY;
  float neg_a[4], bias[4];
  if (decay) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = min(n0 + 4 * g + i, N - 1);
      neg_a[i] = -expf(jb.a_log[n / jb.per]);
      bias[i] = jb.bias[n];
    }
  }
#pragma unroll
  for (int a = 0; a < TT; ++a) {
    const int t = (blockIdx.x * TT + a) * 16 + m;
    if (t >= n_tokens) continue;
    if (decay) {
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[a][i] = neg_a[i] * softplus_f32(acc[a][i] + bias[i]);
    }
    const size_t at = (size_t)t * N + n0 + 4 * g;
    if (VEC && N % 4 == 0) {
      if (n0 + 4 * g >= N) continue;
      if (decay || sizeof(T) == 4) {
        *reinterpret_cast<f32x4*>((float*)jb.out + at) = acc[a];
      } else {
        uint2 o;
        o.x = (uint32_t)f32_to_bf16(acc[a][0]).bits | ((uint32_t)f32_to_bf16(acc[a][1]).bits << 16);
        o.y = (uint32_t)f32_to_bf16(acc[a][2]).bits | ((uint32_t)f32_to_bf16(acc[a][3]).bits << 16);
        *reinterpret_cast<uint2*>((T*)jb.out + at) = o;
      }
      continue;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (n0 + 4 * g + i >= N) continue;
      if (decay) ((float*)jb.out)[at + i] = acc[a][i];
      else ((T*)jb.out)[at + i] = from_f32<T>(acc[a][i]);
    }
  }
}

// x float [T, stride]; job 0: log decays (rank columns at x_off0, w0 [N0, rank0], bias [N0], a_log [N0 / per], out0
// float [T, N0]); job 1 (N1 may be 0): plain sums (w1 [N1, rank1], out1 [T, N1]).  w and out1 of `dtype`.
SHARPI_EXPORT int sharpi_lowrank(const float* x, int stride, int dtype, int n_tokens, int x_off0, int rank0, const void* w0,
                                 int N0, const float* bias, const float* a_log, int per, float* out0, int x_off1, int rank1,
                                 const void* w1, int N1, void* out1, hipStream_t stream) {
  if (n_tokens <= 0) return SHARPI_OK;
  if (N0 < 0 || N1 < 0 || N0 + N1 <= 0) return SHARPI_ERR_ARG;
  if (N0 > 0 && (rank0 <= 0 || x_off0 < 0 || x_off0 + rank0 > stride || !w0 || !bias || !a_log || !out0 || per <= 0 || N0 % per)) return SHARPI_ERR_ARG;
  if (N1 > 0 && (rank1 <= 0 || x_off1 < 0 || x_off1 + rank1 > stride || !w1 || !out1)) return SHARPI_ERR_ARG;
  LowRankJobs jobs;
  jobs.j[0] = LowRankJob{x_off0, rank0, N0, LOWRANK_LOG_DECAY, per > 0 ? per : 1, w0, bias, a_log, out0, ceil_div(N0, 64)};
  jobs.j[1] = LowRankJob{x_off1, rank1, N1, LOWRANK_PLAIN, 1, w1, nullptr, nullptr, out1, ceil_div(N1, 64)};
  const int tt = n_tokens > 16 ? kLrTiles : 1;
  dim3 grid(ceil_div(n_tokens, 16 * tt), jobs.j[0].blocks + jobs.j[1].blocks);
  if (grid.y > 65535) return SHARPI_ERR_ARG;
  auto on16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = stride % 4 == 0 && on16(x) && (N0 == 0 || (rank0 % 16 == 0 && x_off0 % 4 == 0 && on16(w0) && on16(out0))) &&
                   (N1 == 0 || (rank1 % 16 == 0 && x_off1 % 4 == 0 && on16(w1) && on16(out1)));
#define LR(T, V)                                                                                   \
  do {                                                                                             \
    if (tt == 1) lowrank_kernel<T, V, 1><<<grid, 256, 0, stream>>>(x, stride, jobs, n_tokens);     \
    else lowrank_kernel<T, V, kLrTiles><<<grid, 256, 0, stream>>>(x, stride, jobs, n_tokens);      \
  } while (0)
  if (dtype == DT_F32) {
    if (vec) LR(float, true);
    else LR(float, false);
  } else if (dtype == DT_BF16) {
    if (vec) LR(bf16_t, true);
    else LR(bf16_t, false);
  } else {
    return SHARPI_ERR_ARG;
  }
#undef LR
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// ---------------------------------------------------------------------------
// what both forms read
// ---------------------------------------------------------------------------
struct DeltaIn {
  const void* proj; int stride, c_off;           // q | k | v channels side by side from column c_off
  const float* conv_w; int taps; float* ring;    // [channels, taps]; [slots, taps, channels] (null with one tap)
  const float* log_decay;                        // [T, nh * dk]
  const float* beta; int beta_stride, beta_off;  // beta's logit of head h at column beta_off + h
  const int *positions, *state_slots, *cu_tokens;
  float* state;
  int nh, rep, dk, dv, channels, n_q;            // rep: heads a key head; n_q: channels of q (and of k)
  float q_scale;
};

// ---------------------------------------------------------------------------
// steps of single tokens
// ---------------------------------------------------------------------------
template <typename T>
__device__ __forceinline__ float conv_one(const DeltaIn& a, const T* row, const float* ring, int p, int ch, float* now) {
  const float u = to_f32<T>(row[ch]);
  *now = u;
  const float* w = a.conv_w + (size_t)ch * a.taps;
  float acc = 0.f;
  for (int back = a.taps - 1; back > 0; --back)
    if (p >= back) acc = fmaf(w[a.taps - 1 - back], ring[(size_t)((p - back) % a.taps) * a.channels + ch], acc);
  acc = fmaf(w[a.taps - 1], u, acc);
  return acc * sigmoid_f32(acc);
}

template <typename T, int NT>       // NT: 16-row tiles a lane holds of a strip (rows beyond dk stay zero)
__global__ __launch_bounds__(512, NT <= 8 ? 4 : 2) void delta_step_kernel(DeltaIn a, const float* __restrict__ norm_w, float eps,
                                                         const T* __restrict__ gate, T* __restrict__ out) {
  __shared__ __attribute__((aligned(16))) float q_s[NT * 16], k_s[NT * 16], d_s[NT * 16];
  __shared__ float red[3][8];
  extern __shared__ __attribute__((aligned(16))) float vo_s[];      // [dv] values, then [dv] outputs
  const int h = blockIdx.x, e = blockIdx.y, tid = threadIdx.x, nthr = blockDim.x;
  const int lane = tid & 63, w = tid >> 6, nw = nthr >> 6, g = lane >> 4, j = lane & 15;
  const int t = a.cu_tokens[e], p = a.positions[t], slot = a.state_slots[e];
  const int ns = (a.dv + 15) >> 4, nt = (a.dk + 15) >> 4;
  float* st = a.state + ((size_t)slot * a.nh + h) * ns * nt * 256;
  f32x4 S[NT];
  auto fetch = [&](int strip) {
#pragma unroll
    for (int n = 0; n < NT; ++n)
      S[n] = n < nt ? *reinterpret_cast<const f32x4*>(st + ((size_t)strip * nt + n) * 256 + lane * 4) : f32x4{0.f, 0.f, 0.f, 0.f};
  };
  if (w < ns) fetch(w);                    // on its way while q, k, v and the decays are made

  const T* row = (const T*)a.proj + (size_t)t * a.stride + a.c_off;
  float* ring = a.ring ? a.ring + (size_t)slot * a.taps * a.channels : nullptr;
  float* ring_now = ring ? ring + (size_t)(p % a.taps) * a.channels : nullptr;
  const int kh = h / a.rep, q0 = kh * a.dk, k0 = a.n_q + kh * a.dk, v0 = 2 * a.n_q + h * a.dv;
  const bool keeps_qk = ring_now && h % a.rep == 0;
  float qq = 0.f, kk = 0.f, qk = 0.f;
  for (int c = tid; c < NT * 16; c += nthr) {
    float qv = 0.f, kv = 0.f, dc = 1.f;
    if (c < a.dk) {
      float qn, kn;
      qv = conv_one<T>(a, row, ring, p, q0 + c, &qn);
      kv = conv_one<T>(a, row, ring, p, k0 + c, &kn);
      if (keeps_qk) {
        ring_now[q0 + c] = qn;
        ring_now[k0 + c] = kn;
      }
      dc = expf(a.log_decay[(size_t)t * a.nh * a.dk + h * a.dk + c]);
    }
    q_s[c] = qv;
    k_s[c] = kv;
    d_s[c] = dc;
    qq = fmaf(qv, qv, qq);
    kk = fmaf(kv, kv, kk);
    qk = fmaf(qv, kv, qk);
  }
  for (int c = tid; c < a.dv; c += nthr) {
    float vn;
    vo_s[c] = conv_one<T>(a, row, ring, p, v0 + c, &vn);
    if (ring_now) ring_now[v0 + c] = vn;
  }
  qq = wave_sum(qq);
  kk = wave_sum(kk);
  qk = wave_sum(qk);
  if (lane == 0) {
    red[0][w] = qq;
    red[1][w] = kk;
    red[2][w] = qk;
  }
  __syncthreads();
  qq = kk = qk = 0.f;
  for (int i = 0; i < nw; ++i) {
    qq += red[0][i];
    kk += red[1][i];
    qk += red[2][i];
  }
  const float qs = a.q_scale / sqrtf(qq + kUnitFloor), ks = 1.0f / sqrtf(kk + kUnitFloor);
  const float kq = qk * qs * ks;           // k . q of the scaled vectors
  const float beta = sigmoid_f32(a.beta[(size_t)t * a.beta_stride + a.beta_off + h]);
  float* o_s = vo_s + a.dv;
  for (int strip = w; strip < ns; strip += nw) {
    float dotk = 0.f, dotq = 0.f;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const f32x4 d4 = *reinterpret_cast<const f32x4*>(d_s + 16 * n + 4 * g);
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(k_s + 16 * n + 4 * g);
      const f32x4 q4 = *reinterpret_cast<const f32x4*>(q_s + 16 * n + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        S[n][i] *= d4[i];
        dotk = fmaf(S[n][i], k4[i], dotk);
        dotq = fmaf(S[n][i], q4[i], dotq);
      }
      if (n % 2) __builtin_amdgcn_sched_barrier(0);      // (all tiles' operands read ahead would not fit the registers)
    }
    dotk += __shfl_xor(dotk, 16, kWave);
    dotq += __shfl_xor(dotq, 16, kWave);
    dotk += __shfl_xor(dotk, 32, kWave);
    dotq += __shfl_xor(dotq, 32, kWave);
    const int c = strip * 16 + j;
    const float u = c < a.dv ? beta * (vo_s[c] - dotk * ks) : 0.f;
    if (g == 0 && c < a.dv) o_s[c] = fmaf(u, kq, dotq * qs);
    const float uk = u * ks;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      if (n >= nt) continue;
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(k_s + 16 * n + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) S[n][i] = fmaf(k4[i], uk, S[n][i]);
      *reinterpret_cast<f32x4*>(st + ((size_t)strip * nt + n) * 256 + lane * 4) = S[n];
    }
    if (strip + nw < ns) fetch(strip + nw);
  }
  __syncthreads();                         // (also: everybody is done with `red`)
  float ss = 0.f;
  for (int c = tid; c < a.dv; c += nthr) ss = fmaf(o_s[c], o_s[c], ss);
  ss = wave_sum(ss);
  if (lane == 0) red[0][w] = ss;
  __syncthreads();
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += red[0][i];
  const float inv = 1.0f / sqrtf(ss / (float)a.dv + eps);
  const size_t at = (size_t)t * a.nh * a.dv + (size_t)h * a.dv;
  for (int c = tid; c < a.dv; c += nthr) {
    float y = o_s[c] * inv * norm_w[c];
    if (gate) y *= sigmoid_f32(to_f32<T>(gate[at + c]));
    out[at + c] = from_f32<T>(y);
  }
}

// ---------------------------------------------------------------------------
// chunks of 16 tokens
// ---------------------------------------------------------------------------
// chunks int [n, 4] = (entry, first row, tokens, unused).  Per (chunk, head), in floats: W and Qd [dkp / 16][16
// tokens][16 rows], KT [dkp][16], D [dkp], U0 [dvp][16], A [16][16] (dkp, dvp: dk and dv rounded up to 16): every operand of the
// walk's matrix instructions is one contiguous kilobyte.
struct ChunkBuf {
  float *W, *Qd, *KT, *D, *U0, *A;
};

// (TAPS: the convolution's taps, or more: the weights beyond are zero; DKP: room for dk key channels)
template <typename T, int TAPS, int DKP>
__global__ __launch_bounds__(256, DKP <= 128 ? 4 : 2) void delta_chunk_prep_kernel(DeltaIn a, const int* __restrict__ chunks, ChunkBuf b) {
  constexpr int ldk = DKP + 4;             // rows of LDS four banks apart
  extern __shared__ __attribute__((aligned(16))) float smem[];
  constexpr int C = kDcTokens;
  float* q_s = smem;                       // [C][ldk]
  float* k_s = q_s + C * ldk;              // [C][ldk]
  float* b_s = k_s + C * ldk;              // [C][ldk]: running sums of the log decays, in powers of two
  float* L_s = b_s + C * ldk;              // [C][C]
  float* beta_s = L_s + C * C;             // [C]
  float* v_s = beta_s + C;                 // [C][dv]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  // a head's chunks on the die that will walk them, where the heads divide so (blocks are dealt to the dies round robin)
  int h = blockIdx.x % a.nh, chunk = blockIdx.x / a.nh;
  if (a.nh % kDies == 0) {
    const int per = a.nh / kDies, i = blockIdx.x / kDies;
    h = blockIdx.x % kDies + kDies * (i % per);
    chunk = i / per;
  }
  const size_t ch = (size_t)chunk * a.nh + h;
  const int e = chunks[4 * chunk], first = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2];
  const int local0 = first - a.cu_tokens[e], p0 = a.positions[first];
  const int kh = h / a.rep, dkp = (a.dk + 15) & ~15, dvp = (a.dv + 15) & ~15;
  const float* ring = a.ring ? a.ring + (size_t)a.state_slots[e] * a.taps * a.channels : nullptr;
  const T* rows = (const T*)a.proj + (size_t)first * a.stride + a.c_off;

  // q, k, v through the convolution and SiLU: a thread a channel, the last taps - 1 inputs in registers
  for (int idx = tid; idx < 2 * ldk + a.dv; idx += blockDim.x) {
    int chan = -1;
    float* dst;
    int ld;
    if (idx < ldk) {
      dst = q_s + idx;
      ld = ldk;
      if (idx < a.dk) chan = kh * a.dk + idx;
    } else if (idx < 2 * ldk) {
      dst = k_s + idx - ldk;
      ld = ldk;
      if (idx - ldk < a.dk) chan = a.n_q + kh * a.dk + idx - ldk;
    } else {
      dst = v_s + idx - 2 * ldk;
      ld = a.dv;
      chan = 2 * a.n_q + h * a.dv + idx - 2 * ldk;
    }
    if (chan < 0) {                        // columns that pad a row
      for (int t = 0; t < C; ++t) dst[t * ld] = 0.f;
      continue;
    }
    float u[C], wt[TAPS], past[TAPS];
#pragma unroll
    for (int t = 0; t < C; ++t) u[t] = to_f32<T>(rows[(size_t)min(t, n - 1) * a.stride + chan]);   // (no load behind a branch)
#pragma unroll
    for (int back = 0; back < TAPS; ++back) {
      wt[back] = back < a.taps ? a.conv_w[(size_t)chan * a.taps + a.taps - 1 - back] : 0.f;
      past[back] = 0.f;                    // the input `back` tokens before the chunk's first
      if (back > 0 && back < a.taps) {
        if (back <= local0) past[back] = to_f32<T>(*(rows + chan - (ptrdiff_t)back * a.stride));
        else if (back <= p0) past[back] = ring[(size_t)((p0 - back) % a.taps) * a.channels + chan];
      }
    }
#pragma unroll
    for (int t = 0; t < C; ++t) {
      float acc = 0.f;
#pragma unroll
      for (int back = TAPS - 1; back >= 0; --back) acc = fmaf(wt[back], t >= back ? u[t - back < 0 ? 0 : t - back] : past[back - t < 0 ? 0 : back - t], acc);
      dst[t * ld] = t < n ? acc * sigmoid_f32(acc) : 0.f;
    }
  }
  for (int c = tid; c < ldk; c += blockDim.x) {
    float l[C], run = 0.f;
    const float* src = a.log_decay + (size_t)first * a.nh * a.dk + h * a.dk + min(c, a.dk - 1);
#pragma unroll
    for (int t = 0; t < C; ++t) l[t] = src[(size_t)min(t, n - 1) * a.nh * a.dk];
#pragma unroll
    for (int t = 0; t < C; ++t) {
      if (c < a.dk && t < n) run += l[t] * kLog2e;
      b_s[t * ldk + c] = run;
    }
  }
  if (tid < C) beta_s[tid] = tid < n ? sigmoid_f32(a.beta[(size_t)(first + tid) * a.beta_stride + a.beta_off + h]) : 0.f;
  __syncthreads();
  // unit vectors: a wave takes every fourth token's q and k
  for (int t = w; t < C; t += 4) {
    float qq = 0.f, kk = 0.f;
    for (int c = lane; c < a.dk; c += kWave) {
      qq = fmaf(q_s[t * ldk + c], q_s[t * ldk + c], qq);
      kk = fmaf(k_s[t * ldk + c], k_s[t * ldk + c], kk);
    }
    const float qs = a.q_scale / sqrtf(wave_sum(qq) + kUnitFloor), ks = 1.0f / sqrtf(wave_sum(kk) + kUnitFloor);
    for (int c = lane; c < a.dk; c += kWave) {
      q_s[t * ldk + c] *= qs;
      k_s[t * ldk + c] *= ks;
    }
  }
  __syncthreads();
  // the two score matrices: a thread a pair (t, s)
  {
    const int t = tid >> 4, s = tid & 15;
    float l = 0.f, m = 0.f;
    if (s <= t) {
      for (int c = 0; c < dkp; c += 4) {
        const f32x4 bt = *reinterpret_cast<const f32x4*>(b_s + t * ldk + c), bs = *reinterpret_cast<const f32x4*>(b_s + s * ldk + c);
        const f32x4 kt = *reinterpret_cast<const f32x4*>(k_s + t * ldk + c), qt = *reinterpret_cast<const f32x4*>(q_s + t * ldk + c);
        const f32x4 ks = *reinterpret_cast<const f32x4*>(k_s + s * ldk + c);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float x = ks[i] * exp2_f32(bt[i] - bs[i]);
          l = fmaf(kt[i], x, l);
          m = fmaf(qt[i], x, m);
        }
      }
    }
    L_s[t * C + s] = s < t ? l : 0.f;
    b.A[ch * 256 + tid] = m;
  }
  __syncthreads();
  // forward substitution, a thread a column of (W | U0); the other tensors of the walk on the way
  for (int idx = tid; idx < dkp + dvp; idx += blockDim.x) {
    const bool key = idx < dkp;
    const int c = key ? idx : idx - dkp;
    const float* k_c = k_s + c;
    const float* b_c = b_s + c;
    float x[C];
    float* w_out = b.W + ch * C * dkp + (c >> 4) * 256 + (c & 15);
    float* q_out = b.Qd + ch * C * dkp + (c >> 4) * 256 + (c & 15);
#pragma unroll
    for (int t = 0; t < C; ++t) {
      float r;
      if (key) {
        const float decayed = exp2_f32(b_c[t * ldk]);
        r = k_c[t * ldk] * decayed;
        *q_out = q_s[t * ldk + c] * decayed;
        q_out += 16;
      } else {
        r = c < a.dv ? v_s[t * a.dv + c] : 0.f;
      }
      f32x4 L[C / 4];                      // row t (its elements from the diagonal on are zero)
#pragma unroll
      for (int s = 0; s < t; s += 4) L[s / 4] = *reinterpret_cast<const f32x4*>(L_s + t * C + s);
#pragma unroll
      for (int s = 0; s < C; ++s)
        if (s < t) r = fmaf(-L[s / 4][s % 4], x[s], r);
      x[t] = beta_s[t] * r;
      if (key) {
        *w_out = x[t];
        w_out += 16;
      }
      if (t % 2) __builtin_amdgcn_sched_barrier(0);      // (all rows read ahead would not fit the registers)
    }
    if (key) {
      const float total = b_c[(C - 1) * ldk];
      float* kt = b.KT + (ch * dkp + c) * C;
#pragma unroll
      for (int t = 0; t < C; t += 4) {
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = k_c[(t + i) * ldk] * exp2_f32(total - b_c[(t + i) * ldk]);
        *reinterpret_cast<f32x4*>(kt + t) = v;
      }
      b.D[ch * dkp + c] = exp2_f32(total);
    } else {
      float* u0 = b.U0 + (ch * dvp + c) * C;
#pragma unroll
      for (int t = 0; t < C; t += 4) *reinterpret_cast<f32x4*>(u0 + t) = f32x4{x[t], x[t + 1], x[t + 2], x[t + 3]};
    }
  }
}

// Blocks of one (entry, head) go to one die (they read the same W, Qd and KT): with 8 dies dealt round robin, block L
// takes group L % 8 + 8 (L / (8 ns)) and strip (L / 8) % ns.

// Four waves hold the state (TPW 16-row tiles each), a fifth makes the outputs.  Per chunk: P = W S (a partial sum a wave, added
// through LDS by everyone behind the chunk's one barrier), O = Qd S while those sums are on their way, U = U0 - P, S = D S + KT U.
// The partial sums of O are read by the fifth wave behind the NEXT chunk's barrier, with the U it has kept.
constexpr int kDwWaves = 4;

template <typename T, int TPW, int BUFS>      // BUFS - 1: chunks whose operands are requested ahead
__global__ __launch_bounds__(kWave * (kDwWaves + 1), 1) void delta_chunk_walk_kernel(
    DeltaIn a, const int* __restrict__ ent_chunks, ChunkBuf b, float* __restrict__ out, int n_groups) {
  constexpr int C = kDcTokens, NW = kDwWaves;
  __shared__ __attribute__((aligned(16))) f32x4 p_s[2][NW][kWave], o_s[2][NW][kWave];
  const int ns = (a.dv + 15) >> 4, nt = (a.dk + 15) >> 4, dkp = nt * 16, dvp = ns * 16;
  const int group = blockIdx.x % kDies + kDies * (blockIdx.x / (kDies * ns)), strip = (blockIdx.x / kDies) % ns;
  if (group >= n_groups) return;
  const int e = group / a.nh, h = group % a.nh;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, m = lane & 15;
  const int c_first = ent_chunks[2 * e], c_n = ent_chunks[2 * e + 1];
  const int slot = a.state_slots[e];
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  const unsigned at_u = (strip * 16 + m) * C + 4 * g;
  if (w < NW) {
    float* st = a.state + (((size_t)slot * a.nh + h) * ns + strip) * nt * 256;
    f32x4 S[TPW];
    bool has[TPW];
    int tile[TPW];
#pragma unroll
    for (int n = 0; n < TPW; ++n) {
      has[n] = w + n * NW < nt;
      tile[n] = min(w + n * NW, nt - 1);       // (a tile beyond the last: its operands are read, its state stays zero)
      S[n] = has[n] ? *reinterpret_cast<const f32x4*>(st + (size_t)tile[n] * 256 + lane * 4) : zero;
    }
    struct Ops {
      f32x4 W[TPW], Q[TPW], K[TPW], D[TPW], U;
    } buf[BUFS];
    unsigned at_row[TPW], at_kt[TPW], at_d[TPW];
#pragma unroll
    for (int n = 0; n < TPW; ++n) {
      at_row[n] = tile[n] * 256 + m * 16 + 4 * g;
      at_kt[n] = (16 * tile[n] + m) * C + 4 * g;
      at_d[n] = 16 * tile[n] + 4 * g;
    }
    auto fetch = [&](int c, Ops& o) {          // (chunks beyond the last: the last once more, no load behind a branch)
      const size_t ch = (size_t)(c_first + min(c, c_n - 1)) * a.nh + h;
      const float *W = b.W + ch * C * dkp, *Qd = b.Qd + ch * C * dkp, *KT = b.KT + ch * C * dkp, *D = b.D + ch * dkp, *U0 = b.U0 + ch * C * dvp;
#pragma unroll
      for (int n = 0; n < TPW; ++n) {
        o.W[n] = *reinterpret_cast<const f32x4*>(W + at_row[n]);
        o.Q[n] = *reinterpret_cast<const f32x4*>(Qd + at_row[n]);
        o.K[n] = *reinterpret_cast<const f32x4*>(KT + at_kt[n]);
        o.D[n] = *reinterpret_cast<const f32x4*>(D + at_d[n]);
      }
      o.U = *reinterpret_cast<const f32x4*>(U0 + at_u);
    };
    auto one = [&](int c, const Ops& o, Ops& ahead) {
      fetch(c + BUFS - 1, ahead);
      f32x4 P = zero, O = zero;
#pragma unroll
      for (int n = 0; n < TPW; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) P = mfma4(o.W[n][i], S[n][i], P);
      p_s[c & 1][w][lane] = P;
      __syncthreads();
      __builtin_amdgcn_sched_barrier(0);       // (O's products stay behind the barrier: they cover the reads of the shares)
      f32x4 part[NW];
#pragma unroll
      for (int i = 0; i < NW; ++i) part[i] = p_s[c & 1][i][lane];
#pragma unroll
      for (int n = 0; n < TPW; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) O = mfma4(o.Q[n][i], S[n][i], O);
      f32x4 U = o.U;
#pragma unroll
      for (int i = 0; i < NW; ++i) U -= part[i];
#pragma unroll
      for (int n = 0; n < TPW; ++n) {
        S[n] *= o.D[n];
#pragma unroll
        for (int i = 0; i < 4; ++i) S[n] = mfma4(has[n] ? o.K[n][i] : 0.f, U[i], S[n]);
      }
      o_s[c & 1][w][lane] = O;
    };
#pragma unroll
    for (int i = 0; i + 1 < BUFS; ++i) fetch(i, buf[i]);
    int c = 0;
    for (; c + BUFS <= c_n; c += BUFS) {
#pragma unroll
      for (int i = 0; i < BUFS; ++i) one(c + i, buf[i], buf[(i + BUFS - 1) % BUFS]);
    }
#pragma unroll
    for (int i = 0; i + 1 < BUFS; ++i)
      if (c + i < c_n) one(c + i, buf[i], buf[(i + BUFS - 1) % BUFS]);
    __syncthreads();                           // (the last chunk's shares of the outputs are there)
#pragma unroll
    for (int n = 0; n < TPW; ++n)
      if (has[n]) *reinterpret_cast<f32x4*>(st + (size_t)tile[n] * 256 + lane * 4) = S[n];
  } else {
    const int col = strip * 16 + m, row0 = a.cu_tokens[e], len = a.cu_tokens[e + 1] - row0;
    const unsigned at_a = m * 16 + 4 * g;
    f32x4 u[BUFS], A[BUFS], U_before = zero, A_before = zero;
    auto fetch = [&](int c, int i) {
      const size_t ch = (size_t)(c_first + min(c, c_n - 1)) * a.nh + h;
      u[i] = *reinterpret_cast<const f32x4*>(b.U0 + ch * C * dvp + at_u);
      A[i] = *reinterpret_cast<const f32x4*>(b.A + ch * 256 + at_a);
    };
    auto emit = [&](int c) {                   // chunk c's outputs (its P, O and U are known)
      f32x4 y = zero;
#pragma unroll
      for (int i = 0; i < NW; ++i) y += o_s[c & 1][i][lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) y = mfma4(A_before[i], U_before[i], y);
      const int t = c * C + 4 * g;
      float* to = out + (size_t)(row0 + t) * a.nh * a.dv + (size_t)h * a.dv + col;
      if (col < a.dv) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (t + i < len) to[(size_t)i * a.nh * a.dv] = y[i];
      }
    };
    auto one = [&](int c, int i) {
      fetch(c + BUFS - 1, (i + BUFS - 1) % BUFS);
      __syncthreads();                         // chunk c's P, chunk c - 1's O
      f32x4 U = u[i];
#pragma unroll
      for (int j = 0; j < NW; ++j) U -= p_s[c & 1][j][lane];
      if (c > 0) emit(c - 1);
      U_before = U;
      A_before = A[i];
    };
#pragma unroll
    for (int i = 0; i + 1 < BUFS; ++i) fetch(i, i);
    int c = 0;
    for (; c + BUFS <= c_n; c += BUFS) {
#pragma unroll
      for (int i = 0; i < BUFS; ++i) one(c + i, i);
    }
#pragma unroll
    for (int i = 0; i + 1 < BUFS; ++i)
      if (c + i < c_n) one(c + i, i);
    __syncthreads();
    emit(c_n - 1);
  }
  // the convolution's last inputs (everybody who reads the ring has run: the kernel before this one)
  if (a.ring && strip == 0) {
    const int last = a.cu_tokens[e + 1] - 1, len = last + 1 - a.cu_tokens[e], p_last = a.positions[last];
    const int keep = min(len, a.taps - 1), kh = h / a.rep;
    const int n_chan = a.dv + (h % a.rep == 0 ? 2 * a.dk : 0);
    float* ring = a.ring + (size_t)slot * a.taps * a.channels;
    for (int idx = tid; idx < n_chan * keep; idx += blockDim.x) {
      const int back = idx / n_chan, i = idx % n_chan;
      const int chan = i < a.dv ? 2 * a.n_q + h * a.dv + i : i < a.dv + a.dk ? kh * a.dk + i - a.dv : a.n_q + kh * a.dk + i - a.dv - a.dk;
      ring[(size_t)((p_last - back) % a.taps) * a.channels + chan] =
          to_f32<T>(((const T*)a.proj)[(size_t)(last - back) * a.stride + a.c_off + chan]);
    }
  }
}

static int delta_args_ok(const DeltaIn& a, int n_entries) {
  if (a.nh <= 0 || a.rep <= 0 || a.nh % a.rep || a.dk <= 0 || a.dk > 256 || a.dv <= 0 || a.dv > 1024 || a.taps < 1 || a.taps > kDrMaxTaps) return 0;
  if (!a.proj || !a.conv_w || (a.taps > 1 && !a.ring) || !a.log_decay || !a.beta || !a.state || !a.positions || !a.state_slots || !a.cu_tokens) return 0;
  if (a.c_off < 0 || a.c_off + a.channels > a.stride || a.channels != 2 * a.n_q + a.nh * a.dv || a.n_q != (a.nh / a.rep) * a.dk) return 0;
  return a.nh <= 65535 && n_entries <= 65535 && a.beta_off >= 0 && a.beta_off + a.nh <= a.beta_stride;
}

static DeltaIn delta_in(const void* proj, int stride, int c_off, const float* conv_w, int taps, float* ring, const float* log_decay,
                        const float* beta, int beta_stride, int beta_off, const int* positions, const int* state_slots,
                        const int* cu_tokens, float* state, int nh, int nkv, int dk, int dv, float q_scale) {
  const int rep = nkv > 0 ? nh / nkv : 0;
  return DeltaIn{proj, stride, c_off, conv_w, taps, taps > 1 ? ring : nullptr, log_decay, beta, beta_stride, beta_off, positions,
                 state_slots, cu_tokens, state, nh, rep, dk, dv, 2 * nkv * dk + nh * dv, nkv * dk, q_scale};
}

// Every entry one token.  proj [T, stride] of `dtype`: q (nkv dk channels), k, v (nh dv) side by side from c_off;
// conv_w float [channels, taps]; ring float [slots, taps, channels]; log_decay float [T, nh dk]; beta float [T,
// beta_stride]; state float [slots, nh, ceil(dv / 16), ceil(dk / 16), 256]; norm_w float [dv]; gate [T, nh dv] of
// `dtype` (before its sigmoid; null: none); out [T, nh dv] of `dtype`.
SHARPI_EXPORT int sharpi_delta_step(const void* proj, int dtype, int stride, int c_off, const float* conv_w, int taps, float* ring,
                                    const float* log_decay, const float* beta, int beta_stride, int beta_off, const int* positions,
                                    const int* state_slots, const int* cu_tokens, float* state, int n_entries, int nh, int nkv, int dk,
                                    int dv, float q_scale, const float* norm_w, float eps, const void* gate, void* out, hipStream_t stream) {
  if (n_entries <= 0) return SHARPI_OK;
  const DeltaIn a = delta_in(proj, stride, c_off, conv_w, taps, ring, log_decay, beta, beta_stride, beta_off, positions, state_slots,
                             cu_tokens, state, nh, nkv, dk, dv, q_scale);
  if (nkv <= 0 || !delta_args_ok(a, n_entries) || !norm_w || !(eps > 0.f) || !out) return SHARPI_ERR_ARG;
  const int ns = ceil_div(dv, 16);
  dim3 grid(nh, n_entries), block(kWave * (ns < 2 ? 2 : ns < 8 ? ns : 8));
  const size_t lds = 2 * (size_t)dv * sizeof(float);
#define STEP(TV, NT) delta_step_kernel<TV, NT><<<grid, block, lds, stream>>>(a, norm_w, eps, (const TV*)gate, (TV*)out)
#define STEP_BY(TV)                    \
  do {                                 \
    if (dk <= 32) STEP(TV, 2);         \
    else if (dk <= 64) STEP(TV, 4);    \
    else if (dk <= 128) STEP(TV, 8);   \
    else STEP(TV, 16);                 \
  } while (0)
  if (dtype == DT_F32) STEP_BY(float);
  else if (dtype == DT_BF16) STEP_BY(bf16_t);
  else return SHARPI_ERR_ARG;
#undef STEP_BY
#undef STEP
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}

// Entries of any length in chunks: chunks int [n_chunks, 4] = (entry, first row, tokens <= 16, 0), an entry's in order;
// ent_chunks int [n_entries, 2] = (first chunk, chunks); work: scratch floats, sharpi_delta_chunk_floats(..) of them; out
// float [T, nh dv] (neither normed nor gated).
SHARPI_EXPORT long long sharpi_delta_chunk_floats(int n_chunks, int nh, int dk, int dv) {
  const long long dkp = (dk + 15) / 16 * 16, dvp = (dv + 15) / 16 * 16;
  return (long long)n_chunks * nh * (3 * 16 * dkp + dkp + 16 * dvp + 256);
}

SHARPI_EXPORT int sharpi_delta_chunks(const void* proj, int dtype, int stride, int c_off, const float* conv_w, int taps, float* ring,
                                      const float* log_decay, const float* beta, int beta_stride, int beta_off, const int* positions,
                                      const int* state_slots, const int* cu_tokens, float* state, int n_entries, int nh, int nkv, int dk,
                                      int dv, float q_scale, const int* chunks, const int* ent_chunks, int n_chunks, float* work,
                                      float* out, hipStream_t stream) {
  if (n_entries <= 0 || n_chunks <= 0) return SHARPI_OK;
  const DeltaIn a = delta_in(proj, stride, c_off, conv_w, taps, ring, log_decay, beta, beta_stride, beta_off, positions, state_slots,
                             cu_tokens, state, nh, nkv, dk, dv, q_scale);
  if (nkv <= 0 || !delta_args_ok(a, n_entries) || !chunks || !ent_chunks || !work || !out || n_chunks < n_entries) return SHARPI_ERR_ARG;
  if ((dtype != DT_F32 && dtype != DT_BF16) || (long long)n_chunks * nh > 0x7fffffff) return SHARPI_ERR_ARG;
  const int dkp = (dk + 15) / 16 * 16, dvp = (dv + 15) / 16 * 16, nt = dkp / 16, ns = dvp / 16;
  const size_t per = (size_t)n_chunks * nh;
  ChunkBuf b;
  b.W = work;
  b.Qd = b.W + per * 16 * dkp;
  b.KT = b.Qd + per * 16 * dkp;
  b.D = b.KT + per * 16 * dkp;
  b.U0 = b.D + per * dkp;
  b.A = b.U0 + per * 16 * dvp;
  const int dk_room = dk <= 32 ? 32 : dk <= 64 ? 64 : dk <= 128 ? 128 : 256, ldk = dk_room + 4;
  const size_t lds = (size_t)(3 * kDcTokens * ldk + kDcTokens * kDcTokens + kDcTokens + kDcTokens * dv) * sizeof(float);
  if (lds > 160 * 1024) return SHARPI_ERR_ARG;
#define PREP(TV, TAPS, ROOM)                                                                                        \
  do {                                                                                                              \
    auto kern = delta_chunk_prep_kernel<TV, TAPS, ROOM>;                                                            \
    static size_t allowed = 48 * 1024;     /* dynamic LDS this instantiation may take (raised once per size) */     \
    if (lds > allowed) {                                                                                            \
      hipError_t e_ = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
      if (e_ != hipSuccess) return (int)e_;                                                                         \
      allowed = lds;                                                                                                \
    }                                                                                                               \
    kern<<<n_chunks * nh, 256, lds, stream>>>(a, chunks, b);                                                        \
  } while (0)
#define PREP_BY(TV, TAPS)                         \
  do {                                            \
    if (dk_room == 32) PREP(TV, TAPS, 32);        \
    else if (dk_room == 64) PREP(TV, TAPS, 64);   \
    else if (dk_room == 128) PREP(TV, TAPS, 128); \
    else PREP(TV, TAPS, 256);                     \
  } while (0)
  if (dtype == DT_F32) {
    if (taps <= 4) PREP_BY(float, 4);
    else PREP_BY(float, kDrMaxTaps);
  } else {
    if (taps <= 4) PREP_BY(bf16_t, 4);
    else PREP_BY(bf16_t, kDrMaxTaps);
  }
#undef PREP_BY
#undef PREP
  SHARPI_CHECK_LAUNCH();
  const int groups = n_entries * nh;
  const long long blocks = (long long)ceil_div(groups, kDies) * kDies * ns;
  if (blocks > 0x7fffffff) return SHARPI_ERR_ARG;
#define WALK(TV, TPW, BUFS) delta_chunk_walk_kernel<TV, TPW, BUFS><<<(unsigned)blocks, kWave * (kDwWaves + 1), 0, stream>>>(a, ent_chunks, b, out, groups)
#define WALK_BY(TV)                  \
  do {                               \
    if (nt <= 4) WALK(TV, 1, 6);     \
    else if (nt <= 8) WALK(TV, 2, 5);\
    else WALK(TV, 4, 2);             \
  } while (0)
  if (dtype == DT_F32) WALK_BY(float);
  else WALK_BY(bf16_t);
#undef WALK_BY
#undef WALK
  SHARPI_CHECK_LAUNCH();
  return SHARPI_OK;
}
