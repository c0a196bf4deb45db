// Kernels for models that carry per-sequence state besides the paged KV cache (gfx950). Storage of activations
// is bf16 or fp32 (a run-time flag), arithmetic is fp32; recurrent state, residual streams, decays, gates of the
// recurrence and unit norms are fp32 in both modes.
//
//   embed_hash          token embedding * scale + hashed bigram embedding -> S equal fp32 residual streams
//   store_last_token    the step's last token of every sequence -> state (the next step's "previous token")
//   stream_mix_norm     streams <- mix^T streams + out * y, and the next sublayer's input rmsnorm(in . streams) * g
//   poly_norm_act       c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3
//   delta_prep          short conv + SiLU of q/k/v, unit q/k, beta (and the per-head decay) of the gated delta rule
//   conv_state_update   the convolution's trailing inputs -> state
//   gated_delta         the recurrence itself, one workgroup per (sequence, head), the state in registers (four
//                       columns per group of 4 - 16 lanes)
//   qkv_prep            projection bias or short conv, q/k norm, rotate-half rotary (optionally of the values too),
//                       value norm / value mixing, paged cache write
#include "common.h"
#include "lane_reduce.h"
#include "seq_launchers.h"

namespace die {

namespace {

__device__ __forceinline__ float ldv(const void* p, int64_t i, bool f32) {
  return f32 ? reinterpret_cast<const float*>(p)[i] : bf2f(reinterpret_cast<const bf16_t*>(p)[i]);
}
__device__ __forceinline__ void stv(void* p, int64_t i, bool f32, float v) {
  if (f32)
    reinterpret_cast<float*>(p)[i] = v;
  else
    reinterpret_cast<bf16_t*>(p)[i] = f2bf(v);
}
// the value as the activation dtype would hold it
__device__ __forceinline__ float rnd(float v, bool f32) { return f32 ? v : bf2f(f2bf(v)); }
__device__ __forceinline__ float siluf(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }

constexpr int NT = 256;

__device__ __forceinline__ bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
__device__ __forceinline__ bool aligned8(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 7) == 0; }
// 4 consecutive values (element index i a multiple of 4, the address 8- or 16-byte aligned)
__device__ __forceinline__ float4 ld4(const void* p, int64_t i, bool f32) {
  if (f32) return *reinterpret_cast<const float4*>(reinterpret_cast<const float*>(p) + i);
  const uint2 w = *reinterpret_cast<const uint2*>(reinterpret_cast<const bf16_t*>(p) + i);
  return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                     __uint_as_float(w.y & 0xffff0000u));
}
__device__ __forceinline__ void st4(void* p, int64_t i, bool f32, float4 v, float sc) {
  if (f32) {
    *reinterpret_cast<float4*>(reinterpret_cast<float*>(p) + i) = make_float4(v.x * sc, v.y * sc, v.z * sc, v.w * sc);
  } else {
    uint2 w;
    w.x = pack2(v.x * sc, v.y * sc);
    w.y = pack2(v.z * sc, v.w * sc);
    *reinterpret_cast<uint2*>(reinterpret_cast<bf16_t*>(p) + i) = w;
  }
}

// n / d for 0 <= n < 2^21 with inv = 1.0f / d: the nearest a quotient comes to the next integer, 0.5 / d, is far above the
// rounding of the product
__device__ __forceinline__ int qdiv(int n, float inv) { return (int)(((float)n + 0.5f) * inv); }

// sequence of a row: the largest s with cu_q[s] <= row (cu_q == nullptr: the row itself)
__device__ __forceinline__ int seq_of_row(const int* cu_q, int num_seqs, int row) {
  if (cu_q == nullptr) return row;
  int lo = 0, hi = num_seqs - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu_q[mid] <= row)
      lo = mid;
    else
      hi = mid - 1;
  }
  return lo;
}

__global__ void __launch_bounds__(NT) embed_hash_kernel(float* streams, int S, int W, const void* embed,
                                                       const void* bigram, bool f32, const int64_t* ids,
                                                       RaggedRows r, int64_t* prev_tok, float scale,
                                                       int64_t buckets, int64_t mul_prev, int64_t mul_cur) {
  const int row = blockIdx.x;
  const int64_t tok = ids[row];
  int64_t brow = -1;
  if (bigram != nullptr) {
    const int64_t p = r.positions[row];
    if (p <= 0) {
      brow = buckets;
    } else {
      const int s = seq_of_row(r.cu_q, r.num_seqs, row);
      const int first = r.cu_q ? r.cu_q[s] : s;
      const int64_t prev = row > first ? ids[row - 1] : prev_tok[r.state_slots[s]];
      brow = (prev * mul_prev + tok * mul_cur) % buckets;
    }
    if (r.cu_q == nullptr) {
      // one row per sequence: this workgroup is the slot's only reader, so it also stores the new last token
      __syncthreads();
      if (threadIdx.x == 0) prev_tok[r.state_slots[row]] = tok;
    }
  }
  float* out = streams + (int64_t)row * S * W;
  for (int c = threadIdx.x; c < W; c += NT) {
    float x = ldv(embed, tok * W + c, f32) * scale;
    if (brow >= 0) x += ldv(bigram, brow * W + c, f32);
    for (int s = 0; s < S; ++s) out[(int64_t)s * W + c] = x;
  }
}

__global__ void store_last_token_kernel(int64_t* prev_tok, const int64_t* ids, RaggedRows r) {
  const int s = blockIdx.x * blockDim.x + threadIdx.x;
  if (s >= r.num_seqs) return;
  const int last = r.cu_q ? r.cu_q[s + 1] - 1 : s;
  if (r.cu_q && last < r.cu_q[s]) return;
  prev_tok[r.state_slots[s]] = ids[last];
}

constexpr int SMAX = 8;

__global__ void __launch_bounds__(NT) stream_mix_norm_kernel(StreamMixArgs a) {
  __shared__ float red[NT / 64];
  __shared__ float sm[SMAX * SMAX + 2 * SMAX];
  const int S = a.S, W = a.W;
  float* mixw = sm;
  float* outw = sm + SMAX * SMAX;
  float* inw = outw + SMAX;
  if (threadIdx.x < S * S) mixw[threadIdx.x] = a.mix ? a.mix[threadIdx.x] : (threadIdx.x / S == threadIdx.x % S);
  if (threadIdx.x < S) {
    outw[threadIdx.x] = a.outw ? a.outw[threadIdx.x] : 1.0f;
    inw[threadIdx.x] = a.inw ? a.inw[threadIdx.x] : 1.0f;
  }
  __syncthreads();
  const int64_t t = blockIdx.x;
  float* xs = a.streams + t * S * W;
  float ss = 0.f;
  // rows of a multiple of 4 columns: 16-byte accesses, 4 columns per thread and trip; the first KEEP trips keep
  // their u = in . x in registers for the second pass (widths up to 4 * KEEP * NT), later ones re-read the streams
  const bool y_ok = a.y1 == nullptr || (a.ys1 % 4 == 0 && aligned8(a.y1) && (a.y2 == nullptr || (a.ys2 % 4 == 0 && aligned8(a.y2))));
  if (W % 4 == 0 && aligned16(a.streams) && y_ok && (a.h == nullptr || aligned16(a.h))) {
    constexpr int KEEP = 8;
    const int W4 = W / 4;
    float4 ukeep[KEEP];
    auto trip = [&](int c4) -> float4 {
      float4 x[SMAX];
#pragma unroll
      for (int s = 0; s < SMAX; ++s)
        if (s < S) x[s] = reinterpret_cast<const float4*>(xs + (int64_t)s * W)[c4];
      float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
      if (a.y1 != nullptr) {
        float4 y = ld4(a.y1, t * a.ys1 + 4 * c4, a.y_f32);
        y.x *= a.a1, y.y *= a.a1, y.z *= a.a1, y.w *= a.a1;
        if (a.y2 != nullptr) {
          const float4 y2 = ld4(a.y2, t * a.ys2 + 4 * c4, a.y_f32);
          y.x += a.a2 * y2.x, y.y += a.a2 * y2.y, y.z += a.a2 * y2.z, y.w += a.a2 * y2.w;
        }
#pragma unroll
        for (int to = 0; to < SMAX; ++to) {
          if (to < S) {
            const float ow = outw[to];
            float4 n = make_float4(ow * y.x, ow * y.y, ow * y.z, ow * y.w);
#pragma unroll
            for (int s = 0; s < SMAX; ++s) {
              if (s < S) {
                const float m = mixw[s * S + to];
                n.x += m * x[s].x, n.y += m * x[s].y, n.z += m * x[s].z, n.w += m * x[s].w;
              }
            }
            reinterpret_cast<float4*>(xs + (int64_t)to * W)[c4] = n;
            const float iw = inw[to];
            u.x += iw * n.x, u.y += iw * n.y, u.z += iw * n.z, u.w += iw * n.w;
          }
        }
      } else {
#pragma unroll
        for (int s = 0; s < SMAX; ++s) {
          if (s < S) {
            const float iw = inw[s];
            u.x += iw * x[s].x, u.y += iw * x[s].y, u.z += iw * x[s].z, u.w += iw * x[s].w;
          }
        }
      }
      ss += u.x * u.x + u.y * u.y + u.z * u.z + u.w * u.w;
      return u;
    };
#pragma unroll
    for (int it = 0; it < KEEP; ++it) {
      const int c4 = it * NT + threadIdx.x;
      if (c4 < W4) ukeep[it] = trip(c4);
    }
    for (int c4 = KEEP * NT + threadIdx.x; c4 < W4; c4 += NT) trip(c4);
    if (a.h == nullptr) return;
    ss = block_sum<NT>(ss, red);
    const float rs = a.gain[0] / sqrtf(ss / (float)W + a.eps);
#pragma unroll
    for (int it = 0; it < KEEP; ++it) {
      const int c4 = it * NT + threadIdx.x;
      if (c4 < W4) st4(a.h, t * W + 4 * c4, a.h_f32, ukeep[it], rs);
    }
    for (int c4 = KEEP * NT + threadIdx.x; c4 < W4; c4 += NT) {
      float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int s = 0; s < SMAX; ++s) {
        if (s < S) {
          const float4 x = reinterpret_cast<const float4*>(xs + (int64_t)s * W)[c4];  // this thread's own writes
          const float iw = inw[s];
          u.x += iw * x.x, u.y += iw * x.y, u.z += iw * x.z, u.w += iw * x.w;
        }
      }
      st4(a.h, t * W + 4 * c4, a.h_f32, u, rs);
    }
    return;
  }
  for (int c = threadIdx.x; c < W; c += NT) {
    float x[SMAX];
#pragma unroll
    for (int s = 0; s < SMAX; ++s) x[s] = s < S ? xs[(int64_t)s * W + c] : 0.f;
    float u = 0.f;
    if (a.y1 != nullptr) {
      float y = a.a1 * ldv(a.y1, t * a.ys1 + c, a.y_f32);
      if (a.y2 != nullptr) y += a.a2 * ldv(a.y2, t * a.ys2 + c, a.y_f32);
#pragma unroll
      for (int to = 0; to < SMAX; ++to) {
        if (to < S) {
          float n = outw[to] * y;
#pragma unroll
          for (int s = 0; s < SMAX; ++s)
            if (s < S) n += mixw[s * S + to] * x[s];
          xs[(int64_t)to * W + c] = n;
          u += inw[to] * n;
        }
      }
    } else {
#pragma unroll
      for (int s = 0; s < SMAX; ++s)
        if (s < S) u += inw[s] * x[s];
    }
    ss += u * u;
  }
  if (a.h == nullptr) return;
  ss = block_sum<NT>(ss, red);
  const float rs = a.gain[0] / sqrtf(ss / (float)W + a.eps);
  for (int c = threadIdx.x; c < W; c += NT) {
    float u = 0.f;
#pragma unroll
    for (int s = 0; s < SMAX; ++s)
      if (s < S) u += inw[s] * xs[(int64_t)s * W + c];  // this thread's own writes
    stv(a.h, t * W + c, a.h_f32, u * rs);
  }
}

__global__ void __launch_bounds__(NT) poly_norm_act_kernel(void* out, const void* z, int64_t zstride, bool f32,
                                                          const float* coef, float eps, int n) {
  __shared__ float red[NT / 64];
  const int64_t r = blockIdx.x;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  // bf16 rows of a multiple of 8 columns: 16-byte accesses; the first KEEP trips stay in registers between the two
  // passes (rows up to 8 * KEEP * NT wide are read once), wider rows re-read the rest
  constexpr int KEEP = 8;
  if (!f32 && n % 8 == 0 && zstride % 8 == 0 && aligned16(z) && aligned16(out)) {
    const uint4* zr = reinterpret_cast<const uint4*>(reinterpret_cast<const bf16_t*>(z) + r * zstride);
    const int n8 = n / 8;
    uint4 keep[KEEP];
    auto sums = [&](const uint4& v) {
      float f[8];
      unpack8(v, f);
#pragma unroll
      for (int q = 0; q < 8; ++q) {
        const float v2 = f[q] * f[q];
        s2 += v2;
        s4 += v2 * v2;
        s6 += v2 * v2 * v2;
      }
    };
#pragma unroll
    for (int it = 0; it < KEEP; ++it) {
      const int c8 = it * NT + threadIdx.x;
      if (c8 < n8) {
        keep[it] = zr[c8];
        sums(keep[it]);
      }
    }
    for (int c8 = KEEP * NT + threadIdx.x; c8 < n8; c8 += NT) sums(zr[c8]);
    s2 = block_sum<NT>(s2, red);
    s4 = block_sum<NT>(s4, red);
    s6 = block_sum<NT>(s6, red);
    const float r1 = coef[0] / sqrtf(s2 / (float)n + eps), r2 = coef[1] / sqrtf(s4 / (float)n + eps),
                r3 = coef[2] / sqrtf(s6 / (float)n + eps), c3 = coef[3];
    uint4* orow = reinterpret_cast<uint4*>(reinterpret_cast<bf16_t*>(out) + r * n);
    auto apply = [&](const uint4& v) -> uint4 {
      float f[8];
      unpack8(v, f);
#pragma unroll
      for (int q = 0; q < 8; ++q) f[q] = f[q] * r1 + f[q] * f[q] * r2 + f[q] * f[q] * f[q] * r3 + c3;
      return pack8(f);
    };
#pragma unroll
    for (int it = 0; it < KEEP; ++it) {
      const int c8 = it * NT + threadIdx.x;
      if (c8 < n8) orow[c8] = apply(keep[it]);
    }
    for (int c8 = KEEP * NT + threadIdx.x; c8 < n8; c8 += NT) orow[c8] = apply(zr[c8]);
    return;
  }
  for (int c = threadIdx.x; c < n; c += NT) {
    const float v = ldv(z, r * zstride + c, f32);
    const float v2 = v * v;
    s2 += v2;
    s4 += v2 * v2;
    s6 += v2 * v2 * v2;
  }
  s2 = block_sum<NT>(s2, red);
  s4 = block_sum<NT>(s4, red);
  s6 = block_sum<NT>(s6, red);
  const float r1 = coef[0] / sqrtf(s2 / (float)n + eps), r2 = coef[1] / sqrtf(s4 / (float)n + eps),
              r3 = coef[2] / sqrtf(s6 / (float)n + eps), c3 = coef[3];
  for (int c = threadIdx.x; c < n; c += NT) {
    const float v = ldv(z, r * zstride + c, f32);
    stv(out, r * n + c, f32, v * r1 + v * v * r2 + v * v * v * r3 + c3);
  }
}

// ------------------------------------------------------------------------------------------ gated delta rule
constexpr int TAPS_MAX = 16;

// A short causal convolution over each row's own sequence. Row `row` of x is row i of its sequence in this step, at position
// p; inputs before the step come from st [taps - 1, C] (the most recent last), inputs before the sequence's start are
// zero. The channels 8 c8 .. 8 c8 + 7 of the input `back` rows ago (bf16 rows, 16-byte loads):
__device__ __forceinline__ void conv_in8(float* xv, const bf16_t* x, int64_t row, int64_t xstride, int c8, const float* st,
                                         int taps, int C, int i, int64_t p, int back) {
  if (p - back < 0) {
#pragma unroll
    for (int e = 0; e < 8; ++e) xv[e] = 0.f;
  } else if (i - back >= 0) {
    unpack8(*reinterpret_cast<const uint4*>(x + (row - back) * xstride + 8 * c8), xv);
  } else {
    const float4* sp = reinterpret_cast<const float4*>(st + (int64_t)(taps - 1 + i - back) * C + 8 * c8);
    const float4 s0 = sp[0], s1 = sp[1];
    xv[0] = s0.x, xv[1] = s0.y, xv[2] = s0.z, xv[3] = s0.w, xv[4] = s1.x, xv[5] = s1.y, xv[6] = s1.z, xv[7] = s1.w;
  }
}
// One row per sequence: the calling thread is the only reader of its channels' tail, so it shifts it: state row k takes
// row k + 1 (zeros where that lies before the sequence's start), the last one the row's input.
__device__ __forceinline__ void conv8_shift(const bf16_t* x, int64_t row, int64_t xstride, int c8, float* st, int taps,
                                            int C, int64_t p) {
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int k = 0; k + 1 < taps - 1; ++k) {
    const bool live = p - (taps - 2 - k) >= 0;
    float4* dp = reinterpret_cast<float4*>(st + (int64_t)k * C + 8 * c8);
    const float4* sp = reinterpret_cast<const float4*>(st + (int64_t)(k + 1) * C + 8 * c8);
    const float4 t0 = sp[0], t1 = sp[1];
    dp[0] = live ? t0 : zero;
    dp[1] = live ? t1 : zero;
  }
  if (taps > 1) {
    float xv[8];
    unpack8(*reinterpret_cast<const uint4*>(x + row * xstride + 8 * c8), xv);
    float4* dp = reinterpret_cast<float4*>(st + (int64_t)(taps - 2) * C + 8 * c8);
    dp[0] = make_float4(xv[0], xv[1], xv[2], xv[3]);
    dp[1] = make_float4(xv[4], xv[5], xv[6], xv[7]);
  }
}
// rows of a tile: of row rr, its place i in its sequence's rows of this step, its position and its sequence's state
struct ConvRow {
  int i;
  int64_t p;
  float* st;
};
constexpr int CONV_WIN = 4;   // taps held in registers; more are read again for every row
// The convolution of nr consecutive rows for 8 channels, tap-major weights: the weights and the rows (with the CONV_WIN - 1
// rows in front of the tile) are loaded once, all in flight together. put(rr, values): takes a row's 8 results. one_row: a
// step of one row per sequence (nr = 1), whose inputs behind the row are all state; the state then also takes the row.
template <int R, typename F>
__device__ __forceinline__ void conv_rows8(const bf16_t* x, int64_t row0, int nr, int64_t xstride, int c8, const ConvRow* cr,
                                           const float* wt, int taps, int C, bool one_row, F&& put) {
  constexpr int B = CONV_WIN - 1;
  uint4 xr[R + B];   // row row0 - B + j
#pragma unroll
  for (int j = 0; j < R + B; ++j) {
    xr[j] = make_uint4(0, 0, 0, 0);
    if (j < B && (R == 1 || j < CONV_WIN - taps)) continue;   // (single rows: below)
    const int64_t row = row0 + min(j - B, nr - 1);
    xr[j] = *reinterpret_cast<const uint4*>(x + (row < 0 ? 0 : row) * xstride + 8 * c8);
  }
  float w[CONV_WIN][8];
#pragma unroll
  for (int b = 0; b < CONV_WIN; ++b) {   // [taps back]
    const float4* wp = reinterpret_cast<const float4*>(wt + (int64_t)max(0, taps - 1 - b) * C + 8 * c8);
    const float4 w0 = wp[0], w1 = wp[1];
    w[b][0] = w0.x, w[b][1] = w0.y, w[b][2] = w0.z, w[b][3] = w0.w, w[b][4] = w1.x, w[b][5] = w1.y, w[b][6] = w1.z, w[b][7] = w1.w;
  }
  if (R == 1 && one_row && taps <= CONV_WIN) {
    const ConvRow c = cr[0];
    float4 s0[B], s1[B];   // b + 1 rows back
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const int k = taps - 2 - b;
      s0[b] = s1[b] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (k < 0) continue;
      const float4* sp = reinterpret_cast<const float4*>(c.st + (int64_t)k * C + 8 * c8);
      s0[b] = sp[0], s1[b] = sp[1];
    }
    float win[CONV_WIN][8], acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    unpack8(xr[B], win[0]);
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const bool past = c.p - (b + 1) >= 0;   // before the sequence's start: zeros, whatever the slot holds
      const float4 u0 = past ? s0[b] : make_float4(0.f, 0.f, 0.f, 0.f), u1 = past ? s1[b] : make_float4(0.f, 0.f, 0.f, 0.f);
      win[b + 1][0] = u0.x, win[b + 1][1] = u0.y, win[b + 1][2] = u0.z, win[b + 1][3] = u0.w;
      win[b + 1][4] = u1.x, win[b + 1][5] = u1.y, win[b + 1][6] = u1.z, win[b + 1][7] = u1.w;
    }
#pragma unroll
    for (int b = CONV_WIN - 1; b >= 0; --b) {
      if (b < taps) {
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += w[b][e] * win[b][e];
      }
    }
    put(0, acc);
#pragma unroll
    for (int b = 0; b < B; ++b) {   // the input b rows back lands in place taps - 2 - b
      const int k = taps - 2 - b;
      if (k < 0) continue;
      float4* dp = reinterpret_cast<float4*>(c.st + (int64_t)k * C + 8 * c8);
      dp[0] = make_float4(win[b][0], win[b][1], win[b][2], win[b][3]);
      dp[1] = make_float4(win[b][4], win[b][5], win[b][6], win[b][7]);
    }
    return;
  }
  float xf[R + B][8];
#pragma unroll
  for (int j = 0; j < R + B; ++j) unpack8(xr[j], xf[j]);
#pragma unroll
  for (int rr = 0; rr < R; ++rr) {
    if (rr >= nr) break;
    const ConvRow c = cr[rr];
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (R > 1 && taps <= CONV_WIN && c.i >= taps - 1) {   // every input is a row of this step
#pragma unroll
      for (int b = CONV_WIN - 1; b >= 0; --b) {
        if (b < taps) {
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[e] += w[b][e] * xf[rr + B - b][e];
        }
      }
    } else {
      for (int b = taps - 1; b >= 0; --b) {
        float xv[8];
        conv_in8(xv, x, row0 + rr, xstride, c8, c.st, taps, C, c.i, c.p, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += wt[(int64_t)(taps - 1 - b) * C + 8 * c8 + e] * xv[e];
      }
    }
    put(rr, acc);
  }
  if (one_row) conv8_shift(x, row0, xstride, c8, cr[0].st, taps, C, cr[0].p);
}
// Fills cr for rows row0 .. row0 + nr - 1. Every thread looks at its own sequences, so that finding the rows' sequences costs
// one round of loads (a binary search would be a chain of them).
__device__ __forceinline__ void conv_rows_of(ConvRow* cr, int64_t row0, int nr, const RaggedRows& r, float* conv_state, int taps,
                                             int C) {
  auto fill = [&](int rr, int s, int first) {
    cr[rr].i = (int)row0 + rr - first;
    cr[rr].p = r.positions[row0 + rr];
    cr[rr].st = conv_state + (int64_t)r.state_slots[s] * (taps - 1) * C;
  };
  if (r.cu_q == nullptr) {
    for (int rr = threadIdx.x; rr < nr; rr += NT) fill(rr, (int)row0 + rr, (int)row0 + rr);
  } else {
    for (int s = threadIdx.x; s < r.num_seqs; s += NT) {
      const int lo = r.cu_q[s], hi = r.cu_q[s + 1];
      for (int rr = max(0, lo - (int)row0); rr < nr && (int)row0 + rr < hi; ++rr) fill(rr, s, lo);
    }
  }
  __syncthreads();
}
// rows per workgroup: as many as fit 64 KB of LDS (fp32 [R][n]), at most 4; one in a step of one row per sequence
static int conv_tile(const RaggedRows& r, int64_t n) {
  if (r.cu_q == nullptr) return 1;
  const int64_t fit = 64 * 1024 / (4 * n);
  return fit >= 4 ? 4 : (fit >= 2 ? 2 : 1);
}
// the same for one channel; wc / wj: strides of the weight's channel and tap
__device__ __forceinline__ float conv1(const void* x, bool f32, int64_t row, int64_t xstride, int c, const float* st,
                                       const float* w, int64_t wc, int64_t wj, int taps, int C, int i, int64_t p) {
  float acc = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;
    if (p - back < 0) continue;
    const int src = i - back;
    const float xv = src >= 0 ? ldv(x, (row - back) * xstride + c, f32) : st[(int64_t)(taps - 1 + src) * C + c];
    acc += w[c * wc + j * wj] * xv;
  }
  return acc;
}
__device__ __forceinline__ void conv1_shift(const void* x, bool f32, int64_t row, int64_t xstride, int c, float* st,
                                            int taps, int C, int64_t p) {
  for (int k = 0; k + 1 < taps - 1; ++k)
    st[(int64_t)k * C + c] = p - (taps - 2 - k) >= 0 ? st[(int64_t)(k + 1) * C + c] : 0.f;
  if (taps > 1) st[(int64_t)(taps - 2) * C + c] = ldv(x, row * xstride + c, f32);
}

// a lane's share of the sum of squares of a head of d values in LDS, 16 lanes per head (gl: the lane); rows of n values.
// 16 bytes per lane where that is aligned: heads a multiple of the bank count apart then do not collide
__device__ __forceinline__ float lane_sumsq(const float* v, int d, int gl, int n) {
  float ss = 0.f;
  if (((d | n) & 3) == 0) {
    for (int c = 4 * gl; c < d; c += 64) {
      const float4 x = *reinterpret_cast<const float4*>(v + c);
      ss += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
    }
  } else {
    for (int c = gl; c < d; c += 16) ss += v[c] * v[c];
  }
  return ss;
}

template <int R>
__global__ void __launch_bounds__(NT) delta_prep_kernel(float* qkv32, float* bg, const void* x, const void* b,
                                                       const void* a, int64_t xstride, bool f32, const float* conv_w,
                                                       const float* conv_wt, float* conv_state, const float* A_log,
                                                       const float* dt_bias, DeltaShape sh, RaggedRows r) {
  extern __shared__ __attribute__((aligned(16))) float vals[];  // [R][C]
  __shared__ ConvRow cr[R];
  const int64_t row0 = (int64_t)blockIdx.x * R;
  const int nr = min(R, (int)(r.total_rows - row0));
  const int C = sh.channels(), taps = sh.taps;
  conv_rows_of(cr, row0, nr, r, conv_state, taps, C);
  // bf16 steps with the weights also given tap-major ([taps, C]): 8 channels per thread and trip
  const bool wide = conv_wt != nullptr && !f32 && C % 8 == 0 && xstride % 8 == 0 && aligned16(x);
  const bf16_t* xb = reinterpret_cast<const bf16_t*>(x);
  for (int c8 = threadIdx.x; wide && c8 < C / 8; c8 += NT) {
    conv_rows8<R>(xb, row0, nr, xstride, c8, cr, conv_wt, taps, C, r.cu_q == nullptr, [&](int rr, const float* acc) {
      float4* dst = reinterpret_cast<float4*>(vals + rr * C + 8 * c8);
      float v[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = rnd(siluf(rnd(acc[e], false)), false);
      dst[0] = make_float4(v[0], v[1], v[2], v[3]);
      dst[1] = make_float4(v[4], v[5], v[6], v[7]);
    });
  }
  for (int c = threadIdx.x; !wide && c < C; c += NT) {
    for (int rr = 0; rr < nr; ++rr)
      vals[rr * C + c] = rnd(siluf(rnd(conv1(x, f32, row0 + rr, xstride, c, cr[rr].st, conv_w, taps, 1, taps, C, cr[rr].i, cr[rr].p), f32)), f32);
    if (r.cu_q == nullptr) conv1_shift(x, f32, row0, xstride, c, cr[0].st, taps, C, cr[0].p);
  }
  __syncthreads();
  // unit q and k: 16 lanes per head
  const int gl = threadIdx.x & 15, grp = threadIdx.x >> 4;
  const int G = sh.kv_heads, d = sh.dim;
  const float inv_2g = 1.0f / (float)(2 * G);
  for (int u = grp; u < nr * 2 * G; u += NT / 16) {
    const int rr = R == 1 ? 0 : qdiv(u, inv_2g), hh = u - rr * 2 * G;
    float* v = vals + rr * C + hh * d;
    float sc = 1.0f / sqrtf(group_sum<16>(lane_sumsq(v, d, gl, C)) + 1e-6f);
    if (hh < G) sc *= 1.0f / sqrtf((float)d);
    if (((d | C) & 3) == 0) {
      for (int c = 4 * gl; c < d; c += 64) {
        const float4 x = *reinterpret_cast<const float4*>(v + c);
        *reinterpret_cast<float4*>(v + c) = make_float4(x.x * sc, x.y * sc, x.z * sc, x.w * sc);
      }
    } else {
      for (int c = gl; c < d; c += 16) v[c] *= sc;
    }
  }
  __syncthreads();
  if (C % 4 == 0) {
    float4* dst = reinterpret_cast<float4*>(qkv32 + row0 * C);
    for (int c4 = threadIdx.x; c4 < nr * C / 4; c4 += NT) dst[c4] = reinterpret_cast<const float4*>(vals)[c4];
  } else {
    for (int c = threadIdx.x; c < nr * C; c += NT) qkv32[row0 * C + c] = vals[c];
  }
  const int H = sh.heads;
  const float inv_h = 1.0f / (float)H;
  for (int u = threadIdx.x; u < nr * H; u += NT) {
    const int rr = R == 1 ? 0 : qdiv(u, inv_h), h = u - rr * H;
    const int64_t row = row0 + rr;
    const float beta = sigmoidf(ldv(b, row * xstride + h, f32));
    if (a == nullptr) {   // the decay is the recurrence kernel's (per key channel)
      bg[row * H + h] = beta;
      continue;
    }
    const float sp = softplus_of<false>(ldv(a, row * xstride + h, f32) + dt_bias[h]);
    bg[row * 2 * H + h] = beta;
    bg[row * 2 * H + H + h] = expf(-expf(A_log[h]) * sp);
  }
}

__global__ void __launch_bounds__(NT) conv_state_update_kernel(float* conv_state, const void* x, int64_t xstride,
                                                              bool f32, DeltaShape sh, RaggedRows r) {
  const int s = blockIdx.y;
  const int c = blockIdx.x * NT + threadIdx.x;
  const int C = sh.channels(), taps = sh.taps;
  if (c >= C) return;
  const int q0 = r.cu_q ? r.cu_q[s] : s;
  const int L = r.cu_q ? r.cu_q[s + 1] - q0 : 1;
  if (L <= 0) return;
  const int64_t p0 = r.positions[q0];
  float* st = conv_state + (int64_t)r.state_slots[s] * (taps - 1) * C;
  float old[TAPS_MAX];
#pragma unroll
  for (int k = 0; k < TAPS_MAX; ++k) old[k] = k < taps - 1 ? st[(int64_t)k * C + c] : 0.f;
  for (int k = 0; k < taps - 1; ++k) {
    const int idx = L - 1 - (taps - 2 - k);  // row of the step that lands in place k
    float v = 0.f;
    if (idx >= 0) {
      v = ldv(x, (int64_t)(q0 + idx) * xstride + c, f32);
    } else if (p0 + idx >= 0) {
      const int ok = taps - 1 + idx;
#pragma unroll
      for (int m = 0; m < TAPS_MAX; ++m)
        if (m == ok) v = old[m];
    }
    st[(int64_t)k * C + c] = v;
  }
}

constexpr int TB = 16;  // tokens staged per trip, at most

// 4 consecutive values at p[i + c] of a row piece of n values (c a multiple of 4), zeros beyond it. VEC (n and the row's
// start multiples of 4, the base aligned): one 8- / 16-byte load without a branch around it, so that a run of these stays
// in flight together.
template <bool F32, bool VEC> __device__ __forceinline__ float4 ld4z(const void* p, int64_t i, int c, int n) {
  if constexpr (VEC) {
    const float4 v = ld4(p, i + (c < n ? c : 0), F32);
    return c < n ? v : make_float4(0.f, 0.f, 0.f, 0.f);
  } else {
    float f[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) f[e] = c + e < n ? ldv(p, i + c + e, F32) : 0.f;
    return make_float4(f[0], f[1], f[2], f[3]);
  }
}

// One workgroup per (sequence, head). The state S [dim, vdim] lives in registers for the whole step: a group of LN lanes
// holds 4 columns, lane l of it the rows 4 LN m + 4 l + i (m < M, i < 4) — 16 M values per lane, LN M 4 >= dim. A token
// costs a lane 4 multiply-adds per value and two sums over its group (S^T k and S^T q, on DPP adds); k, q (and with CD
// the decays) are read from LDS as consecutive float4s, one read per 16 values of the state. Up to TB tokens are staged
// per trip, the next trip's rows are already in flight; the read-outs of a trip are normed and gated afterwards, one wave
// per token. NE: float4s of q (and of k) per thread and trip. CD: a decay per key channel, computed while a trip is staged. VEC: dim, vdim and the row strides are multiples
// of 4.
template <int LN, int M, int NE, bool F32, bool CD, bool VEC>
__global__ void __launch_bounds__(M > 2 && NE == 1 ? 512 : 1024) gated_delta_kernel(GatedDeltaArgs a, RaggedRows r, int TT) {
  const DeltaShape& sh = a.sh;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int DPAD = 4 * LN * M, NV = 4;
  const int d = sh.dim, dv = sh.vdim, H = sh.heads, G = sh.kv_heads, C = sh.channels();
  const int dvp = (dv + 3) & ~3;
  float* qs = sm;                  // [TB][DPAD], zero beyond dim
  float* ks = qs + TB * DPAD;      // [TB][DPAD]
  float* gs = ks + TB * DPAD;      // [TB][DPAD] with CD: decays
  float* vs = gs + (CD ? TB * DPAD : 0);   // [TB][dvp]
  float* os = vs + TB * dvp;       // [TB][dvp]
  float* bs = os + TB * dvp;       // [TB][2]: beta, decay per head
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x, nthr = blockDim.x;
  const int l = tid % LN, j0 = 4 * (tid / LN);
  const int kh = h / (H / G);
  const int q0 = r.cu_q ? r.cu_q[s] : s;
  const int L = r.cu_q ? r.cu_q[s + 1] - q0 : 1;
  if (L <= 0) return;
  const bool fresh = r.positions[q0] <= 0;
  const bool live = j0 < dv;
  float* st = a.state + ((int64_t)r.state_slots[s] * H + h) * d * dv;
  const float expA = CD ? expf(a.A_log[h]) : 0.f;
  const int bgw = CD ? H : 2 * H;

  // a trip's rows in registers on their way to LDS
  float4 rq[NE], rk[NE], rz[NE], rv[NV];
  float2 rb;
  // (a thread without a row of its own loads the trip's last one and does not store it)
  auto fetch = [&](int t0) {
    const int nb = min(TT, L - t0);
#pragma unroll
    for (int u = 0; u < NE; ++u) {
      const int e = tid + u * nthr, tt = e / (DPAD / 4), c = 4 * (e % (DPAD / 4));
      const int64_t row = q0 + t0 + min(tt, nb - 1);
      rq[u] = ld4z<true, VEC>(a.qkv32, row * C + kh * d, c, d);
      rk[u] = ld4z<true, VEC>(a.qkv32, row * C + G * d + kh * d, c, d);
      if (CD) rz[u] = ld4z<F32, VEC>(a.z, row * a.zstride + h * d, c, d);
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      if (u * LN >= TB) break;   // a trip's values fill at most TB / LN float4s per thread
      const int e = tid + u * nthr, tt = e / (dvp / 4), c = 4 * (e % (dvp / 4));
      rv[u] = ld4z<true, VEC>(a.qkv32, (int64_t)(q0 + t0 + min(tt, nb - 1)) * C + 2 * G * d + h * dv, c, dv);
    }
    const float* b = a.bg + (int64_t)(q0 + t0 + min(tid, nb - 1)) * bgw + h;
    rb = make_float2(b[0], CD ? 0.f : b[H]);
  };
  float4 zb[NE];
#pragma unroll
  for (int u = 0; u < NE; ++u)
    if (CD) zb[u] = ld4z<true, VEC>(a.z_bias, h * d, 4 * ((tid + u * nthr) % (DPAD / 4)), d);
  auto decay1 = [&](float z, int c) { return c < d ? exp_of<!F32>(-expA * softplus_of<!F32>(z)) : 0.f; };
  auto stage = [&](int nb) {
#pragma unroll
    for (int u = 0; u < NE; ++u) {
      const int e = tid + u * nthr, tt = e / (DPAD / 4), c = 4 * (e % (DPAD / 4));
      if (tt < nb) {
        *reinterpret_cast<float4*>(qs + tt * DPAD + c) = rq[u];
        *reinterpret_cast<float4*>(ks + tt * DPAD + c) = rk[u];
        if (CD)
          *reinterpret_cast<float4*>(gs + tt * DPAD + c) =
              make_float4(decay1(rz[u].x + zb[u].x, c), decay1(rz[u].y + zb[u].y, c + 1), decay1(rz[u].z + zb[u].z, c + 2),
                          decay1(rz[u].w + zb[u].w, c + 3));
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      if (u * LN >= TB) break;
      const int e = tid + u * nthr, tt = e / (dvp / 4), c = 4 * (e % (dvp / 4));
      if (tt < nb) *reinterpret_cast<float4*>(vs + tt * dvp + c) = rv[u];
    }
    if (tid < nb) *reinterpret_cast<float2*>(bs + 2 * tid) = rb;
  };

  fetch(0);
  float S[M][4][4];   // [m][i][column]
#pragma unroll
  for (int m = 0; m < M; ++m)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 4 * LN * m + 4 * l + i;
      float4 v = ld4z<true, VEC>(st, (int64_t)min(row, d - 1) * dv, j0, dv);
      if (fresh || row >= d) v = make_float4(0.f, 0.f, 0.f, 0.f);   // (a new sequence reads its slot but not its content)
      S[m][i][0] = v.x, S[m][i][1] = v.y, S[m][i][2] = v.z, S[m][i][3] = v.w;
    }
  const int lane = tid & 63, wave = tid >> 6, nwaves = nthr >> 6;
  for (int t0 = 0; t0 < L; t0 += TT) {
    const int nb = min(TT, L - t0);
    stage(nb);
    __syncthreads();
    if (t0 + TT < L) fetch(t0 + TT);
    for (int tt = 0; tt < nb; ++tt) {
      const float2 bg = *reinterpret_cast<const float2*>(bs + 2 * tt);
      const float4 v4 = live ? *reinterpret_cast<const float4*>(vs + tt * dvp + j0) : make_float4(0.f, 0.f, 0.f, 0.f);
      const float4* kt = reinterpret_cast<const float4*>(ks + tt * DPAD) + l;
      const float4* qt = reinterpret_cast<const float4*>(qs + tt * DPAD) + l;
      const float4* gt = reinterpret_cast<const float4*>(gs + tt * DPAD) + l;
      float kk[M][4], dot[4] = {0.f, 0.f, 0.f, 0.f}, o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int m = 0; m < M; ++m) {
        const float4 k4 = kt[LN * m], g4 = CD ? gt[LN * m] : make_float4(bg.y, bg.y, bg.y, bg.y);
        const float gg[4] = {g4.x, g4.y, g4.z, g4.w};
        kk[m][0] = k4.x, kk[m][1] = k4.y, kk[m][2] = k4.z, kk[m][3] = k4.w;
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            S[m][i][c] *= gg[i];
            dot[c] += S[m][i][c] * kk[m][i];
          }
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) dot[c] = group_sum<LN>(dot[c]);
      const float u[4] = {bg.x * (v4.x - dot[0]), bg.x * (v4.y - dot[1]), bg.x * (v4.z - dot[2]), bg.x * (v4.w - dot[3])};
#pragma unroll
      for (int m = 0; m < M; ++m) {
        const float4 q4 = qt[LN * m];
        const float qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            S[m][i][c] += kk[m][i] * u[c];
            o[c] += S[m][i][c] * qq[i];
          }
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) o[c] = group_sum<LN>(o[c]);
      if (l == 0 && live) *reinterpret_cast<float4*>(os + tt * dvp + j0) = make_float4(o[0], o[1], o[2], o[3]);
    }
    __syncthreads();
    for (int tt = wave; tt < nb; tt += nwaves) {
      float ss = 0.f;
      for (int c = lane; c < dv; c += 64) ss += os[tt * dvp + c] * os[tt * dvp + c];
      ss = wave_sum(ss);
      const float rs = a.mult / sqrtf(ss / (float)dv + a.eps);
      const int64_t row = q0 + t0 + tt;
      for (int c = lane; c < dv; c += 64) {
        const float gt = ldv(a.gate, row * a.gstride + h * dv + c, F32);
        stv(a.out, row * a.ostride + h * dv + c, F32,
            os[tt * dvp + c] * rs * a.norm_w[c] * (a.gate_sigmoid ? sigmoidf(gt) : siluf(gt)));
      }
    }
  }
  if (!live) return;
#pragma unroll
  for (int m = 0; m < M; ++m)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 4 * LN * m + 4 * l + i;
      if (row >= d) continue;
      float* p = st + (int64_t)row * dv + j0;
      if constexpr (VEC) {
        *reinterpret_cast<float4*>(p) = make_float4(S[m][i][0], S[m][i][1], S[m][i][2], S[m][i][3]);
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (j0 + c < dv) p[c] = S[m][i][c];
      }
    }
}

// --------------------------------------------------------------------------------------------------- qkv prep
// One workgroup per R rows (R > 1 with a convolution only, which then reads its weights once for all of them).
template <int R, bool CONV>
__global__ void __launch_bounds__(NT) qkv_prep_kernel(QkvPrepArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[NT / 64];
  __shared__ ConvRow cr[CONV ? R : 1];
  const int H = a.heads, G = a.kv_heads, d = a.dim, dv = a.vdim;
  const int nq = H * d, nk = G * d, nv = G * dv, C = nq + nk + nv;
  float* qv = sm;               // row rr: [q | k | v] at rr * C
  float* kv = qv + nq;
  float* vv = kv + nk;
  // cosine / sine of the rows' rotation angles, shared by the heads: keys and queries, then values
  const int half = a.rot_dims / 2, vhalf = a.v_inv_freq != nullptr ? dv / 2 : 0, nang = half + vhalf;
  float* ct = sm + R * C;
  float* snt = ct + R * nang;
  const int64_t t0 = (int64_t)blockIdx.x * R;
  const int nr = R == 1 ? 1 : min(R, (int)(a.T - t0));
  const bool f32 = a.f32;
  // cache row of key/value head 0 (head g: g * block_size further; a block's interior is head-major), < 0: not written
  __shared__ int64_t crow[R];
  if (threadIdx.x < nr) {
    const int64_t slot = a.slots[t0 + threadIdx.x];
    const int64_t blk = slot / a.block_size;
    crow[threadIdx.x] = slot < 0 ? -1 : blk * G * a.block_size + (slot - blk * a.block_size);
  }
  const float inv_ang = 1.0f / (float)max(1, nang), inv_half = 1.0f / (float)max(1, half), inv_vhalf = 1.0f / (float)max(1, vhalf),
              inv_hg = 1.0f / (float)(H + G), inv_g = 1.0f / (float)G, inv_d = 1.0f / (float)d, inv_dv = 1.0f / (float)dv;
  for (int e = threadIdx.x; e < nr * nang; e += NT) {
    const int rr = R == 1 ? 0 : qdiv(e, inv_ang), i = e - rr * nang;
    const bool kq = i < half;
    float sn, cs;
    sincosf((float)a.positions[t0 + rr] * (kq ? a.inv_freq[i] : a.v_inv_freq[i - half]), &sn, &cs);
    const float gain = kq ? a.rot_gain : 1.0f;
    ct[e] = cs * gain;
    snt[e] = sn * gain;
  }
  float sq = 0.f, sk = 0.f;   // sums of squares over the whole projections (used with R == 1)
  float lam = 0.f;
  if (a.v_lambda != nullptr) lam = a.v_lambda[0];
  // bf16 with head sizes that are multiples of 8: 16-byte loads and stores, 8 values per thread and trip
  const bool v_is_k = a.v == nullptr;   // values = keys as projected
  const bool wide = !f32 && d % 8 == 0 && dv % 8 == 0 && a.xstride % 8 == 0 && aligned16(a.q) && aligned16(a.k) &&
                    aligned16(a.v) && aligned16(a.q_out) && aligned16(a.cache) &&
                    (a.v_first == nullptr || (a.vfstride % 8 == 0 && aligned16(a.v_first)));
  if (CONV) {
    // short convolution over the sequence of the channels q | k | v (adjacent columns)
    conv_rows_of(cr, t0, nr, a.r, a.conv_state, a.taps, C);
    const bf16_t* xb = reinterpret_cast<const bf16_t*>(a.q);
    for (int c8 = threadIdx.x; wide && c8 < C / 8; c8 += NT) {
      conv_rows8<R>(xb, t0, nr, a.xstride, c8, cr, a.conv_wt, a.taps, C, a.r.cu_q == nullptr, [&](int rr, const float* acc) {
        float4* dst = reinterpret_cast<float4*>(qv + rr * C + 8 * c8);
        dst[0] = make_float4(acc[0], acc[1], acc[2], acc[3]);
        dst[1] = make_float4(acc[4], acc[5], acc[6], acc[7]);
        if (R == 1) {
          float ss = 0.f;
#pragma unroll
          for (int e = 0; e < 8; ++e) ss += acc[e] * acc[e];
          if (8 * c8 < nq)
            sq += ss;
          else if (8 * c8 < nq + nk)
            sk += ss;
        }
      });
    }
    for (int c = threadIdx.x; !wide && c < C; c += NT) {
      for (int rr = 0; rr < nr; ++rr) {
        const float x = conv1(a.q, f32, t0 + rr, a.xstride, c, cr[rr].st, a.conv_wt, 1, C, a.taps, C, cr[rr].i, cr[rr].p);
        qv[rr * C + c] = x;
        if (c < nq)
          sq += x * x;
        else if (c < nq + nk)
          sk += x * x;
      }
      if (a.r.cu_q == nullptr) conv1_shift(a.q, f32, t0, a.xstride, c, cr[0].st, a.taps, C, cr[0].p);
    }
  } else if (wide) {
    const bf16_t* qp = reinterpret_cast<const bf16_t*>(a.q) + t0 * a.xstride;
    const bf16_t* kp = reinterpret_cast<const bf16_t*>(a.k) + t0 * a.xstride;
    const bf16_t* vp = reinterpret_cast<const bf16_t*>(a.v) + t0 * a.xstride;
    for (int c8 = threadIdx.x; c8 < (v_is_k ? nq + nk : C) / 8; c8 += NT) {
      const int c = 8 * c8;
      float f[8];
      unpack8(*reinterpret_cast<const uint4*>(c < nq ? qp + c : (c < nq + nk ? kp + c - nq : vp + c - nq - nk)), f);
      if (a.bias != nullptr) {
        const float4* bp = reinterpret_cast<const float4*>(a.bias + c);
        const float4 b0 = bp[0], b1 = bp[1];
        f[0] += b0.x, f[1] += b0.y, f[2] += b0.z, f[3] += b0.w, f[4] += b1.x, f[5] += b1.y, f[6] += b1.z, f[7] += b1.w;
      }
      if (c < nq + nk) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
        if (c < nq)
          sq += ss;
        else
          sk += ss;
      } else if (a.v_lambda != nullptr) {
        float g8[8];
        unpack8(*reinterpret_cast<const uint4*>(reinterpret_cast<const bf16_t*>(a.v_first) + t0 * a.vfstride + c - nq - nk), g8);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = (1.0f - lam) * f[e] + lam * g8[e];
      }
      float4* dst = reinterpret_cast<float4*>(qv + c);   // qv, kv and vv are adjacent
      dst[0] = make_float4(f[0], f[1], f[2], f[3]);
      dst[1] = make_float4(f[4], f[5], f[6], f[7]);
    }
  } else {
    for (int c = threadIdx.x; c < nq; c += NT) {
      const float x = ldv(a.q, t0 * a.xstride + c, f32) + (a.bias != nullptr ? a.bias[c] : 0.f);
      qv[c] = x;
      sq += x * x;
    }
    for (int c = threadIdx.x; c < nk; c += NT) {
      const float x = ldv(a.k, t0 * a.xstride + c, f32) + (a.bias != nullptr ? a.bias[nq + c] : 0.f);
      kv[c] = x;
      sk += x * x;
    }
    for (int c = threadIdx.x; c < (v_is_k ? 0 : nv); c += NT) {
      float x = ldv(a.v, t0 * a.xstride + c, f32) + (a.bias != nullptr ? a.bias[nq + nk + c] : 0.f);
      if (a.v_lambda != nullptr) x = (1.0f - lam) * x + lam * ldv(a.v_first, t0 * a.vfstride + c, f32);
      vv[c] = x;
    }
  }
  const bool per_head = a.q_norm != nullptr && a.head_norm;
  auto rotate = [&]() {
    for (int e = threadIdx.x; e < nr * (H + G) * half; e += NT) {
      const int hr = qdiv(e, inv_half), i = e - hr * half;
      const int rr = R == 1 ? 0 : qdiv(hr, inv_hg), hd = hr - rr * (H + G);
      float* base = (hd < H ? qv + hd * d : kv + (hd - H) * d) + rr * C;
      const float cs = ct[rr * nang + i], sn = snt[rr * nang + i];
      const float u = base[i], v = base[i + half];
      base[i] = u * cs - v * sn;
      base[i + half] = v * cs + u * sn;
    }
  };
  // query temperature of row rr
  auto temperature = [&](int rr) {
    return 1.0f + a.q_temp_coef * logf((float)((a.positions[t0 + rr] + 1) / a.q_temp_every) + 1.0f);
  };
  const bool rot_first = per_head && a.norm_after_rot;
  if (a.rot_dims > 0 && rot_first) {
    __syncthreads();   // every thread's loads are in LDS
    rotate();
  }
  if (v_is_k && !per_head) {
    __syncthreads();
    for (int c = threadIdx.x; c < nk; c += NT) vv[c] = kv[c];
  }
  if (per_head) {
    // 16 lanes per head, 16 heads at a time: sum of squares, then one pass that also keeps the raw key as the value
    // (values taken from the keys) and folds the query temperature into the q heads' factor
    __syncthreads();
    const int grp = threadIdx.x >> 4, gl = threadIdx.x & 15;
    for (int u = grp; u < nr * (H + G); u += NT / 16) {
      const int rr = R == 1 ? 0 : qdiv(u, inv_hg), hd = u - rr * (H + G);
      float* base = (hd < H ? qv + hd * d : kv + (hd - H) * d) + rr * C;
      const float* w = hd < H ? a.q_norm : a.k_norm;
      float* raw = (v_is_k && hd >= H) ? vv + (hd - H) * d : nullptr;
      float rs = 1.0f / sqrtf(group_sum<16>(lane_sumsq(base, d, gl, C)) / (float)d + a.eps);
      if (hd < H && a.q_temp_coef != 0.f) rs *= temperature(rr);
      if (((d | C) & 3) == 0) {
        for (int c = 4 * gl; c < d; c += 64) {
          const float4 x = *reinterpret_cast<const float4*>(base + c), ww = *reinterpret_cast<const float4*>(w + c);
          if (raw != nullptr) *reinterpret_cast<float4*>(raw + c) = x;
          *reinterpret_cast<float4*>(base + c) = make_float4(x.x * rs * ww.x, x.y * rs * ww.y, x.z * rs * ww.z, x.w * rs * ww.w);
        }
        continue;
      }
      for (int c = gl; c < d; c += 16) {
        const float x = base[c];
        if (raw != nullptr) raw[c] = x;
        base[c] = x * rs * w[c];
      }
    }
  } else if (a.q_norm != nullptr) {   // over the whole projection (R == 1)
    __shared__ float redk[NT / 64];
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((threadIdx.x & 63) == 0) {
      red[threadIdx.x >> 6] = sq;
      redk[threadIdx.x >> 6] = sk;
    }
    __syncthreads();   // (every thread's loads are in LDS, too)
    sq = sk = 0.f;
#pragma unroll
    for (int i = 0; i < NT / 64; ++i) {
      sq += red[i];
      sk += redk[i];
    }
    const float rq = 1.0f / sqrtf(sq / (float)nq + a.eps), rk = 1.0f / sqrtf(sk / (float)nk + a.eps);
    if (((nq | nk) & 3) == 0 && aligned16(a.q_norm) && aligned16(a.k_norm)) {
      for (int c = 4 * threadIdx.x; c < nq + nk; c += 4 * NT) {   // (qv and kv are adjacent)
        const float4 x = *reinterpret_cast<const float4*>(qv + c);
        const float4 ww = *reinterpret_cast<const float4*>(c < nq ? a.q_norm + c : a.k_norm + (c - nq));
        const float rs = c < nq ? rq : rk;
        *reinterpret_cast<float4*>(qv + c) = make_float4(x.x * rs * ww.x, x.y * rs * ww.y, x.z * rs * ww.z, x.w * rs * ww.w);
      }
    } else {
      for (int c = threadIdx.x; c < nq; c += NT) qv[c] *= rq * a.q_norm[c];
      for (int c = threadIdx.x; c < nk; c += NT) kv[c] *= rk * a.k_norm[c];
    }
  }
  __syncthreads();
  if (a.q_temp_coef != 0.f && !per_head) {
    for (int rr = 0; rr < nr; ++rr) {
      const float qm = temperature(rr);
      for (int c = threadIdx.x; c < nq; c += NT) qv[rr * C + c] *= qm;
    }
    __syncthreads();
  }
  if (a.rot_dims > 0 && !rot_first) rotate();
  for (int e = threadIdx.x; e < nr * G * vhalf; e += NT) {   // rotated values
    const int rg = qdiv(e, inv_vhalf), i = e - rg * vhalf, rr = R == 1 ? 0 : qdiv(rg, inv_g);
    float* base = vv + rr * C + (rg - rr * G) * dv;
    const float cs = ct[rr * nang + half + i], sn = snt[rr * nang + half + i];
    const float u = base[i], v = base[i + vhalf];
    base[i] = u * cs - v * sn;
    base[i + vhalf] = v * cs + u * sn;
  }
  if (a.v_unit) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int rg = wave; rg < nr * G; rg += NT / 64) {
      const int rr = R == 1 ? 0 : qdiv(rg, inv_g);
      float* base = vv + rr * C + (rg - rr * G) * dv;
      float ss = 0.f;
      for (int c = lane; c < dv; c += 64) ss += base[c] * base[c];
      ss = wave_sum(ss);
      const float rs = 1.0f / sqrtf(ss / (float)dv + a.eps);
      for (int c = lane; c < dv; c += 64) base[c] *= rs;
    }
  }
  __syncthreads();
  for (int rr = 0; rr < nr; ++rr) {
    const int64_t t = t0 + rr;
    const int64_t row = crow[rr];
    const float* q = qv + rr * C;
    if (wide) {
      bf16_t* qo = reinterpret_cast<bf16_t*>(a.q_out) + t * nq;
      bf16_t* cb = reinterpret_cast<bf16_t*>(a.cache);
      for (int c8 = threadIdx.x; c8 < C / 8; c8 += NT) {
        const int c = 8 * c8;
        const uint4 w = pack8(q + c);
        if (c < nq) {
          *reinterpret_cast<uint4*>(qo + c) = w;
        } else if (row >= 0) {
          const int k = c - nq;
          const int g = k < nk ? qdiv(k, inv_d) : qdiv(k - nk, inv_dv);
          const int e = k < nk ? k - g * d : d + (k - nk) - g * dv;
          *reinterpret_cast<uint4*>(cb + (row + (int64_t)g * a.block_size) * (d + dv) + e) = w;
        }
      }
      continue;
    }
    for (int c = threadIdx.x; c < nq; c += NT) stv(a.q_out, t * nq + c, f32, q[c]);
    if (row < 0) continue;
    for (int k = threadIdx.x; k < nk + nv; k += NT) {
      const int g = k < nk ? qdiv(k, inv_d) : qdiv(k - nk, inv_dv);
      const int e = k < nk ? k - g * d : d + (k - nk) - g * dv;
      stv(a.cache, (row + (int64_t)g * a.block_size) * (d + dv) + e, f32, q[nq + k]);
    }
  }
}

bool rows_ok(const RaggedRows& r) { return r.positions != nullptr && r.state_slots != nullptr && r.num_seqs >= 0; }

}  // namespace

hipError_t launch_embed_hash(float* streams, int S, int W, const void* embed, const void* bigram, bool f32,
                             const int64_t* ids, RaggedRows r, int64_t* prev_tok, float scale, int64_t buckets,
                             int64_t mul_prev, int64_t mul_cur, hipStream_t s) {
  if (r.total_rows == 0) return hipSuccess;
  if (S < 1 || W < 1 || (bigram != nullptr && (buckets < 1 || prev_tok == nullptr || !rows_ok(r))))
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(embed_hash_kernel, dim3(r.total_rows), dim3(NT), 0, s, streams, S, W, embed, bigram, f32, ids, r,
                     prev_tok, scale, buckets, mul_prev, mul_cur);
  return hipGetLastError();
}

hipError_t launch_store_last_token(int64_t* prev_tok, const int64_t* ids, RaggedRows r, hipStream_t s) {
  if (r.num_seqs == 0 || r.cu_q == nullptr) return hipSuccess;  // one row per sequence: embed_hash stored it
  if (!rows_ok(r)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(store_last_token_kernel, dim3((r.num_seqs + 63) / 64), dim3(64), 0, s, prev_tok, ids, r);
  return hipGetLastError();
}

hipError_t launch_stream_mix_norm(const StreamMixArgs& a, hipStream_t s) {
  if (a.T == 0) return hipSuccess;
  if (a.S < 1 || a.S > SMAX || a.W < 1 || (a.h != nullptr && a.gain == nullptr)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(stream_mix_norm_kernel, dim3(a.T), dim3(NT), 0, s, a);
  return hipGetLastError();
}

hipError_t launch_poly_norm_act(void* out, const void* z, int64_t zstride, bool f32, const float* coef, float eps,
                                int rows, int n, hipStream_t s) {
  if (rows == 0) return hipSuccess;
  if (n < 1) return hipErrorInvalidValue;
  hipLaunchKernelGGL(poly_norm_act_kernel, dim3(rows), dim3(NT), 0, s, out, z, zstride, f32, coef, eps, n);
  return hipGetLastError();
}

static bool delta_ok(const DeltaShape& sh) {
  return sh.heads >= 1 && sh.kv_heads >= 1 && sh.heads % sh.kv_heads == 0 && sh.dim >= 1 && sh.dim <= 256 &&
         sh.vdim >= 1 && sh.vdim <= 256 && sh.taps >= 1 && sh.taps <= TAPS_MAX;
}

hipError_t launch_delta_prep(float* qkv32, float* bg, const void* x, const void* b, const void* a, int64_t xstride,
                             bool f32, const float* conv_w, const float* conv_wt, float* conv_state,
                             const float* A_log, const float* dt_bias, DeltaShape sh, RaggedRows r, hipStream_t s) {
  if (r.total_rows == 0) return hipSuccess;
  if (!delta_ok(sh) || !rows_ok(r)) return hipErrorInvalidValue;
  const int R = conv_tile(r, sh.channels());
  const size_t lds = sizeof(float) * R * sh.channels();
  if (lds > 150 * 1024) return hipErrorInvalidValue;
  auto* fn = R == 4 ? delta_prep_kernel<4> : (R == 2 ? delta_prep_kernel<2> : delta_prep_kernel<1>);
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(fn, dim3((r.total_rows + R - 1) / R), dim3(NT), lds, s, qkv32, bg, x, b, a, xstride, f32, conv_w,
                     conv_wt, conv_state, A_log, dt_bias, sh, r);
  return hipGetLastError();
}

hipError_t launch_conv_state_update(float* conv_state, const void* x, int64_t xstride, bool f32, DeltaShape sh,
                                    RaggedRows r, hipStream_t s) {
  if (r.num_seqs == 0 || sh.taps <= 1 || r.cu_q == nullptr) return hipSuccess;  // one row each: delta_prep did it
  if (!delta_ok(sh) || !rows_ok(r)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(conv_state_update_kernel, dim3((sh.channels() + NT - 1) / NT, r.num_seqs), dim3(NT), 0, s,
                     conv_state, x, xstride, f32, sh, r);
  return hipGetLastError();
}

template <int LN, int M, int NE, bool F32, bool CD, bool VEC> static hipError_t launch_ne(const GatedDeltaArgs& a, RaggedRows r, hipStream_t s) {
  const int groups = (a.sh.vdim + 3) / 4;
  const int nthr = (LN * groups + 63) / 64 * 64;
  // tokens per trip: what NE float4s of q and k per thread can hold
  int tt = NE * nthr / (LN * M);
  tt = tt > TB ? TB : tt;
  const size_t lds = sizeof(float) * (TB * ((CD ? 3 : 2) * 4 * LN * M + 2 * 4 * groups) + 2 * TB);
  auto* fn = gated_delta_kernel<LN, M, NE, F32, CD, VEC>;
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(fn, dim3(a.sh.heads, r.num_seqs), dim3(nthr), lds, s, a, r, tt);
  return hipGetLastError();
}
template <int LN, int M, bool F32, bool CD, bool VEC>
static hipError_t launch_gd(const GatedDeltaArgs& a, RaggedRows r, hipStream_t s) {
  // one float4 per thread where that holds 8 tokens or more (and, for the larger states, the workgroup has at most 512
  // threads, so that a lane may use 256 registers)
  const int groups = (a.sh.vdim + 3) / 4;
  return groups >= 8 * M && (M <= 2 || LN * groups <= 512) ? launch_ne<LN, M, 1, F32, CD, VEC>(a, r, s)
                                                           : launch_ne<LN, M, 2, F32, CD, VEC>(a, r, s);
}
template <int LN, int M> static hipError_t launch_gd(const GatedDeltaArgs& a, RaggedRows r, hipStream_t s) {
  auto a16 = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool vec = a.sh.dim % 4 == 0 && a.sh.vdim % 4 == 0 && a16(a.qkv32) && a16(a.state) && a16(a.z_bias) &&
                   (a.z == nullptr || (a.zstride % 4 == 0 && a16(a.z)));
  if (a.f32) {
    if (a.z != nullptr)
      return vec ? launch_gd<LN, M, true, true, true>(a, r, s) : launch_gd<LN, M, true, true, false>(a, r, s);
    return vec ? launch_gd<LN, M, true, false, true>(a, r, s) : launch_gd<LN, M, true, false, false>(a, r, s);
  }
  if (a.z != nullptr)
    return vec ? launch_gd<LN, M, false, true, true>(a, r, s) : launch_gd<LN, M, false, true, false>(a, r, s);
  return vec ? launch_gd<LN, M, false, false, true>(a, r, s) : launch_gd<LN, M, false, false, false>(a, r, s);
}

hipError_t launch_gated_delta(const GatedDeltaArgs& a, RaggedRows r, hipStream_t s) {
  if (r.num_seqs == 0 || r.total_rows == 0) return hipSuccess;
  if (!delta_ok(a.sh) || !rows_ok(r) || (a.z != nullptr && (a.z_bias == nullptr || a.A_log == nullptr)))
    return hipErrorInvalidValue;
  if (a.sh.dim <= 16) return launch_gd<4, 1>(a, r, s);
  if (a.sh.dim <= 32) return launch_gd<8, 1>(a, r, s);
  if (a.sh.dim <= 64) return launch_gd<16, 1>(a, r, s);
  if (a.sh.dim <= 128) return launch_gd<16, 2>(a, r, s);
  if (a.sh.dim <= 192) return launch_gd<16, 3>(a, r, s);
  return launch_gd<16, 4>(a, r, s);
}

hipError_t launch_qkv_prep(const QkvPrepArgs& a, hipStream_t s) {
  if (a.T == 0) return hipSuccess;
  if (a.heads < 1 || a.kv_heads < 1 || a.heads % a.kv_heads != 0 || a.dim < 1 || a.vdim < 1 || a.rot_dims < 0 ||
      a.rot_dims > a.dim || (a.rot_dims & 1) || a.block_size < 1 || (a.rot_dims > 0 && a.inv_freq == nullptr) ||
      ((a.q_norm == nullptr) != (a.k_norm == nullptr)) || (a.v_lambda != nullptr && a.v_first == nullptr) ||
      (a.v == nullptr && (a.vdim != a.dim || a.v_lambda != nullptr)) || (a.head_norm && a.q_norm == nullptr) ||
      (a.q_temp_coef != 0.f && a.q_temp_every < 1))
    return hipErrorInvalidValue;
  if (a.v_inv_freq != nullptr && ((a.vdim & 1) || a.v_unit || a.v == nullptr)) return hipErrorInvalidValue;
  if (a.conv_wt != nullptr && (a.bias != nullptr || a.v == nullptr || a.v_lambda != nullptr || a.taps < 1 ||
                               a.taps > TAPS_MAX || !rows_ok(a.r) || (a.taps > 1 && a.conv_state == nullptr)))
    return hipErrorInvalidValue;
  if (a.bias != nullptr && (a.v == nullptr || a.v_lambda != nullptr)) return hipErrorInvalidValue;
  const size_t C = (size_t)a.heads * a.dim + (size_t)a.kv_heads * (a.dim + a.vdim);   // (150 KB of LDS bound every index below 2^21)
  const bool conv = a.conv_wt != nullptr;
  const int R = conv && (a.q_norm == nullptr || a.head_norm) ? conv_tile(a.r, C) : 1;
  const size_t lds = sizeof(float) * R * (C + a.rot_dims + (a.v_inv_freq != nullptr ? a.vdim : 0));
  if (lds > 150 * 1024) return hipErrorInvalidValue;
  auto* fn = !conv ? qkv_prep_kernel<1, false>
                   : (R == 4 ? qkv_prep_kernel<4, true> : (R == 2 ? qkv_prep_kernel<2, true> : qkv_prep_kernel<1, true>));
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(fn, dim3((a.T + R - 1) / R), dim3(NT), lds, s, a);
  return hipGetLastError();
}

}  // namespace die
