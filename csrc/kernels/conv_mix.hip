// Kernels for layers whose sublayers read a convolved input (gfx950). Storage of activations is bf16 or fp32, arithmetic
// is fp32; the residual, the norms and the convolution's rows and state are fp32 in both modes.
//
//   conv_norm        residual sum, RMS norm and the causal convolution over the normed rows, one launch (any of the three
//                    may be absent)
//   rot_head_gate    attention output turned back by the query's position, sigmoid gate per head, scale
#include "common.h"
#include "conv_launchers.h"
#include "lane_reduce.h"

namespace die {

namespace {

constexpr int NT = 256;
constexpr int TAPS_MAX = 16;
constexpr int CONV_RB = 4;   // rows per step of a prompt-sized conv_norm

__device__ __forceinline__ float ldv(const void* p, int64_t i, bool f32) {
  return f32 ? reinterpret_cast<const float*>(p)[i] : bf2f(reinterpret_cast<const bf16_t*>(p)[i]);
}
__device__ __forceinline__ void stv(void* p, int64_t i, bool f32, float v) {
  if (f32)
    reinterpret_cast<float*>(p)[i] = v;
  else
    reinterpret_cast<bf16_t*>(p)[i] = f2bf(v);
}
// VEC (1 or 4) consecutive values
template <int VEC> struct Vals {
  float v[VEC];
};
template <int VEC> __device__ __forceinline__ Vals<VEC> ldf(const float* p) {
  Vals<VEC> r;
  if constexpr (VEC == 4) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    r.v[0] = x.x, r.v[1] = x.y, r.v[2] = x.z, r.v[3] = x.w;
  } else {
    r.v[0] = p[0];
  }
  return r;
}
template <int VEC> __device__ __forceinline__ void stf(float* p, const Vals<VEC>& r) {
  if constexpr (VEC == 4)
    *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else
    p[0] = r.v[0];
}
template <int VEC, bool F32> __device__ __forceinline__ Vals<VEC> lda(const void* p, int64_t i) {
  if constexpr (F32) return ldf<VEC>(reinterpret_cast<const float*>(p) + i);
  Vals<VEC> r;
  const bf16_t* q = reinterpret_cast<const bf16_t*>(p) + i;
  if constexpr (VEC == 4) {
    const uint2 w = *reinterpret_cast<const uint2*>(q);
    r.v[0] = __uint_as_float(w.x << 16), r.v[1] = __uint_as_float(w.x & 0xffff0000u);
    r.v[2] = __uint_as_float(w.y << 16), r.v[3] = __uint_as_float(w.y & 0xffff0000u);
  } else {
    r.v[0] = bf2f(q[0]);
  }
  return r;
}
// the sublayer's output: one row piece, or the sum of its partial sums
template <int VEC, bool F32> __device__ __forceinline__ Vals<VEC> ldy(const ConvNormArgs& a, int64_t i) {
  Vals<VEC> r = lda<VEC, F32>(a.y, i);
  if constexpr (F32) {
    for (int s = 1; s < a.yslabs; ++s) {
      const Vals<VEC> p = lda<VEC, F32>(a.y, i + s * a.yslab);
#pragma unroll
      for (int e = 0; e < VEC; ++e) r.v[e] += p.v[e];
    }
  }
  return r;
}
template <int VEC> __device__ __forceinline__ void sta(void* p, int64_t i, bool f32, const Vals<VEC>& r) {
  if (f32) {
    stf<VEC>(reinterpret_cast<float*>(p) + i, r);
    return;
  }
  bf16_t* q = reinterpret_cast<bf16_t*>(p) + i;
  if constexpr (VEC == 4) {
    uint2 w;
    w.x = pack2(r.v[0], r.v[1]);
    w.y = pack2(r.v[2], r.v[3]);
    *reinterpret_cast<uint2*>(q) = w;
  } else {
    q[0] = f2bf(r.v[0]);
  }
}

// The general form (any width, alignment and number of taps). One workgroup per (sequence, tile of R rows). It walks its
// rows in order and keeps the last taps - 1 normed rows in an LDS ring (row i in slot i mod (taps - 1)); a column belongs to
// one thread from load to store, so the ring needs no barrier. A tile that does not start its sequence first recomputes the taps - 1 rows in front of it from resid_in and
// y (which is why the residual is not updated in place then). The first tile alone reads the sequence's convolution
// state; it also writes it, at its end, after recomputing the step's last rows where they are not its own. The next
// row's loads are issued before the current row's reduction.
template <int TR, int VEC, bool YF32>
__global__ void __launch_bounds__(NT) conv_norm_kernel(ConvNormArgs a, RaggedRows r, int R, int tiles) {
  extern __shared__ __attribute__((aligned(16))) float ring[];   // [taps - 1][W]
  __shared__ float red[NT / 64];
  const int s = blockIdx.x / tiles, tile = blockIdx.x % tiles, tid = threadIdx.x;
  const int W = a.W, H = a.conv_wt != nullptr ? a.taps - 1 : 0;   // H: rows of history
  const int q0 = r.cu_q ? r.cu_q[s] : s;
  const int L = r.cu_q ? r.cu_q[s + 1] - q0 : 1;
  const int i0 = tile * R;
  if (i0 >= L) return;
  const int i1 = min(i0 + R, L);
  const int hs = max(0, i0 - H);
  // rows visited: hs .. i1 - 1, then (first tile of a longer step) the step's last H rows for the state
  const bool keeper = tile == 0 && H > 0;
  const int n1 = i1 - hs, n2 = keeper && L > i1 ? min(H, L) : 0;
  const int64_t p0 = H > 0 ? r.positions[q0] : 0;
  float* st = H > 0 ? a.conv_state + (int64_t)r.state_slots[s] * H * W : nullptr;

  Vals<VEC> x[TR], nx[TR], ny[TR];
  auto row_of = [&](int n) { return n < n1 ? hs + n : L - n2 + (n - n1); };
  auto load = [&](int n) {
    const int64_t row = q0 + row_of(n);
#pragma unroll
    for (int t = 0; t < TR; ++t) {
      const int c = VEC * (t * NT + tid);
      if (c < W) {
        if (a.resid_in != nullptr) {
          nx[t] = ldf<VEC>(a.resid_in + row * W + c);
        } else {
#pragma unroll
          for (int e = 0; e < VEC; ++e) nx[t].v[e] = 0.f;
        }
        if (a.y != nullptr) ny[t] = ldy<VEC, YF32>(a, row * a.ystride + c);
      }
    }
  };
  load(0);
  for (int n = 0; n < n1 + n2; ++n) {
    const int i = row_of(n);
    const bool own = n < n1 && i >= i0;
    const int64_t row = q0 + i;
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < TR; ++t) {
      const int c = VEC * (t * NT + tid);
      if (c < W) {
        x[t] = nx[t];
        if (a.y != nullptr) {
#pragma unroll
          for (int e = 0; e < VEC; ++e) x[t].v[e] += ny[t].v[e];
          if (own && a.resid_out != nullptr) stf<VEC>(a.resid_out + row * W + c, x[t]);
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss += x[t].v[e] * x[t].v[e];
      }
    }
    if (n + 1 < n1 + n2) load(n + 1);
    float rs = 1.0f;
    if (a.w != nullptr) {
      ss = block_sum<NT>(ss, red);
      rs = 1.0f / sqrtf(ss / (float)W + a.eps);
    }
    const int64_t p = p0 + i;
#pragma unroll
    for (int t = 0; t < TR; ++t) {
      const int c = VEC * (t * NT + tid);
      if (c >= W) continue;
      if (a.w != nullptr) {
        const Vals<VEC> w = ldf<VEC>(a.w + c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[t].v[e] *= rs * w.v[e];
      }
      if (own) {
        Vals<VEC> o = x[t];
        if (a.conv_wt != nullptr) {
          const Vals<VEC> wc = ldf<VEC>(a.conv_wt + (int64_t)H * W + c);
#pragma unroll
          for (int e = 0; e < VEC; ++e) o.v[e] += wc.v[e] * x[t].v[e];
          for (int b = 1; b <= H; ++b) {   // b rows back
            if (p - b < 0) break;
            const int src = i - b;
            const Vals<VEC> past = src >= 0 ? ldf<VEC>(ring + (src % H) * W + c) : ldf<VEC>(st + (int64_t)(H + src) * W + c);
            const Vals<VEC> wb = ldf<VEC>(a.conv_wt + (int64_t)(H - b) * W + c);
#pragma unroll
            for (int e = 0; e < VEC; ++e) o.v[e] += wb.v[e] * past.v[e];
          }
        }
        sta<VEC>(a.h, row * a.hstride + c, a.h_f32, o);
      }
      if (H > 0) stf<VEC>(ring + (i % H) * W + c, x[t]);
    }
  }
  if (!keeper) return;
#pragma unroll
  for (int t = 0; t < TR; ++t) {
    const int c = VEC * (t * NT + tid);
    if (c >= W) continue;
    for (int k = 0; k < H; ++k) {
      const int i = L - H + k;   // the row that lands in place k; before the step: from the old state, rows ahead of k
      Vals<VEC> v;
#pragma unroll
      for (int e = 0; e < VEC; ++e) v.v[e] = 0.f;
      if (i >= 0)
        v = ldf<VEC>(ring + (i % H) * W + c);
      else if (p0 + i >= 0)
        v = ldf<VEC>(st + (int64_t)(H + i) * W + c);
      stf<VEC>(st + (int64_t)k * W + c, v);
    }
  }
}

template <int TR, int VEC> hipError_t launch_cn(const ConvNormArgs& a, RaggedRows r, int R, int tiles, hipStream_t s) {
  const size_t lds = sizeof(float) * (size_t)(a.conv_wt != nullptr ? a.taps - 1 : 0) * a.W;
  if (lds > 150 * 1024) return hipErrorInvalidValue;
  auto* fn = a.y_f32 ? conv_norm_kernel<TR, VEC, true> : conv_norm_kernel<TR, VEC, false>;
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(fn, dim3((unsigned)((int64_t)tiles * r.num_seqs)), dim3(NT), lds, s, a, r, R, tiles);
  return hipGetLastError();
}

// Up to 4 taps, widths of a multiple of 4 up to 8 NT: the same walk with everything a column needs in registers — its
// norm and convolution weights, the H = taps - 1 normed rows behind the current one (from the sequence's state at its
// first tile) — and RB rows per step, whose loads are in flight during the step before and whose sums of squares share
// one barrier.
template <int NTH, int TR, int H, int RB, bool YF32>
__global__ void __launch_bounds__(NTH) conv_norm_reg_kernel(ConvNormArgs a, RaggedRows r, int R, int tiles) {
  constexpr int NW = NTH / 64;
  __shared__ float red[2][RB][NW];
  const int s = blockIdx.x / tiles, tile = blockIdx.x % tiles, tid = threadIdx.x;
  const int W = a.W;
  const int q0 = r.cu_q ? r.cu_q[s] : s;
  const int L = r.cu_q ? r.cu_q[s + 1] - q0 : 1;
  const int i0 = tile * R;
  if (i0 >= L) return;
  const int i1 = min(i0 + R, L);
  const int hs = max(0, i0 - H);
  // rows visited: hs .. i1 - 1, then (first tile of a longer step) the step's last H rows for the state
  const bool keeper = tile == 0 && H > 0;
  const int n1 = i1 - hs, n2 = keeper && L > i1 ? min(H, L) : 0, nn = n1 + n2;
  const bool has_y = a.y != nullptr;
  auto row_of = [&](int n) { return n < n1 ? hs + n : L - n2 + (n - n1); };

  Vals<4> nx[RB][TR], ny[RB][TR];
  auto load = [&](int n) {
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      const int64_t row = q0 + row_of(min(n + b, nn - 1));   // beyond the last row: loaded and not used
#pragma unroll
      for (int t = 0; t < TR; ++t) {
        const int c = min(4 * (t * NTH + tid), W - 4);
        if (a.resid_in != nullptr)
          nx[b][t] = ldf<4>(a.resid_in + row * W + c);
        else
          nx[b][t].v[0] = nx[b][t].v[1] = nx[b][t].v[2] = nx[b][t].v[3] = 0.f;
        if (has_y) ny[b][t] = ldy<4, YF32>(a, row * a.ystride + c);
      }
    }
  };
  load(0);
  Vals<4> w[TR], cw[H + 1][TR], past[H > 0 ? H : 1][TR];   // past[b]: b + 1 rows back
  const bool conv = a.conv_wt != nullptr;
  const int64_t p0 = H > 0 ? r.positions[q0] : 0;
  float* st = H > 0 ? a.conv_state + (int64_t)r.state_slots[s] * H * W : nullptr;
#pragma unroll
  for (int t = 0; t < TR; ++t) {
    const int c = min(4 * (t * NTH + tid), W - 4);
    if (a.w != nullptr)
      w[t] = ldf<4>(a.w + c);
    else
      w[t].v[0] = w[t].v[1] = w[t].v[2] = w[t].v[3] = 1.0f;
#pragma unroll
    for (int b = 0; b <= H; ++b) {   // cw[b]: weights of the row b back
      if (conv) cw[b][t] = ldf<4>(a.conv_wt + (int64_t)(H - b) * W + c);
    }
#pragma unroll
    for (int b = 0; b < H; ++b) {
      past[b][t] = ldf<4>(st + (int64_t)(H - 1 - b) * W + c);
      if (tile > 0 || p0 - (b + 1) < 0) {   // before the sequence's start; later tiles visit these rows first
#pragma unroll
        for (int e = 0; e < 4; ++e) past[b][t].v[e] = 0.f;
      }
    }
  }
  int buf = 0;
  for (int n = 0; n < nn; n += RB, buf ^= 1) {
    Vals<4> x[RB][TR];
    float ss[RB];
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      const int i = row_of(min(n + b, nn - 1));
      const bool own = n + b < n1 && i >= i0;
      ss[b] = 0.f;
#pragma unroll
      for (int t = 0; t < TR; ++t) {
        const int c = 4 * (t * NTH + tid);
        x[b][t] = nx[b][t];
        if (has_y) {
#pragma unroll
          for (int e = 0; e < 4; ++e) x[b][t].v[e] += ny[b][t].v[e];
          if (own && c < W && a.resid_out != nullptr) stf<4>(a.resid_out + (int64_t)(q0 + i) * W + c, x[b][t]);
        }
        if (c < W) {
#pragma unroll
          for (int e = 0; e < 4; ++e) ss[b] += x[b][t].v[e] * x[b][t].v[e];
        }
      }
    }
    if (n + RB < nn) load(n + RB);
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      float v = group_sum<16>(ss[b]);
      v += __shfl_xor(v, 16, 64);
      v = xor32_sum(v);
      if ((tid & 63) == 0) red[buf][b][tid >> 6] = v;
    }
    __syncthreads();   // (the other buffer is written next, so one barrier per step is enough)
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      if (n + b >= nn) break;
      const int i = row_of(n + b);
      const bool own = n + b < n1 && i >= i0;
      float tot = 0.f;
#pragma unroll
      for (int k = 0; k < NW; ++k) tot += red[buf][b][k];
      const float rs = a.w != nullptr ? 1.0f / sqrtf(tot / (float)W + a.eps) : 1.0f;
#pragma unroll
      for (int t = 0; t < TR; ++t) {
        const int c = 4 * (t * NTH + tid);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[b][t].v[e] *= rs * w[t].v[e];
        if (own && c < W) {
          Vals<4> o = x[b][t];
          if (conv) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              o.v[e] += cw[0][t].v[e] * x[b][t].v[e];
#pragma unroll
              for (int k = 0; k < H; ++k) o.v[e] += cw[k + 1][t].v[e] * past[k][t].v[e];
            }
          }
          sta<4>(a.h, (int64_t)(q0 + i) * a.hstride + c, a.h_f32, o);
        }
#pragma unroll
        for (int k = H - 1; k > 0; --k) past[k][t] = past[k - 1][t];
        if (H > 0) past[0][t] = x[b][t];
      }
    }
  }
  if (!keeper) return;
#pragma unroll
  for (int t = 0; t < TR; ++t) {
    const int c = 4 * (t * NTH + tid);
    if (c >= W) continue;
#pragma unroll
    for (int k = 0; k < H; ++k) stf<4>(st + (int64_t)k * W + c, past[H - 1 - k][t]);
  }
}

template <int NTH, int TR, int H, int RB> hipError_t launch_cr(const ConvNormArgs& a, RaggedRows r, int R, int tiles, hipStream_t s) {
  auto* fn = a.y_f32 ? conv_norm_reg_kernel<NTH, TR, H, RB, true> : conv_norm_reg_kernel<NTH, TR, H, RB, false>;
  hipLaunchKernelGGL(fn, dim3((unsigned)((int64_t)tiles * r.num_seqs)), dim3(NTH), 0, s, a, r, R, tiles);
  return hipGetLastError();
}
template <int H, int RB> hipError_t launch_cr(const ConvNormArgs& a, RaggedRows r, int R, int tiles, hipStream_t s) {
  if (a.W <= 1024) return launch_cr<256, 1, H, RB>(a, r, R, tiles, s);
  if (a.W <= 2048) return launch_cr<512, 1, H, RB>(a, r, R, tiles, s);
  if (a.W <= 4096) return launch_cr<1024, 1, H, RB>(a, r, R, tiles, s);
  return launch_cr<1024, 2, H, RB>(a, r, R, tiles, s);
}
template <int RB> hipError_t launch_cr(const ConvNormArgs& a, RaggedRows r, int R, int tiles, hipStream_t s) {
  switch (a.conv_wt != nullptr ? a.taps : 1) {
    case 1: return launch_cr<0, RB>(a, r, R, tiles, s);
    case 2: return launch_cr<1, RB>(a, r, R, tiles, s);
    case 3: return launch_cr<2, RB>(a, r, R, tiles, s);
    default: return launch_cr<3, RB>(a, r, R, tiles, s);
  }
}

// One workgroup per token: the token's gates and rotation angles once in LDS, then 4 + 4 (or 1 + 1) output columns of a
// pair of halves per thread and trip.
__global__ void __launch_bounds__(NT) rot_head_gate_kernel(RotHeadGateArgs a, bool vec) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int64_t t = blockIdx.x;
  const int H = a.heads, V = a.vdim, half = V / 2;
  const bool f32 = a.f32;
  float* ct = sm;                                        // [half] cos, [half] sin
  float* snt = ct + (a.inv_freq != nullptr ? half : 0);
  float* gates = snt + (a.inv_freq != nullptr ? half : 0);   // [H]
  for (int h = threadIdx.x; h < H; h += NT) gates[h] = a.mult / (1.0f + expf(-ldv(a.g, t * a.gstride + h, f32)));
  if (a.inv_freq != nullptr) {
    const float p = (float)a.positions[t];
    for (int i = threadIdx.x; i < half; i += NT) {
      float sn, cs;
      sincosf(p * a.inv_freq[i], &sn, &cs);
      ct[i] = cs;
      snt[i] = sn;
    }
  }
  __syncthreads();
  const int64_t ob = t * H * V, wb = t * a.ostride;
  if (a.inv_freq == nullptr) {
    if (vec) {
      for (int e = 4 * threadIdx.x; e < H * V; e += 4 * NT) {
        Vals<4> u = f32 ? lda<4, true>(a.o, ob + e) : lda<4, false>(a.o, ob + e);
        const float gt = gates[e / V];
#pragma unroll
        for (int q = 0; q < 4; ++q) u.v[q] *= gt;
        sta<4>(a.out, wb + e, f32, u);
      }
    } else {
      for (int e = threadIdx.x; e < H * V; e += NT) stv(a.out, wb + e, f32, ldv(a.o, ob + e, f32) * gates[e / V]);
    }
    return;
  }
  if (vec) {
    const int q4 = half / 4;
    for (int e = threadIdx.x; e < H * q4; e += NT) {
      const int h = e / q4, i = 4 * (e % q4), c = h * V + i;
      const Vals<4> u = f32 ? lda<4, true>(a.o, ob + c) : lda<4, false>(a.o, ob + c);
      const Vals<4> v = f32 ? lda<4, true>(a.o, ob + c + half) : lda<4, false>(a.o, ob + c + half);
      const float gt = gates[h];
      Vals<4> x, y;
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const float cs = ct[i + q], sn = snt[i + q];
        x.v[q] = (u.v[q] * cs + v.v[q] * sn) * gt;
        y.v[q] = (v.v[q] * cs - u.v[q] * sn) * gt;
      }
      sta<4>(a.out, wb + c, f32, x);
      sta<4>(a.out, wb + c + half, f32, y);
    }
    return;
  }
  for (int e = threadIdx.x; e < H * half; e += NT) {
    const int h = e / half, i = e % half, c = h * V + i;
    const float u = ldv(a.o, ob + c, f32), v = ldv(a.o, ob + c + half, f32), gt = gates[h];
    stv(a.out, wb + c, f32, (u * ct[i] + v * snt[i]) * gt);
    stv(a.out, wb + c + half, f32, (v * ct[i] - u * snt[i]) * gt);
  }
}

bool a16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace

hipError_t launch_conv_norm(const ConvNormArgs& a, RaggedRows r0, hipStream_t s) {
  RaggedRows r = r0;
  if (r.total_rows == 0 || r.num_seqs == 0) return hipSuccess;
  const bool conv = a.conv_wt != nullptr;
  if (a.W < 1 || a.h == nullptr || a.hstride < a.W || (a.y == nullptr && a.resid_in == nullptr) ||
      (conv && (a.w == nullptr || a.resid_in == nullptr || (a.y != nullptr && a.resid_out == nullptr))) ||
      (a.y != nullptr && (a.yslabs < 1 || (a.yslabs > 1 && !a.y_f32))))
    return hipErrorInvalidValue;
  if (conv && (a.taps < 1 || a.taps > TAPS_MAX || r.positions == nullptr || r.state_slots == nullptr || a.max_q < 1 ||
               (a.taps > 1 && a.conv_state == nullptr)))
    return hipErrorInvalidValue;
  int R = 1, tiles = 1;
  if (!conv) {   // rows are independent
    r.cu_q = nullptr;
    r.num_seqs = r.total_rows;
  } else if (r.cu_q != nullptr) {
    // rows per workgroup: about four workgroups per CU, at most 32 visited rows; at least the history, and together with
    // it (a tile visits both) a multiple of the rows per step
    const int H = a.taps - 1;
    R = r.total_rows / (4 * num_cus());
    R = R < 1 ? 1 : (R > 32 - H ? 32 - H : R);
    if (R < H) R = H;
    R = (R + H + CONV_RB - 1) / CONV_RB * CONV_RB - H;
    tiles = (a.max_q + R - 1) / R;
    if (a.y != nullptr && tiles > 1 && a.resid_out == a.resid_in) return hipErrorInvalidValue;
  }
  if ((int64_t)tiles * r.num_seqs > 0x7fffffff) return hipErrorInvalidValue;
  const bool vec = a.W % 4 == 0 && a.hstride % 4 == 0 && a16(a.resid_in) && a16(a.w) && a16(a.h) && (!conv || (a16(a.conv_wt) && a16(a.conv_state))) &&
                   (a.y == nullptr || (a16(a.resid_out) && a16(a.y) && a.ystride % 4 == 0 && (a.yslabs == 1 || a.yslab % 4 == 0)));
  if (vec && a.W <= 8192 && (!conv || a.taps <= 4))
    return r.cu_q != nullptr ? launch_cr<CONV_RB>(a, r, R, tiles, s) : launch_cr<1>(a, r, R, tiles, s);
  if (vec) {
    if (a.W <= 4 * NT) return launch_cn<1, 4>(a, r, R, tiles, s);
    if (a.W <= 8 * NT) return launch_cn<2, 4>(a, r, R, tiles, s);
    if (a.W <= 16 * NT) return launch_cn<4, 4>(a, r, R, tiles, s);
    if (a.W <= 32 * NT) return launch_cn<8, 4>(a, r, R, tiles, s);
    return a.W <= 64 * NT ? launch_cn<16, 4>(a, r, R, tiles, s) : hipErrorInvalidValue;
  }
  if (a.W <= 4 * NT) return launch_cn<4, 1>(a, r, R, tiles, s);
  if (a.W <= 16 * NT) return launch_cn<16, 1>(a, r, R, tiles, s);
  return a.W <= 64 * NT ? launch_cn<64, 1>(a, r, R, tiles, s) : hipErrorInvalidValue;
}

hipError_t launch_rot_head_gate(const RotHeadGateArgs& a, hipStream_t s) {
  if (a.T == 0) return hipSuccess;
  if (a.heads < 1 || a.vdim < 1 || (a.inv_freq != nullptr && ((a.vdim & 1) || a.positions == nullptr)))
    return hipErrorInvalidValue;
  const int unit = a.inv_freq != nullptr ? a.vdim / 2 : a.vdim;
  const bool vec = unit % 4 == 0 && a.ostride % 4 == 0 && a16(a.o) && a16(a.out);
  const size_t lds = sizeof(float) * ((size_t)a.heads + (a.inv_freq != nullptr ? a.vdim : 0));
  if (lds > 48 * 1024) return hipErrorInvalidValue;
  hipLaunchKernelGGL(rot_head_gate_kernel, dim3(a.T), dim3(NT), lds, s, a, vec);
  return hipGetLastError();
}

}  // namespace die
