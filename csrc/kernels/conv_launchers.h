// Host launchers of the kernels for layers whose sublayers read a convolved input ("Canon" layers): the residual sum,
// the pre-norm and a short causal convolution over the normed rows in one launch, and the epilogue of attention over
// rotated values (the output turned back, a sigmoid gate per head). Raw pointers + an explicit stream, no allocation and
// no synchronisation: every launcher is hipGraph-capturable. `f32` selects the storage type of activations (false:
// bf16); norm and convolution weights, the convolution's state and the residual are always fp32.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

#include "seq_launchers.h"

namespace die {

struct ConvNormArgs {
  const float* resid_in;   // [T, W], or nullptr: zeros (x = y)
  float* resid_out;        // [T, W]: resid_in + y; not written without y, or nullptr: not kept. May equal resid_in only
                           // where no other row reads the row: without a convolution, or with one row per sequence
  const void* y;           // [T, W], row stride ystride, or nullptr
  int64_t ystride;
  bool y_f32;
  int yslabs;              // fp32 y as the sum of this many partial sums, yslab elements apart (else 1)
  int64_t yslab;
  const float* w;          // [W], or nullptr: no norm, n = x (without a convolution)
  float eps;
  const float* conv_wt;    // [taps, W], tap-major, the current row's weights last; nullptr: no convolution
  float* conv_state;       // [slots, taps - 1, W]: the last normed rows before the step, the most recent last
  int taps;
  void* h;                 // [T, W], row stride hstride
  int64_t hstride;
  bool h_f32;
  int W, max_q;            // max_q: most rows of one sequence in this step
};
// x = resid_in + y; n = x / sqrt(mean(x^2) + eps) * w; h[t] = n[t] + sum_j conv_wt[j] * n[t - (taps - 1) + j] over the
// row's own sequence, zeros before its start. conv_state takes the sequence's last taps - 1 rows of n.
hipError_t launch_conv_norm(const ConvNormArgs& a, RaggedRows r, hipStream_t s);

// out[t, h, :] = mult * sigmoid(g[t, h]) * o[t, h, :]; with inv_freq [vdim / 2] every pair (i, i + vdim / 2) of o is first
// turned by -positions[t] * inv_freq[i]. o contiguous; out and g with row strides.
struct RotHeadGateArgs {
  void* out;
  int64_t ostride;
  const void* o;           // [T, H * vdim]
  const void* g;           // [T, H]
  int64_t gstride;
  bool f32;
  const int64_t* positions;
  const float* inv_freq;
  float mult;
  int T, heads, vdim;
};
hipError_t launch_rot_head_gate(const RotHeadGateArgs& a, hipStream_t s);

}  // namespace die
