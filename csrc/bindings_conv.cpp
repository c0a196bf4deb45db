// Torch bindings of the convolved-input kernels (csrc/kernels/conv_mix.hip); registered into src/_Cmix by
// register_conv_ops(). Shapes, dtypes, devices and index ranges that the host can see are validated here; the launchers
// trust them.
#include <ATen/hip/HIPContext.h>
#include <c10/hip/HIPStream.h>
#include <torch/extension.h>

#include "kernels/conv_launchers.h"

using at::Tensor;
using OptTensor = c10::optional<Tensor>;

namespace {

inline hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define HIP_OK(call)                                                                                   \
  do {                                                                                                  \
    hipError_t e_ = (call);                                                                             \
    TORCH_CHECK(e_ == hipSuccess, "HIP launch failed: ", hipGetErrorString(e_), " (", #call, ")");      \
  } while (0)

bool is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, name, " must be bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}

void check_rows(const Tensor& t, const char* name) {
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1, name, " must be [rows, n] with unit inner stride");
}

void check_c(const Tensor& t, at::ScalarType d, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == d && t.is_contiguous(), name, ": wrong device / dtype / layout");
}

const float* f32_vec(const OptTensor& t, int64_t n, const char* name) {
  if (!t.has_value()) return nullptr;
  check_c(*t, at::kFloat, name);
  TORCH_CHECK(t->numel() == n, name, ": expected ", n, " values, got ", t->numel());
  return t->data_ptr<float>();
}

void conv_norm(Tensor h, OptTensor resid_in, OptTensor resid_out, OptTensor y, OptTensor w, double eps, OptTensor conv_wt,
               OptTensor conv_state, int64_t max_q, OptTensor positions, OptTensor cu_q, OptTensor state_slots) {
  check_rows(h, "h");
  const int64_t T = h.size(0), W = h.size(1);
  TORCH_CHECK(resid_in.has_value() || y.has_value(), "resid_in or y");
  TORCH_CHECK(!conv_wt.has_value() || (w.has_value() && resid_in.has_value()), "a convolution runs over the normed residual");
  die::ConvNormArgs a;
  a.resid_in = nullptr;
  if (resid_in.has_value()) {
    check_c(*resid_in, at::kFloat, "resid_in");
    TORCH_CHECK(resid_in->sizes() == h.sizes(), "resid_in [T, W]");
    a.resid_in = resid_in->data_ptr<float>();
  }
  a.resid_out = nullptr;
  a.y = nullptr;
  a.ystride = 0;
  a.y_f32 = false;
  a.yslabs = 1;
  a.yslab = 0;
  if (y.has_value()) {
    a.y_f32 = is_f32(*y, "y");
    if (y->dim() == 3) {
      TORCH_CHECK(a.y_f32 && y->is_contiguous() && y->size(0) >= 1 && y->size(1) == T && y->size(2) == W,
                  "y as partial sums: fp32 [n, T, W] contiguous");
      a.yslabs = (int)y->size(0);
      a.yslab = T * W;
      a.ystride = W;
    } else {
      check_rows(*y, "y");
      TORCH_CHECK(y->size(0) == T && y->size(1) == W, "y [T, W]");
      a.ystride = y->stride(0);
    }
    TORCH_CHECK(resid_out.has_value() || !conv_wt.has_value(), "y needs resid_out");
    a.y = y->data_ptr();
    if (resid_out.has_value()) {
      check_c(*resid_out, at::kFloat, "resid_out");
      TORCH_CHECK(resid_out->sizes() == h.sizes(), "resid_out [T, W]");
      a.resid_out = resid_out->data_ptr<float>();
    }
  }
  a.w = f32_vec(w, W, "w");
  a.eps = (float)eps;
  a.h_f32 = is_f32(h, "h");
  a.h = h.data_ptr();
  a.hstride = h.stride(0);
  a.W = (int)W;
  a.max_q = (int)max_q;
  a.conv_wt = nullptr;
  a.conv_state = nullptr;
  a.taps = 0;
  die::RaggedRows r{nullptr, nullptr, nullptr, (int)T, (int)T};
  if (conv_wt.has_value()) {
    check_c(*conv_wt, at::kFloat, "conv_wt");
    TORCH_CHECK(conv_wt->dim() == 2 && conv_wt->size(1) == W && conv_wt->size(0) >= 1 && conv_wt->size(0) <= 16,
                "conv_wt [taps, W], taps <= 16");
    a.taps = (int)conv_wt->size(0);
    a.conv_wt = conv_wt->data_ptr<float>();
    TORCH_CHECK(conv_state.has_value() && positions.has_value() && state_slots.has_value(),
                "a convolution needs its state and the step's rows");
    check_c(*conv_state, at::kFloat, "conv_state");
    TORCH_CHECK(conv_state->dim() == 3 && conv_state->size(1) == a.taps - 1 && conv_state->size(2) == W,
                "conv_state [slots, taps - 1, W]");
    a.conv_state = conv_state->data_ptr<float>();
    check_c(*positions, at::kLong, "positions");
    check_c(*state_slots, at::kInt, "state_slots");
    TORCH_CHECK(positions->numel() >= T, "positions [T]");
    r.positions = positions->data_ptr<int64_t>();
    r.state_slots = state_slots->data_ptr<int>();
    if (cu_q.has_value()) {
      check_c(*cu_q, at::kInt, "cu_q");
      TORCH_CHECK(cu_q->numel() >= 2 && max_q >= 1, "cu_q [S + 1], max_q >= 1");
      r.cu_q = cu_q->data_ptr<int>();
      r.num_seqs = (int)cu_q->numel() - 1;
    }
    TORCH_CHECK(state_slots->numel() >= r.num_seqs, "state_slots [S]");
  }
  HIP_OK(die::launch_conv_norm(a, r, cur_stream()));
}

void rot_head_gate(Tensor out, Tensor o, Tensor g, int64_t heads, int64_t vdim, OptTensor positions, OptTensor inv_freq,
                   double mult) {
  die::RotHeadGateArgs a;
  a.f32 = is_f32(o, "o");
  TORCH_CHECK(o.dim() == 2 && o.is_contiguous() && o.size(1) == heads * vdim, "o [T, H * vdim] contiguous");
  const int64_t T = o.size(0);
  check_rows(g, "g");
  check_rows(out, "out");
  TORCH_CHECK(is_f32(g, "g") == a.f32 && is_f32(out, "out") == a.f32 && g.size(0) == T && g.size(1) == heads &&
                  out.sizes() == o.sizes(),
              "g [T, H], out [T, H * vdim], one dtype");
  a.out = out.data_ptr();
  a.ostride = out.stride(0);
  a.o = o.data_ptr();
  a.g = g.data_ptr();
  a.gstride = g.stride(0);
  a.positions = nullptr;
  a.inv_freq = nullptr;
  if (inv_freq.has_value()) {
    TORCH_CHECK(vdim % 2 == 0 && positions.has_value(), "a rotation needs an even vdim and the positions");
    check_c(*positions, at::kLong, "positions");
    TORCH_CHECK(positions->numel() >= T, "positions [T]");
    a.positions = positions->data_ptr<int64_t>();
    a.inv_freq = f32_vec(inv_freq, vdim / 2, "inv_freq");
  }
  a.mult = (float)mult;
  a.T = (int)T;
  a.heads = (int)heads;
  a.vdim = (int)vdim;
  HIP_OK(die::launch_rot_head_gate(a, cur_stream()));
}

}  // namespace

void register_conv_ops(pybind11::module& m) {
  m.def("conv_norm", &conv_norm);
  m.def("rot_head_gate", &rot_head_gate);
}
