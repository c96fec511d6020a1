// Torch bindings for the rows of parallel residual streams (hyperrows32.hip),
// the gated recurrence (gru_scan.hip) and the short convolution
// (short_conv.hip). Every shape a kernel or its grid assumes is checked here
// on the host before the launch; VALUES inside index tensors are bounded in
// the kernels.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

void embed_streams_launch(float*, const long*, const void*, int, int, int, long, float, int, hipStream_t);
void stream_step_launch(float*, const void*, const void*, long, const float*, const float*, const float*, const float*, const float*, void*, const float*, void*, void*, const int*, const int*, const int*, int, int, int, int, int, int, float, int, hipStream_t);
void token_shift_launch(void*, const void*, const float*, void*, const int*, const int*, const int*, const int*, const int*, int, int, int, int, int, int, hipStream_t);
void gru_scan_launch(void*, const void*, long, int, int, int, int, const float*, const float*, float*, const int*, const int*, const int*, const int*, const int*, float*, int, int, int, int, int, hipStream_t);
int stream_step_max_streams();
int stream_step_max_width();

#define HIP_CHECK_LAST()                                                     \
  do {                                                                       \
    hipError_t e_ = hipGetLastError();                                       \
    TORCH_CHECK(e_ == hipSuccess, "HIP kernel launch failed: ",              \
                hipGetErrorString(e_));                                      \
  } while (0)

namespace {

using at::Tensor;
using OptTensor = c10::optional<Tensor>;

hipStream_t cur_stream(const Tensor& t) {
  return c10::hip::getCurrentHIPStream(t.device().index()).stream();
}

void chk(const Tensor& t, const char* name, at::ScalarType ty) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.scalar_type() == ty, name, " has the wrong dtype");
  TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
}

// bf16 -> 1, fp32 -> 0
int act_kind(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
  if (t.scalar_type() == at::kBFloat16) return 1;
  TORCH_CHECK(t.scalar_type() == at::kFloat, name, " must be bf16 or fp32");
  return 0;
}

// a [T, C] view whose rows may be strided (a column slice of a projection)
int view_kind(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.dim() == 2 && (t.size(1) == 1 || t.stride(1) == 1) &&
              t.stride(0) >= t.size(1), name, " must be a row-major 2-d view");
  if (t.scalar_type() == at::kBFloat16) return 1;
  TORCH_CHECK(t.scalar_type() == at::kFloat, name, " must be bf16 or fp32");
  return 0;
}

// the per-sequence view: first row, rows, state slot of every sequence
int seq_view(const Tensor& seq_first, const Tensor& seq_rows,
             const Tensor& state_slots, const Tensor& pos32, int T) {
  chk(seq_first, "seq_first", at::kInt);
  chk(seq_rows, "seq_rows", at::kInt);
  chk(state_slots, "state_slots", at::kInt);
  chk(pos32, "pos32", at::kInt);
  const int nseq = seq_first.numel();
  TORCH_CHECK(nseq >= 1 && seq_rows.numel() == nseq &&
              state_slots.numel() == nseq && pos32.numel() == T);
  return nseq;
}

const float* vec(const OptTensor& t, const char* name, long n) {
  TORCH_CHECK(t.has_value(), name, " is missing");
  chk(*t, name, at::kFloat);
  TORCH_CHECK(t->numel() == n, name, " has the wrong size");
  return t->data_ptr<float>();
}

void embed_streams(Tensor x, Tensor tokens, Tensor embed, double scale) {
  chk(x, "x", at::kFloat);
  chk(tokens, "tokens", at::kLong);
  const int bf = act_kind(embed, "embed");
  TORCH_CHECK(x.dim() == 3 && embed.dim() == 2 && embed.size(1) == x.size(2));
  TORCH_CHECK(tokens.numel() == x.size(0) && embed.size(0) >= 1);
  embed_streams_launch(x.data_ptr<float>(), tokens.data_ptr<long>(),
                       embed.data_ptr(), (int)x.size(0), (int)x.size(1),
                       (int)x.size(2), embed.size(0), (float)scale, bf,
                       cur_stream(x));
  HIP_CHECK_LAST();
}

void stream_step(Tensor x, OptTensor a, OptTensor gate, OptTensor gate_b,
                 OptTensor mix, OptTensor out_w, OptTensor in_w,
                 OptTensor norm_w, double eps, OptTensor h, OptTensor hs,
                 OptTensor mu, OptTensor prev, OptTensor row_seq,
                 OptTensor state_slots, OptTensor pos32) {
  chk(x, "x", at::kFloat);
  TORCH_CHECK(x.dim() == 3);
  const int T = x.size(0), S = x.size(1), W = x.size(2);
  TORCH_CHECK(S >= 1 && S <= stream_step_max_streams() && W >= 1 &&
              W <= stream_step_max_width(), "stream sizes unsupported");
  TORCH_CHECK(a.has_value() || in_w.has_value(), "nothing to close or open");
  int bf = -1;
  auto kind = [&](int k) {
    TORCH_CHECK(bf < 0 || bf == k, "operands must share a dtype");
    bf = k;
  };
  const void *ap = nullptr, *gp = nullptr;
  long ld_gate = W;
  const float *gb = nullptr, *mp = nullptr, *op = nullptr, *ip = nullptr,
              *np = nullptr, *mup = nullptr;
  void *hp = nullptr, *hsp = nullptr, *pp = nullptr;
  const int *rs = nullptr, *sl = nullptr, *ps = nullptr;
  int nseq = 1, nslots = 1, M = 1;
  if (a.has_value()) {
    kind(act_kind(*a, "a"));
    TORCH_CHECK(a->dim() == 2 && a->size(0) == T && a->size(1) == W);
    ap = a->data_ptr();
    mp = vec(mix, "mix", (long)S * S);
    op = vec(out_w, "out_w", S);
    if (gate.has_value()) {
      kind(view_kind(*gate, "gate"));
      TORCH_CHECK(gate->size(0) == T && gate->size(1) == W);
      gp = gate->data_ptr();
      ld_gate = gate->stride(0);
      if (gate_b.has_value()) gb = vec(gate_b, "gate_b", W);
    }
  }
  if (in_w.has_value()) {
    ip = vec(in_w, "in_w", S);
    np = vec(norm_w, "norm_w", W);
    TORCH_CHECK(h.has_value());
    kind(act_kind(*h, "h"));
    TORCH_CHECK(h->dim() == 2 && h->size(0) == T && h->size(1) == W);
    hp = h->data_ptr();
    if (hs.has_value()) {
      TORCH_CHECK(prev.has_value() && row_seq.has_value() &&
                  state_slots.has_value() && pos32.has_value());
      kind(act_kind(*hs, "hs"));
      kind(act_kind(*prev, "prev"));
      TORCH_CHECK(mu.has_value() && mu->numel() >= W && mu->numel() % W == 0);
      M = mu->numel() / W;
      TORCH_CHECK(hs->numel() == (long)M * T * W && prev->dim() == 2 &&
                  prev->size(0) >= 1 && prev->size(1) == W);
      chk(*row_seq, "row_seq", at::kInt);
      chk(*state_slots, "state_slots", at::kInt);
      chk(*pos32, "pos32", at::kInt);
      nseq = state_slots->numel();
      TORCH_CHECK(row_seq->numel() == T && pos32->numel() == T && nseq == T,
                  "the shift in this pass takes one row per sequence");
      mup = vec(mu, "mu", (long)M * W);
      hsp = hs->data_ptr();
      pp = prev->data_ptr();
      nslots = prev->size(0);
      rs = row_seq->data_ptr<int>();
      sl = state_slots->data_ptr<int>();
      ps = pos32->data_ptr<int>();
    }
  }
  stream_step_launch(x.data_ptr<float>(), ap, gp, ld_gate, gb, mp, op, ip, np,
                     hp, mup, hsp, pp, rs, sl, ps, nseq, nslots, M, T, S, W,
                     (float)eps, bf, cur_stream(x));
  HIP_CHECK_LAST();
}

void token_shift(Tensor hs, Tensor h, Tensor mu, Tensor prev, Tensor seq_first,
                 Tensor seq_rows, Tensor state_slots, Tensor row_seq,
                 Tensor pos32) {
  const int bf = act_kind(h, "h");
  TORCH_CHECK(act_kind(hs, "hs") == bf && act_kind(prev, "prev") == bf,
              "operands must share a dtype");
  chk(mu, "mu", at::kFloat);
  chk(row_seq, "row_seq", at::kInt);
  TORCH_CHECK(h.dim() == 2 && prev.dim() == 2 && prev.size(1) == h.size(1) &&
              prev.size(0) >= 1);
  TORCH_CHECK(hs.data_ptr() != h.data_ptr(), "hs must not alias h");
  const int T = h.size(0), W = h.size(1);
  TORCH_CHECK(mu.numel() >= W && mu.numel() % W == 0 && row_seq.numel() == T);
  const int M = mu.numel() / W;
  TORCH_CHECK(hs.numel() == (long)M * T * W, "one plane of hs per shift");
  const int nseq = seq_view(seq_first, seq_rows, state_slots, pos32, T);
  token_shift_launch(hs.data_ptr(), h.data_ptr(), mu.data_ptr<float>(),
                     prev.data_ptr(), seq_first.data_ptr<int>(),
                     seq_rows.data_ptr<int>(), state_slots.data_ptr<int>(),
                     row_seq.data_ptr<int>(), pos32.data_ptr<int>(), nseq,
                     (int)prev.size(0), M, T, W, bf, cur_stream(h));
  HIP_CHECK_LAST();
}

void gru_scan(Tensor y, Tensor src, long col_z, long col_u, long col_g,
              Tensor z_b, Tensor u_b, Tensor state, Tensor seq_first,
              Tensor seq_rows, Tensor state_slots, Tensor pos32,
              OptTensor runs) {
  const int bf = act_kind(y, "y");
  TORCH_CHECK(view_kind(src, "src") == bf, "y and src must share a dtype");
  chk(z_b, "z_b", at::kFloat);
  chk(u_b, "u_b", at::kFloat);
  chk(state, "state", at::kFloat);
  TORCH_CHECK(y.dim() == 2 && src.size(0) == y.size(0));
  const int T = y.size(0), N = y.size(1);
  const long W = src.size(1);
  TORCH_CHECK(N >= 1 && z_b.numel() == N && u_b.numel() == N);
  TORCH_CHECK(col_z >= 0 && col_z + N <= W && col_u >= 0 && col_u + N <= W &&
              col_g >= 0 && col_g + N <= W, "columns outside the source");
  TORCH_CHECK(state.dim() >= 2 && state.size(0) >= 1 &&
              state.numel() == state.size(0) * N, "state must be [slots, N]");
  TORCH_CHECK((uintptr_t)src.data_ptr() % 16 == 0, "src must be aligned");
  const int nseq = seq_view(seq_first, seq_rows, state_slots, pos32, T);
  const int* rp = nullptr;
  float* wp = nullptr;
  int nruns = nseq;
  Tensor ws;
  if (runs.has_value()) {
    chk(*runs, "runs", at::kInt);
    TORCH_CHECK(runs->dim() == 2 && runs->size(1) == 4);
    nruns = runs->size(0);
    rp = runs->data_ptr<int>();
    ws = at::empty({(long)nruns, 3L, (long)N},
                   at::TensorOptions().dtype(at::kFloat).device(y.device()));
    wp = ws.data_ptr<float>();
  }
  gru_scan_launch(y.data_ptr(), src.data_ptr(), src.stride(0), (int)col_z,
                  (int)col_u, (int)col_g, N, z_b.data_ptr<float>(),
                  u_b.data_ptr<float>(), state.data_ptr<float>(),
                  seq_first.data_ptr<int>(), seq_rows.data_ptr<int>(),
                  state_slots.data_ptr<int>(), pos32.data_ptr<int>(), rp, wp,
                  nruns, nseq, (int)state.size(0), T, bf, cur_stream(y));
  HIP_CHECK_LAST();
}

}  // namespace

#include "short_conv_binding.h"

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_streams", &embed_streams);
  m.def("stream_step", &stream_step);
  m.def("token_shift", &token_shift);
  m.def("gru_scan", &gru_scan);
  m.def("short_conv", &short_conv);
}
