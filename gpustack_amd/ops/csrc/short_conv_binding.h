// Torch binding of the short convolution (short_conv.hip), shared by the
// libraries that carry it. Every shape the kernels or their grids assume is
// checked here on the host; values inside index tensors are bounded in the
// kernels. Uses the including file's chk / act_kind / view_kind / seq_view.
#pragma once

void short_conv_launch(void*, const void*, long, int, int, int, const float*, const float*, void*, const int*, const int*, const int*, const int*, const int*, int, int, int, int, int, int, hipStream_t);
int conv_max_taps();

namespace {

void short_conv(Tensor out, Tensor src, long col0, Tensor w, OptTensor b,
                OptTensor conv_state, Tensor seq_first, Tensor seq_rows,
                Tensor state_slots, Tensor row_seq, Tensor pos32, bool silu,
                bool single) {
  const int bf = act_kind(out, "out");
  TORCH_CHECK(view_kind(src, "src") == bf, "out and src must share a dtype");
  chk(w, "w", at::kFloat);
  chk(row_seq, "row_seq", at::kInt);
  TORCH_CHECK(out.dim() == 2 && w.dim() == 2);
  const int T = out.size(0), C = out.size(1), taps = w.size(1);
  TORCH_CHECK(src.size(0) == T && col0 >= 0 && col0 + C <= src.size(1));
  TORCH_CHECK(w.size(0) == C && taps >= 1 && taps <= conv_max_taps(),
              "weights must be [channels, taps <= 16]");
  const float* bp = nullptr;
  if (b.has_value()) {
    chk(*b, "b", at::kFloat);
    TORCH_CHECK(b->numel() == C);
    bp = b->data_ptr<float>();
  }
  void* sp = nullptr;
  int nslots = 1;
  if (taps > 1) {
    TORCH_CHECK(conv_state.has_value(), "the convolution keeps inputs");
    TORCH_CHECK(act_kind(*conv_state, "conv_state") == bf,
                "out, src and the state must share a dtype");
    TORCH_CHECK(conv_state->dim() == 3 && conv_state->size(1) == taps - 1 &&
                conv_state->size(2) == C && conv_state->size(0) >= 1,
                "state must be [slots, taps - 1, channels]");
    sp = conv_state->data_ptr();
    nslots = conv_state->size(0);
  }
  const int nseq = seq_view(seq_first, seq_rows, state_slots, pos32, T);
  TORCH_CHECK(row_seq.numel() == T);
  TORCH_CHECK(!single || nseq == T, "one row per sequence");
  short_conv_launch(out.data_ptr(), src.data_ptr(), src.stride(0), (int)col0,
                    C, taps, w.data_ptr<float>(), bp, sp,
                    seq_first.data_ptr<int>(), seq_rows.data_ptr<int>(),
                    state_slots.data_ptr<int>(), row_seq.data_ptr<int>(),
                    pos32.data_ptr<int>(), nseq, nslots, T, bf, silu ? 1 : 0,
                    single ? 1 : 0, cur_stream(src));
  HIP_CHECK_LAST();
}

}  // namespace
