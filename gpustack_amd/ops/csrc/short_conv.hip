// Short causal convolution per channel over a ragged batch (gfx950), with
// or without a bias and SiLU.
//
//   out[t, c] = act(b[c] + sum_k w[c, k] * in_c(t - (taps - 1 - k)))
//
// Sequence s brings rows seq_first[s] .. seq_first[s] + seq_rows[s] - 1; the
// inputs before them come from the last taps - 1 inputs kept in the
// sequence's state slot, inputs before position 0 are zero. A second launch
// moves the slot on (it must not race with the reads); where every sequence
// brings one row (a decode step), one launch does both, since a lane then
// owns its (slot, channel).
#include "common.h"

namespace {

template <typename T> DEVICE_INLINE float ld(const T* p);
template <> DEVICE_INLINE float ld<float>(const float* p) { return *p; }
template <> DEVICE_INLINE float ld<unsigned short>(const unsigned short* p) {
  return bf2f(*p);
}
template <typename T> DEVICE_INLINE void st(T* p, float v);
template <> DEVICE_INLINE void st<float>(float* p, float v) { *p = v; }
template <> DEVICE_INLINE void st<unsigned short>(unsigned short* p, float v) {
  *p = f2bf(v);
}

constexpr int MAX_TAPS = 16;

struct ConvArgs {
  long ld_src;
  int col0, C, taps, silu;
  const float* w;          // [C, taps]
  const float* b;          // [C] or null
  const int* seq_first;
  const int* seq_rows;
  const int* state_slots;
  const int* row_seq;
  const int* pos32;
  int nseq, nslots, T;
};

DEVICE_INLINE float act(float v, int silu) {
  return silu ? v / (1.0f + expf(-v)) : v;
}

// grid (T, ceil(C / 256)): one lane per (row, channel).
template <typename TS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    TS* __restrict__ out, const TS* __restrict__ src,
    const TS* __restrict__ conv_state, ConvArgs p) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.C) return;
  const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
  const int first = min(max(p.seq_first[s], 0), t);
  const int i = t - first;                   // row index inside the portion
  const int pos = max(p.pos32[t], 0);
  const int slot = min(max(p.state_slots[s], 0), p.nslots - 1);
  const int keep = p.taps - 1;
  const TS* stp = conv_state + (long)slot * keep * p.C;
  float acc = p.b != nullptr ? p.b[c] : 0.f;
  for (int k = 0; k < p.taps; ++k) {
    const int d = keep - k;                  // how far back this tap looks
    float v = 0.f;
    if (i - d >= 0)
      v = ld(src + (long)(t - d) * p.ld_src + p.col0 + c);
    else if (pos - d >= 0)
      v = ld(stp + (long)(keep + i - d) * p.C + c);
    acc += p.w[(long)c * p.taps + k] * v;
  }
  st(out + (long)t * p.C + c, act(acc, p.silu));
}

// Every sequence brings exactly one row: the lane that convolves a channel
// also shifts that channel's kept inputs by one. grid (T, ceil(C / 256)).
template <typename TS>
__global__ __launch_bounds__(256) void short_conv_step_kernel(
    TS* __restrict__ out, const TS* __restrict__ src,
    TS* __restrict__ conv_state, ConvArgs p) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.C) return;
  const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
  const int pos = max(p.pos32[t], 0);
  const int slot = min(max(p.state_slots[s], 0), p.nslots - 1);
  const int keep = p.taps - 1;
  TS* stp = conv_state + (long)slot * keep * p.C + c;
  float acc = p.b != nullptr ? p.b[c] : 0.f;
  const TS x = src[(long)t * p.ld_src + p.col0 + c];
  for (int k = 0; k < keep; ++k) {
    TS v = 0;
    if (pos - (keep - k) >= 0) v = stp[(long)k * p.C];
    if (k > 0) stp[(long)(k - 1) * p.C] = v;
    acc += p.w[(long)c * p.taps + k] * ld(&v);
  }
  if (keep > 0) stp[(long)(keep - 1) * p.C] = x;
  acc += p.w[(long)c * p.taps + keep] * ld(&x);
  st(out + (long)t * p.C + c, act(acc, p.silu));
}

// The same for bf16 rows whose channel count, first column and row stride
// are multiples of 8: a lane takes 8 neighbouring channels of RB rows in a
// row with 16-byte loads, its TAPS x 8 weights in registers.
// grid (ceil(T / RB), ceil(C / 8 / 256)).
constexpr int RB = 8;

template <int TAPS>
__global__ __launch_bounds__(256) void short_conv_vec_kernel(
    unsigned short* __restrict__ out, const unsigned short* __restrict__ src,
    const unsigned short* __restrict__ conv_state, ConvArgs p) {
  const int C = p.C;
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= C) return;
  constexpr int keep = TAPS - 1;
  float wr[TAPS][8], br[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    br[e] = p.b != nullptr ? p.b[c + e] : 0.f;
#pragma unroll
    for (int k = 0; k < TAPS; ++k) wr[k][e] = p.w[(long)(c + e) * TAPS + k];
  }
  const int t_end = min(p.T, (int)(blockIdx.x + 1) * RB);
  for (int t = blockIdx.x * RB; t < t_end; ++t) {
    const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
    const int first = min(max(p.seq_first[s], 0), t);
    const int i = t - first;
    const int pos = max(p.pos32[t], 0);
    const int slot = min(max(p.state_slots[s], 0), p.nslots - 1);
    const unsigned short* stp = conv_state + (long)slot * keep * C;
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = br[e];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) {
      const int d = keep - k;
      u16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (i - d >= 0)
        v = *reinterpret_cast<const u16x8*>(src + (long)(t - d) * p.ld_src +
                                            p.col0 + c);
      else if (pos - d >= 0)
        v = *reinterpret_cast<const u16x8*>(stp + (long)(keep + i - d) * C + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] += wr[k][e] * bf2f(v[e]);
    }
    u16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = f2bf(act(acc[e], p.silu));
    *reinterpret_cast<u16x8*>(out + (long)t * C + c) = o;
  }
}

// grid (nseq, ceil(C / 256)): the slot's new last inputs, after every read
// of the old ones (stream order).
template <typename TS>
__global__ __launch_bounds__(256) void conv_state_update_kernel(
    const TS* __restrict__ src, TS* __restrict__ conv_state, ConvArgs p) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.C) return;
  const int first = p.seq_first[s], n = p.seq_rows[s];
  if (first < 0 || n < 1 || first + n > p.T) return;
  const int hist = max(p.pos32[first], 0);
  const int slot = min(max(p.state_slots[s], 0), p.nslots - 1);
  const int keep = p.taps - 1;
  TS* stp = conv_state + (long)slot * keep * p.C;
  TS fresh[MAX_TAPS];
  for (int j = 0; j < keep; ++j) {
    const int i = n - (keep - j);            // local row of new entry j
    TS v = 0;
    if (i >= 0)
      v = src[(long)(first + i) * p.ld_src + p.col0 + c];
    else if (hist + i >= 0)
      v = stp[(long)(keep + i) * p.C + c];
    fresh[j] = v;
  }
  for (int j = 0; j < keep; ++j) stp[(long)j * p.C + c] = fresh[j];
}

template <typename TS>
void run(void* out, const void* src, void* conv_state, const ConvArgs& p,
         int single, hipStream_t s) {
  const dim3 grid(p.T, (p.C + 255) / 256), sgrid(p.nseq, (p.C + 255) / 256);
  const TS* sp = (const TS*)src;
  TS* cs = (TS*)conv_state;
  if (single) {
    short_conv_step_kernel<TS><<<grid, 256, 0, s>>>((TS*)out, sp, cs, p);
    return;
  }
  bool done = false;
  if constexpr (sizeof(TS) == 2) {
    // few rows: one lane per (row, channel) makes more workgroups
    const bool vec = p.C % 8 == 0 && p.col0 % 8 == 0 && p.ld_src % 8 == 0 &&
                     (long)p.T * p.C >= (1 << 20);
    const dim3 vgrid((p.T + RB - 1) / RB, (p.C / 8 + 255) / 256);
    if (vec && p.taps >= 2 && p.taps <= 5) {
      done = true;
      switch (p.taps) {
        case 2: short_conv_vec_kernel<2><<<vgrid, 256, 0, s>>>((TS*)out, sp, cs, p); break;
        case 3: short_conv_vec_kernel<3><<<vgrid, 256, 0, s>>>((TS*)out, sp, cs, p); break;
        case 4: short_conv_vec_kernel<4><<<vgrid, 256, 0, s>>>((TS*)out, sp, cs, p); break;
        default: short_conv_vec_kernel<5><<<vgrid, 256, 0, s>>>((TS*)out, sp, cs, p); break;
      }
    }
  }
  if (!done) short_conv_kernel<TS><<<grid, 256, 0, s>>>((TS*)out, sp, cs, p);
  if (p.taps > 1)
    conv_state_update_kernel<TS><<<sgrid, 256, 0, s>>>(sp, cs, p);
}

}  // namespace

int conv_max_taps() { return MAX_TAPS; }

// single: every sequence brings one row (T == nseq)
void short_conv_launch(void* out, const void* src, long ld_src, int col0,
                       int C, int taps, const float* w, const float* b,
                       void* conv_state, const int* seq_first,
                       const int* seq_rows, const int* state_slots,
                       const int* row_seq, const int* pos32, int nseq,
                       int nslots, int T, int bf, int silu, int single,
                       hipStream_t s) {
  if (T <= 0 || nseq <= 0) return;
  ConvArgs p;
  p.ld_src = ld_src; p.col0 = col0; p.C = C; p.taps = taps; p.silu = silu;
  p.w = w; p.b = b; p.seq_first = seq_first; p.seq_rows = seq_rows;
  p.state_slots = state_slots; p.row_seq = row_seq; p.pos32 = pos32;
  p.nseq = nseq; p.nslots = nslots; p.T = T;
  if (bf) run<unsigned short>(out, src, conv_state, p, single, s);
  else run<float>(out, src, conv_state, p, single, s);
}
