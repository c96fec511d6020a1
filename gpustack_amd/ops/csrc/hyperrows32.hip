// Row kernels of a residual made of S parallel fp32 streams (gfx950).
//
//   embed_streams : x[t, s] = embed[token_t] * scale for every stream
//   stream_step   : closes one sublayer and opens the next,
//                     y = a * sigmoid(gate + gate_b)
//                     x_t <- sum_s mix[s, t] x_s + out[t] * y
//                     u = sum_s in[s] x_s;  h = rmsnorm(u) * norm_w
//                   reading and writing the streams once; for batches of
//                   single rows the token shift of h in the same pass
//   token_shift   : hs = h + (h_prev - h) * mu, h_prev the row before in the
//                   sequence, kept in a state slot between steps; for one
//                   or several mu, each with a plane of hs of its own
//
// The streams x [T, S, W] are updated in place; one workgroup handles a row,
// a lane reads a channel of ALL streams before it writes any. Norms, gates
// and streams are fp32 whatever the GEMM dtype; h and hs leave in that dtype.
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
template <typename T> struct Vec4;
template <> struct Vec4<float> {
  static DEVICE_INLINE void load(const float* p, float* o) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
    o[0] = v[0]; o[1] = v[1]; o[2] = v[2]; o[3] = v[3];
  }
  static DEVICE_INLINE void store(float* p, const float* o) {
    *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
  }
};
template <> struct Vec4<unsigned short> {
  static DEVICE_INLINE void load(const unsigned short* p, float* o) {
    const u16x4 v = *reinterpret_cast<const u16x4*>(p);
    o[0] = bf2f(v[0]); o[1] = bf2f(v[1]); o[2] = bf2f(v[2]); o[3] = bf2f(v[3]);
  }
  static DEVICE_INLINE void store(unsigned short* p, const float* o) {
    *reinterpret_cast<u16x4*>(p) = u16x4{f2bf(o[0]), f2bf(o[1]), f2bf(o[2]), f2bf(o[3])};
  }
};

DEVICE_INLINE float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

constexpr int MAX_STREAMS = 32;

template <int THREADS>
DEVICE_INLINE float block_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < THREADS / 64; ++i) s += red[i];
  return s;
}

struct StepArgs {
  float* x;                // [T, S, W]
  const void* a;           // [T, W] or null: nothing to close
  const void* gate;        // [T, W] rows ld_gate apart, or null: no gate
  long ld_gate;
  const float* gate_b;     // [W] or null
  const float* mix;        // [S, S], from x to
  const float* out;        // [S]
  const float* in;         // [S] or null: nothing to open
  const float* norm_w;     // [W]
  void* h;                 // [T, W]
  const float* mu;         // [M, W] or null: no token shift
  void* hs;                // [M, T, W]
  void* prev;              // [nslots, W]
  const int* row_seq;
  const int* slots;
  const int* pos32;
  int nseq, nslots, M, T, S, W;
  float eps;
};

// slot and "has a previous row" of a single-row sequence
DEVICE_INLINE void shift_row(const StepArgs& p, long t, long& slot, bool& has) {
  const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
  slot = min(max(p.slots[s], 0), p.nslots - 1);
  has = p.pos32[t] > 0;
}

// W % 4 == 0 and W <= NV * 4 * THREADS: four consecutive channels per lane
// and step; u stays in registers between the sum of squares and the store.
template <typename TA, int S, int NV, int THREADS>
__global__ __launch_bounds__(THREADS) void stream_step_vec_kernel(StepArgs p) {
  __shared__ float red[THREADS / 64];
  const long t = blockIdx.x;
  const int W = p.W;
  float* xr = p.x + t * S * W;
  const TA* ar = (const TA*)p.a;
  const TA* gr = (const TA*)p.gate;
  float mix[S][S], ow[S], iw[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    iw[s] = p.in != nullptr ? p.in[s] : 0.f;
    ow[s] = ar != nullptr ? p.out[s] : 0.f;
#pragma unroll
    for (int q = 0; q < S; ++q) mix[s][q] = ar != nullptr ? p.mix[s * S + q] : 0.f;
  }
  float keep[NV][4];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = (threadIdx.x + j * THREADS) * 4;
    float u[4] = {0.f, 0.f, 0.f, 0.f};
    if (i < W) {
      float xo[S][4];
#pragma unroll
      for (int s = 0; s < S; ++s) Vec4<float>::load(xr + (long)s * W + i, xo[s]);
      if (ar != nullptr) {
        float y[4];
        Vec4<TA>::load(ar + t * W + i, y);
        if (gr != nullptr) {
          float g[4], b[4] = {0.f, 0.f, 0.f, 0.f};
          Vec4<TA>::load(gr + t * p.ld_gate + i, g);
          if (p.gate_b != nullptr) Vec4<float>::load(p.gate_b + i, b);
#pragma unroll
          for (int k = 0; k < 4; ++k) y[k] *= sigmoid_f(g[k] + b[k]);
        }
#pragma unroll
        for (int q = 0; q < S; ++q) {
          float n[4];
#pragma unroll
          for (int k = 0; k < 4; ++k) n[k] = ow[q] * y[k];
#pragma unroll
          for (int s = 0; s < S; ++s)
#pragma unroll
            for (int k = 0; k < 4; ++k) n[k] += mix[s][q] * xo[s][k];
          Vec4<float>::store(xr + (long)q * W + i, n);
#pragma unroll
          for (int k = 0; k < 4; ++k) u[k] += iw[q] * n[k];
        }
      } else {
#pragma unroll
        for (int s = 0; s < S; ++s)
#pragma unroll
          for (int k = 0; k < 4; ++k) u[k] += iw[s] * xo[s][k];
      }
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      keep[j][k] = u[k];
      ss += u[k] * u[k];
    }
  }
  if (p.in == nullptr) return;
  const float inv = 1.0f / sqrtf(block_sum<THREADS>(ss, red) / (float)W + p.eps);
  long slot = 0;
  bool has = false;
  if (p.mu != nullptr) shift_row(p, t, slot, has);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = (threadIdx.x + j * THREADS) * 4;
    if (i < W) {
      float w[4], o[4];
      Vec4<float>::load(p.norm_w + i, w);
#pragma unroll
      for (int k = 0; k < 4; ++k) o[k] = keep[j][k] * inv * w[k];
      Vec4<TA>::store((TA*)p.h + t * W + i, o);
      if (p.mu != nullptr) {
        TA* pp = (TA*)p.prev + slot * W + i;
        float m[4], q[4] = {0.f, 0.f, 0.f, 0.f};
        if (has) Vec4<TA>::load(pp, q);
        Vec4<TA>::store(pp, o);
        // the row as the GEMM dtype holds it, as in a longer portion
        if constexpr (sizeof(TA) == 2) {
#pragma unroll
          for (int k = 0; k < 4; ++k) o[k] = bf2f(f2bf(o[k]));
        }
        for (int b = 0; b < p.M; ++b) {
          float r[4];
          Vec4<float>::load(p.mu + (long)b * W + i, m);
#pragma unroll
          for (int k = 0; k < 4; ++k) r[k] = o[k] + (q[k] - o[k]) * m[k];
          Vec4<TA>::store((TA*)p.hs + ((long)b * p.T + t) * W + i, r);
        }
      }
    }
  }
}

// Any width up to the LDS row (W floats) and up to MAX_STREAMS streams.
template <typename TA>
__global__ __launch_bounds__(256) void stream_step_kernel(StepArgs p) {
  extern __shared__ float us[];                // [W]
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int W = p.W, S = p.S;
  float* xr = p.x + t * S * W;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) {
    float xo[MAX_STREAMS];
    for (int s = 0; s < S; ++s) xo[s] = xr[(long)s * W + i];
    float u = 0.f;
    if (p.a != nullptr) {
      float y = ld((const TA*)p.a + t * W + i);
      if (p.gate != nullptr) {
        float g = ld((const TA*)p.gate + t * p.ld_gate + i);
        if (p.gate_b != nullptr) g += p.gate_b[i];
        y *= sigmoid_f(g);
      }
      for (int q = 0; q < S; ++q) {
        float n = p.out[q] * y;
        for (int s = 0; s < S; ++s) n += p.mix[s * S + q] * xo[s];
        xr[(long)q * W + i] = n;
        if (p.in != nullptr) u += p.in[q] * n;
      }
    } else {
      for (int s = 0; s < S; ++s) u += p.in[s] * xo[s];
    }
    us[i] = u;
    ss += u * u;
  }
  if (p.in == nullptr) return;
  const float inv = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)W + p.eps);
  long slot = 0;
  bool has = false;
  if (p.mu != nullptr) shift_row(p, t, slot, has);
  for (int i = threadIdx.x; i < W; i += 256) {   // a lane's own us[i]
    TA o;
    st(&o, us[i] * inv * p.norm_w[i]);
    ((TA*)p.h)[t * W + i] = o;
    if (p.mu != nullptr) {
      TA* pp = (TA*)p.prev + slot * W + i;
      const float q = has ? ld(pp) : 0.f, v = ld(&o);
      *pp = o;
      for (int b = 0; b < p.M; ++b)
        st((TA*)p.hs + ((long)b * p.T + t) * W + i,
           v + (q - v) * p.mu[(long)b * W + i]);
    }
  }
}

struct ShiftArgs {
  const float* mu;
  const int* seq_first;
  const int* seq_rows;
  const int* slots;
  const int* row_seq;
  const int* pos32;
  int nseq, nslots, M, T, W;
};

// grid (T, ceil(W / (256 * V))): a lane takes V channels of one row. The
// lane of a sequence's first row reads the slot and then puts the step's
// last row there: nobody else touches that (slot, channel).
template <typename TA, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(
    TA* __restrict__ hs, const TA* __restrict__ h, TA* __restrict__ prev,
    ShiftArgs p) {
  const long t = blockIdx.x;
  const int i = (blockIdx.y * 256 + threadIdx.x) * V;
  const int W = p.W;
  if (i >= W) return;
  const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
  const int first = p.seq_first[s];
  typedef TA vec_t __attribute__((ext_vector_type(V)));
  const vec_t cur = *reinterpret_cast<const vec_t*>(h + t * W + i);
  vec_t old = 0;
  if (t > first) {
    old = *reinterpret_cast<const vec_t*>(h + (t - 1) * W + i);
  } else {
    const long slot = min(max(p.slots[s], 0), p.nslots - 1);
    vec_t* pp = reinterpret_cast<vec_t*>(prev + slot * W + i);
    if (p.pos32[t] > 0) old = *pp;
    const long last = min(max(t + p.seq_rows[s] - 1, t), (long)p.T - 1);
    *pp = *reinterpret_cast<const vec_t*>(h + last * W + i);
  }
  for (int b = 0; b < p.M; ++b) {
    const float* mu = p.mu + (long)b * W + i;
    vec_t o;
#pragma unroll
    for (int k = 0; k < V; ++k) {
      const TA cv = cur[k], ov = old[k];
      const float c = ld(&cv), q = ld(&ov);
      TA r;
      st(&r, c + (q - c) * mu[k]);
      o[k] = r;
    }
    *reinterpret_cast<vec_t*>(hs + ((long)b * p.T + t) * W + i) = o;
  }
}

template <typename TA>
__global__ __launch_bounds__(256) void token_shift_any_kernel(
    TA* __restrict__ hs, const TA* __restrict__ h, TA* __restrict__ prev,
    ShiftArgs p) {
  const long t = blockIdx.x;
  const int i = blockIdx.y * 256 + threadIdx.x;
  const int W = p.W;
  if (i >= W) return;
  const int s = min(max(p.row_seq[t], 0), p.nseq - 1);
  const TA cur = h[t * W + i];
  TA old = 0;
  if (t > p.seq_first[s]) {
    old = h[(t - 1) * W + i];
  } else {
    const long slot = min(max(p.slots[s], 0), p.nslots - 1);
    TA* pp = prev + slot * W + i;
    if (p.pos32[t] > 0) old = *pp;
    const long last = min(max(t + p.seq_rows[s] - 1, t), (long)p.T - 1);
    *pp = h[last * W + i];
  }
  const float c = ld(&cur), q = ld(&old);
  for (int b = 0; b < p.M; ++b)
    st(hs + ((long)b * p.T + t) * W + i, c + (q - c) * p.mu[(long)b * W + i]);
}

template <typename TW>
__global__ __launch_bounds__(256) void embed_streams_kernel(
    float* __restrict__ x, const long* __restrict__ tokens,
    const TW* __restrict__ embed, int S, int W, long vocab, float scale) {
  const long t = blockIdx.x;
  const long tok = min(max(tokens[t], 0L), vocab - 1);   // never read outside
  const TW* e = embed + tok * W;
  float* xr = x + t * S * W;
  for (int i = threadIdx.x; i < W; i += 256) {
    const float v = ld(e + i) * scale;
    for (int s = 0; s < S; ++s) xr[(long)s * W + i] = v;
  }
}

template <typename TA, int S>
void step_pick(const StepArgs& p, int T, hipStream_t s) {
  const int W = p.W;
  // few rows: a row's work spread over more waves
  if (T <= 512 && W > 1024 && W <= 4096)
    stream_step_vec_kernel<TA, S, 1, 1024><<<T, 1024, 0, s>>>(p);
  else if (T <= 512 && W > 4096)
    stream_step_vec_kernel<TA, S, 2, 1024><<<T, 1024, 0, s>>>(p);
  else if (W <= 1024)
    stream_step_vec_kernel<TA, S, 1, 256><<<T, 256, 0, s>>>(p);
  else if (W <= 2048)
    stream_step_vec_kernel<TA, S, 2, 256><<<T, 256, 0, s>>>(p);
  else if (W <= 4096)
    stream_step_vec_kernel<TA, S, 4, 256><<<T, 256, 0, s>>>(p);
  else
    stream_step_vec_kernel<TA, S, 8, 256><<<T, 256, 0, s>>>(p);
}

template <typename TA>
void step_run(const StepArgs& p, int T, hipStream_t s) {
  if (p.W % 4 == 0 && p.W <= 8192 && p.S <= 6 && p.ld_gate % 4 == 0 &&
      (uintptr_t)p.gate % (4 * sizeof(TA)) == 0) {
    switch (p.S) {
      case 1: step_pick<TA, 1>(p, T, s); return;
      case 2: step_pick<TA, 2>(p, T, s); return;
      case 3: step_pick<TA, 3>(p, T, s); return;
      case 4: step_pick<TA, 4>(p, T, s); return;
      case 5: step_pick<TA, 5>(p, T, s); return;
      default: step_pick<TA, 6>(p, T, s); return;
    }
  }
  const size_t smem = (size_t)p.W * sizeof(float);
  if (smem > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)stream_step_kernel<TA>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)smem);
  stream_step_kernel<TA><<<T, 256, smem, s>>>(p);
}

template <typename TA>
void shift_run(void* hs, const void* h, void* prev, const ShiftArgs& p,
               hipStream_t s) {
  constexpr int V = 16 / sizeof(TA);
  if (p.W % V == 0)
    token_shift_kernel<TA, V><<<dim3(p.T, (p.W / V + 255) / 256), 256, 0, s>>>(
        (TA*)hs, (const TA*)h, (TA*)prev, p);
  else
    token_shift_any_kernel<TA><<<dim3(p.T, (p.W + 255) / 256), 256, 0, s>>>(
        (TA*)hs, (const TA*)h, (TA*)prev, p);
}

}  // namespace

int stream_step_max_streams() { return MAX_STREAMS; }
int stream_step_max_width() { return 38 * 1024; }   // LDS row of the any-size path

void embed_streams_launch(float* x, const long* tokens, const void* embed,
                          int T, int S, int W, long vocab, float scale, int bf,
                          hipStream_t s) {
  if (T <= 0) return;
  if (bf)
    embed_streams_kernel<unsigned short><<<T, 256, 0, s>>>(
        x, tokens, (const unsigned short*)embed, S, W, vocab, scale);
  else
    embed_streams_kernel<float><<<T, 256, 0, s>>>(
        x, tokens, (const float*)embed, S, W, vocab, scale);
}

void stream_step_launch(float* x, const void* a, const void* gate, long ld_gate,
                        const float* gate_b, const float* mix, const float* out,
                        const float* in, const float* norm_w, void* h,
                        const float* mu, void* hs, void* prev,
                        const int* row_seq, const int* slots, const int* pos32,
                        int nseq, int nslots, int M, int T, int S, int W,
                        float eps, int bf, hipStream_t s) {
  if (T <= 0) return;
  StepArgs p;
  p.x = x; p.a = a; p.gate = gate; p.ld_gate = ld_gate; p.gate_b = gate_b;
  p.mix = mix; p.out = out; p.in = in; p.norm_w = norm_w; p.h = h; p.mu = mu;
  p.hs = hs; p.prev = prev; p.row_seq = row_seq; p.slots = slots;
  p.pos32 = pos32; p.nseq = nseq; p.nslots = nslots; p.M = M; p.T = T;
  p.S = S; p.W = W; p.eps = eps;
  if (bf) step_run<unsigned short>(p, T, s);
  else step_run<float>(p, T, s);
}

void token_shift_launch(void* hs, const void* h, const float* mu, void* prev,
                        const int* seq_first, const int* seq_rows,
                        const int* slots, const int* row_seq, const int* pos32,
                        int nseq, int nslots, int M, int T, int W, int bf,
                        hipStream_t s) {
  if (T <= 0 || nseq <= 0) return;
  ShiftArgs p;
  p.mu = mu; p.seq_first = seq_first; p.seq_rows = seq_rows; p.slots = slots;
  p.row_seq = row_seq; p.pos32 = pos32; p.nseq = nseq; p.nslots = nslots;
  p.M = M; p.T = T; p.W = W;
  if (bf) shift_run<unsigned short>(hs, h, prev, p, s);
  else shift_run<float>(hs, h, prev, p, s);
}
