// Gated recurrence with one state value per channel and sequence (gfx950).
//
//   S_t = (1 - z_t) S_(t-1) + z_t c_t,    y_t = S_t * silu(g_t)
//   z = sigmoid(zp + b_z);  c = u + 1/2 (u >= 0) or sigmoid(u), u = up + b_u
//
// zp, up and g are column blocks of one projection row; gates, candidates
// and the state are fp32. The state [slots, N] is read where a sequence's
// first row of the step sits behind position 0 and starts from zero
// otherwise; it is written back after the last row.
//
// A run of rows is walked by lanes that own VC neighbouring channels each,
// so every row is one coalesced load per column block. Long prompts are cut
// into runs (host-built list: first row, rows, sequence, index of the
// sequence's first run): a first pass leaves every run's (A, B), the
// recurrence S -> A S + B of all its rows, and the second walks the rows
// again from the carry that its predecessors' pairs give. The state a prompt
// portion starts from is passed on by the first pass, since the second pass's
// last run overwrites the slot.
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

// hardware exponential and reciprocal, each within a few ulp of fp32; an
// overflowing exponential gives rcp(inf) = 0
DEVICE_INLINE float sigmoid_f(float z) {
  return __builtin_amdgcn_rcpf(1.0f + __expf(-z));
}
DEVICE_INLINE float candidate(float u) {
  return u >= 0.f ? u + 0.5f : sigmoid_f(u);
}

struct GruArgs {
  long ld_src;
  int col_z, col_u, col_g, N;
  const float* z_b;        // [N]
  const float* u_b;        // [N]
  float* state;            // [nslots, N]
  const int* seq_first;
  const int* seq_rows;
  const int* slots;
  const int* pos32;
  const int* runs;         // [nruns, 4] or null: one run per sequence
  float* ws;               // [nruns, 3, N]: A, B, carried-in state
  int nruns, nseq, nslots, T;
};

struct Run {
  int row0, rows, seq, first;
  bool ok;
};

DEVICE_INLINE Run run_of(const GruArgs& p, int r) {
  Run o;
  if (p.runs != nullptr) {
    const int* q = p.runs + 4L * r;
    o.row0 = q[0]; o.rows = q[1]; o.seq = q[2]; o.first = q[3];
  } else {
    o.row0 = p.seq_first[r]; o.rows = p.seq_rows[r]; o.seq = r; o.first = r;
  }
  o.ok = o.row0 >= 0 && o.rows >= 1 && o.row0 + o.rows <= p.T && o.seq >= 0 &&
         o.seq < p.nseq && o.first >= 0 && o.first <= r;
  return o;
}

// VC neighbouring channels of a row as fp32
template <typename TS, int VC>
DEVICE_INLINE void load_v(const TS* p, float* o) {
  if constexpr (VC == 1) {
    o[0] = ld(p);
  } else {
    typedef TS vec_t __attribute__((ext_vector_type(VC)));
    const vec_t v = *reinterpret_cast<const vec_t*>(p);
#pragma unroll
    for (int k = 0; k < VC; ++k) { const TS e = v[k]; o[k] = ld(&e); }
  }
}
template <typename TS, int VC>
DEVICE_INLINE void store_v(TS* p, const float* f) {
  if constexpr (VC == 1) {
    st(p, f[0]);
  } else {
    typedef TS vec_t __attribute__((ext_vector_type(VC)));
    vec_t v;
#pragma unroll
    for (int k = 0; k < VC; ++k) { TS e; st(&e, f[k]); v[k] = e; }
    *reinterpret_cast<vec_t*>(p) = v;
  }
}

constexpr int THREADS = 64;    // one wave: many small workgroups
constexpr int UNROLL = 8;      // rows whose loads are in flight together

// grid (nruns, ceil(N / (64 * VC)))
template <typename TS, int VC>
__global__ __launch_bounds__(THREADS) void gru_run_summary_kernel(
    const TS* __restrict__ src, GruArgs p) {
  const Run r = run_of(p, blockIdx.x);
  const int c = (blockIdx.y * THREADS + threadIdx.x) * VC;
  if (!r.ok || c >= p.N) return;
  float zb[VC], ub[VC], A[VC], B[VC];
#pragma unroll
  for (int k = 0; k < VC; ++k) {
    zb[k] = p.z_b[c + k];
    ub[k] = p.u_b[c + k];
    A[k] = 1.f;
    B[k] = 0.f;
  }
  const TS* base = src + (long)r.row0 * p.ld_src + c;
  for (int i0 = 0; i0 < r.rows; i0 += UNROLL) {
    float z[UNROLL][VC], u[UNROLL][VC];
#pragma unroll
    for (int j = 0; j < UNROLL; ++j) {
      const long i = min(i0 + j, r.rows - 1);
      load_v<TS, VC>(base + i * p.ld_src + p.col_z, z[j]);
      load_v<TS, VC>(base + i * p.ld_src + p.col_u, u[j]);
    }
#pragma unroll
    for (int j = 0; j < UNROLL; ++j) {
      if (i0 + j < r.rows) {
#pragma unroll
        for (int k = 0; k < VC; ++k) {
          const float zz = sigmoid_f(z[j][k] + zb[k]);
          const float keep = 1.0f - zz;
          A[k] *= keep;
          B[k] = keep * B[k] + zz * candidate(u[j][k] + ub[k]);
        }
      }
    }
  }
  float* w = p.ws + (long)blockIdx.x * 3 * p.N + c;
#pragma unroll
  for (int k = 0; k < VC; ++k) {
    w[k] = A[k];
    w[p.N + k] = B[k];
  }
  if (r.first == (int)blockIdx.x) {
    const long slot = min(max(p.slots[r.seq], 0), p.nslots - 1);
    const bool has = p.pos32[r.row0] > 0;
#pragma unroll
    for (int k = 0; k < VC; ++k)
      w[2 * p.N + k] = has ? p.state[slot * p.N + c + k] : 0.f;
  }
}

template <typename TS, int VC>
__global__ __launch_bounds__(THREADS) void gru_run_kernel(
    TS* __restrict__ y, const TS* __restrict__ src, GruArgs p) {
  const int me = blockIdx.x;
  const Run r = run_of(p, me);
  const int c = (blockIdx.y * THREADS + threadIdx.x) * VC;
  if (!r.ok || c >= p.N) return;
  const int N = p.N;
  const long slot = min(max(p.slots[r.seq], 0), p.nslots - 1);
  float* sp = p.state + slot * N + c;
  float zb[VC], ub[VC], S[VC];
#pragma unroll
  for (int k = 0; k < VC; ++k) {
    zb[k] = p.z_b[c + k];
    ub[k] = p.u_b[c + k];
  }
  if (p.ws != nullptr) {
    const float* w = p.ws + (long)r.first * 3 * N + c;
#pragma unroll
    for (int k = 0; k < VC; ++k) S[k] = w[2 * N + k];
#pragma unroll 4
    for (int q = r.first; q < me; ++q) {
      const float* v = p.ws + (long)q * 3 * N + c;
#pragma unroll
      for (int k = 0; k < VC; ++k) S[k] = v[k] * S[k] + v[N + k];
    }
  } else {
    const bool has = p.pos32[r.row0] > 0;
#pragma unroll
    for (int k = 0; k < VC; ++k) S[k] = has ? sp[k] : 0.f;
  }
  const TS* base = src + (long)r.row0 * p.ld_src + c;
  TS* yo = y + (long)r.row0 * N + c;
  for (int i0 = 0; i0 < r.rows; i0 += UNROLL) {
    float z[UNROLL][VC], u[UNROLL][VC], g[UNROLL][VC];
#pragma unroll
    for (int j = 0; j < UNROLL; ++j) {
      const long i = min(i0 + j, r.rows - 1);
      load_v<TS, VC>(base + i * p.ld_src + p.col_z, z[j]);
      load_v<TS, VC>(base + i * p.ld_src + p.col_u, u[j]);
      load_v<TS, VC>(base + i * p.ld_src + p.col_g, g[j]);
    }
#pragma unroll
    for (int j = 0; j < UNROLL; ++j) {
      if (i0 + j < r.rows) {
        float o[VC];
#pragma unroll
        for (int k = 0; k < VC; ++k) {
          const float zz = sigmoid_f(z[j][k] + zb[k]);
          S[k] = (1.0f - zz) * S[k] + zz * candidate(u[j][k] + ub[k]);
          o[k] = S[k] * g[j][k] * sigmoid_f(g[j][k]);
        }
        store_v<TS, VC>(yo + (long)(i0 + j) * N, o);
      }
    }
  }
  if (r.row0 + r.rows == p.seq_first[r.seq] + p.seq_rows[r.seq]) {
#pragma unroll
    for (int k = 0; k < VC; ++k) sp[k] = S[k];
  }
}

template <typename TS, int VC>
void run(void* y, const void* src, const GruArgs& p, hipStream_t s) {
  const dim3 grid(p.nruns, (p.N + THREADS * VC - 1) / (THREADS * VC));
  if (p.ws != nullptr)
    gru_run_summary_kernel<TS, VC><<<grid, THREADS, 0, s>>>((const TS*)src, p);
  gru_run_kernel<TS, VC><<<grid, THREADS, 0, s>>>((TS*)y, (const TS*)src, p);
}

}  // namespace

// runs null: one run per sequence (nruns == nseq), no workspace
void gru_scan_launch(void* y, const void* src, long ld_src, int col_z,
                     int col_u, int col_g, int N, const float* z_b,
                     const float* u_b, float* state, const int* seq_first,
                     const int* seq_rows, const int* slots, const int* pos32,
                     const int* runs, float* ws, int nruns, int nseq,
                     int nslots, int T, int bf, hipStream_t s) {
  if (T <= 0 || nruns <= 0) return;
  GruArgs p;
  p.ld_src = ld_src; p.col_z = col_z; p.col_u = col_u; p.col_g = col_g;
  p.N = N; p.z_b = z_b; p.u_b = u_b; p.state = state; p.seq_first = seq_first;
  p.seq_rows = seq_rows; p.slots = slots; p.pos32 = pos32; p.runs = runs;
  p.ws = ws; p.nruns = nruns; p.nseq = nseq; p.nslots = nslots; p.T = T;
  auto fits = [&](int v) {
    return N % v == 0 && ld_src % v == 0 && col_z % v == 0 && col_u % v == 0 &&
           col_g % v == 0;
  };
  // wide lanes pay once there are enough of them to fill the chip
  const bool many = (long)nruns * N >= 4L * 64 * 1024;
  if (bf) {
    if (many && fits(4)) run<unsigned short, 4>(y, src, p, s);
    else if (fits(2)) run<unsigned short, 2>(y, src, p, s);
    else run<unsigned short, 1>(y, src, p, s);
  } else {
    if (fits(2)) run<float, 2>(y, src, p, s);
    else run<float, 1>(y, src, p, s);
  }
}
