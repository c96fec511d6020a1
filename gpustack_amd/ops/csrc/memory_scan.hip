// Matrix memories: one fp32 state S [N x P] per head and sequence, written by
// k v^T and read by q, in three forms of decay (gfx950).
//
//   CONST : S_t = a S + k v^T                 y = S_t^T q      a per head
//   CHAN  : S_t = diag(w_t) S + k v^T         y = (S_(t-1) + diag(u) k v^T)^T q
//           w_t = exp(-exp(z_t + w0)) per head and state row
//   GATED : S_t = a_t S + b_t k v^T           y = S_t^T q, to be divided by
//           max(|n_t . q|, exp(-m_t)) + 1e-6, n_t = a_t n + b_t k, with a_t =
//           exp(f + m_(t-1) - m_t), b_t = exp(i - m_t), m_t = max(f + m_(t-1), i)
//
// q and k may turn with the row's position (channel i with i + half) and carry
// a constant factor. S lives in the sequence's slot of a state pool [slots, H,
// N, P]; n and m in [slots, H, N + 1] beside it. A batch is ragged: sequence s
// brings rows seq_first[s] .. + seq_rows[s] - 1; the position of its first row
// says whether the slot is read (> 0) or everything starts from zero.
//
//   rope_table       : cos / sin of every row's angles, once per step
//   memory_gates     : GATED, prompts: a wave per (sequence, head) turns 64
//                      rows' gates into (a, b) with a max-plus prefix scan
//   memory_scan      : prompts. TPP neighbouring lanes share two value
//                      channels, NR state rows each, in registers; rows are
//                      staged through LDS and walked in order, the next
//                      row's operands on their way while one is worked on.
//                      GATED: one more workgroup per (sequence, head) walks n
//                      as a state whose value is always 1
//   memory_step      : single rows (decode): one pass over the state
#include "common.h"

namespace {

template <typename T> DEVICE_INLINE float ld(const T* p);
template <> DEVICE_INLINE float ld<float>(const float* p) { return *p; }
template <> DEVICE_INLINE float ld<unsigned short>(const unsigned short* p) {
  return bf2f(*p);
}

enum { CONST_DECAY = 0, CHAN_DECAY = 1, GATED = 2 };

struct MemArgs {
  const void *q, *k, *v;         // [T, H * N] / [T, H * P] rows ld_* apart
  long ld_q, ld_k, ld_v;
  float q_scale, k_scale;
  int H, N, P;
  const float* decay;            // CONST: [H]
  const void* chan;              // CHAN: [T, H * N] rows ld_c apart
  long ld_c;
  const float* w0;               // CHAN: [H, N]
  const float* u;                // CHAN: [H, N]
  const float* rot;              // [T, 2, half] cos | sin, or null
  const float* inv_freq;         // [half]
  int half;
  const void* gates;             // GATED: [T, 2 H] rows ld_g apart: i | f
  long ld_g;
  const float *i_b, *f_b;        // GATED: [H]
  float cap;
  float* ab;                     // GATED, prompts: [T, H, 3] a, b, exp(-m)
  float* rden;                   // GATED: [T, H] 1 / denominator, left to the
                                 // reader of y
  float* state;                  // [nslots, H, N, P]
  float* extra;                  // GATED: [nslots, H, N + 1]
  const int* seq_first;
  const int* seq_rows;
  const int* slots;
  const int* pos32;
  int nslots, T, vec;
};

DEVICE_INLINE float log_sigmoid_f(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}
DEVICE_INLINE float capped(float z, float cap) { return cap * tanhf(z / cap); }

template <int CTRL>
DEVICE_INLINE float dpp_add(float x) {
  return x + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
      0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
// sum over TPP = 8 or 16 neighbouring lanes: quads, then mirrored halves
template <int TPP>
DEVICE_INLINE float lanes_sum(float x) {
  x = dpp_add<0xB1>(x);          // lane ^ 1
  x = dpp_add<0x4E>(x);          // lane ^ 2
  x = dpp_add<0x141>(x);         // mirror within 8
  if constexpr (TPP == 16) x = dpp_add<0x140>(x);   // mirror within 16
  return x;
}

struct SeqView {
  int first, n;
  long slot;
  bool has, ok;
};
DEVICE_INLINE SeqView view_of(const MemArgs& p, int s) {
  SeqView o;
  o.first = p.seq_first[s];
  o.n = p.seq_rows[s];
  o.ok = o.first >= 0 && o.n >= 1 && o.first + o.n <= p.T;
  o.slot = min(max(p.slots[s], 0), p.nslots - 1);
  o.has = o.ok && p.pos32[o.first] > 0;
  return o;
}

__global__ __launch_bounds__(64) void rope_table_kernel(
    float* __restrict__ out, const int* __restrict__ pos32,
    const float* __restrict__ inv_freq, int half) {
  const long t = blockIdx.x;
  const float pos = (float)pos32[t];
  for (int i = threadIdx.x; i < half; i += 64) {
    float s, c;
    sincosf(pos * inv_freq[i], &s, &c);
    out[(t * 2) * half + i] = c;
    out[(t * 2 + 1) * half + i] = s;
  }
}

// ---- GATED: the gates of a prompt ---------------------------------------------

template <typename TS>
__global__ __launch_bounds__(64) void memory_gates_kernel(MemArgs p) {
  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const SeqView sv = view_of(p, s);
  if (!sv.ok) return;
  const int H = p.H;
  float* mp = p.extra + (sv.slot * H + h) * (p.N + 1) + p.N;
  float m_in = sv.has ? *mp : 0.f;
  const float ib = p.i_b[h], fb = p.f_b[h];
  float zi = 0.f, zf = 0.f;
  auto fetch = [&](int c0) {
    if (c0 + lane < sv.n) {
      const TS* g = (const TS*)p.gates + (long)(sv.first + c0 + lane) * p.ld_g + h;
      zi = ld(g);
      zf = ld(g + H);
    }
  };
  fetch(0);
  for (int c0 = 0; c0 < sv.n; c0 += 64) {
    const int rows = min(64, sv.n - c0);
    float gi = -INFINITY, gf = 0.f;        // rows past the end keep m
    if (lane < rows) {
      gi = capped(zi + ib, p.cap);
      gf = log_sigmoid_f(capped(zf + fb, p.cap));
    }
    fetch(c0 + 64);
    float F = gf, I = gi;                  // m -> max(F + m, I)
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const float fp = __shfl_up(F, d, WAVE_SIZE), ip = __shfl_up(I, d, WAVE_SIZE);
      if (lane >= d) {
        I = fmaxf(ip + F, I);
        F += fp;
      }
    }
    const float m = fmaxf(F + m_in, I);
    float before = __shfl_up(m, 1, WAVE_SIZE);
    if (lane == 0) before = m_in;
    if (lane < rows) {
      float* o = p.ab + ((long)(sv.first + c0 + lane) * H + h) * 3;
      o[0] = expf(gf + before - m);
      o[1] = expf(gi - m);
      o[2] = expf(-m);
    }
    m_in = __shfl(m, rows - 1, WAVE_SIZE);
  }
  if (lane == 0) *mp = m_in;
}

// ---- prompts ------------------------------------------------------------------

constexpr int VC = 2;                       // value channels per lane

constexpr int scan_lds(int mode, int nr, int tpp, int ch) {
  return 2 * ch * ((mode == CHAN_DECAY ? 3 : 2) * tpp * (nr + 4)
                   + 256 / tpp * VC + 4) * 4;
}
// rows staged per pass: as many of 16, 8, 4, 2 as keep the LDS small
constexpr int scan_rows(int mode, int nr, int tpp) {
  int ch = 16;
  while (ch > 2 && scan_lds(mode, nr, tpp, ch) > 56 * 1024) ch /= 2;
  return ch;
}

// one row's operands of a lane
template <int MODE, int NR>
struct RowOps {
  f32x4 k[NR / 4], q[NR / 4], w[MODE == CHAN_DECAY ? NR / 4 : 1];
  float v[VC], a, b;
};

// grid (nseq, H, ceil(P / channels per workgroup)), GATED one more in z;
// blockDim 64 .. 256
template <typename TS, int MODE, int NR, int TPP>
__global__ __launch_bounds__(256) void memory_scan_kernel(
    float* __restrict__ y, MemArgs p) {
  constexpr int CH = scan_rows(MODE, NR, TPP);
  constexpr int NS = NR + 4;               // floats between two lanes' slices
  constexpr int ROW = TPP * NS;
  constexpr int WROW = MODE == CHAN_DECAY ? ROW : 4;
  constexpr int PBM = 256 / TPP * VC;
  __shared__ __attribute__((aligned(16))) float ks[2][CH][ROW];
  __shared__ __attribute__((aligned(16))) float qs[2][CH][ROW];
  __shared__ __attribute__((aligned(16))) float ws[2][CH][WROW];
  __shared__ __attribute__((aligned(16))) float vs[2][CH][PBM];
  __shared__ float sc[2][CH][4];           // a, b, exp(-m), bonus
  const int s = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x, nthr = blockDim.x;
  const int PB = nthr / TPP * VC, p0 = blockIdx.z * PB;
  const int ns = tid % TPP, pl = (tid / TPP) * VC;
  const SeqView sv = view_of(p, s);
  if (!sv.ok) return;
  const int H = p.H, N = p.N, half = p.half;
  // the normaliser: a state of one channel whose value is 1
  const bool norm = MODE == GATED && blockIdx.z + 1 == gridDim.z;
  const int P = norm ? 1 : p.P;
  const int pc = norm ? pl : p0 + pl;
  float* sp = norm ? p.extra + (sv.slot * H + h) * (long)(N + 1)
                   : p.state + (sv.slot * H + h) * (long)N * P;
  float S[VC][NR];
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const int nn = ns * NR + j;
#pragma unroll
    for (int c = 0; c < VC; ++c)
      S[c][j] = sv.has && nn < N && pc + c < P ? sp[(long)nn * P + pc + c] : 0.f;
  }
  if (norm)
    for (int i = tid; i < 2 * CH * PBM; i += nthr) (&vs[0][0][0])[i] = 1.f;
  // state rows past N keep k = q = w = 0
  for (int i = tid; i < 2 * CH * ROW; i += nthr) {
    (&ks[0][0][0])[i] = 0.f;
    (&qs[0][0][0])[i] = 0.f;
    if constexpr (MODE == CHAN_DECAY) (&ws[0][0][0])[i] = 0.f;
  }
  __syncthreads();
  auto at = [](int nn) { return (nn / NR) * NS + nn % NR; };
  const float* w0 = MODE == CHAN_DECAY ? p.w0 + (long)h * N : nullptr;
  const float* ub = MODE == CHAN_DECAY ? p.u + (long)h * N : nullptr;

  auto stage = [&](int buf, int c0) {
    const int rows = min(CH, sv.n - c0);
    const long t0 = sv.first + c0;
    if (sizeof(TS) == 2 && p.vec) {
      // 8 channels per lane and step
      const int nvec = N / 8, np = half > 0 ? nvec - half / 8 : nvec;
      for (int i = tid; i < rows * np; i += nthr) {
        const int r = i / np;
        int e = (i % np) * 8;
        const bool turn = e < half;
        if (!turn) e += half;              // the pairs' second halves are done
        const long t = t0 + r;
        const unsigned short* qp = (const unsigned short*)p.q + t * p.ld_q + (long)h * N + e;
        const unsigned short* kp = (const unsigned short*)p.k + t * p.ld_k + (long)h * N + e;
        const u16x8 q8 = *reinterpret_cast<const u16x8*>(qp);
        const u16x8 k8 = *reinterpret_cast<const u16x8*>(kp);
        u16x8 q9 = q8, k9 = k8;
        if (turn) {
          q9 = *reinterpret_cast<const u16x8*>(qp + half);
          k9 = *reinterpret_cast<const u16x8*>(kp + half);
        }
        u16x8 z8 = q8;
        if constexpr (MODE == CHAN_DECAY)
          z8 = *reinterpret_cast<const u16x8*>(
              (const unsigned short*)p.chan + t * p.ld_c + (long)h * N + e);
#pragma unroll
        for (int g = 0; g < 2; ++g) {
          f32x4 qo, ko, q2, k2, wo, cs, sn;
          if (turn) {
            cs = *reinterpret_cast<const f32x4*>(p.rot + t * 2 * half + e + g * 4);
            sn = *reinterpret_cast<const f32x4*>(p.rot + (t * 2 + 1) * half + e + g * 4);
          }
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            float q = bf2f(q8[g * 4 + x]), k = bf2f(k8[g * 4 + x]);
            if (turn) {
              const float qb = bf2f(q9[g * 4 + x]), kb = bf2f(k9[g * 4 + x]);
              const float qa = q, ka = k;
              q = qa * cs[x] - qb * sn[x];
              q2[x] = (qb * cs[x] + qa * sn[x]) * p.q_scale;
              k = ka * cs[x] - kb * sn[x];
              k2[x] = (kb * cs[x] + ka * sn[x]) * p.k_scale;
            }
            qo[x] = q * p.q_scale;
            ko[x] = k * p.k_scale;
            if constexpr (MODE == CHAN_DECAY)
              wo[x] = expf(-expf(bf2f(z8[g * 4 + x]) + w0[e + g * 4 + x]));
          }
          const int o = at(e + g * 4);
          *reinterpret_cast<f32x4*>(&qs[buf][r][o]) = qo;
          *reinterpret_cast<f32x4*>(&ks[buf][r][o]) = ko;
          if constexpr (MODE == CHAN_DECAY)
            *reinterpret_cast<f32x4*>(&ws[buf][r][o]) = wo;
          if (turn) {
            const int o2 = at(e + half + g * 4);
            *reinterpret_cast<f32x4*>(&qs[buf][r][o2]) = q2;
            *reinterpret_cast<f32x4*>(&ks[buf][r][o2]) = k2;
          }
        }
      }
      for (int i = tid; !norm && i < rows * (PB / 8); i += nthr) {
        const int r = i / (PB / 8), c = (i % (PB / 8)) * 8;
        u16x8 v8 = {0, 0, 0, 0, 0, 0, 0, 0};
        if (p0 + c < P)
          v8 = *reinterpret_cast<const u16x8*>(
              (const unsigned short*)p.v + (t0 + r) * p.ld_v + (long)h * P + p0 + c);
#pragma unroll
        for (int x = 0; x < 8; ++x) vs[buf][r][c + x] = bf2f(v8[x]);
      }
    } else {
      for (int i = tid; i < rows * N; i += nthr) {
        const int r = i / N, e = i % N;
        const long t = t0 + r;
        const TS* qp = (const TS*)p.q + t * p.ld_q + (long)h * N;
        const TS* kp = (const TS*)p.k + t * p.ld_k + (long)h * N;
        float q = ld(qp + e), k = ld(kp + e);
        if (e < 2 * half) {
          const bool lo = e < half;
          const int f = lo ? e : e - half, o = lo ? e + half : e - half;
          const float c = p.rot[t * 2 * half + f];
          const float sn = p.rot[(t * 2 + 1) * half + f] * (lo ? -1.f : 1.f);
          q = q * c + ld(qp + o) * sn;
          k = k * c + ld(kp + o) * sn;
        }
        qs[buf][r][at(e)] = q * p.q_scale;
        ks[buf][r][at(e)] = k * p.k_scale;
        if constexpr (MODE == CHAN_DECAY)
          ws[buf][r][at(e)] = expf(-expf(
              ld((const TS*)p.chan + t * p.ld_c + (long)h * N + e) + w0[e]));
      }
      for (int i = tid; !norm && i < rows * PB; i += nthr) {
        const int r = i / PB, c = i % PB;
        vs[buf][r][c] = p0 + c < P
            ? ld((const TS*)p.v + (t0 + r) * p.ld_v + (long)h * P + p0 + c) : 0.f;
      }
    }
    if constexpr (MODE == GATED) {
      if (tid < rows) {
        const float* g = p.ab + ((t0 + tid) * H + h) * 3;
        sc[buf][tid][0] = g[0];
        sc[buf][tid][1] = g[1];
        sc[buf][tid][2] = g[2];
      }
    }
  };

  const float a_const = MODE == CONST_DECAY ? p.decay[h] : 0.f;
  int buf = 0;
  for (int c0 = 0; c0 < sv.n; c0 += CH, buf ^= 1) {
    const int rows = min(CH, sv.n - c0);
    stage(buf, c0);
    __syncthreads();
    if constexpr (MODE == CHAN_DECAY) {
      // sum_n q u k of every row, eight lanes a row
      const int l = tid & 7;
      for (int r = tid >> 3; r < CH; r += nthr >> 3) {
        float d = 0.f;
        if (r < rows)
          for (int e = l; e < N; e += 8) {
            const int o = at(e);
            d += qs[buf][r][o] * ub[e] * ks[buf][r][o];
          }
        d = lanes_sum<8>(d);
        if (l == 0) sc[buf][r][3] = d;
      }
      __syncthreads();
    }
    const float* kb = &ks[buf][0][ns * NS];
    const float* qb = &qs[buf][0][ns * NS];
    const float* wb = &ws[buf][0][MODE == CHAN_DECAY ? ns * NS : 0];
    auto fetch = [&](int r, RowOps<MODE, NR>& o) {
#pragma unroll
      for (int j = 0; j < NR / 4; ++j) {
        o.k[j] = *reinterpret_cast<const f32x4*>(kb + r * ROW + j * 4);
        o.q[j] = *reinterpret_cast<const f32x4*>(qb + r * ROW + j * 4);
        if constexpr (MODE == CHAN_DECAY)
          o.w[j] = *reinterpret_cast<const f32x4*>(wb + r * ROW + j * 4);
      }
#pragma unroll
      for (int c = 0; c < VC; ++c) o.v[c] = vs[buf][r][pl + c];
      o.a = MODE == GATED ? sc[buf][r][0] : a_const;
      o.b = MODE == GATED ? sc[buf][r][1] : 1.f;
    };
    // a lane keeps the sums of one row in TPP and stores them together
    float out[VC];
#pragma unroll
    for (int c = 0; c < VC; ++c) out[c] = 0.f;
    auto work = [&](int r, const RowOps<MODE, NR>& o) {
      float acc[VC], bv[VC];
#pragma unroll
      for (int c = 0; c < VC; ++c) {
        acc[c] = 0.f;
        bv[c] = MODE == GATED ? o.b * o.v[c] : o.v[c];
      }
#pragma unroll
      for (int j = 0; j < NR / 4; ++j)
#pragma unroll
        for (int x = 0; x < 4; ++x)
#pragma unroll
          for (int c = 0; c < VC; ++c) {
            float& st = S[c][j * 4 + x];
            if constexpr (MODE == CHAN_DECAY) {
              acc[c] += st * o.q[j][x];
              st = o.w[j][x] * st + o.k[j][x] * bv[c];
            } else {
              st = o.a * st + o.k[j][x] * bv[c];
              acc[c] += st * o.q[j][x];
            }
          }
      const bool mine = (r & (TPP - 1)) == ns;
#pragma unroll
      for (int c = 0; c < VC; ++c) {
        acc[c] = lanes_sum<TPP>(acc[c]);
        out[c] = mine ? acc[c] : out[c];
      }
      if ((r & (TPP - 1)) == TPP - 1 || r == rows - 1) {
        const int rf = (r & ~(TPP - 1)) + ns;
        if (rf <= r) {
          const long t = sv.first + c0 + rf;
          if (norm) {
            if (pc == 0)
              p.rden[t * H + h] =
                  1.0f / (fmaxf(fabsf(out[0]), sc[buf][rf][2]) + 1e-6f);
          } else {
            float* yo = y + t * H * P + (long)h * P + pc;
#pragma unroll
            for (int c = 0; c < VC; ++c) {
              float o2 = out[c];
              if constexpr (MODE == CHAN_DECAY)
                o2 += vs[buf][rf][pl + c] * sc[buf][rf][3];
              if (pc + c < P) yo[c] = o2;
            }
          }
        }
      }
    };
    if constexpr (NR <= 16) {
      RowOps<MODE, NR> o0, o1;
      fetch(0, o0);
      for (int r = 0; r < rows; r += 2) {
        fetch(min(r + 1, CH - 1), o1);
        work(r, o0);
        if (r + 1 < rows) {
          fetch(min(r + 2, CH - 1), o0);
          work(r + 1, o1);
        }
      }
    } else {
      RowOps<MODE, NR> o0;
      for (int r = 0; r < rows; ++r) {
        fetch(r, o0);
        work(r, o0);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const int nn = ns * NR + j;
#pragma unroll
    for (int c = 0; c < VC; ++c)
      if (nn < N && pc + c < P) sp[(long)nn * P + pc + c] = S[c][j];
  }
}

// ---- single rows (decode) -----------------------------------------------------

DEVICE_INLINE float block_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

// grid (nseq, H), P % 4 == 0 and P <= 1024: a lane owns 4 neighbouring value
// channels of every RP-th state row. More rows of a sequence, should a batch
// bring them, are walked one after the other.
template <typename TS, int MODE>
__global__ __launch_bounds__(256) void memory_step_kernel(
    float* __restrict__ y, MemArgs p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int N = p.N, P = p.P, P4 = P / 4, RP = 256 / P4, H = p.H;
  float* vs = sm;                 // [P]
  float* part = vs + P;           // [RP][P]
  float* ks = part + RP * P;      // [N]
  float* qs = ks + N;             // [N]
  float* ws = qs + N;             // [N] with CHAN_DECAY
  __shared__ float red[4];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const SeqView sv = view_of(p, s);
  if (!sv.ok) return;
  const int cg = tid % P4, r0 = tid / P4, half = p.half;
  float* sp = p.state + (sv.slot * H + h) * (long)N * P;
  float* ex = MODE == GATED ? p.extra + (sv.slot * H + h) * (long)(N + 1) : nullptr;
  for (int r = 0; r < sv.n; ++r) {
    const long t = sv.first + r;
    const bool fresh = !sv.has && r == 0;        // start from zero
    __syncthreads();
    // the first touch of the state does not wait for the row
    f32x4 S0 = {0.f, 0.f, 0.f, 0.f};
    if (r0 < RP && r0 < N && !fresh)
      S0 = *reinterpret_cast<const f32x4*>(sp + (long)r0 * P + cg * 4);
    float a = 1.f, b = 1.f, m = 0.f;
    if constexpr (MODE == CONST_DECAY) a = p.decay[h];
    if constexpr (MODE == GATED) {
      const TS* g = (const TS*)p.gates + t * p.ld_g + h;
      const float gi = capped(ld(g) + p.i_b[h], p.cap);
      const float gf = log_sigmoid_f(capped(ld(g + H) + p.f_b[h], p.cap));
      const float m_old = fresh ? 0.f : ex[N];
      m = fmaxf(gf + m_old, gi);
      a = expf(gf + m_old - m);
      b = expf(gi - m);
    }
    const TS* qp = (const TS*)p.q + t * p.ld_q + (long)h * N;
    const TS* kp = (const TS*)p.k + t * p.ld_k + (long)h * N;
    float dot = 0.f;
    for (int e = tid; e < N; e += 256) {
      float q = ld(qp + e), k = ld(kp + e);
      if (e < 2 * half) {
        const bool lo = e < half;
        const int f = lo ? e : e - half, o = lo ? e + half : e - half;
        float sn, c;
        sincosf((float)p.pos32[t] * p.inv_freq[f], &sn, &c);
        if (lo) sn = -sn;
        q = q * c + ld(qp + o) * sn;
        k = k * c + ld(kp + o) * sn;
      }
      q *= p.q_scale;
      k *= p.k_scale;
      qs[e] = q;
      ks[e] = k;
      if constexpr (MODE == CHAN_DECAY) {
        ws[e] = expf(-expf(ld((const TS*)p.chan + t * p.ld_c + (long)h * N + e)
                           + p.w0[(long)h * N + e]));
        dot += q * p.u[(long)h * N + e] * k;
      }
      if constexpr (MODE == GATED) {
        const float n = a * (fresh ? 0.f : ex[e]) + b * k;
        ex[e] = n;
        dot += n * q;
      }
    }
    for (int e = tid; e < P; e += 256)
      vs[e] = ld((const TS*)p.v + t * p.ld_v + (long)h * P + e);
    float total = 0.f;
    if constexpr (MODE == CONST_DECAY) __syncthreads();
    else total = block_sum(dot, red);
    if constexpr (MODE == GATED) {
      // every lane has read the old maximum before the sum's barriers
      if (tid == 0) ex[N] = m;
    }
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (r0 < RP) {
      const f32x4 v4 = *reinterpret_cast<const f32x4*>(vs + cg * 4);
      for (int nn = r0; nn < N; nn += RP) {
        f32x4* sa = reinterpret_cast<f32x4*>(sp + (long)nn * P + cg * 4);
        f32x4 S = nn == r0 ? S0 : fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *sa;
        const float q = qs[nn], k = MODE == GATED ? b * ks[nn] : ks[nn];
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          if constexpr (MODE == CHAN_DECAY) {
            acc[x] += S[x] * q;
            S[x] = ws[nn] * S[x] + k * v4[x];
          } else {
            S[x] = a * S[x] + k * v4[x];
            acc[x] += S[x] * q;
          }
        }
        *sa = S;
      }
      *reinterpret_cast<f32x4*>(part + r0 * P + cg * 4) = acc;
    }
    __syncthreads();
    if (MODE == GATED && tid == 0)
      p.rden[t * H + h] = 1.0f / (fmaxf(fabsf(total), expf(-m)) + 1e-6f);
    for (int e = tid; e < P; e += 256) {
      float o = MODE == CHAN_DECAY ? total * vs[e] : 0.f;
      const int nr = min(RP, N);
      for (int x = 0; x < nr; ++x) o += part[x * P + e];
      y[t * H * P + (long)h * P + e] = o;
    }
  }
}

template <typename TS, int MODE, int NR, int TPP>
void scan_go(float* y, const MemArgs& p, int nseq, hipStream_t s) {
  const int per_wave = 64 / TPP * VC;
  const int waves = min(4, (p.P + per_wave - 1) / per_wave);
  const int pb = waves * per_wave;
  memory_scan_kernel<TS, MODE, NR, TPP>
      <<<dim3(nseq, p.H, (p.P + pb - 1) / pb + (MODE == GATED ? 1 : 0)),
         waves * 64, 0, s>>>(y, p);
}

template <typename TS, int MODE>
int scan_pick(float* y, const MemArgs& p, int nseq, hipStream_t s) {
  // lanes per channel pair: 16 where the batch would leave SIMDs without a
  // wave, or the state needs them
  const long waves = (long)nseq * p.H * ((p.P + 15) / 16);
  const bool wide = p.N > 256 || (p.N >= 64 && waves < 1024);
#define MEM_CASE(NRV, TPPV) \
  if (p.N <= NRV * TPPV) { scan_go<TS, MODE, NRV, TPPV>(y, p, nseq, s); return 1; }
  if (!wide) {
    MEM_CASE(4, 8) MEM_CASE(8, 8) MEM_CASE(16, 8) MEM_CASE(32, 8)
  }
  MEM_CASE(4, 16) MEM_CASE(8, 16) MEM_CASE(16, 16) MEM_CASE(32, 16)
#undef MEM_CASE
  return 0;
}

template <typename TS, int MODE>
int mem_run(float* y, const MemArgs& p, int nseq, int single, hipStream_t s) {
  const int P4 = p.P / 4;
  if (single && p.P % 4 == 0 && P4 <= 256) {
    const size_t smem = (size_t)(3 * p.N + p.P + (256 / P4) * p.P) * sizeof(float);
    memory_step_kernel<TS, MODE><<<dim3(nseq, p.H), 256, smem, s>>>(y, p);
    return 1;
  }
  if constexpr (MODE == GATED)
    memory_gates_kernel<TS><<<dim3(nseq, p.H), 64, 0, s>>>(p);
  return scan_pick<TS, MODE>(y, p, nseq, s);
}

template <typename TS>
int mem_mode(float* y, const MemArgs& p, int mode, int nseq, int single,
             hipStream_t s) {
  switch (mode) {
    case CONST_DECAY: return mem_run<TS, CONST_DECAY>(y, p, nseq, single, s);
    case CHAN_DECAY: return mem_run<TS, CHAN_DECAY>(y, p, nseq, single, s);
    default: return mem_run<TS, GATED>(y, p, nseq, single, s);
  }
}

}  // namespace

int memory_scan_max_state() { return 512; }

// the caller needs the gates' workspace (ab) unless the step kernel runs
int memory_scan_steps(int P, int single) {
  return single && P % 4 == 0 && P / 4 <= 256;
}

void rope_table_launch(float* out, const int* pos32, const float* inv_freq,
                       int T, int half, hipStream_t s) {
  if (T <= 0 || half <= 0) return;
  rope_table_kernel<<<T, 64, 0, s>>>(out, pos32, inv_freq, half);
}

int memory_scan_launch(
    float* y, const void* q, long ld_q, const void* k, long ld_k,
    const void* v, long ld_v, float q_scale, float k_scale, int H, int N, int P,
    int mode, const float* decay, const void* chan, long ld_c, const float* w0,
    const float* u, const float* rot, const float* inv_freq, int half,
    const void* gates, long ld_g, const float* i_b, const float* f_b, float cap,
    float* ab, float* rden, float* state, float* extra, const int* seq_first,
    const int* seq_rows, const int* slots, const int* pos32, int nseq,
    int nslots, int T, int bf, int single, hipStream_t s) {
  if (T <= 0 || nseq <= 0) return 1;
  MemArgs p;
  p.q = q; p.k = k; p.v = v; p.ld_q = ld_q; p.ld_k = ld_k; p.ld_v = ld_v;
  p.q_scale = q_scale; p.k_scale = k_scale; p.H = H; p.N = N; p.P = P;
  p.decay = decay; p.chan = chan; p.ld_c = ld_c; p.w0 = w0; p.u = u;
  p.rot = rot; p.inv_freq = inv_freq; p.half = half; p.gates = gates;
  p.ld_g = ld_g; p.i_b = i_b; p.f_b = f_b; p.cap = cap; p.ab = ab;
  p.rden = rden; p.state = state; p.extra = extra; p.seq_first = seq_first;
  p.seq_rows = seq_rows; p.slots = slots; p.pos32 = pos32; p.nslots = nslots;
  p.T = T;
  auto al = [](const void* x, long ldx) {
    return (uintptr_t)x % 16 == 0 && ldx % 8 == 0;
  };
  p.vec = bf && N % 8 == 0 && P % 8 == 0 && half % 8 == 0 && al(q, ld_q) &&
          al(k, ld_k) && al(v, ld_v) && (chan == nullptr || al(chan, ld_c)) &&
          (uintptr_t)rot % 16 == 0;
  return bf ? mem_mode<unsigned short>(y, p, mode, nseq, single, s)
            : mem_mode<float>(y, p, mode, nseq, single, s);
}
