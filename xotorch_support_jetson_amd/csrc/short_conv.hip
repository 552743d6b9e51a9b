// Stages in front of the recurrences and convolved attention of bias-free layer-norm sandwich blocks (gfx950):
//
//   conv_prep          causal convolutions over time, per channel; then per unit of channels (a head, or a piece of a run)
//                      SiLU and a unit length or a weighted RMS norm; the per-request state of last inputs
//   recurrence_gates   step sizes, low-rank channel decays and low-rank output gates of the channel-decay delta rule
//   ssd_steps          step sizes and decays of an SSD mixer
//
// P is a fused projection's fp32 output [T, ldp]; "column offset" arguments address its slices.  Everything here is fp32.
#include "mixer_util.h"

namespace xot {
namespace {
using namespace mix;

constexpr int CONV_SILU = 1, CONV_UNIT = 2, CONV_UNIT_SCALED = 4, CONV_RMS = 8, CONV_MAX = 256;  // ops.reference.conv_units
constexpr int CTB = 8;  // tokens whose inputs are in flight together (runs of tokens)

// A wave per (run of tokens, unit): lane l holds the unit's channels VW l .. VW l + VW - 1, the filter, and the last TAPS - 1
// inputs, which slide along the run (at the start of a run or a sequence they come from P or the sequence's state).  TAPS 0:
// any filter length, taps read from memory again for every token.  SINGLE: every sequence has one new token, whose wave also
// writes the state (else conv_tail_k does, after every token has read it).
struct ConvArgs {
  const float* P;  // [S][T][ldp], slabs ss apart
  int ldp, S;
  int64_t ss;
  int x_off;
  const float *conv_w, *conv_b;
  int taps, C;
  const int* units;
  int NU;
  const float* norm_w;
  int norm_n;
  float* conv_state;
  const int *state_slots, *cu;
  int B, T, run;
  float eps;
  float* out;
};

template <int TAPS, int VW, bool SINGLE>
__device__ __forceinline__ void conv_body(const ConvArgs& A, int bx, int by) {
  const float* __restrict__ P = A.P;
  const float* __restrict__ conv_w = A.conv_w;
  const float* __restrict__ conv_b = A.conv_b;
  const float* __restrict__ norm_w = A.norm_w;
  const int* __restrict__ units = A.units;
  const int* __restrict__ state_slots = A.state_slots;
  const int* __restrict__ cu = A.cu;
  float* __restrict__ conv_state = A.conv_state;
  float* __restrict__ out = A.out;
  const int ldp = A.ldp, S = A.S, x_off = A.x_off, taps_rt = A.taps, C = A.C, NU = A.NU, norm_n = A.norm_n, B = A.B, T = A.T, run = SINGLE ? 1 : A.run;
  constexpr int NT = SINGLE ? 1 : CTB;  // tokens whose inputs are in flight together
  const int64_t ss = A.ss;
  const float eps = A.eps;
  const int unit = by * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (unit >= NU) return;  // (wave-uniform; no workgroup barrier below)
  const int taps = TAPS ? TAPS : taps_rt;
  const int c0 = min(max(units[4 * unit], 0), C), n = min(min(max(units[4 * unit + 1], 0), 64 * VW), C - c0);
  if (n <= 0) return;
  const int kind = units[4 * unit + 2], nw = units[4 * unit + 3];
  const bool rms = (kind & CONV_RMS) && norm_w && nw >= 0 && nw + n <= norm_n;
  const int l0 = lane * VW;
  constexpr int TW = TAPS ? TAPS : 1;
  float w[TW][VW], bias[VW], g[VW];
  bool in[VW];
#pragma unroll
  for (int e = 0; e < VW; ++e) {
    in[e] = l0 + e < n;
    const int c = c0 + (in[e] ? l0 + e : 0);
    bias[e] = conv_b && in[e] ? conv_b[c] : 0.0f;
    g[e] = rms && in[e] ? norm_w[nw + l0 + e] : 1.0f;
    if constexpr (TAPS == 4) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(conv_w + (int64_t)c * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) w[j][e] = in[e] ? a[j] : 0.0f;
    } else {
#pragma unroll
      for (int j = 0; j < TAPS; ++j) w[j][e] = in[e] ? conv_w[(int64_t)c * TAPS + j] : 0.0f;
    }
  }
  // vector loads where every row of the unit starts on a boundary and the unit is whole vectors
  const bool vec = VW > 1 && (ldp % VW == 0) && (ss % VW == 0) && ((x_off + c0) % VW == 0) && (C % VW == 0) && (c0 % VW == 0) && (n % VW == 0);
  auto ldv = [&](const float* p, float* v) {  // p: the unit's first channel of a row
    if (vec) {
      if constexpr (VW == 4) {
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        if (in[0]) x = *reinterpret_cast<const f32x4*>(p + l0);
        v[0] = x[0]; v[1] = x[1]; v[2] = x[2]; v[3] = x[3];
      } else if constexpr (VW == 2) {
        typedef float f32x2_c __attribute__((ext_vector_type(2)));
        f32x2_c x = {0.f, 0.f};
        if (in[0]) x = *reinterpret_cast<const f32x2_c*>(p + l0);
        v[0] = x[0]; v[1] = x[1];
      }
    } else {
#pragma unroll
      for (int e = 0; e < VW; ++e) v[e] = in[e] ? p[l0 + e] : 0.0f;
    }
  };
  auto stv = [&](float* p, const float* v) {
    if (vec) {
      if (!in[0]) return;
      if constexpr (VW == 4) {
        *reinterpret_cast<f32x4*>(p + l0) = f32x4{v[0], v[1], v[2], v[3]};
      } else if constexpr (VW == 2) {
        typedef float f32x2_c __attribute__((ext_vector_type(2)));
        *reinterpret_cast<f32x2_c*>(p + l0) = f32x2_c{v[0], v[1]};
      }
    } else {
#pragma unroll
      for (int e = 0; e < VW; ++e)
        if (in[e]) p[l0 + e] = v[e];
    }
  };

  // a row of P, which may still be S split-K slabs
  auto ldp_row = [&](const float* p, float* v) {
    if (S == 1) {
      ldv(p, v);
      return;
    }
#pragma unroll
    for (int e = 0; e < VW; ++e) v[e] = 0.0f;
    for (int k0 = 0; k0 < S; k0 += 8) {  // (eight slabs in flight; those past the last repeat it, unused)
      float a[8][VW];
#pragma unroll
      for (int k = 0; k < 8; ++k) ldv(p + min(k0 + k, S - 1) * ss, a[k]);
#pragma unroll
      for (int k = 0; k < 8; ++k)
#pragma unroll
        for (int e = 0; e < VW; ++e) v[e] += k0 + k < S ? a[k][e] : 0.0f;
    }
  };

  const int t0 = bx * run, t1 = min(T, t0 + run);
  int b = SINGLE ? t0 : seq_of(cu, B, t0), slot = state_slots[b], tstart = cu[b], tend = cu[b + 1];
  // input of the sequence's token `local` (negative: before this step) for the unit's channels
  auto input = [&](int local, float* v) {
    if (local >= 0) {
      ldp_row(P + (int64_t)(tstart + local) * ldp + x_off + c0, v);
    } else if (slot >= 0) {
      ldv(conv_state + ((int64_t)slot * (taps - 1) + (taps - 1 + local)) * C + c0, v);
    } else {
#pragma unroll
      for (int e = 0; e < VW; ++e) v[e] = 0.0f;
    }
  };
  constexpr int HN = TAPS > 1 ? TAPS - 1 : 1;
  float hist[HN][VW];
  bool fresh = true;
  for (int tb = t0; tb < t1; tb += NT) {
    const int nt = min(NT, t1 - tb);
    float x[NT][VW], y[NT][VW];
    bool ok[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) ldp_row(P + (int64_t)(tb + min(i, nt - 1)) * ldp + x_off + c0, x[i]);
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      ok[i] = false;
      if (i >= nt) continue;
      const int t = tb + i;
      while (!SINGLE && t >= tend && b + 1 < B) {  // (sequences without new tokens are passed over)
        ++b;
        slot = state_slots[b];
        tstart = cu[b];
        tend = cu[b + 1];
        fresh = true;
      }
      ok[i] = slot >= 0;
      const int local = t - tstart;
      if (TAPS > 1 && fresh) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) input(local - (TAPS - 1) + j, hist[j]);
        fresh = false;
      }
#pragma unroll
      for (int e = 0; e < VW; ++e) y[i][e] = bias[e];
      if (TAPS) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
          for (int e = 0; e < VW; ++e) y[i][e] += w[j][e] * hist[j][e];
#pragma unroll
        for (int e = 0; e < VW; ++e) y[i][e] += w[TW - 1][e] * x[i][e];
#pragma unroll
        for (int j = 0; j + 1 < TAPS - 1; ++j)
#pragma unroll
          for (int e = 0; e < VW; ++e) hist[j][e] = hist[j + 1][e];
        if (TAPS > 1) {
#pragma unroll
          for (int e = 0; e < VW; ++e) hist[HN - 1][e] = x[i][e];
        }
      } else {
        for (int j = 0; j < taps; ++j) {
          float v[VW];
          input(local - (taps - 1) + j, v);
#pragma unroll
          for (int e = 0; e < VW; ++e)
            if (in[e]) y[i][e] += conv_w[(int64_t)(c0 + l0 + e) * taps + j] * v[e];
        }
      }
      if (kind & CONV_SILU) {
#pragma unroll
        for (int e = 0; e < VW; ++e) y[i][e] = siluf_(y[i][e]);
      }
    }
    if (kind & ~CONV_SILU) {
      float s[NT];
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        s[i] = 0.0f;
#pragma unroll
        for (int e = 0; e < VW; ++e) s[i] += ok[i] && in[e] ? y[i][e] * y[i][e] : 0.0f;
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1)
#pragma unroll
        for (int i = 0; i < NT; ++i) s[i] += __shfl_xor(s[i], o, 64);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const float k = kind & CONV_RMS ? 1.0f / sqrtf(s[i] / (float)n + eps)
                                        : 1.0f / sqrtf(s[i] + 1e-6f) * (kind & CONV_UNIT_SCALED ? 1.0f / sqrtf((float)n) : 1.0f);
#pragma unroll
        for (int e = 0; e < VW; ++e) y[i][e] *= k * g[e];
      }
    }
#pragma unroll
    for (int i = 0; i < NT; ++i)
      if (ok[i]) stv(out + (int64_t)(tb + i) * C + c0, y[i]);
    if (SINGLE && ok[0]) {  // (run 1: the inputs after this token are the next step's history)
      float* st = conv_state + (int64_t)slot * (taps - 1) * C + c0;
      if (TAPS) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) stv(st + (int64_t)j * C, hist[j]);
      } else {
        for (int j = 0; j + 1 < taps - 1; ++j) {
          float v[VW];
          ldv(st + (int64_t)(j + 1) * C, v);
          stv(st + (int64_t)j * C, v);
        }
        if (taps > 1) stv(st + (int64_t)(taps - 2) * C, x[0]);
      }
    }
  }
}

template <int TAPS, int VW, bool SINGLE>
__global__ __launch_bounds__(256) void conv_prep_k(ConvArgs a) {
  conv_body<TAPS, VW, SINGLE>(a, blockIdx.x, blockIdx.y);
}

// the last taps - 1 inputs of every sequence -> its state slot
__global__ void conv_tail_k(const float* __restrict__ P, int ldp, int S, int64_t ss, int x_off, int C, int taps,
                            float* __restrict__ conv_state,
                            const int* __restrict__ state_slots, const int* __restrict__ cu) {
  const int b = blockIdx.x;
  const int slot = state_slots[b], n = cu[b + 1] - cu[b];
  if (slot < 0 || n <= 0) return;
  float* st = conv_state + (int64_t)slot * (taps - 1) * C;
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < C; c += gridDim.y * blockDim.x)
    for (int i = 0; i < taps - 1; ++i) {  // ascending: entry i takes the old entry i + n (> i) or a token of this step
      const int s = n - (taps - 1) + i;
      st[(int64_t)i * C + c] = s >= 0 ? slab1(P + (int64_t)(cu[b] + s) * ldp + x_off + c, S, ss) : st[(int64_t)(i + n) * C + c];
    }
}

// ------------------------------------------------------------------ gates
// Workgroup = (GTOK tokens, job): job 0 the step sizes beta, then blocks of 64 decay channels, then blocks of 64 output-gate
// channels.  The tokens' rank rows lie in LDS; four neighbouring lanes share a channel, each sums a quarter of its weight row
// (in pieces of eight) for all the tokens.
constexpr int GTOK = 8;

struct GateArgs {
  const float* P;
  int ldp, S;
  int64_t ss;
  int T, b_off;
  float* beta;
  int H, a1_off;
  const void* a2;
  int ra;
  const float *dt_bias, *A_log;
  int d;
  float* decay;
  int g1_off;
  const void* g2;
  int rg, ng;
  float* gate;
};

template <typename WT>
__device__ __forceinline__ void gates_body(const GateArgs& A, int bx, int by, float* ys) {  // ys: LDS [GTOK][rank]
  const float* __restrict__ P = A.P;
  const WT* __restrict__ a2 = (const WT*)A.a2;
  const WT* __restrict__ g2 = (const WT*)A.g2;
  const float* __restrict__ dt_bias = A.dt_bias;
  const float* __restrict__ A_log = A.A_log;
  float* __restrict__ beta = A.beta;
  float* __restrict__ decay = A.decay;
  float* __restrict__ gate = A.gate;
  const int ldp = A.ldp, S = A.S, T = A.T, b_off = A.b_off, H = A.H, a1_off = A.a1_off, ra = A.ra, d = A.d, g1_off = A.g1_off,
            rg = A.rg, ng = A.ng;
  const int64_t ss = A.ss;
  const int t0 = bx * GTOK, nt = min(GTOK, T - t0), HD = H * d, nab = (HD + 63) / 64;
  int job = by;
  if (job == 0) {
    for (int e = threadIdx.x; e < nt * H; e += 256) {
      const int t = t0 + e / H, h = e % H;
      beta[(int64_t)t * H + h] = sigmoidf_(slab1(P + (int64_t)t * ldp + b_off + h, S, ss));
    }
    return;
  }
  --job;
  const bool dec = job < nab;
  const int part = threadIdx.x & 3, c = (dec ? job : job - nab) * 64 + (threadIdx.x >> 2), nc = dec ? HD : ng;
  const int rank = dec ? ra : rg, off = dec ? a1_off : g1_off;
  const WT* w = (dec ? a2 : g2) + (int64_t)min(c, nc - 1) * rank;
  const float rate = dec ? expf(A_log[min(c, nc - 1) / d]) : 0.0f, bias = dec ? dt_bias[min(c, nc - 1)] : 0.0f;
  // the first four pieces of the lane's weight row are on their way while the rank rows are summed
  const bool pieces = (rank & 7) == 0;
  float wv[4][8];
  if (pieces) {
#pragma unroll
    for (int k = 0; k < 4; ++k) ld8(w + min(8 * part + 32 * k, rank - 8), wv[k]);
  }
  // the rank rows: four elements a thread and eight slabs in flight at a time, without branches around the loads
  const int ne = GTOK * rank;
  for (int e0 = 0; e0 < ne; e0 += 1024) {
    const float* p[4];
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int e = min(e0 + (int)threadIdx.x + 256 * j, ne - 1), i = e / rank;
      p[j] = P + (int64_t)(t0 + min(i, nt - 1)) * ldp + off + e - i * rank;
      v[j] = 0.0f;
    }
    for (int k0 = 0; k0 < S; k0 += 8) {
      float a[8][4];
#pragma unroll
      for (int k = 0; k < 8; ++k)
#pragma unroll
        for (int j = 0; j < 4; ++j) a[k][j] = p[j][min(k0 + k, S - 1) * ss];
#pragma unroll
      for (int k = 0; k < 8; ++k)
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] += k0 + k < S ? a[k][j] : 0.0f;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int e = e0 + threadIdx.x + 256 * j;
      if (e < ne) ys[e] = v[j];
    }
  }
  __syncthreads();
  float z[GTOK];
#pragma unroll
  for (int i = 0; i < GTOK; ++i) z[i] = 0.0f;
  if (pieces) {
    auto add = [&](const float* v, int r) {
#pragma unroll
      for (int i = 0; i < GTOK; ++i) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(ys + i * rank + r), b = *reinterpret_cast<const f32x4*>(ys + i * rank + r + 4);
        z[i] += v[0] * a[0] + v[1] * a[1] + v[2] * a[2] + v[3] * a[3] + v[4] * b[0] + v[5] * b[1] + v[6] * b[2] + v[7] * b[3];
      }
    };
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (8 * part + 32 * k < rank) add(wv[k], 8 * part + 32 * k);
    for (int r = 8 * part + 128; r < rank; r += 32) {
      float v[8];
      ld8(w + r, v);
      add(v, r);
    }
  } else {
    for (int r = part; r < rank; r += 4) {
      const float v = ldf(w + r);
#pragma unroll
      for (int i = 0; i < GTOK; ++i) z[i] += v * ys[i * rank + r];
    }
  }
#pragma unroll
  for (int i = 0; i < GTOK; ++i) {
    z[i] += __shfl_xor(z[i], 1, 64);
    z[i] += __shfl_xor(z[i], 2, 64);
  }
  if (c >= nc) return;
#pragma unroll
  for (int i = 0; i < GTOK; ++i) {
    if (i >= nt || (i & 3) != part) continue;  // (the four lanes of a channel share the writes)
    if (dec) decay[(int64_t)(t0 + i) * HD + c] = expf(-rate * softplusf_(z[i] + bias));
    else gate[(int64_t)(t0 + i) * ng + c] = z[i];
  }
}

template <typename WT>
__global__ __launch_bounds__(256) void recurrence_gates_k(GateArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ys[];
  gates_body<WT>(a, blockIdx.x, blockIdx.y, ys);
}

// Decays from finished products za [T, >= HD] (prompts: a GEMM made them) and the step sizes; W channels a thread.
template <int W>
__global__ __launch_bounds__(256) void channel_decay_k(const float* __restrict__ P, int ldp, int S, int64_t ss, int T, int b_off,
                                                       float* __restrict__ beta, int H, const float* __restrict__ za, int ldz,
                                                       const float* __restrict__ dt_bias, const float* __restrict__ A_log, int d,
                                                       float* __restrict__ decay) {
  const int t0 = blockIdx.x * GTOK, nt = min(GTOK, T - t0), HD = H * d;
  if (blockIdx.y == 0) {
    for (int e = threadIdx.x; e < nt * H; e += 256) {
      const int t = t0 + e / H, h = e % H;
      beta[(int64_t)t * H + h] = sigmoidf_(slab1(P + (int64_t)t * ldp + b_off + h, S, ss));
    }
    return;
  }
  const int c = ((blockIdx.y - 1) * 256 + threadIdx.x) * W;
  if (c >= HD) return;  // (W > 1: HD is a multiple of W)
  float rate[W], bias[W], z[GTOK][W];
#pragma unroll
  for (int e = 0; e < W; ++e) {
    rate[e] = -expf(A_log[(c + e) / d]);
    bias[e] = dt_bias[c + e];
  }
#pragma unroll
  for (int i = 0; i < GTOK; ++i) {
    const float* p = za + (int64_t)(t0 + min(i, nt - 1)) * ldz + c;
    if constexpr (W == 4) *reinterpret_cast<f32x4*>(z[i]) = *reinterpret_cast<const f32x4*>(p);
    else z[i][0] = *p;
  }
#pragma unroll
  for (int i = 0; i < GTOK; ++i) {
    if (i >= nt) continue;
#pragma unroll
    for (int e = 0; e < W; ++e) z[i][e] = expf(rate[e] * softplusf_(z[i][e] + bias[e]));
    float* o = decay + (int64_t)(t0 + i) * HD + c;
    if constexpr (W == 4) *reinterpret_cast<f32x4*>(o) = *reinterpret_cast<f32x4*>(z[i]);
    else *o = z[i][0];
  }
}

struct StepArgs {
  const float* P;
  int ldp, S;
  int64_t ss;
  int dt_off;
  const float *dt_bias, *A_log;
  int H, total;
  float *dt, *decay;
};

__device__ __forceinline__ void steps_body(const StepArgs& a, int e) {
  if (e >= a.total) return;
  const int t = e / a.H, h = e - t * a.H;
  const float s = softplusf_(slab1(a.P + (int64_t)t * a.ldp + a.dt_off + h, a.S, a.ss) + a.dt_bias[h]);
  a.dt[e] = s;
  a.decay[e] = expf(-expf(a.A_log[h]) * s);
}

__global__ __launch_bounds__(256) void ssd_steps_k(StepArgs a) { steps_body(a, blockIdx.x * 256 + threadIdx.x); }

// Single-token steps: the gates (or step sizes) and the convolutions read the same projection and do not depend on each
// other, so one launch does both; the gates' workgroups, the longer ones, come first.
template <int TAPS, int VW, typename WT>
__global__ __launch_bounds__(256) void conv_gates_k(ConvArgs c, GateArgs g, StepArgs s, int n_gate, int gate_x, int n_step) {
  extern __shared__ __attribute__((aligned(16))) float ys[];
  int b = blockIdx.x;
  if (b < n_gate) {
    gates_body<WT>(g, b % gate_x, b / gate_x, ys);
    return;
  }
  b -= n_gate;
  if (b < n_step) {
    steps_body(s, b * 256 + threadIdx.x);
    return;
  }
  b -= n_step;
  conv_body<TAPS, VW, true>(c, b % c.T, b / c.T);
}

// ------------------------------------------------------------------ host side
using OptT = c10::optional<at::Tensor>;

ConvArgs conv_args(const at::Tensor& P, int64_t x_off, const at::Tensor& conv_w, const OptT& conv_b, const at::Tensor& units,
                   const OptT& norm_w, at::Tensor& conv_state, const at::Tensor& state_slots, const at::Tensor& cu_q, double eps,
                   at::Tensor& out, int64_t width) {
  const Slabs p = slabs_of(P, "P");
  const int64_t T = p.T, B = state_slots.numel();
  f32c(conv_w, "conv_w");
  f32c(conv_state, "conv_state");
  f32c(out, "out");
  i32c(units, "units");
  i32c(state_slots, "state_slots");
  i32c(cu_q, "cu_q");
  MCHECK(conv_w.dim() == 2 && units.dim() == 2 && units.size(1) == 4, "conv_w must be [C, taps], units [n, 4]");
  const int64_t C = conv_w.size(0), taps = conv_w.size(1);
  MCHECK(taps >= 1 && (taps == 1 || (conv_state.dim() == 3 && conv_state.size(1) == taps - 1 && conv_state.size(2) == C)),
         "conv_state must be [slots, taps - 1, C]");
  MCHECK(out.dim() == 2 && out.size(0) == T && out.size(1) == C && cu_q.numel() == B + 1, "conv_prep: shape mismatch");
  cols_ok(p, x_off, C, "conv inputs");
  MCHECK(width >= 1 && width <= CONV_MAX, "a unit holds at most ", CONV_MAX, " channels");
  ConvArgs a{};
  a.P = p.p;
  a.ldp = p.ld;
  a.S = p.S;
  a.ss = p.ss;
  a.x_off = (int)x_off;
  a.conv_w = conv_w.data_ptr<float>();
  if (conv_b.has_value()) {
    f32c(*conv_b, "conv_b");
    MCHECK(conv_b->numel() == C, "conv_b must hold a number per channel");
    a.conv_b = conv_b->data_ptr<float>();
  }
  a.taps = (int)taps;
  a.C = (int)C;
  a.units = units.data_ptr<int>();
  a.NU = (int)units.size(0);
  if (norm_w.has_value()) {
    f32c(*norm_w, "norm_w");
    a.norm_w = norm_w->data_ptr<float>();
    a.norm_n = (int)norm_w->numel();
  }
  // (units lie inside the C channels by construction, ops.reference.conv_units; the kernel clamps them all the same)
  a.conv_state = conv_state.data_ptr<float>();
  a.state_slots = state_slots.data_ptr<int>();
  a.cu = cu_q.data_ptr<int>();
  a.B = (int)B;
  a.T = (int)T;
  a.eps = (float)eps;
  a.out = out.data_ptr<float>();
  return a;
}

GateArgs gate_args(const Slabs& p, int64_t b_off, at::Tensor& beta, int64_t a1_off, const OptT& a2, const at::Tensor& dt_bias,
                   const at::Tensor& A_log, at::Tensor& decay, int64_t g1_off, const OptT& g2, const OptT& gate, bool* bf) {
  const int64_t T = p.T, H = A_log.numel(), HD = dt_bias.numel();
  f32c(beta, "beta");
  f32c(dt_bias, "dt_bias");
  f32c(A_log, "A_log");
  f32c(decay, "decay");
  MCHECK(H > 0 && HD % H == 0 && beta.numel() == T * H && decay.numel() == T * HD, "recurrence_gates: shape mismatch");
  cols_ok(p, b_off, H, "step sizes");
  auto second = [&](const OptT& w, int64_t off, int64_t rows, const char* what) {
    MCHECK(w.has_value() && w->is_cuda() && is_act(*w) && w->is_contiguous() && w->dim() == 2 && w->size(0) == rows, what,
           " must be contiguous [channels, rank]");
    cols_ok(p, off, w->size(1), what);
    MCHECK(w->size(1) >= 1 && w->size(1) <= 1024, what, ": rank above 1024");
    *bf = w->scalar_type() == at::kBFloat16;
    return w->size(1);
  };
  GateArgs a{};
  a.P = p.p;
  a.ldp = p.ld;
  a.S = p.S;
  a.ss = p.ss;
  a.T = (int)T;
  a.b_off = (int)b_off;
  a.beta = beta.data_ptr<float>();
  a.H = (int)H;
  a.a1_off = (int)a1_off;
  a.ra = (int)second(a2, a1_off, HD, "a2");
  a.a2 = a2->data_ptr();
  a.dt_bias = dt_bias.data_ptr<float>();
  a.A_log = A_log.data_ptr<float>();
  a.d = (int)(HD / H);
  a.decay = decay.data_ptr<float>();
  a.g1_off = (int)g1_off;
  if (gate.has_value()) {
    f32c(*gate, "gate");
    MCHECK(gate->dim() == 2 && gate->size(0) == T, "gate must be [T, channels]");
    const bool abf = *bf;
    a.ng = (int)gate->size(1);
    a.rg = (int)second(g2, g1_off, a.ng, "g2");
    MCHECK(abf == *bf, "a2 and g2 must have one dtype");
    a.g2 = g2->data_ptr();
    a.gate = gate->data_ptr<float>();
  }
  return a;
}
inline unsigned gate_jobs(const GateArgs& a) { return (unsigned)(1 + (a.H * a.d + 63) / 64 + (a.ng + 63) / 64); }
inline size_t gate_lds(const GateArgs& a) { return (size_t)GTOK * std::max(a.ra, a.rg) * sizeof(float); }

StepArgs step_args(const Slabs& p, int64_t dt_off, const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& dt, at::Tensor& decay) {
  const int64_t T = p.T, H = A_log.numel();
  f32c(dt_bias, "dt_bias");
  f32c(A_log, "A_log");
  f32c(dt, "dt");
  f32c(decay, "decay");
  MCHECK(dt_bias.numel() == H && dt.numel() == T * H && decay.numel() == T * H, "ssd_steps: shape mismatch");
  cols_ok(p, dt_off, H, "dt");
  StepArgs a{};
  a.P = p.p;
  a.ldp = p.ld;
  a.S = p.S;
  a.ss = p.ss;
  a.dt_off = (int)dt_off;
  a.dt_bias = dt_bias.data_ptr<float>();
  a.A_log = A_log.data_ptr<float>();
  a.H = (int)H;
  a.total = (int)(T * H);
  a.dt = dt.data_ptr<float>();
  a.decay = decay.data_ptr<float>();
  return a;
}

// GO(TAPS, VW) for the filter length and the unit width of a launch
#define CONV_PICK(GO)                     \
  switch (a.taps) {                       \
    case 1: CONV_WIDTH(GO, 1); break;     \
    case 2: CONV_WIDTH(GO, 2); break;     \
    case 3: CONV_WIDTH(GO, 3); break;     \
    case 4: CONV_WIDTH(GO, 4); break;     \
    default: CONV_WIDTH(GO, 0); break;    \
  }
#define CONV_WIDTH(GO, TAPS)      \
  if (width <= 64) GO(TAPS, 1);   \
  else if (width <= 128) GO(TAPS, 2); \
  else GO(TAPS, 4)

void conv_prep(const at::Tensor& P, int64_t x_off, const at::Tensor& conv_w, const OptT& conv_b, const at::Tensor& units,
               const OptT& norm_w, at::Tensor& conv_state, const at::Tensor& state_slots, const at::Tensor& cu_q, double eps,
               at::Tensor& out, int64_t max_qlen, int64_t width) {
  ConvArgs a = conv_args(P, x_off, conv_w, conv_b, units, norm_w, conv_state, state_slots, cu_q, eps, out, width);
  if (a.T == 0 || a.B == 0 || a.NU == 0) return;
  const bool single = max_qlen == 1 && a.T == a.B;
  a.run = single ? 1 : a.T >= 1024 ? 32 : CTB;
  const dim3 grid((unsigned)((a.T + a.run - 1) / a.run), (unsigned)((a.NU + 3) / 4));
#define CP_GO(TAPS, VW)                                                      \
  do {                                                                       \
    if (single) conv_prep_k<TAPS, VW, true><<<grid, 256, 0, stream()>>>(a);  \
    else conv_prep_k<TAPS, VW, false><<<grid, 256, 0, stream()>>>(a);        \
  } while (0)
  CONV_PICK(CP_GO)
#undef CP_GO
  if (a.taps > 1 && !single)
    conv_tail_k<<<dim3((unsigned)a.B, (unsigned)((a.C + 255) / 256)), 256, 0, stream()>>>(
        a.P, a.ldp, a.S, a.ss, a.x_off, a.C, a.taps, a.conv_state, a.state_slots, a.cu);
}

// A step of single tokens (T == B): conv_prep together with recurrence_gates (beta given) or ssd_steps (dt given).
void conv_prep_gates(const at::Tensor& P, int64_t x_off, const at::Tensor& conv_w, const OptT& conv_b, const at::Tensor& units,
                     const OptT& norm_w, at::Tensor& conv_state, const at::Tensor& state_slots, const at::Tensor& cu_q, double eps,
                     at::Tensor& out, int64_t width, int64_t b_off, const OptT& beta, int64_t a1_off, const OptT& a2,
                     const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& decay, int64_t g1_off, const OptT& g2,
                     const OptT& gate, int64_t dt_off, const OptT& dt) {
  ConvArgs a = conv_args(P, x_off, conv_w, conv_b, units, norm_w, conv_state, state_slots, cu_q, eps, out, width);
  MCHECK(a.T == a.B, "conv_prep_gates: every sequence has one new token");
  MCHECK(beta.has_value() != dt.has_value(), "conv_prep_gates: either the delta rule's gates or the step sizes");
  if (a.T == 0 || a.NU == 0) return;
  a.run = 1;
  const Slabs p = slabs_of(P, "P");
  GateArgs g{};
  StepArgs s{};
  bool bf = false;
  int n_gate = 0, gate_x = 1, n_step = 0;
  size_t lds = 0;
  if (beta.has_value()) {
    at::Tensor bt = *beta;
    g = gate_args(p, b_off, bt, a1_off, a2, dt_bias, A_log, decay, g1_off, g2, gate, &bf);
    gate_x = (a.T + GTOK - 1) / GTOK;
    n_gate = gate_x * (int)gate_jobs(g);
    lds = gate_lds(g);
  } else {
    at::Tensor d = *dt;
    s = step_args(p, dt_off, dt_bias, A_log, d, decay);
    n_step = (s.total + 255) / 256;
  }
  const unsigned grid = (unsigned)(n_gate + n_step + a.T * ((a.NU + 3) / 4));
#define CG_GO(TAPS, VW)                                                                                              \
  do {                                                                                                               \
    if (bf) conv_gates_k<TAPS, VW, uint16_t><<<grid, 256, lds, stream()>>>(a, g, s, n_gate, gate_x, n_step);         \
    else conv_gates_k<TAPS, VW, float><<<grid, 256, lds, stream()>>>(a, g, s, n_gate, gate_x, n_step);               \
  } while (0)
  CONV_PICK(CG_GO)
#undef CG_GO
}
#undef CONV_PICK
#undef CONV_WIDTH

void recurrence_gates(const at::Tensor& P, int64_t b_off, at::Tensor& beta, int64_t a1_off, const OptT& a2,
                      const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& decay, int64_t g1_off, const OptT& g2,
                      const OptT& gate, const OptT& za) {
  const Slabs p = slabs_of(P, "P");
  const int64_t T = p.T, H = A_log.numel(), HD = dt_bias.numel();
  if (T == 0) return;
  if (za.has_value()) {
    f32c(beta, "beta");
    f32c(dt_bias, "dt_bias");
    f32c(A_log, "A_log");
    f32c(decay, "decay");
    MCHECK(H > 0 && HD % H == 0 && beta.numel() == T * H && decay.numel() == T * HD, "recurrence_gates: shape mismatch");
    cols_ok(p, b_off, H, "step sizes");
    const int ldz = ld_of(*za, "za");
    MCHECK(za->size(0) == T && za->size(1) >= HD && !gate.has_value(), "za must be [T, >= H d], and the gate made with it");
    const int64_t d = HD / H;
    const bool vec = HD % 4 == 0 && ldz % 4 == 0 && (reinterpret_cast<uintptr_t>(za->data_ptr()) & 15) == 0 &&
                     (reinterpret_cast<uintptr_t>(decay.data_ptr()) & 15) == 0;
    const int64_t per = vec ? 1024 : 256;
    const dim3 grid((unsigned)((T + GTOK - 1) / GTOK), (unsigned)(1 + (HD + per - 1) / per));
#define CD_GO(W)                                                                                                             \
  channel_decay_k<W><<<grid, 256, 0, stream()>>>(p.p, p.ld, p.S, p.ss, (int)T, (int)b_off, beta.data_ptr<float>(), (int)H,   \
                                                 za->data_ptr<float>(), ldz, dt_bias.data_ptr<float>(),                      \
                                                 A_log.data_ptr<float>(), (int)d, decay.data_ptr<float>())
    if (vec) CD_GO(4);
    else CD_GO(1);
#undef CD_GO
    return;
  }
  bool bf = false;
  const GateArgs a = gate_args(p, b_off, beta, a1_off, a2, dt_bias, A_log, decay, g1_off, g2, gate, &bf);
  const dim3 grid((unsigned)((T + GTOK - 1) / GTOK), gate_jobs(a));
  if (bf) recurrence_gates_k<uint16_t><<<grid, 256, gate_lds(a), stream()>>>(a);
  else recurrence_gates_k<float><<<grid, 256, gate_lds(a), stream()>>>(a);
}

void ssd_steps(const at::Tensor& P, int64_t dt_off, const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& dt,
               at::Tensor& decay) {
  const Slabs p = slabs_of(P, "P");
  if (p.T == 0) return;
  const StepArgs a = step_args(p, dt_off, dt_bias, A_log, dt, decay);
  ssd_steps_k<<<(unsigned)((a.total + 255) / 256), 256, 0, stream()>>>(a);
}

}  // namespace

void bind_short_conv(pybind11::module& m) {
  m.def("conv_prep", &conv_prep);
  m.def("conv_prep_gates", &conv_prep_gates);
  m.def("recurrence_gates", &recurrence_gates);
  m.def("ssd_steps", &ssd_steps);
}

}  // namespace xot
