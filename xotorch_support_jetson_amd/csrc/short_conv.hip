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
constexpr int CTB = 8;  // tokens whose inputs are in flight together

// A wave per (run of tokens, unit): lane l holds the unit's channels VW l .. VW l + VW - 1, the filter, and the last TAPS - 1
// inputs, which slide along the run (at the start of a run or a sequence they come from P or the sequence's state).  TAPS 0:
// any filter length, taps read from memory again for every token.  single: every sequence has one new token, whose wave also
// writes the state (else conv_tail_k does, after every token has read it).
template <int TAPS, int VW>
__global__ __launch_bounds__(256) void conv_prep_k(const float* __restrict__ P, int ldp, int S, int64_t ss, int x_off,
                                                   const float* __restrict__ conv_w,
                                                   const float* __restrict__ conv_b, int taps_rt, int C,
                                                   const int* __restrict__ units, int NU, const float* __restrict__ norm_w,
                                                   int norm_n, float* __restrict__ conv_state,
                                                   const int* __restrict__ state_slots, const int* __restrict__ cu, int B, int T,
                                                   int run, int single, float eps, float* __restrict__ out) {
  const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (unit >= NU) return;  // (wave-uniform; no workgroup barrier below)
  const int taps = TAPS ? TAPS : taps_rt;
  const int c0 = min(max(units[4 * unit], 0), C), n = min(min(max(units[4 * unit + 1], 0), 64 * VW), C - c0);
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
    ldv(p, v);
    for (int k0 = 1; k0 < S; k0 += 4) {  // (four slabs in flight; those past the last repeat it, unused)
      float a[4][VW];
#pragma unroll
      for (int k = 0; k < 4; ++k) ldv(p + min(k0 + k, S - 1) * ss, a[k]);
#pragma unroll
      for (int k = 0; k < 4; ++k)
#pragma unroll
        for (int e = 0; e < VW; ++e) v[e] += k0 + k < S ? a[k][e] : 0.0f;
    }
  };

  const int t0 = blockIdx.x * run, t1 = min(T, t0 + run);
  int b = single ? t0 : seq_of(cu, B, t0), slot = state_slots[b], tstart = cu[b], tend = cu[b + 1];
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
  for (int tb = t0; tb < t1; tb += CTB) {
    const int nt = min(CTB, t1 - tb);
    float x[CTB][VW], y[CTB][VW];
    bool ok[CTB];
#pragma unroll
    for (int i = 0; i < CTB; ++i)
      if (i == 0 || !single) ldp_row(P + (int64_t)(tb + min(i, nt - 1)) * ldp + x_off + c0, x[i]);
#pragma unroll
    for (int i = 0; i < CTB; ++i) {
      ok[i] = false;
      if (i >= nt) continue;
      const int t = tb + i;
      while (t >= tend && b + 1 < B) {  // (sequences without new tokens are passed over)
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
      float s[CTB];
#pragma unroll
      for (int i = 0; i < CTB; ++i) {
        s[i] = 0.0f;
#pragma unroll
        for (int e = 0; e < VW; ++e) s[i] += ok[i] && in[e] ? y[i][e] * y[i][e] : 0.0f;
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1)
#pragma unroll
        for (int i = 0; i < CTB; ++i) s[i] += __shfl_xor(s[i], o, 64);
#pragma unroll
      for (int i = 0; i < CTB; ++i) {
        const float k = kind & CONV_RMS ? 1.0f / sqrtf(s[i] / (float)n + eps)
                                        : 1.0f / sqrtf(s[i] + 1e-6f) * (kind & CONV_UNIT_SCALED ? 1.0f / sqrtf((float)n) : 1.0f);
#pragma unroll
        for (int e = 0; e < VW; ++e) y[i][e] *= k * g[e];
      }
    }
#pragma unroll
    for (int i = 0; i < CTB; ++i)
      if (ok[i]) stv(out + (int64_t)(tb + i) * C + c0, y[i]);
    if (single && ok[0]) {  // (run 1: the inputs after this token are the next step's history)
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

template <typename WT>
__global__ __launch_bounds__(256) void recurrence_gates_k(const float* __restrict__ P, int ldp, int S, int64_t ss, int T, int b_off,
                                                          float* __restrict__ beta, int H, int a1_off, const WT* __restrict__ a2,
                                                          int ra, const float* __restrict__ dt_bias,
                                                          const float* __restrict__ A_log, int d, float* __restrict__ decay,
                                                          int g1_off, const WT* __restrict__ g2, int rg, int ng,
                                                          float* __restrict__ gate) {
  extern __shared__ __attribute__((aligned(16))) float ys[];  // [GTOK][rank]
  const int t0 = blockIdx.x * GTOK, nt = min(GTOK, T - t0), HD = H * d, nab = (HD + 63) / 64;
  int job = blockIdx.y;
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
  // the rank rows: four elements a thread and four slabs in flight at a time, without branches around the loads
  const int ne = GTOK * rank;
  for (int e0 = 0; e0 < ne; e0 += 1024) {
    const float* p[4];
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int e = min(e0 + (int)threadIdx.x + 256 * j, ne - 1), i = e / rank;
      p[j] = P + (int64_t)(t0 + min(i, nt - 1)) * ldp + off + e - i * rank;
      v[j] = *p[j];
    }
    for (int k0 = 1; k0 < S; k0 += 4) {
      float a[4][4];
#pragma unroll
      for (int k = 0; k < 4; ++k)
#pragma unroll
        for (int j = 0; j < 4; ++j) a[k][j] = p[j][min(k0 + k, S - 1) * ss];
#pragma unroll
      for (int k = 0; k < 4; ++k)
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
  if ((rank & 7) == 0) {
#pragma unroll 4
    for (int r = 8 * part; r < rank; r += 32) {
      float v[8];
      ld8(w + r, v);
#pragma unroll
      for (int i = 0; i < GTOK; ++i) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(ys + i * rank + r), b = *reinterpret_cast<const f32x4*>(ys + i * rank + r + 4);
        z[i] += v[0] * a[0] + v[1] * a[1] + v[2] * a[2] + v[3] * a[3] + v[4] * b[0] + v[5] * b[1] + v[6] * b[2] + v[7] * b[3];
      }
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

__global__ void ssd_steps_k(const float* __restrict__ P, int ldp, int S, int64_t ss, int dt_off, const float* __restrict__ dt_bias,
                            const float* __restrict__ A_log, int H, int total, float* __restrict__ dt, float* __restrict__ decay) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= total) return;
  const int t = e / H, h = e - t * H;
  const float s = softplusf_(slab1(P + (int64_t)t * ldp + dt_off + h, S, ss) + dt_bias[h]);
  dt[e] = s;
  decay[e] = expf(-expf(A_log[h]) * s);
}

// ------------------------------------------------------------------ host side
void conv_prep(const at::Tensor& P, int64_t x_off, const at::Tensor& conv_w, const c10::optional<at::Tensor>& conv_b,
               const at::Tensor& units, const c10::optional<at::Tensor>& norm_w, at::Tensor& conv_state,
               const at::Tensor& state_slots, const at::Tensor& cu_q, double eps, at::Tensor& out, int64_t max_qlen,
               int64_t width) {
  const Slabs p = slabs_of(P, "P");
  const int64_t T = p.T, B = state_slots.numel();
  f32c(conv_w, "conv_w");
  f32c(conv_state, "conv_state");
  f32c(out, "out");
  i32c(units, "units");
  i32c(state_slots, "state_slots");
  i32c(cu_q, "cu_q");
  MCHECK(conv_w.dim() == 2 && units.dim() == 2 && units.size(1) == 4, "conv_w must be [C, taps], units [n, 4]");
  const int64_t C = conv_w.size(0), taps = conv_w.size(1), NU = units.size(0);
  if (T == 0 || B == 0 || NU == 0) return;
  MCHECK(taps >= 1 && (taps == 1 || (conv_state.dim() == 3 && conv_state.size(1) == taps - 1 && conv_state.size(2) == C)),
         "conv_state must be [slots, taps - 1, C]");
  MCHECK(out.dim() == 2 && out.size(0) == T && out.size(1) == C && cu_q.numel() == B + 1, "conv_prep: shape mismatch");
  cols_ok(p, x_off, C, "conv inputs");
  MCHECK(width >= 1 && width <= CONV_MAX, "a unit holds at most ", CONV_MAX, " channels");
  const float *bp = nullptr, *np = nullptr;
  int nn = 0;
  if (conv_b.has_value()) {
    f32c(*conv_b, "conv_b");
    MCHECK(conv_b->numel() == C, "conv_b must hold a number per channel");
    bp = conv_b->data_ptr<float>();
  }
  if (norm_w.has_value()) {
    f32c(*norm_w, "norm_w");
    np = norm_w->data_ptr<float>();
    nn = (int)norm_w->numel();
  }
  // (units lie inside the C channels by construction, ops.reference.conv_units; the kernel clamps them all the same)
  const bool single = max_qlen == 1 && T == B;
  const int run = single ? 1 : T >= 1024 ? 32 : CTB;
  const dim3 grid((unsigned)((T + run - 1) / run), (unsigned)((NU + 3) / 4));
#define CP_VW(TAPS, VW)                                                                                                      \
  conv_prep_k<TAPS, VW><<<grid, 256, 0, stream()>>>(                                                                         \
      p.p, p.ld, p.S, p.ss, (int)x_off, conv_w.data_ptr<float>(), bp, (int)taps, (int)C, units.data_ptr<int>(), (int)NU, \
      np, nn, conv_state.data_ptr<float>(), state_slots.data_ptr<int>(), cu_q.data_ptr<int>(), (int)B, (int)T, run,          \
      (int)single, (float)eps, out.data_ptr<float>())
#define CP_GO(TAPS)                        \
  if (width <= 64) CP_VW(TAPS, 1);         \
  else if (width <= 128) CP_VW(TAPS, 2);   \
  else CP_VW(TAPS, 4)
  switch (taps) {
    case 1: CP_GO(1); break;
    case 2: CP_GO(2); break;
    case 3: CP_GO(3); break;
    case 4: CP_GO(4); break;
    default: CP_GO(0); break;
  }
#undef CP_GO
#undef CP_VW
  if (taps > 1 && !single)
    conv_tail_k<<<dim3((unsigned)B, (unsigned)((C + 255) / 256)), 256, 0, stream()>>>(
        p.p, p.ld, p.S, p.ss, (int)x_off, (int)C, (int)taps, conv_state.data_ptr<float>(), state_slots.data_ptr<int>(),
        cu_q.data_ptr<int>());
}

void recurrence_gates(const at::Tensor& P, int64_t b_off, at::Tensor& beta, int64_t a1_off, const c10::optional<at::Tensor>& a2,
                      const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& decay, int64_t g1_off,
                      const c10::optional<at::Tensor>& g2, const c10::optional<at::Tensor>& gate,
                      const c10::optional<at::Tensor>& za) {
  const Slabs p = slabs_of(P, "P");
  const int64_t T = p.T, H = A_log.numel(), HD = dt_bias.numel();
  if (T == 0) return;
  f32c(beta, "beta");
  f32c(dt_bias, "dt_bias");
  f32c(A_log, "A_log");
  f32c(decay, "decay");
  MCHECK(H > 0 && HD % H == 0 && beta.numel() == T * H && decay.numel() == T * HD, "recurrence_gates: shape mismatch");
  cols_ok(p, b_off, H, "step sizes");
  if (za.has_value()) {
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
  auto second = [&](const c10::optional<at::Tensor>& w, int64_t off, int64_t rows, const char* what) {
    MCHECK(w.has_value() && w->is_cuda() && is_act(*w) && w->is_contiguous() && w->dim() == 2 && w->size(0) == rows, what,
           " must be contiguous [channels, rank]");
    cols_ok(p, off, w->size(1), what);
    MCHECK(w->size(1) >= 1 && w->size(1) <= 1024, what, ": rank above 1024");
    bf = w->scalar_type() == at::kBFloat16;
    return w->size(1);
  };
  const int64_t ra = second(a2, a1_off, HD, "a2");
  int64_t rg = 0, ng = 0;
  if (gate.has_value()) {
    f32c(*gate, "gate");
    MCHECK(gate->dim() == 2 && gate->size(0) == T, "gate must be [T, channels]");
    ng = gate->size(1);
    const bool abf = bf;
    rg = second(g2, g1_off, ng, "g2");
    MCHECK(abf == bf, "a2 and g2 must have one dtype");
  }
  const dim3 grid((unsigned)((T + GTOK - 1) / GTOK), (unsigned)(1 + (HD + 63) / 64 + (ng + 63) / 64));
  const size_t lds = (size_t)GTOK * std::max(ra, rg) * sizeof(float);
#define RG_GO(WT)                                                                                                            \
  recurrence_gates_k<WT><<<grid, 256, lds, stream()>>>(                                                                      \
      p.p, p.ld, p.S, p.ss, (int)T, (int)b_off, beta.data_ptr<float>(), (int)H, (int)a1_off, (const WT*)a2->data_ptr(),      \
      (int)ra, dt_bias.data_ptr<float>(), A_log.data_ptr<float>(), (int)(HD / H), decay.data_ptr<float>(), (int)g1_off,      \
      ng ? (const WT*)g2->data_ptr() : nullptr, (int)rg, (int)ng, ng ? gate->data_ptr<float>() : nullptr)
  if (bf) RG_GO(uint16_t);
  else RG_GO(float);
#undef RG_GO
}

void ssd_steps(const at::Tensor& P, int64_t dt_off, const at::Tensor& dt_bias, const at::Tensor& A_log, at::Tensor& dt,
               at::Tensor& decay) {
  const Slabs p = slabs_of(P, "P");
  const int64_t T = p.T, H = A_log.numel();
  if (T == 0) return;
  f32c(dt_bias, "dt_bias");
  f32c(A_log, "A_log");
  f32c(dt, "dt");
  f32c(decay, "decay");
  MCHECK(dt_bias.numel() == H && dt.numel() == T * H && decay.numel() == T * H, "ssd_steps: shape mismatch");
  cols_ok(p, dt_off, H, "dt");
  ssd_steps_k<<<(unsigned)((T * H + 255) / 256), 256, 0, stream()>>>(p.p, p.ld, p.S, p.ss, (int)dt_off, dt_bias.data_ptr<float>(),
                                                                    A_log.data_ptr<float>(), (int)H, (int)(T * H),
                                                                    dt.data_ptr<float>(), decay.data_ptr<float>());
}

}  // namespace

void bind_short_conv(pybind11::module& m) {
  m.def("conv_prep", &conv_prep);
  m.def("recurrence_gates", &recurrence_gates);
  m.def("ssd_steps", &ssd_steps);
}

}  // namespace xot
