// Matrix-core attention over a sliding window or the query's chunk, with an optional per-head sink, on plain paged caches
// (K [pages, G, 64, d], V^T [pages, Gv, dv, 64], bf16): the kernels behind attn_window_pool for steps without pooled blocks.
//
//   window_prefill_k   prompt portions: a workgroup owns 256 (token, head of the group) rows of one (sequence, kv head), so
//                      a page is read once for all query heads of the group
//   window_decode_k    single tokens: a workgroup owns one (sequence, kv head, share of the pages), its waves deal the
//                      pages among themselves and merge through LDS; window_merge_k adds up the shares
//
// Both compute transposed scores S^T = K Q^T (keys x rows): a lane's accumulator rows are keys of ONE query row, so the
// running maximum and denominator are per lane (the four lanes of a row agree on the maximum through two shuffles and keep
// partial denominators).  The key order 32 kk + 8 (c / 4) + 4 hf + c % 4 of the tiles makes the exponentials, rounded to
// bf16, come out in the B-operand layout of O^T += V^T P^T.  Scores, maxima, sums: fp32 (base-2 exponentials).
#include "mixer_util.h"

namespace xot {
namespace {
using namespace mix;

constexpr float L2E_W = 1.4426950408889634f;
constexpr float NEG_W = -3.0e38f;

// the first token a query at position pos sees
__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
  const int lo = window > 0 ? max(0, pos - window + 1) : 0;
  return chunk > 0 ? max(lo, pos - pos % chunk) : lo;
}

// key `key` is seen by the query at `pos` whose window / chunk starts at lo; the first `keep` tokens stay visible
__device__ __forceinline__ bool seen(int key, int pos, int lo, int keep) { return key <= pos && (key >= lo || key < keep); }

// two probabilities in one dword of bf16
__device__ __forceinline__ uint32_t pack2(float a, float b) {
  typedef __bf16 bf16x2_w __attribute__((ext_vector_type(2)));
  typedef float f32x2_w __attribute__((ext_vector_type(2)));
  return __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2_w{a, b}), bf16x2_w));
}

// ------------------------------------------------------------------ prompt portions
// XOR swizzle of a K row's 16-byte granules in LDS (conflict-free fragment reads): the 12 granules of a 96-wide row keep
// their group of four
template <int DK>
__device__ __forceinline__ int k_swz(int r) {
  return DK == 128  ? (3 * (r & 1)) | (((r >> 1) & 1) << 2) | (((r >> 3) & 1) << 3)
         : DK == 96 ? (r >> 3) & 3
                    : (r & 1) | (((r >> 1) & 1) << 1) | (((r >> 3) & 1) << 2);
}

// 8 waves, two 16-row blocks each.  Pages arrive by LDS-DMA in a three-deep ring (two in flight), swizzled through the
// per-lane source addresses.  Waves skip pages none of their rows sees; the latest rows' workgroups start first, those of
// one (sequence, kv head) on one XCD.
template <int DK, int DV, typename OT, bool CAP>
__global__ __launch_bounds__(512, 1) void window_prefill_k(
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc,
    const int* __restrict__ block_tables, int width, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
    const float* __restrict__ sink, float scale_l2, int window, int chunk, OT* __restrict__ out, int ldo, int H, int G, int Gv,
    int num_pages, int keep, float inv_cap2, float cap_l2) {
  constexpr int KS = DK / 32, NDT = DV / 16;
  constexpr int KGPR = DK / 8;                                     // 16-byte granules of a K row
  constexpr int KEL = PAGE_TOK * DK, VEL = PAGE_TOK * DV;          // elements of a page's images
  constexpr int NCHK = KEL / 512, NCH = (KEL + VEL) / 512;         // 1 KB LDS-DMA chunks (K then V^T)
  static_assert(NCH % 8 == 0 && DK % 32 == 0 && DV % 16 == 0, "chunks split over 8 waves");
  constexpr int CPW = NCH / 8;
  extern __shared__ __attribute__((aligned(16))) uint16_t smem[];  // [3][K page | V^T page]
  int tile, kvh, b;
  {
    const int nwg = gridDim.x * gridDim.y * gridDim.z;
    int lin = blockIdx.x + gridDim.x * (blockIdx.y + gridDim.y * blockIdx.z);
    const int xcd = lin & 7, qq = nwg >> 3, rr = nwg & 7;
    lin = (xcd < rr ? xcd * (qq + 1) : rr * (qq + 1) + (xcd - rr) * qq) + (lin >> 3);
    tile = gridDim.x - 1 - lin % gridDim.x;
    lin /= gridDim.x;
    kvh = lin % gridDim.y;
    b = lin / gridDim.y;
  }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int g = lane >> 4, c = lane & 15;
  const int rep = H / G, gv = kvh / (G / Gv);
  const int q0 = cu_q[b], qlen = cu_q[b + 1] - q0;
  const int nrows = qlen * rep, row0 = tile * 256;
  const int ctx = min(ctx_lens[b], width * PAGE_TOK);
  if (row0 >= nrows || ctx < qlen) return;  // (the whole workgroup; ctx 0: a padding row)
  const int pos0 = ctx - qlen;

  s16x8 qf[2][KS];  // lane (g, c): row c of block blk, dims 32 s + 8 g .. + 8
  int qpos[2], qlo[2];
  float m[2], l[2];
#pragma unroll
  for (int blk = 0; blk < 2; ++blk) {
    const int row = row0 + 32 * wave + 16 * blk + c;
    const bool ok = row < nrows;
    const int ti = ok ? row / rep : 0, h = kvh * rep + (ok ? row % rep : 0);
    qpos[blk] = ok ? pos0 + ti : -1;
    qlo[blk] = ok ? first_seen(pos0 + ti, window, chunk) : 0;
    const uint16_t* qp = q + ((int64_t)(q0 + ti) * H + h) * DK + 8 * g;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const s16x8 v = ld16(qp + 32 * s);
      qf[blk][s] = ok ? v : s16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
    m[blk] = sink ? sink[h] * L2E_W : NEG_W;
    l[blk] = sink && g == 0 ? 1.0f : 0.0f;  // (partial denominators: one of the row's four lanes counts the sink)
  }
  const int last_row = min(nrows, row0 + 256) - 1;
  const int p_first = first_seen(pos0 + row0 / rep, window, chunk) / PAGE_TOK;
  const int p_end = (pos0 + last_row / rep) / PAGE_TOK + 1;
  // pages in order: those of kept first tokens before the window, then p_first on
  const int nkp = min((keep + PAGE_TOK - 1) / PAGE_TOK, p_first), nit = nkp + p_end - p_first;
  auto page_at = [&](int i) { return i < nkp ? i : p_first + i - nkp; };
  // the wave's rows: the last key any of them sees, the first row's position, the first key of the first / last row
  const int wr0 = row0 + 32 * wave, wr1 = min(nrows - 1, wr0 + 31);
  const bool live = wr1 >= wr0;
  const int wmax = live ? pos0 + wr1 / rep : -1, wmin = pos0 + wr0 / rep;
  const int wlo_first = live ? first_seen(wmin, window, chunk) : 0, wlo_last = live ? first_seen(wmax, window, chunk) : 0;

  f32x4 o[2][NDT];
#pragma unroll
  for (int blk = 0; blk < 2; ++blk)
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) o[blk][dt] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int* bt = block_tables + (int64_t)b * width;
  auto issue = [&](int p, int buf) {
    const int64_t page = min(max(bt[p], 0), num_pages - 1);
    const uint16_t* kb = kc + (page * G + kvh) * KEL;
    const uint16_t* vb = vc + (page * Gv + gv) * VEL;
    uint16_t* dst = smem + buf * (KEL + VEL);
#pragma unroll
    for (int i = 0; i < CPW; ++i) {
      const int ch = wave * CPW + i;
      const uint16_t* src;
      if (ch < NCHK) {
        const int P = ch * 64 + lane, r = P / KGPR, j = (P % KGPR) ^ k_swz<DK>(r);
        src = kb + (r * KGPR + j) * 8;
      } else {
        const int P = (ch - NCHK) * 64 + lane, r = P >> 3, j = (P & 7) ^ (r & 7);  // V^T image rows: 64 keys = 8 granules
        src = vb + (r * 8 + j) * 8;
      }
      __builtin_amdgcn_global_load_lds((__attribute__((address_space(1))) void*)src,
                                       (__attribute__((address_space(3))) void*)(dst + ch * 512), 16, 0, 0);
    }
  };
  int kofs[4][KS];  // fragment addresses inside a page image, fixed per lane
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = 32 * (j >> 1) + 8 * (c >> 2) + 4 * (j & 1) + (c & 3);
#pragma unroll
    for (int s = 0; s < KS; ++s) kofs[j][s] = r * DK + 8 * ((4 * s + g) ^ k_swz<DK>(r));
  }
  int vofs[2];
#pragma unroll
  for (int kk = 0; kk < 2; ++kk) vofs[kk] = c * PAGE_TOK + 8 * ((4 * kk + g) ^ (c & 7));

  auto score = [&](const uint16_t* Ks, int key0, s16x8(&pf)[2][2], float(&alpha)[2]) {
    f32x4 st[2][4];
#pragma unroll
    for (int blk = 0; blk < 2; ++blk)
#pragma unroll
      for (int j = 0; j < 4; ++j) st[blk][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int KPF = 4, NKS = 4 * KS;  // K fragments KPF steps ahead of their MFMAs
    s16x8 ka[KPF];
#pragma unroll
    for (int t = 0; t < KPF - 1; ++t) ka[t] = ld16(Ks + kofs[t & 3][t >> 2]);
#pragma unroll
    for (int t = 0; t < NKS; ++t) {
      if (t + KPF - 1 < NKS) ka[(t + KPF - 1) % KPF] = ld16(Ks + kofs[(t + KPF - 1) & 3][(t + KPF - 1) >> 2]);
      const int j = t & 3, s = t >> 2;
      st[0][j] = mfma16(ka[t % KPF], qf[0][s], st[0][j]);
      st[1][j] = mfma16(ka[t % KPF], qf[1][s], st[1][j]);
      __builtin_amdgcn_sched_barrier(0);
    }
    if constexpr (CAP) {
#pragma unroll
      for (int blk = 0; blk < 2; ++blk)
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r) st[blk][j][r] = capped_l2(st[blk][j][r] * scale_l2, inv_cap2, cap_l2);
    }
    const float sc = CAP ? 1.0f : scale_l2;
    const bool masked = key0 + PAGE_TOK - 1 > wmin || key0 < wlo_last;  // (wave-uniform)
#pragma unroll
    for (int blk = 0; blk < 2; ++blk) {
      if (masked) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = key0 + 32 * (j >> 1) + 8 * g + 4 * (j & 1) + r;
            st[blk][j][r] = seen(key, qpos[blk], qlo[blk], keep) ? st[blk][j][r] * sc : -INFINITY;
          }
      } else if constexpr (!CAP) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r) st[blk][j][r] *= sc;
      }
      float mt = NEG_W;
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) mt = fmaxf(mt, st[blk][j][r]);
      mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
      mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
      const float mn = fmaxf(m[blk], mt);
      alpha[blk] = __builtin_amdgcn_exp2f(m[blk] - mn);
      m[blk] = mn;
      float ls = 0.f;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        u32x4 pw;
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          const float p0 = __builtin_amdgcn_exp2f(st[blk][2 * kk + (e >> 2)][e & 3] - mn);
          const float p1 = __builtin_amdgcn_exp2f(st[blk][2 * kk + (e >> 2)][(e & 3) + 1] - mn);
          pw[e >> 1] = pack2(p0, p1);
          ls += p0 + p1;
        }
        pf[blk][kk] = __builtin_bit_cast(s16x8, pw);
      }
      l[blk] = l[blk] * alpha[blk] + ls;
    }
  };
  auto accumulate = [&](const uint16_t* Vs, const s16x8(&pf)[2][2], const float(&alpha)[2]) {
    if (__ballot(alpha[0] != 1.f || alpha[1] != 1.f)) {  // (the running maxima stop moving after a row's first pages)
#pragma unroll
      for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          o[0][dt][r] *= alpha[0];
          o[1][dt][r] *= alpha[1];
        }
    }
    constexpr int VPF = 3;
    s16x8 va[VPF][2];
#pragma unroll
    for (int t = 0; t < VPF - 1; ++t)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) va[t][kk] = ld16(Vs + vofs[kk] + 16 * t * PAGE_TOK);
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
      if (dt + VPF - 1 < NDT) {
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) va[(dt + VPF - 1) % VPF][kk] = ld16(Vs + vofs[kk] + 16 * (dt + VPF - 1) * PAGE_TOK);
      }
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        o[0][dt] = mfma16(va[dt % VPF][kk], pf[0][kk], o[0][dt]);
        o[1][dt] = mfma16(va[dt % VPF][kk], pf[1][kk], o[1][dt]);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
  };

  // ring: page i + 2 is issued once every wave is past page i - 1
  issue(page_at(0), 0);
  if (nit > 1) issue(page_at(1), 1);
  for (int i = 0; i < nit; ++i) {
    const int buf = i % 3;
    if (i + 1 < nit)
      asm volatile("s_waitcnt vmcnt(%0)" ::"n"(CPW) : "memory");  // this wave's share of page i has landed
    else
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (i + 2 < nit) issue(page_at(i + 2), (i + 2) % 3);
    const int key0 = page_at(i) * PAGE_TOK;
    if (key0 > wmax || (key0 + PAGE_TOK <= wlo_first && key0 >= keep)) continue;  // (wave-uniform) no row of this wave sees the page
    const uint16_t* Ks = smem + buf * (KEL + VEL);
    s16x8 pf[2][2];
    float alpha[2];
    score(Ks, key0, pf, alpha);
    accumulate(Ks + KEL, pf, alpha);
  }

#pragma unroll
  for (int blk = 0; blk < 2; ++blk) {  // o[blk][dt][r] = O[row c of the block][dim 16 dt + 4 g + r]
    float L = l[blk];
    L += __shfl_xor(L, 16, 64);
    L += __shfl_xor(L, 32, 64);
    const int row = row0 + 32 * wave + 16 * blk + c;
    if (row < nrows) {
      OT* op = out + (int64_t)(q0 + row / rep) * ldo + (kvh * rep + row % rep) * DV + 4 * g;
      const float inv = L > 0.f ? 1.f / L : 0.f;
#pragma unroll
      for (int dt = 0; dt < NDT; ++dt) {
        if constexpr (sizeof(OT) == 4) {
          *reinterpret_cast<f32x4*>(op + 16 * dt) = f32x4{o[blk][dt][0] * inv, o[blk][dt][1] * inv, o[blk][dt][2] * inv, o[blk][dt][3] * inv};
        } else {
          s16x4 v;
#pragma unroll
          for (int r = 0; r < 4; ++r) v[r] = (short)f2bf(o[blk][dt][r] * inv);
          *reinterpret_cast<s16x4*>(op + 16 * dt) = v;
        }
      }
    }
  }
}

// ------------------------------------------------------------------ single tokens
// WDW waves; rows = the group's query heads (at most 16).  K and V^T fragments go straight from global memory to registers
// (page p's values and page p + 1's keys are in flight under page p's scores); d <= 32 NK and dv <= 32 NK, multiples of 8
// (RAG: smaller than the tiles, missing dims are zeros).  nsplit > 1: share blockIdx.z of the visible pages, unnormalised
// sums and (maximum, denominator) into part [T][G][nsplit][rep][dv + 2].
constexpr int WDW = 8;

template <int NK, bool RAG, typename OT, bool CAP>
__global__ __launch_bounds__(64 * WDW, 1) void window_decode_k(
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc,
    const int* __restrict__ block_tables, int width, const int* __restrict__ ctx_lens, const float* __restrict__ sink,
    float scale_l2, int window, int chunk, OT* __restrict__ out, int ldo, int H, int G, int Gv, int d_rt, int dv_rt,
    int num_pages, float* __restrict__ part, int nsplit, int keep, float inv_cap2, float cap_l2) {
  constexpr int NDT = NK * 2;
  const int d = RAG ? d_rt : NK * 32, dv = RAG ? dv_rt : NK * 32;
  extern __shared__ float sm[];  // merge: [WDW][rep][dv + 2]
  const int b = blockIdx.x, kvh = blockIdx.y, sp = blockIdx.z;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int g = lane >> 4, c = lane & 15;
  const int rep = H / G, gv = kvh / (G / Gv), ms = dv + 2;
  const int ctx = min(ctx_lens[b], width * PAGE_TOK);
  if (ctx <= 0) {  // padding row of a captured decode batch: zeros, so that nothing downstream reads stale memory
    if (nsplit == 1)
      for (int e = threadIdx.x; e < rep * dv; e += blockDim.x) stf(out + (int64_t)b * ldo + kvh * rep * dv + e, 0.0f);
    return;
  }
  const int pos = ctx - 1, lo = first_seen(pos, window, chunk);
  // visible pages in order: those of kept first tokens before the window, then the window's or chunk's own
  const int pa = lo / PAGE_TOK, nkp = min((keep + PAGE_TOK - 1) / PAGE_TOK, pa), np = nkp + pos / PAGE_TOK + 1 - pa;
  auto page_at = [&](int i) { return i < nkp ? i : pa + i - nkp; };
  // this share's pages [s0, s1) of the np visible ones
  const int s0 = (int)((int64_t)np * sp / nsplit), s1 = (int)((int64_t)np * (sp + 1) / nsplit);
  const s16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  s16x8 qf[NK];
  {
    const uint16_t* qp = q + ((int64_t)b * H + kvh * rep + min(c, rep - 1)) * d + 8 * g;
#pragma unroll
    for (int s = 0; s < NK; ++s) qf[s] = c < rep && (!RAG || 32 * s + 8 * g < d) ? ld16(qp + 32 * s) : zero;
  }
  const bool first = wave == 0 && sp == 0 && sink;
  float m = first && c < rep ? sink[kvh * rep + c] * L2E_W : NEG_W;
  float l = first && g == 0 ? 1.0f : 0.0f;
  f32x4 o[NDT];
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int* bt = block_tables + (int64_t)b * width;
  s16x8 kf[4][NK];
  auto load_k = [&](int i) {
    const uint16_t* kb = kc + ((int64_t)min(max(bt[page_at(i)], 0), num_pages - 1) * G + kvh) * PAGE_TOK * d + 8 * g;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = 32 * (j >> 1) + 8 * (c >> 2) + 4 * (j & 1) + (c & 3);
#pragma unroll
      for (int s = 0; s < NK; ++s) kf[j][s] = !RAG || 32 * s + 8 * g < d ? ld16(kb + r * d + 32 * s) : zero;
    }
  };
  int p = s0 + wave;
  if (p < s1) load_k(p);
  for (; p < s1; p += WDW) {
    const uint16_t* vb = vc + ((int64_t)min(max(bt[page_at(p)], 0), num_pages - 1) * Gv + gv) * PAGE_TOK * dv + 8 * g;
    s16x8 vf[NDT][2];
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        vf[dt][kk] = !RAG || 16 * dt + c < dv ? ld16(vb + (16 * dt + c) * PAGE_TOK + 32 * kk) : zero;
    f32x4 st[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      st[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < NK; ++s) st[j] = mfma16(kf[j][s], qf[s], st[j]);
    }
    if (p + WDW < s1) load_k(p + WDW);
    const int key0 = page_at(p) * PAGE_TOK;
    float mt = NEG_W;
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = key0 + 32 * (j >> 1) + 8 * g + 4 * (j & 1) + r;
        const float t = CAP ? capped_l2(st[j][r] * scale_l2, inv_cap2, cap_l2) : st[j][r] * scale_l2;
        st[j][r] = seen(key, pos, lo, keep) ? t : -INFINITY;
        mt = fmaxf(mt, st[j][r]);
      }
    mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    const float mn = fmaxf(m, mt), alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    float ls = 0.f;
    s16x8 pf[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      u32x4 pw;
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const float p0 = __builtin_amdgcn_exp2f(st[2 * kk + (e >> 2)][e & 3] - mn);
        const float p1 = __builtin_amdgcn_exp2f(st[2 * kk + (e >> 2)][(e & 3) + 1] - mn);
        pw[e >> 1] = pack2(p0, p1);
        ls += p0 + p1;
      }
      pf[kk] = __builtin_bit_cast(s16x8, pw);
    }
    l = l * alpha + ls;
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
#pragma unroll
      for (int r = 0; r < 4; ++r) o[dt][r] *= alpha;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) o[dt] = mfma16(vf[dt][kk], pf[kk], o[dt]);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (c < rep) {
    float* mine = sm + (wave * rep + c) * ms;
    if (g == 0) {
      mine[0] = m;
      mine[1] = l;
    }
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (!RAG || 16 * dt + 4 * g + r < dv) mine[2 + 16 * dt + 4 * g + r] = o[dt][r];
  }
  __syncthreads();
  for (int e = threadIdx.x; e < rep * dv; e += blockDim.x) {
    const int r = e / dv, i = e - r * dv;
    float M = NEG_W;
#pragma unroll
    for (int w = 0; w < WDW; ++w) M = fmaxf(M, sm[(w * rep + r) * ms]);
    float L = 0.f, a = 0.f;
#pragma unroll
    for (int w = 0; w < WDW; ++w) {
      const float* s = sm + (w * rep + r) * ms;
      const float f = __builtin_amdgcn_exp2f(s[0] - M);
      L += s[1] * f;
      a += s[2 + i] * f;
    }
    if (nsplit == 1) {
      stf(out + (int64_t)b * ldo + (kvh * rep + r) * dv + i, L > 0.f ? a / L : 0.f);
    } else {
      float* pt = part + ((((int64_t)b * G + kvh) * nsplit + sp) * rep + r) * ms;
      pt[2 + i] = a;
      if (i == 0) {
        pt[0] = M;
        pt[1] = L;
      }
    }
  }
}

// out[b, head] = sum over the shares of e^(m - M) a / sum of e^(m - M) l
template <typename OT>
__global__ __launch_bounds__(256) void window_merge_k(const float* __restrict__ part, const int* __restrict__ ctx_lens,
                                                      OT* __restrict__ out, int ldo, int rep, int dv, int nsplit, int G) {
  const int b = blockIdx.x, kvh = blockIdx.y, ms = dv + 2;
  const bool live = ctx_lens[b] > 0;
  const float* base = part + ((int64_t)b * G + kvh) * nsplit * rep * ms;
  for (int e = threadIdx.x; e < rep * dv; e += blockDim.x) {
    const int r = e / dv, i = e - r * dv;
    float M = NEG_W, L = 0.f, a = 0.f;
    if (live) {
      for (int s = 0; s < nsplit; ++s) M = fmaxf(M, base[(s * rep + r) * ms]);
      for (int s = 0; s < nsplit; ++s) {
        const float* t = base + (s * rep + r) * ms;
        const float f = __builtin_amdgcn_exp2f(t[0] - M);
        L += t[1] * f;
        a += t[2 + i] * f;
      }
    }
    stf(out + (int64_t)b * ldo + (kvh * rep + r) * dv + i, L > 0.f ? a / L : 0.f);
  }
}

struct WinArgs {
  const at::Tensor &q, &k, &v, &bt, &cu, &ctx;
  const float* sink;
  float scale_l2;
  int window, chunk, ldo, keep;
  float inv_cap2, cap_l2;  // softcap (0: none)
};

template <int DK, int DV, typename OT, bool CAP>
void go_prefill(const WinArgs& a, at::Tensor& out, int64_t max_qlen) {
  const int H = (int)a.q.size(1), G = (int)a.k.size(1), Gv = (int)a.v.size(1);
  constexpr int SMEM = 3 * (DK + DV) * PAGE_TOK * 2;
  auto kern = window_prefill_k<DK, DV, OT, CAP>;
  static bool attr = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, SMEM) == hipSuccess;
  (void)attr;
  const dim3 grid((unsigned)((max_qlen * (H / G) + 255) / 256), (unsigned)G, (unsigned)a.ctx.numel());
  kern<<<grid, 512, SMEM, stream()>>>((const uint16_t*)a.q.data_ptr(), (const uint16_t*)a.k.data_ptr(),
                                      (const uint16_t*)a.v.data_ptr(), a.bt.data_ptr<int>(), (int)a.bt.size(1),
                                      a.cu.data_ptr<int>(), a.ctx.data_ptr<int>(), a.sink, a.scale_l2, a.window, a.chunk,
                                      (OT*)out.data_ptr(), a.ldo, H, G, Gv, (int)a.k.size(0), a.keep, a.inv_cap2, a.cap_l2);
}

template <int NK, bool RAG, typename OT, bool CAP>
void go_decode(const WinArgs& a, at::Tensor& out, float* part, int nsplit) {
  const int H = (int)a.q.size(1), G = (int)a.k.size(1), Gv = (int)a.v.size(1), dv = (int)a.v.size(2), B = (int)a.ctx.numel();
  const int smem = WDW * (H / G) * (dv + 2) * 4;
  auto kern = window_decode_k<NK, RAG, OT, CAP>;
  static bool attr = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize,
                                         WDW * 16 * (32 * NK + 2) * 4) == hipSuccess;
  (void)attr;
  kern<<<dim3(B, G, nsplit), 64 * WDW, smem, stream()>>>(
      (const uint16_t*)a.q.data_ptr(), (const uint16_t*)a.k.data_ptr(), (const uint16_t*)a.v.data_ptr(), a.bt.data_ptr<int>(),
      (int)a.bt.size(1), a.ctx.data_ptr<int>(), a.sink, a.scale_l2, a.window, a.chunk, (OT*)out.data_ptr(), a.ldo, H, G, Gv,
      (int)a.q.size(2), dv, (int)a.k.size(0), part, nsplit, a.keep, a.inv_cap2, a.cap_l2);
  if (nsplit > 1)
    window_merge_k<OT><<<dim3(B, G), 256, 0, stream()>>>(part, a.ctx.data_ptr<int>(), (OT*)out.data_ptr(), a.ldo, H / G, dv,
                                                         nsplit, G);
}

}  // namespace

// The matrix-core path of attn_window_pool (csrc/hybrid.hip, which has checked shapes and dtypes): bf16 queries and caches,
// no pooled blocks.  Returns false when these kernels do not take the step.
bool window_attention(const at::Tensor& q, const at::Tensor& k_cache, const at::Tensor& v_cache, const at::Tensor& block_tables,
                      const at::Tensor& cu_q, const at::Tensor& ctx_lens, const float* sink, double scale, int64_t window,
                      int64_t chunk, int64_t keep, double softcap, at::Tensor& out, int64_t ldo, int64_t max_qlen) {
  const int64_t T = q.size(0), H = q.size(1), d = q.size(2), G = k_cache.size(1), dv = v_cache.size(2), B = ctx_lens.numel();
  const int64_t rep = H / G, width = block_tables.size(1);
  const bool o32 = out.scalar_type() == at::kFloat;
  const WinArgs a{q, k_cache, v_cache, block_tables, cu_q, ctx_lens, sink, (float)(scale * L2E_W), (int)window, (int)chunk, (int)ldo,
                  (int)keep, (float)(softcap > 0 ? 2.0 / softcap : 0.0), (float)(softcap * L2E_W)};
  const bool cap = softcap > 0;
  if (max_qlen == 1 && T == B && rep <= 16 && d % 8 == 0 && dv % 8 == 0 && d <= 128 && dv <= 128) {
    // shares of the visible pages: enough workgroups for the 256 CUs, at least two pages per wave of a share
    int64_t pages = width;
    if (chunk > 0) pages = std::min(pages, (chunk + 63) / 64 + 1);
    if (window > 0) pages = std::min(pages, (window + 63) / 64 + 1);
    pages = std::min(width, pages + (keep + 63) / 64);
    const int64_t nsplit = std::max<int64_t>(1, std::min<int64_t>((256 + B * G - 1) / (B * G), pages / (2 * WDW)));
    at::Tensor part;
    if (nsplit > 1) part = at::empty({B * G * nsplit * rep * (dv + 2)}, q.options().dtype(at::kFloat));
    float* pp = nsplit > 1 ? part.data_ptr<float>() : nullptr;
    const int64_t n = (std::max(d, dv) + 31) / 32;
    const bool rag = d != 32 * n || dv != 32 * n;
#define WD_CAP(NK, RAG, OT)                                                \
  (cap ? go_decode<NK, RAG, OT, true>(a, out, pp, (int)nsplit)              \
       : go_decode<NK, RAG, OT, false>(a, out, pp, (int)nsplit))
#define WD_OT(NK, RAG) (o32 ? WD_CAP(NK, RAG, float) : WD_CAP(NK, RAG, uint16_t))
#define WD_GO(NK) (rag ? WD_OT(NK, true) : WD_OT(NK, false))
    switch (n) {
      case 1: WD_GO(1); break;
      case 2: WD_GO(2); break;
      case 3: WD_GO(3); break;
      default: WD_GO(4); break;
    }
#undef WD_GO
#undef WD_OT
#undef WD_CAP
    return true;
  }
  if (max_qlen >= 16 && ldo % 4 == 0) {
#define WP_GO(DK, DV)                                            \
  if (d == DK && dv == DV) {                                     \
    if (o32 && cap) go_prefill<DK, DV, float, true>(a, out, max_qlen); \
    else if (o32) go_prefill<DK, DV, float, false>(a, out, max_qlen);  \
    else if (cap) go_prefill<DK, DV, uint16_t, true>(a, out, max_qlen); \
    else go_prefill<DK, DV, uint16_t, false>(a, out, max_qlen);  \
    return true;                                                 \
  }
    WP_GO(64, 64)
    WP_GO(96, 96)
    WP_GO(128, 128)
    WP_GO(64, 128)
    WP_GO(128, 64)
#undef WP_GO
  }
  return false;
}

}  // namespace xot
