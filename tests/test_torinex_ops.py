"""The ops behind Torinex's layers, one mechanism at a time, against the functions of tests/torinex_oracle.py: the torch
twins on the CPU and, marked gpu, the HIP kernels in float32 and bfloat16 (the activations' dtype; norms, scores and
router scores are float32 in both)."""
import pytest
import torch

import torinex_oracle as oracle
from xotorch_support_jetson_amd.models.weights import _pair_order, interleave_gate_up
from xotorch_support_jetson_amd.ops import kernels as K
from xotorch_support_jetson_amd.ops.rope import build_cos_sin

RUNS = [pytest.param("cpu", torch.float32, id="cpu-f32"),
        pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=pytest.mark.gpu),
        pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)]
F64 = torch.float64


def rnd(*shape, seed=0, scale=1.0):
  return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def close(got, want, tol, what=""):
  err = (got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-9)
  assert err < tol, f"{what}: off by {float(err):.3g}"


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("D", [40, 1030, 2050, 4200])
def test_result_norm_with_bias_and_stream_copy(dev, dtype, D):
  """x += rms_norm(y + bias) * w and the stream itself as the next operand; y rows wider than D; padding untouched."""
  T, eps = 5, 1e-4
  x, y, yb, w = rnd(T, D, seed=1), rnd(T, D + 24, seed=2), rnd(D, seed=3), rnd(D, seed=4)
  want = x.double() + oracle.rms_norm(y[:, :D].double() + yb.double(), w.double(), eps)
  xd, out = x.clone().to(dev), torch.zeros(T, D + 8, dtype=dtype, device=dev)
  K.sandwich_add_norm(xd, y.to(dev), w.to(dev), None, eps, out, yb=yb.to(dev))
  close(xd, want, 1e-5, "stream")
  close(out[:, :D], want, 1e-6 if dtype == torch.float32 else 5e-3, "copy")
  assert float(out[:, D:].abs().max()) == 0.0
  out.zero_()
  K.sandwich_add_norm(xd, None, None, None, eps, out)  # nothing added
  close(out[:, :D], want, 1e-5 if dtype == torch.float32 else 5e-3, "copy alone")


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("own", [True, False])
@pytest.mark.parametrize("H,G,d,dv,R", [(4, 2, 16, 24, 16), (6, 3, 12, 20, 6), (2, 1, 96, 40, 64), (5, 5, 8, 8, 0), (3, 1, 72, 72, 40)])
def test_projection_norms_rotation_and_store(dev, dtype, own, H, G, d, dv, R):
  """Biases, one weighted norm over all of q (and of k), then the interleaved rotation (rows, biases and norm weights
  reordered per head as the loader does), the paged write; a token without a slot writes nothing."""
  T, eps, base, pos0 = 9, 1e-3, 300.0, 61
  t = {}
  for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
    t[n], t[n + ".b"], t[n + ".norm"] = rnd(rows, 32, seed=len(t), scale=0.3), rnd(rows, seed=len(t) + 1), 1.0 + rnd(rows, seed=len(t) + 2, scale=0.2)
  h = rnd(pos0 + T, 32, seed=30)
  m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "rot": {"base": base, "dims": R}}
  t64 = {k: v.double() for k, v in t.items()}
  wq = oracle.queries(h.double(), m, t64, "", eps)[pos0:]
  wk, wv = (a[pos0:] for a in oracle.keys_values(h.double(), m, t64, "", eps))
  order = _pair_order(d, R)

  def rows(w, heads):
    return w.reshape(heads, d, *w.shape[1:])[:, order].reshape(w.shape)
  W = torch.cat([rows(t["q"], H)] + ([rows(t["k"], G), t["v"]] if own else []))
  b = torch.cat([rows(t["q.b"], H)] + ([rows(t["k.b"], G), t["v.b"]] if own else []))
  P = (h[pos0:].double() @ W.double().T).float().to(dev)
  q = torch.empty(T, H, d, dtype=dtype, device=dev)
  kc = torch.full((4, G, 64, d), 7.0, dtype=dtype, device=dev)
  vc = torch.full((4, G, dv, 64), 7.0, dtype=dtype, device=dev)
  pages = [2, 0]
  slots = torch.tensor([pages[(pos0 + i) // 64] * 64 + (pos0 + i) % 64 for i in range(T)])
  slots[4] = -1
  tab = build_cos_sin(R, 128, base, None, torch.device(dev)) if R else torch.zeros(1, 0, device=dev)
  K.qk_norm_rope_store(P, b.to(dev), 0, H * d if own else -1, (H + G) * d if own else -1, H, G, d, dv, R,
                       torch.arange(pos0, pos0 + T, dtype=torch.int32, device=dev), tab, slots.to(dev), eps, False, q, kc, vc,
                       rows(t["q.norm"], H).to(dev), rows(t["k.norm"], G).to(dev) if own else None)
  tol = 1e-5 if dtype == torch.float32 else 1e-2
  close(q, wq[..., order], tol, "q")
  if not own:
    assert float(kc.min()) == float(kc.max()) == 7.0 and float(vc.min()) == float(vc.max()) == 7.0
    return
  for i in range(T):
    s = int(slots[i])
    if s >= 0:
      close(kc[s // 64, :, s % 64], wk[i][:, order], tol, f"k {i}")
      close(vc[s // 64, :, :, s % 64], wv[i], tol, f"v {i}")
  free = pages[(pos0 + 4) // 64] * 64 + (pos0 + 4) % 64
  assert float(kc[free // 64, :, free % 64].max()) == 7.0


CASES = [  # H, G, d, dv, chunk, context lengths, new tokens
  (8, 2, 16, 24, 37, [150, 131], [19, 1]), (4, 2, 96, 96, 100, [150, 201], [101, 1]), (2, 1, 128, 128, 64, [129, 70], [129, 6]),
  (4, 4, 32, 64, 200, [199, 201], [40, 40]), (6, 3, 72, 40, 50, [101, 50], [101, 50]), (3, 3, 64, 64, 1, [70, 33], [70, 1]),
  (16, 2, 64, 64, 130, [261, 260], [1, 1]), (5, 1, 12, 20, 9, [64, 65], [2, 1]), (2, 2, 96, 32, 0, [80, 20], [80, 20]),
  (8, 1, 128, 64, 300, [310, 290, 5, 301], [1, 1, 1, 1]), (32, 2, 96, 96, 1000, [640, 3], [1, 1]), (4, 1, 40, 40, 64, [700, 64], [1, 1]),
  (6, 1, 120, 88, 250, [500, 499, 251], [1, 1, 1]), (1, 1, 8, 8, 128, [127, 128, 129], [1, 1, 1]), (24, 1, 64, 128, 77, [154, 155], [1, 1]),
]


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("H,G,d,dv,chunk,n,new", CASES)
def test_chunk_attention(dev, dtype, H, G, d, dv, chunk, n, new):
  """Softmax with one in the denominator inside the query's chunk, over scrambled pages whose unused places hold large
  values; portions and single tokens, key and value sizes apart, a strong key in front of every chunk edge."""
  B, need = len(n), [-(-x // 64) for x in n]
  perm = torch.randperm(sum(need) + 2, generator=torch.Generator().manual_seed(5)).tolist()
  width = max(need) + 1
  tables, at = torch.zeros(B, width, dtype=torch.int32), 0
  for b in range(B):
    tables[b, :need[b]] = torch.tensor(perm[at:at + need[b]], dtype=torch.int32)
    at += need[b]
  kc = torch.full((sum(need) + 2, G, 64, d), 100.0, dtype=dtype)
  vc = torch.full((sum(need) + 2, G, dv, 64), 100.0, dtype=dtype)
  ks, vs = [], []
  for b in range(B):
    k, v = rnd(n[b], G, d, seed=10 + b), rnd(n[b], G, dv, seed=20 + b)
    if chunk:
      k[chunk - 1::chunk] *= 3.0  # (the last key of a chunk scores far up or down)
    k, v = k.to(dtype), v.to(dtype)
    for p in range(n[b]):
      kc[tables[b, p // 64], :, p % 64], vc[tables[b, p // 64], :, :, p % 64] = k[p], v[p]
    ks.append(k.double())
    vs.append(v.double())
  q = torch.cat([rnd(new[b], H, d, seed=30 + b) for b in range(B)]).to(dtype)
  cu = torch.tensor([0] + torch.tensor(new).cumsum(0).tolist(), dtype=torch.int32)
  out = torch.full((sum(new), H * dv + 8), 3.0, dtype=dtype, device=dev)
  scale = 0.5 / d ** 0.5
  K.attn_window_pool(q.to(dev), kc.to(dev), vc.to(dev), None, None, tables.to(dev), cu.to(dev),
                     torch.tensor(n, dtype=torch.int32, device=dev), torch.zeros(H, device=dev), scale, 0, 0, out[:, :H * dv],
                     max_qlen=max(new), chunk=chunk)
  for b in range(B):
    got = out[cu[b]:cu[b + 1], :H * dv].double().cpu().reshape(new[b], H, dv)
    for i in range(new[b]):
      p = n[b] - new[b] + i
      js = [j for j in range(n[b]) if oracle.sees(p, j, chunk)]
      for h in range(0, H, max(1, H // 4)):
        w = oracle.softmax_plus_one((ks[b][js, h // (H // G)] @ q[cu[b] + i, h].double()) * scale)
        close(got[i, h], w @ vs[b][js, h // (H // G)], 1e-4 if dtype == torch.float32 else 2.5e-2, f"sequence {b} token {p} head {h}")
  assert float(out[:, H * dv:].min()) == 3.0


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("E,top,groups,keep", [(10, 2, 2, 1), (6, 3, 3, 2), (4, 2, 4, 3), (48, 9, 8, 3), (5, 5, 1, 1), (1, 1, 1, 1), (40, 2, 20, 1)])
def test_grouped_softmax_routing(dev, E, top, groups, keep):
  """Softmax over all experts, the groups ranked by their largest score, weights as they are (they do not sum to one)."""
  T = 40
  z = rnd(T, E, seed=E) * 2.0
  out = K.moe_route_ds(z.to(dev), None, top, groups, keep, 1, False, False, 1.0)
  topw, topi = out[0].reshape(T, top).cpu(), out[1].reshape(T, top).cpu()
  for t in range(T):
    idx, w = oracle.route(z[t].double(), {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}})
    got = dict(zip(topi[t].tolist(), topw[t].tolist()))
    assert sorted(got) == sorted(idx), f"token {t}: experts {sorted(got)} for {sorted(idx)}"
    for e, we in zip(idx, w):
      assert abs(got[e] - we) < 1e-5


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_gelu_of_a_projection_times_a_table_slice(dev, dtype):
  T, n, V, cols, col0 = 11, 20, 30, 64, 41
  P, table = rnd(T, 40, seed=1, scale=2.0), rnd(V, cols, seed=2).to(dtype)
  ids = torch.tensor([0, 29, 3, 3, 7, 1, 2, 28, 5, 6, 4], dtype=torch.int32)
  out = torch.zeros(T, n + 12, dtype=dtype, device=dev)
  K.gelu_gather_mul(P.to(dev), 5, table.to(dev), ids.to(dev), col0, n, out)
  want = oracle.gelu_tanh(P[:, 5:5 + n].double()) * table[ids.long(), col0:col0 + n].double()
  close(out[:, :n], want, 1e-5 if dtype == torch.float32 else 1e-2)
  assert float(out[:, n:].abs().max()) == 0.0


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_clamped_gate_of_the_shared_expert(dev, dtype):
  T, n, lim = 6, 24, 0.7
  P = rnd(T, 64, seed=1, scale=2.0)
  out = torch.zeros(T, n, dtype=dtype, device=dev)
  K.glu_act(P.to(dev), 3, 33, n, True, lim, out)
  t = {"gate": torch.eye(n, dtype=F64), "up": torch.eye(n, dtype=F64), "down": torch.eye(n, dtype=F64)}
  g, u = P[:, 3:3 + n].double(), P[:, 33:33 + n].double()
  want = torch.stack([oracle.clamped_expert(torch.cat([g[i], u[i]])[None],
                                            {"gate": torch.cat([t["gate"], 0 * t["gate"]], 1), "up": torch.cat([0 * t["up"], t["up"]], 1),
                                             "down": t["down"]}, "", lim)[0] for i in range(T)])
  close(out, want, 1e-5 if dtype == torch.float32 else 1e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("T,E,k,F,D,bm", [(5, 6, 2, 128, 128, 0), (40, 4, 2, 128, 256, 0), (300, 3, 1, 256, 256, 0), (600, 4, 2, 256, 256, 256),
                                          (600, 4, 2, 256, 256, 2256), (300, 3, 2, 256, 256, 1128), (400, 2, 2, 256, 256, 2192)])
@pytest.mark.parametrize("shuffled", [False, True])
def test_grouped_gemm_with_the_clamped_epilogue(T, E, k, F, D, bm, shuffled):
  """The experts' gate / up products with the clamped gate applied in the GEMM's epilogue, both grouped GEMM kernels."""
  from xotorch_support_jetson_amd.ops._ext import require
  from xotorch_support_jetson_amd.ops.weights_layout import shuffle_for_stream
  if bm and not shuffled:
    pytest.skip("the tall tiles read pre-shuffled weights")
  lim = 0.9
  x = rnd(T, D, seed=1).bfloat16()
  g, u = rnd(E, F, D, seed=2, scale=D ** -0.5 * 2).bfloat16(), rnd(E, F, D, seed=3, scale=D ** -0.5 * 2).bfloat16()
  idx = torch.randint(0, E, (T, k), generator=torch.Generator().manual_seed(4)).sort(1).values
  flat = idx.reshape(-1)
  order = torch.argsort(flat, stable=True)
  tok = (order // k).int()
  off = torch.cat([torch.zeros(1, dtype=torch.long), torch.bincount(flat, minlength=E).cumsum(0)]).int()
  W = torch.stack([interleave_gate_up(g[e], u[e]) for e in range(E)]).cuda()
  if shuffled:
    W = torch.stack([shuffle_for_stream(W[e].contiguous()) for e in range(E)])
  act = torch.full((T * k, F), 9.0, dtype=torch.bfloat16, device="cuda")
  require().gemm_moe(x.cuda(), W, act, off.cuda(), tok.cuda(), K.EPI["clamp_glu"], T, shuffled, 1, bm, lim)
  act = act.double().cpu()
  t = {"down": torch.eye(F, dtype=F64)}
  for e in range(E):
    lo, hi = int(off[e]), int(off[e + 1])
    want = oracle.clamped_expert(x[tok[lo:hi].long()].double(), dict(t, gate=g[e].double(), up=u[e].double()), "", lim)
    if hi > lo:
      close(act[lo:hi], want, 1e-2, f"expert {e}")


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 5, 40, 130, 300, 520, 2100])
@pytest.mark.parametrize("N,D", [(256, 128), (512, 384), (768, 256)])
def test_gemm_with_the_feed_forward_epilogues(M, N, D):
  """relu^2 and the clamped gate in the epilogue of the dense projections, every kernel configuration the policy would try."""
  from xotorch_support_jetson_amd.ops import linear as L
  lim = 0.9
  x = rnd(M, D, seed=1).bfloat16()
  w = rnd(N, D, seed=2, scale=D ** -0.5 * 2).bfloat16()
  up = torch.relu(x.double() @ w.double().T) ** 2
  g, u = w[:N // 2], w[N // 2:]
  glu = oracle.clamped_expert(x.double(), {"gate": g.double(), "up": u.double(), "down": torch.eye(N // 2, dtype=F64)}, "", lim)
  for epi, wt, want in (("relu2", w, up), ("clamp_glu", interleave_gate_up(g, u), glu)):
    ws = L.to_stream_layout(wt.contiguous().cuda())
    xd = x.cuda()
    close(L.linear(xd, ws, epi=epi, epi_arg=lim), want, 1.5e-2, f"{epi} as chosen")
    cands = [("stream",) + c for c in L.policy._stream_cands(M, N, D, epi)] if M <= 512 else []
    if M >= 65:
      cands += [c for c in L.policy._big_cands(M, N, D) if c[1] in (2256, 128, 4256)]
    for cfg in cands:
      out = torch.full((M, want.shape[1]), 7.0, dtype=torch.bfloat16, device="cuda")
      L._shuffled_call(xd, ws, None, None, epi, out, cfg, lim)
      close(out, want, 1.5e-2, f"{epi} {cfg}")


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 30])
def test_split_projection_read_as_slabs(M):
  """A split-K projection left unreduced: the consumers' sums equal the reduced product's results."""
  from xotorch_support_jetson_amd.ops import linear as L
  D, N, n = 1024, 256, 200
  x, w = rnd(M, D, seed=1).bfloat16().cuda(), L.to_stream_layout(rnd(N, D, seed=2, scale=D ** -0.5).bfloat16().cuda())
  key = ("sh", L._m_bucket(M), N, D, "none", False, str(torch.float32))
  keep = L.policy.table.get(key)
  try:
    L.policy.table[key] = ("stream", 1, 4)
    full = L.linear(x, w, out_dtype=torch.float32).clone()
    res = {}
    for name, P in (("slabs", L.linear_slabs(x, w)), ("reduced", full)):
      assert (P.dim() == 3) == (name == "slabs")
      h, o = rnd(M, n, seed=3).cuda(), torch.zeros(M, n, dtype=torch.bfloat16, device="cuda")
      K.sandwich_add_norm(h, P, rnd(n, seed=4).cuda(), None, 1e-5, o, yb=rnd(n, seed=5).cuda())
      e = torch.zeros(M, 64, dtype=torch.bfloat16, device="cuda")
      K.gelu_gather_mul(P, 100, rnd(9, 64, seed=6).bfloat16().cuda(), torch.arange(M, dtype=torch.int32, device="cuda") % 9, 3, 60, e)
      q = torch.empty(M, 4, 24, dtype=torch.bfloat16, device="cuda")
      kc, vc = (torch.zeros(1, 2, *s, dtype=torch.bfloat16, device="cuda") for s in ((64, 24), (20, 64)))
      K.qk_norm_rope_store(P, rnd(N, seed=7).cuda(), 0, 96, 144, 4, 2, 24, 20, 16, torch.arange(M, dtype=torch.int32, device="cuda"),
                           build_cos_sin(16, 64, 100.0, None, torch.device("cuda")), torch.arange(M, device="cuda"), 1e-5, False, q,
                           kc, vc, rnd(96, seed=8).cuda(), rnd(48, seed=9).cuda())
      res[name] = [t.double().cpu() for t in (h, o, e, q, kc, vc)]
    for a, b in zip(res["slabs"], res["reduced"]):
      close(a, b, 8e-3)
  finally:
    if keep is None:
      L.policy.table.pop(key, None)
    else:
      L.policy.table[key] = keep


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_values_of_many_tokens_are_stored_through_tiles(dtype):
  """300 tokens of several sequences at scrambled slots (some without one): keys and values as one by one."""
  T, H, G, d, dv = 300, 6, 3, 8, 40
  P = rnd(T, H * d + G * (d + dv), seed=1).cuda()
  slots = torch.randperm(384, generator=torch.Generator().manual_seed(2))[:T].cuda()
  slots[::17] = -1
  pos, tab = torch.arange(T, dtype=torch.int32, device="cuda") % 100, build_cos_sin(8, 100, 100.0, None, torch.device("cuda"))
  res = []
  for step in (T, 50):  # (50 tokens at a time: written by the rotation kernel itself)
    q = torch.empty(T, H, d, dtype=dtype, device="cuda")
    kc, vc = torch.full((6, G, 64, d), 5.0, dtype=dtype, device="cuda"), torch.full((6, G, dv, 64), 5.0, dtype=dtype, device="cuda")
    for lo in range(0, T, step):
      s = slice(lo, lo + step)
      K.qk_norm_rope_store(P[s], None, 0, H * d, (H + G) * d, H, G, d, dv, 8, pos[s], tab, slots[s].contiguous(), 1e-5, False, q[s], kc, vc,
                           torch.ones(H * d, device="cuda"), torch.ones(G * d, device="cuda"))
    res.append((q, kc, vc))
  for a, b in zip(*res):
    assert torch.equal(a, b)
  ok = (slots >= 0).cpu()
  s = slots.cpu()[ok]
  want = P[:, (H + G) * d:].cpu()[ok].reshape(-1, G, dv).to(dtype)
  assert torch.equal(res[0][2].cpu()[s // 64, :, :, s % 64], want)
