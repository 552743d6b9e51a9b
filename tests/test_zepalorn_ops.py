"""The ops behind Zepalorn's layers, one mechanism at a time, against the functions of tests/zepalorn_oracle.py: the torch
twins on the CPU and, marked gpu, the HIP kernels in float32 and bfloat16 (the activations' dtype; norms, scores, gates
and states are float32 in both)."""
import math

import pytest
import torch

import zepalorn_oracle as oracle
from xotorch_support_jetson_amd.models.config import WindowAttnSpec
from xotorch_support_jetson_amd.ops import kernels as K
from xotorch_support_jetson_amd.ops.reference import CONV_RMS, CONV_SILU, CONV_UNIT, CONV_UNIT_SCALED, conv_units
from xotorch_support_jetson_amd.ops.rope import build_cos_sin

RUNS = [pytest.param("cpu", torch.float32, id="cpu-f32"),
        pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=pytest.mark.gpu),
        pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)]
DEVS = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
F64 = torch.float64


def rnd(*shape, seed=0, scale=1.0):
  return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def close(got, want, tol, what=""):
  err = (got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-9)
  assert err < tol, f"{what}: off by {float(err):.3g}"


def cuts(lens, dev):
  return torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32, device=dev)


# ------------------------------------------------------------------ norms
@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("D", [36, 41, 1030, 2052, 4200, 8300])
def test_layer_norm_without_bias(dev, dtype, D):
  """x += LN(y) * wb and out = LN(x) * wn; a large common offset separates the layer norm from an RMS norm."""
  T, eps = 5, 1e-3
  x, y, wb, wn = rnd(T, D, seed=1) + 3.0, rnd(T, D + 8, seed=2) - 5.0, rnd(D, seed=3), rnd(D, seed=4)
  want = x.double() + oracle.layer_norm(y[:, :D].double(), wb.double(), eps)
  xd, out = x.clone().to(dev), torch.zeros(T, D + 4, dtype=dtype, device=dev)
  K.sandwich_add_norm(xd, y.to(dev), wb.to(dev), wn.to(dev), eps, out, layer=True)
  close(xd, want, 1e-5, "stream")
  close(out[:, :D], oracle.layer_norm(want, wn.double(), eps), 1e-5 if dtype == torch.float32 else 5e-3, "next operand")
  assert float(out[:, D:].abs().max()) == 0.0


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("D,S", [(40, 1), (96, 3), (1033, 2), (2048, 6), (3000, 1), (4400, 5)])
def test_mean_of_two_normed_rows(dev, D, S):
  T, eps = 4, 1e-4
  y1, y2, w = rnd(T, D, seed=1), rnd(S, T, D + 4, seed=2), rnd(2, D, seed=3)
  if dev == "cpu":
    y2 = y2.sum(0, keepdim=True)
  want = 0.5 * (oracle.rms(y1.double(), eps) * w[0].double() + oracle.rms(y2.double().sum(0)[:, :D], eps) * w[1].double())
  out = torch.empty(T, D, device=dev)
  K.pair_norm_mean(y1.to(dev), (y2 if y2.shape[0] > 1 else y2[0]).to(dev), w.to(dev), eps, out)
  close(out, want, 1e-5)


# ------------------------------------------------------------------ short convolutions
def _conv_want(x, w, b, parts, norm_w, eps):
  y, out, c0 = oracle.short_conv(x, w, b), [], 0
  for part in parts:
    n, kind = part[0], part[1]
    u = y[:, c0:c0 + n]
    u = oracle.silu(u) if kind & CONV_SILU else u
    if kind & (CONV_UNIT | CONV_UNIT_SCALED):
      u = u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6) * (n ** -0.5 if kind & CONV_UNIT_SCALED else 1.0)
    elif kind & CONV_RMS:
      u = oracle.rms(u, eps) * norm_w[part[2]:part[2] + n]
    out.append(u)
    c0 += n
  return torch.cat(out, 1)


CONVS = [
  [(24, CONV_SILU | CONV_UNIT_SCALED)] * 2 + [(24, CONV_SILU | CONV_UNIT)] * 2 + [(72, CONV_SILU)],
  [(16, CONV_RMS, 0)] * 3 + [(16, CONV_RMS, 16)] + [(300, 0), (77, CONV_SILU)],
  [(128, CONV_SILU | CONV_UNIT_SCALED), (128, CONV_SILU | CONV_UNIT), (256, CONV_SILU)],
  [(200, CONV_RMS, 0), (256, CONV_UNIT)], [(7, CONV_SILU), (3, CONV_UNIT), (5, CONV_RMS, 9)], [(600, CONV_SILU)],
]


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("n", range(len(CONVS)))
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_convolutions_in_portions(dev, n, taps):
  """Three sequences in unequal portions (down to one token, shorter than the filter, none at all, a step of single tokens)
  continue from their states; another slot's state and an inactive sequence's stay as they were."""
  parts, eps, off = CONVS[n], 1e-4, 3
  C = sum(p[0] for p in parts)
  units, width = conv_units(parts, C)
  assert int(units[:, 1].max()) <= width and int(units[:, 1].sum()) == C
  w, b, nw = rnd(C, taps, seed=1), (rnd(C, seed=2) if n % 2 else None), rnd(256, seed=3)
  seqs = [rnd(30, C + off + 2, seed=10 + i) for i in range(3)]
  want = [_conv_want(s[:, off:off + C].double(), w.double(), None if b is None else b.double(), parts, nw.double(), eps) for s in seqs]
  state = torch.full((6, taps - 1, C), 9.0, device=dev)
  slots = [4, 0, 2]
  for s in slots:
    state[s] = 0.0
  at, live = [0, 0, 0], torch.tensor(slots + [-1], dtype=torch.int32, device=dev)
  for lens in ([7, 1, 2], [1, 0, 20], [1, 1, 1], [20, 3, 1], [1, 25, 6]):
    lens = [min(k, 30 - a) for k, a in zip(lens, at)]
    P = torch.cat([s[a:a + k] for s, a, k in zip(seqs, at, lens)] + [rnd(1, C + off + 2, seed=50)]).to(dev)
    T = P.shape[0]
    if dev != "cpu" and lens[0] == 20:  # as split-K slabs
      part = rnd(2, T, P.shape[1], seed=60).to(dev)
      P = torch.stack([part[0], P - part[0] - part[1], part[1]])
    out = torch.full((T, C), 5.0, device=dev)
    K.conv_prep(P, off, w.to(dev), None if b is None else b.to(dev), units.to(dev), nw.to(dev), state, live, cuts(lens + [1], dev), eps,
                out, max_qlen=max(lens), width=width)
    o = 0
    for i in range(3):
      if lens[i]:
        close(out[o:o + lens[i]], want[i][at[i]:at[i] + lens[i]], 2e-5, f"taps {taps}, sequence {i}, tokens {at[i]}..")
      o += lens[i]
      at[i] += lens[i]
    assert float(out[o:].min()) == 5.0
  if taps > 1:
    assert float(state[[1, 3, 5]].min()) == float(state[[1, 3, 5]].max()) == 9.0
    for i, s in enumerate(slots):
      close(state[s], seqs[i][at[i] - (taps - 1):at[i], off:off + C].double(), 1e-5, "state")


@pytest.mark.gpu
def test_convolutions_of_many_tokens():
  """Runs of 32 tokens a wave, sequence borders inside them."""
  lens, taps, parts = [700, 1, 333, 2, 100], 4, CONVS[0]
  C = sum(p[0] for p in parts)
  units, width = conv_units(parts, C)
  w, nw = rnd(C, taps, seed=1), rnd(1, seed=3)
  P = rnd(sum(lens), C, seed=4)
  out, state = torch.empty(sum(lens), C, device="cuda:0"), torch.zeros(5, taps - 1, C, device="cuda:0")
  K.conv_prep(P.cuda(), 0, w.cuda(), None, units.cuda(), None, state, torch.arange(5, dtype=torch.int32, device="cuda:0"), cuts(lens, "cuda:0"),
              1e-5, out, max_qlen=700, width=width)
  o = 0
  for n in lens:
    close(out[o:o + n], _conv_want(P[o:o + n].double(), w.double(), None, parts, nw.double(), 1e-5), 2e-5, f"{n} tokens")
    o += n


def test_conv_units_refuse_what_does_not_fit():
  with pytest.raises(ValueError):
    conv_units([(300, CONV_RMS, 0)], 300)
  with pytest.raises(ValueError):
    conv_units([(30, 0)], 31)


# ------------------------------------------------------------------ gates
@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("H,d,dv,ra,rg,T", [(3, 20, 12, 24, 8, 5), (2, 64, 96, 128, 40, 19), (1, 1, 1, 1, 3, 9), (4, 130, 7, 7, 160, 8), (2, 32, 64, 512, 16, 1)])
def test_gates_of_the_channel_delta_rule(dev, dtype, H, d, dv, ra, rg, T):
  P = rnd(T, ra + rg + H + 5, seed=1)
  a2, g2 = rnd(H * d, ra, seed=2, scale=ra ** -0.5).to(dtype), rnd(H * dv, rg, seed=3, scale=rg ** -0.5).to(dtype)
  dt_bias, A_log = rnd(H * d, seed=4, scale=4.0), rnd(H, seed=5)
  z = P[:, :ra].double() @ a2.double().T + dt_bias.double()
  want = torch.exp(-torch.exp(A_log.double())[None, :, None] * torch.log1p(torch.exp(z)).reshape(T, H, d)).reshape(T, -1)
  args = dict(device=dev)
  beta, decay, gate = torch.empty(T, H, **args), torch.empty(T, H * d, **args), torch.empty(T, H * dv, **args)
  Pd = P.to(dev)
  if dev != "cpu" and T == 19:
    part = rnd(4, *P.shape, seed=9).to(dev)
    Pd = torch.cat([part, (Pd - part.sum(0))[None]])
  K.recurrence_gates(Pd, ra + rg, beta, 0, a2.to(dev), dt_bias.to(dev), A_log.to(dev), decay, ra, g2.to(dev), gate)
  close(beta, torch.sigmoid(P[:, ra + rg:ra + rg + H].double()), 1e-5, "beta")
  close(decay, want, 1e-5, "decay")
  close(gate, P[:, ra:ra + rg].double() @ g2.double().T, 2e-5, "gate")
  beta2, decay2 = torch.empty_like(beta), torch.empty_like(decay)
  za = torch.cat([(z - dt_bias.double()).float(), torch.full((T, 4), 7.0)], 1).to(dev)
  K.recurrence_gates(Pd, ra + rg, beta2, 0, None, dt_bias.to(dev), A_log.to(dev), decay2, 0, None, None, za=za)
  close(beta2, beta.double().cpu(), 1e-6, "beta beside a finished product")
  close(decay2, want, 1e-5, "decay of a finished product")


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("kind", ["gates", "steps"])
@pytest.mark.parametrize("taps", [1, 3, 4, 7])
def test_single_tokens_do_convolutions_and_gates_at_once(dev, dtype, kind, taps):
  """One call for convolutions and gates (or step sizes) gives what the separate ones give, states included; a padding row
  (slot -1) keeps its hands off the states."""
  T, H, d, dv, ra, rg, C = 11, 3, 20, 24, 40, 12, 2 * 20 + 90
  parts = [(20, CONV_SILU | CONV_UNIT), (20, CONV_RMS, 3), (90, CONV_SILU)]
  units, width = conv_units(parts, C)
  n = C + ra + rg + 2 * H
  P, w, nw = rnd(T, n, seed=1).to(dev), rnd(C, taps, seed=2).to(dev), rnd(30, seed=3).to(dev)
  if dev != "cpu":
    P = torch.stack([P * 0.5, P * 0.25, P * 0.25])
  slots = torch.tensor([3, 0, 7, 1, -1, 2, 9, 8, 4, 10, 5], dtype=torch.int32, device=dev)
  state = rnd(12, taps - 1, C, seed=4).to(dev)
  dt_bias, A_log = rnd(H * d if kind == "gates" else H, seed=5).to(dev), rnd(H, seed=6).to(dev)
  a2, g2 = rnd(H * d, ra, seed=7).to(dev, dtype), rnd(H * dv, rg, seed=8).to(dev, dtype)

  def outs():
    s = {"out": torch.full((T, C), 2.0, device=dev), "state": state.clone(), "decay": torch.zeros(T, dt_bias.numel(), device=dev),
         "first": torch.zeros(T, H, device=dev), "gate": torch.zeros(T, H * dv, device=dev)}
    args = (C, s["first"], C + H, a2, dt_bias, A_log, s["decay"], C + H + ra, g2, s["gate"]) if kind == "gates" else \
      (C, dt_bias, A_log, s["first"], s["decay"])
    return s, args
  both, args = outs()
  conv = (0, w, None, units.to(dev), nw)
  K.conv_prep(P, *conv, both["state"], slots, cuts([1] * T, dev), 1e-5, both["out"], max_qlen=1, width=width, **{kind: args})
  apart, args = outs()
  K.conv_prep(P, *conv, apart["state"], slots, cuts([1] * T, dev), 1e-5, apart["out"], max_qlen=1, width=width)
  (K.recurrence_gates if kind == "gates" else K.ssd_steps)(P, *args)
  for k in both:
    assert torch.equal(both[k], apart[k]), k
  assert torch.equal(both["state"][[6, 11]], state[[6, 11]]) and float(both["out"][4].min()) == 2.0


@pytest.mark.parametrize("dev", DEVS)
def test_ssd_steps(dev):
  T, H = 7, 5
  P, b, A = rnd(T, 12, seed=1, scale=5.0), rnd(H, seed=2), rnd(H, seed=3)
  dt, decay = torch.empty(T, H, device=dev), torch.empty(T, H, device=dev)
  K.ssd_steps(P.to(dev), 4, b.to(dev), A.to(dev), dt, decay)
  want = torch.log1p(torch.exp(P[:, 4:9].double() + b.double()))
  close(dt, want, 1e-5)
  close(decay, torch.exp(-torch.exp(A.double()) * want), 1e-5)


# ------------------------------------------------------------------ recurrences
def _recurrence_case(dev, H, G, d, dv, lens, chan, seed=0):
  T = sum(lens)
  q, k = rnd(T, G * d, seed=seed + 1, scale=d ** -0.5), torch.nn.functional.normalize(rnd(T, G, d, seed=seed + 2), dim=-1).reshape(T, -1)
  v, beta = rnd(T, H * dv, seed=seed + 3), torch.rand(T, H, generator=torch.Generator().manual_seed(seed + 4))
  g = 1.0 - 0.4 * torch.rand(T, H * (d if chan else 1), generator=torch.Generator().manual_seed(seed + 5)) ** 2
  return q, k, v, g, beta


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 24, 40), (3, 3, 7, 5), (2, 1, 128, 130), (1, 1, 2, 1), (2, 2, 64, 64), (2, 1, 200, 33)])
def test_delta_rule_with_channel_decays(dev, H, G, d, dv):
  """Two steps of three sequences over their slots; the state's key rows decay one by one, not all alike."""
  lens = [21, 1, 30]
  q, k, v, g, beta = _recurrence_case(dev, H, G, d, dv, lens, True)
  state, slots = torch.full((5, H, dv, d), 3.0, device=dev), [3, 1, 4]
  for s in slots:
    state[s] = 0.0
  src, o, want = [h // (H // G) for h in range(H)], 0, []
  for n in lens:
    s = slice(o, o + n)
    want.append(oracle.channel_delta_state(q[s].double().reshape(n, G, d)[:, src], k[s].double().reshape(n, G, d)[:, src],
                                           v[s].double().reshape(n, H, dv), g[s].double().reshape(n, H, d), beta[s].double()))
    o += n
  got, first = [[], [], []], [9, 0, 30]
  for lo, hi in ((None, first), (first, lens)):
    idx, ln = [], []
    for i in range(3):
      a, e = (lo[i] if lo else 0), hi[i]
      base = sum(lens[:i])
      idx += list(range(base + a, base + e))
      ln.append(e - a)
    out = torch.empty(len(idx), H * dv, device=dev)
    K.linear_recurrence(q[idx].to(dev), k[idx].to(dev), v[idx].to(dev), g[idx].to(dev), beta[idx].to(dev), 1.0, state,
                        torch.tensor(slots, dtype=torch.int32, device=dev), cuts(ln, dev), out)
    for i, part in enumerate(out.cpu().split(ln)):
      got[i].append(part)
  for i in range(3):
    close(torch.cat(got[i]).reshape(lens[i], H, dv), want[i], 2e-5, f"sequence {i}")
  assert float(state[[0, 2]].min()) == float(state[[0, 2]].max()) == 3.0


@pytest.mark.gpu
@pytest.mark.parametrize("rule", ["delta", "ssd"])
def test_recurrences_with_two_channels_a_thread(rule):
  """Enough (sequence, head, channel block) workgroups for the kernel that keeps two value channels per thread, with value
  channels that do not fill its last block."""
  B, L, H, G, d, dv = 16, 16, 16, 8, 12, 72
  q, k, v, g, beta = _recurrence_case("cuda:0", H, G, d, dv, [L] * B, rule == "delta")
  state, out = torch.zeros(B, H, dv, d, device="cuda:0"), torch.empty(B * L, H * dv, device="cuda:0")
  K.linear_recurrence(q.cuda(), k.cuda(), v.cuda(), g.cuda(), beta.cuda(), 1.0, state, torch.arange(B, dtype=torch.int32, device="cuda:0"),
                      cuts([L] * B, "cuda:0"), out, plain=rule == "ssd")
  src = [h // (H // G) for h in range(H)]
  for b in (0, 7, 15):
    s = slice(b * L, b * L + L)
    qq, kk, vv = q[s].double().reshape(L, G, d)[:, src], k[s].double().reshape(L, G, d)[:, src], v[s].double().reshape(L, H, dv)
    if rule == "delta":
      want = oracle.channel_delta_state(qq, kk, vv, g[s].double().reshape(L, H, d), beta[s].double())
    else:
      want, S = torch.zeros(L, H, dv, dtype=F64), torch.zeros(H, d, dv, dtype=F64)
      for t in range(L):
        S = g[s][t].double()[:, None, None] * S + torch.einsum("hd,hv->hdv", kk[t], vv[t] * beta[s][t].double()[:, None])
        want[t] = torch.einsum("hdv,hd->hv", S, qq[t])
    close(out[s].reshape(L, H, dv), want, 2e-5, f"sequence {b}")


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("H,dv,groups,S", [(6, 8, 2, 1), (4, 64, 4, 3), (3, 7, 3, 1), (8, 128, 1, 1), (2, 12, 1, 2)])
def test_ssd_skip_gate_and_grouped_norm(dev, dtype, H, dv, groups, S):
  """The convolved rows are the last columns of wider ones; the gate may lie in split-K slabs."""
  T, inner, eps = 5, H * dv, 1e-3
  o, x, D, w, z = rnd(T, inner, seed=1), rnd(T, inner + 20, seed=2), rnd(H, seed=3), rnd(inner, seed=4), rnd(T, inner + 8, seed=5)
  y = (o.double() + (x[:, 8:8 + inner].double().reshape(T, H, dv) * D.double()[None, :, None]).reshape(T, inner)) * oracle.silu(z[:, 4:4 + inner].double())
  want = oracle.rms(y.reshape(T, groups, -1), eps).reshape(T, inner) * w.double()
  P = z.to(dev)
  if S > 1 and dev != "cpu":
    part = rnd(S - 1, *z.shape, seed=9).to(dev)
    P = torch.cat([part, (P - part.sum(0))[None]])
  out = torch.zeros(T, inner + 4, dtype=dtype, device=dev)
  K.ssd_gate_norm(o.to(dev), x.to(dev)[:, 8:], D.to(dev), P, 4, w.to(dev), groups, eps, out)
  close(out[:, :inner], want, 2e-5 if dtype == torch.float32 else 6e-3)
  assert float(out[:, inner:].abs().max()) == 0.0


# ------------------------------------------------------------------ rotation, attention
@pytest.mark.parametrize("rot", [
  {"base": 20000.0, "dims": 32, "scaling": {"factor": 6.0, "original": 4096, "fast": 24.0, "slow": 1.0}},
  {"base": 500.0, "dims": 6, "scaling": {"factor": 3.0, "original": 64, "fast": 4.0, "slow": 2.0}},
  {"base": 1e6, "dims": 64, "scaling": {"factor": 1.0, "original": 4096, "fast": 32.0, "slow": 1.0}},
  {"base": 100.0, "dims": 4, "scaling": {"factor": 4.0, "original": 1000000, "fast": 1.0, "slow": 0.5}},  # (hi below lo)
  {"base": 10000.0, "dims": 16, "scaling": {"factor": 2.0, "original": 1, "fast": 3.0, "slow": 3.0}},
  {"base": 10000.0, "dims": 16}])
def test_yarn_table(rot):
  sc = rot.get("scaling")
  a = WindowAttnSpec(1, 1, 64, 64, 0, 0, rot["dims"], rot["base"],
                     ("yarn", sc["factor"], sc["original"], sc["fast"], sc["slow"]) if sc else None, 1.0)
  tab = build_cos_sin(rot["dims"], 300, rot["base"], a.rope_scaling(), "cpu").double()
  f, m = oracle.frequencies(rot)
  ang = torch.arange(300, dtype=F64)[:, None] * f[None, :]
  assert (tab - torch.cat([torch.cos(ang), torch.sin(ang)], 1) * m).abs().max() < 1e-6


CASES = [  # H, G, d, dv, window, chunk, keep, softcap, context lengths, new tokens
  (6, 2, 64, 64, 37, 0, 5, 0.0, [150, 131], [100, 1]), (6, 2, 64, 64, 37, 0, 70, 0.0, [250, 90], [1, 1]),
  (8, 2, 16, 24, 21, 0, 3, 0.0, [150, 40], [60, 1]), (6, 3, 72, 40, 65, 0, 1, 4.0, [180, 66], [80, 30]),
  (4, 1, 128, 128, 0, 90, 0, 3.0, [200, 91], [110, 91]), (4, 1, 128, 128, 0, 90, 0, 3.0, [200, 91, 180], [1, 1, 1]),
  (5, 5, 12, 20, 9, 0, 130, 0.0, [300, 64], [70, 3]), (2, 1, 128, 64, 64, 0, 64, 0.0, [400, 65], [150, 20]),
  (16, 1, 96, 96, 100, 0, 5, 2.0, [700, 260], [1, 1]), (3, 1, 40, 40, 1, 0, 2, 0.0, [70, 3], [70, 3]),
  (1, 1, 8, 8, 0, 5, 0, 1.5, [33, 70], [2, 5]), (4, 4, 32, 32, 200, 0, 10, 0.0, [150, 5], [150, 5]), (2, 2, 64, 64, 0, 64, 0, 30.0, [640, 1], [1, 1]),
]


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("H,G,d,dv,window,chunk,keep,cap,n,new", CASES)
def test_window_attention_with_kept_tokens_and_capped_scores(dev, dtype, H, G, d, dv, window, chunk, keep, cap, n, new):
  """Over scrambled pages whose unused places hold large values: prompts, short portions and single tokens, strong keys at the
  kept tokens' edge (the last kept one and the first that is not) and at every window's edge by way of many queries."""
  B, need = len(n), [-(-x // 64) for x in n]
  perm = torch.randperm(sum(need) + 2, generator=torch.Generator().manual_seed(5)).tolist()
  width = max(need) + 1
  tables, at = torch.zeros(B, width, dtype=torch.int32), 0
  for b in range(B):
    tables[b, :need[b]] = torch.tensor(perm[at:at + need[b]], dtype=torch.int32)
    at += need[b]
  kc = torch.full((sum(need) + 2, G, 64, d), 50.0, dtype=dtype)
  vc = torch.full((sum(need) + 2, G, dv, 64), 50.0, dtype=dtype)
  ks, vs = [], []
  for b in range(B):
    k, v = rnd(n[b], G, d, seed=10 + b), rnd(n[b], G, dv, seed=20 + b)
    for p in (keep - 1, keep):
      if 0 <= p < n[b]:
        k[p] *= 4.0
    k[7::11] *= 2.5
    k, v = k.to(dtype), v.to(dtype)
    for p in range(n[b]):
      kc[tables[b, p // 64], :, p % 64], vc[tables[b, p // 64], :, :, p % 64] = k[p], v[p]
    ks.append(k.double())
    vs.append(v.double())
  q = torch.cat([rnd(new[b], H, d, seed=30 + b) for b in range(B)]).to(dtype)
  cu = cuts(new, "cpu")
  scale = (2.0 if cap else 0.7) / d ** 0.5
  out = torch.full((sum(new), H * dv + 8), 3.0, dtype=dtype, device=dev)
  K.attn_window_pool(q.to(dev), kc.to(dev), vc.to(dev), None, None, tables.to(dev), cu.to(dev),
                     torch.tensor(n, dtype=torch.int32, device=dev), None, scale, window, 0, out[:, :H * dv], max_qlen=max(new),
                     chunk=chunk, keep=keep, softcap=cap)
  for b in range(B):
    got = out[cu[b]:cu[b + 1], :H * dv].double().cpu().reshape(new[b], H, dv)
    for i in range(0, new[b], 1 if new[b] < 40 else 3):
      p = n[b] - new[b] + i
      js = [j for j in range(n[b]) if (oracle.sees_chunk(p, j, chunk) if chunk else oracle.sees_window(p, j, window, keep))]
      for h in range(0, H, max(1, H // 3)):
        s = (ks[b][js, h // (H // G)] @ q[cu[b] + i, h].double()) * scale
        s = cap * torch.tanh(s / cap) if cap else s
        close(got[i, h], torch.softmax(s, 0) @ vs[b][js, h // (H // G)], 1e-4 if dtype == torch.float32 else 3e-2,
              f"sequence {b} token {p} head {h}")
  assert float(out[:, H * dv:].min()) == 3.0


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_capped_scores_far_beyond_the_cap(dev, dtype):
  """Scores of hundreds, both signs: equal weights among those at +cap, e^(-2 cap) for those at -cap."""
  n, d, cap = 40, 32, 1.5
  k = torch.ones(n, d)
  k[::2] = -1.0
  v = rnd(n, d, seed=1).to(dtype)
  kc, vc = torch.zeros(1, 1, 64, d, dtype=dtype), torch.zeros(1, 1, d, 64, dtype=dtype)
  kc[0, 0, :n], vc[0, 0, :, :n] = k.to(dtype), v.T
  for new in (1, 20):
    q = torch.full((new, 1, d), 20.0).to(dtype)
    out = torch.empty(new, d, dtype=dtype, device=dev)
    K.attn_window_pool(q.to(dev), kc.to(dev), vc.to(dev), None, None, torch.zeros(1, 1, dtype=torch.int32, device=dev), cuts([new], dev),
                       torch.tensor([n], dtype=torch.int32, device=dev), None, 1.0, 0, 0, out, max_qlen=new, softcap=cap)
    w = torch.tensor([math.exp(-2 * cap) if j % 2 == 0 else 1.0 for j in range(n)], dtype=F64)
    close(out[-1], (w[:, None] * v.double()).sum(0) / w.sum(), 1e-4 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("limit", [0.7, 5.0])
def test_clamped_gate_of_interleaved_columns(dev, dtype, limit):
  from xotorch_support_jetson_amd.models.transformer import ShardModel
  T, F = 5, 48
  g, u = rnd(T, F, seed=1, scale=2.0), rnd(T, F, seed=2, scale=2.0)
  P = torch.stack([g.view(T, 3, 16), u.view(T, 3, 16)], 2).reshape(T, 2 * F)
  out = torch.empty(T, F, dtype=dtype, device=dev)
  ShardModel._glu_tiles(P.to(dev), True, limit, out)
  gg, uu = torch.clamp(g.double(), max=limit), torch.clamp(u.double(), -limit, limit)
  close(out, gg * torch.sigmoid(1.702 * gg) * (uu + 1.0), 1e-5 if dtype == torch.float32 else 6e-3)
