"""Zepalorn in the framework against the plain implementation in tests/zepalorn_oracle.py.

Every test makes its own small configuration and random checkpoint tensors, runs them through the serving runner (paged
caches and state slots per layer, batched steps; HIP kernels and HIP-graph decode on a GPU, the torch twins on the CPU) and
compares logits at every position with the oracle's float64 run over the whole sequence.  Each body runs on the CPU and,
marked gpu, on cuda:0 in float32 and bfloat16.
"""
import asyncio
import json

import numpy as np
import pytest
import torch

import zepalorn_oracle as oracle
from xotorch_support_jetson_amd.inference.shard import Shard
from xotorch_support_jetson_amd.models.config import TINY_ZEPALORN, from_hf_config
from xotorch_support_jetson_amd.models.weights import mixed_weights, needed_files, random_mixed_tensors
from xotorch_support_jetson_amd.runtime.runner import ShardRunner

RUNS = [pytest.param("cpu", torch.float32, id="cpu-f32"),
        pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=pytest.mark.gpu),
        pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)]
TOL = {torch.float32: 2e-4, torch.bfloat16: 6e-2}
YARN = {"factor": 4.0, "original": 128, "fast": 16.0, "slow": 1.0}


def rot(dims, base=10000.0, scaling=YARN):
  r = {"base": base, "dims": dims}
  return dict(r, scaling=scaling) if scaling else r


def delta(heads=4, kv_heads=2, dim=16, vdim=24, conv=3, rank=12, gate_rank=20):
  return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "rank": rank, "gate_rank": gate_rank}


def attention(heads=6, kv_heads=2, dim=16, vdim=8, window=20, keep=3, scale=0.3, r=None):
  m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot(8) if r is None else r}
  if window:
    m["mask"] = {"size": window, "keep_first": keep}
  if not m["rot"]:
    del m["rot"]
  return m


def pair(heads=4, kv_heads=1, dim=24, vdim=16, conv=2, chunk=37, cap=8.0, scale=0.25, r=None, rheads=6, rvdim=8, state=20, groups=3, rconv=4,
         norm_groups=2):
  left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale, "rot": rot(16, 5000.0) if r is None else r,
          "mask": {"size": chunk}, "softcap": cap}
  for k in ("rot", "softcap"):
    if not left[k]:
      del left[k]
  return {"left": left, "right": {"heads": rheads, "vdim": rvdim, "state": state, "groups": groups, "conv": rconv, "norm_groups": norm_groups}}


def dense(ff=72, limit=1.2):
  return {"kind": "dense", "ff": ff, "limit": limit}


def layer(kind, mixer, mlp=None, of=None):
  out = {"type": kind, "mixer": mixer, "mlp": mlp}
  if of is not None:
    out["weights_of"] = of
  return out


def config(layers, width=64, vocab=96, eps=1e-5, scale=4.0):
  return {"architecture": "Zepalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


SMALL = config([layer("channel_delta", delta(), dense()), layer("attention", attention(), dense(56, 2.0)),
                layer("channel_delta", delta(), dense(), of=0), layer("parallel", pair(), dense(40)),
                layer("attention", attention(), dense(56, 2.0), of=1), layer("parallel", pair(), dense(40), of=3)])
_ORACLE = {}


class Rig:
  """A configuration + random tensors in the runner and in the oracle."""

  def __init__(self, cfg, dev, dtype, seed=1, pages=24, slots=4, tweak=None, graphs=None):
    self.cfg, self.dev, self.dtype = cfg, torch.device(dev), dtype
    self.c = from_hf_config(cfg)
    self.tensors = random_mixed_tensors(self.c, seed)
    if tweak:
      tweak(self.tensors)
    self.key = None if tweak else (json.dumps(cfg, sort_keys=True), seed)
    shard = Shard("t", 0, self.c.num_layers - 1, self.c.num_layers)
    w = mixed_weights(self.c, shard, self.tensors.__getitem__, self.dev, dtype)
    self.runner = ShardRunner(self.c, shard, self.dev, weights=w, num_pages=pages, max_batch=slots, max_ctx=pages * 64,
                              dtype=dtype, use_graphs=graphs)
    self.V = self.c.vocab_size
    self.memo = {}

  def tokens(self, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, self.V, (n,), generator=g).tolist()

  def want(self, toks):
    memo = self.memo if self.key is None else _ORACLE.setdefault(self.key, {})
    k = tuple(toks)
    if k not in memo:
      memo[k] = oracle.forward(self.cfg, self.tensors, toks)
    return memo[k]

  def step(self, entries):
    """entries [(rid, tokens)] -> logits of every token of the step, split per entry."""
    rids = [r for r, _ in entries]
    qlens = [len(t) for _, t in entries]
    flat = [t for _, ts in entries for t in ts]
    out = self.runner.forward(rids, qlens, torch.tensor(flat, dtype=torch.int32), logit_rows=list(range(len(flat))))
    return list(out.double().cpu().split(qlens))

  def run_alone(self, rid, toks, cuts):
    """One request in portions of the given sizes (the last size repeats); logits at every position."""
    outs, lo, i = [], 0, 0
    while lo < len(toks):
      n = min(cuts[min(i, len(cuts) - 1)], len(toks) - lo)
      outs.append(self.step([(rid, toks[lo:lo + n])])[0])
      lo, i = lo + n, i + 1
    self.runner.free(rid)
    return torch.cat(outs)

  def check(self, got, toks, what=""):
    want = self.want(toks)
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    worst = int(err.argmax())
    assert err.max() < TOL[self.dtype], f"{what}: position {worst} of {len(toks)} is off by {float(err.max()):.3g}"


def moves(a, b, by=0.05):
  return (a - b).abs().max() > by * b.abs().max()


# ------------------------------------------------------------------ whole prompts, portions, decoding
@pytest.mark.parametrize("dev,dtype", RUNS)
def test_whole_prompt(dev, dtype):
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(110, 3)
  rig.check(rig.run_alone("a", toks, [len(toks)]), toks, "whole prompt")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_long_prompt(dev, dtype):
  """Enough tokens for the second projections of the low-rank gates to run as GEMMs, in one step and cut in the middle."""
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(300, 13)
  rig.check(rig.run_alone("a", toks, [300]), toks, "one step")
  rig.check(rig.run_alone("a", toks, [270, 1, 2, 1]), toks, "a long portion, then short ones")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_residual_stream_after_every_layer(dev, dtype):
  """The stream after each layer, read off by running the first layers only."""
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(40, 4)
  trail = []
  oracle.forward(rig.cfg, rig.tensors, toks, trail)
  model = rig.runner.model
  all_runs = model.runs
  assert len(trail) == len(all_runs) == 6
  model.shard = Shard("t", 0, 4, rig.c.num_layers)  # (not the last layer: forward returns the hidden state)
  try:
    for n in range(1, len(all_runs) + 1):
      model.runs = all_runs[:n]
      x = rig.runner.forward(["a"], [len(toks)], torch.tensor(toks, dtype=torch.int32)).double().cpu()
      rig.runner.free("a")
      err = (x - trail[n - 1]).abs().max() / trail[n - 1].abs().max()
      assert err < (1e-4 if dtype == torch.float32 else 3e-2), f"after layer {n - 1}: {float(err):.3g}"
  finally:
    model.runs = all_runs


MECHANISMS = {
  "channel-delta": config([layer("channel_delta", delta())], 48, 60),
  "shared-tensors": config([layer("channel_delta", delta(2, 1, 8, 8)), layer("channel_delta", delta(2, 1, 8, 8), of=0),
                            layer("channel_delta", delta(2, 1, 8, 8), of=1)], 48, 60),
  "kept-tokens": config([layer("attention", attention(4, 2, 16, 32, window=9, keep=5))], 48, 60),
  "parallel": config([layer("parallel", pair())], 48, 60),
  "clamped-ff": config([layer("attention", attention(1, 1, 8, 8, window=4, keep=0), dense(56, 0.4))], 48, 60),
}


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("kind", list(MECHANISMS))
def test_each_mechanism_alone(dev, dtype, kind):
  rig = Rig(MECHANISMS[kind], dev, dtype, seed=7)
  toks = rig.tokens(80, 5)
  rig.check(rig.run_alone("a", toks, [len(toks)]), toks, f"{kind}: prompt")
  rig.check(rig.run_alone("a", toks, [30, 2, 1, 1, 17, 1]), toks, f"{kind}: portions and decoding")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_first_tokens(dev, dtype):
  """Sequences of one to six tokens: shorter than the filters, at and just past the kept tokens."""
  rig = Rig(SMALL, dev, dtype)
  for n in range(1, 7):
    toks = rig.tokens(n, 10 + n)
    rig.check(rig.run_alone("a", toks, [n]), toks, f"{n}-token prompt")
    rig.check(rig.run_alone("a", toks, [1]), toks, f"{n} tokens one by one")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_prefill_against_decoding(dev, dtype):
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(110, 3)
  whole = rig.run_alone("a", toks, [len(toks)])
  single = rig.run_alone("b", toks, [1])
  rig.check(single, toks, "token by token")
  assert (whole - single).abs().max() < TOL[dtype] * whole.abs().max()


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("cuts", [[2], [3, 2, 5, 1, 1, 7], [47, 1, 1, 17, 2], [64, 1], [63, 2, 1], [100, 1], [19, 2, 16, 2, 35, 2]])
def test_portions(dev, dtype, cuts):
  """A prompt cut anywhere (inside pages, windows, chunks and filters, at their edges, down to two tokens)."""
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(110, 3)
  rig.check(rig.run_alone("a", toks, cuts), toks, f"portions {cuts}")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_long_decoding(dev, dtype):
  """A short prompt, then 150 single tokens: pages, windows and chunks are crossed while decoding."""
  rig = Rig(SMALL, dev, dtype)
  toks = rig.tokens(165, 6)
  rig.check(rig.run_alone("a", toks, [15, 1]), toks, "long decoding")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_graph_decoding_matches_eager(dtype):
  """Single-token steps replayed from a captured HIP graph (no logit rows asked: the runner's decode path) give the
  logits of the eager steps, replay after replay, with eager prompt steps of another request in between; three requests
  in a batch bucket of four leave a padding row."""
  rig = Rig(SMALL, "cuda:0", dtype, graphs=True)
  toks = [rig.tokens(70, 8 + i) for i in range(3)]
  want = [rig.run_alone(f"e{i}", t, [30, 1]) for i, t in enumerate(toks)]
  rids = ["g0", "g1", "g2"]
  for r, t in zip(rids, toks):
    rig.runner.forward([r], [30], torch.tensor(t[:30], dtype=torch.int32))
  for i in range(30, 70):
    out = rig.runner.forward(rids, [1] * 3, torch.tensor([t[i] for t in toks], dtype=torch.int32)).double().cpu()
    for b in range(3):
      assert (out[b] - want[b][i]).abs().max() < TOL[dtype] * want[b][i].abs().max(), f"step {i}, request {b}"
    if i % 7 == 0:
      rig.run_alone("other", rig.tokens(30, i), [30])
  for r in rids:
    rig.runner.free(r)


# ------------------------------------------------------------------ batches, pages, slots
@pytest.mark.parametrize("dev,dtype", RUNS)
def test_mixed_batches_match_alone(dev, dtype):
  """Unequal requests in one step (portions beside single tokens, a request that sits a step out) give each the
  logits it gets alone."""
  rig = Rig(SMALL, dev, dtype, pages=12)
  seqs = {"a": rig.tokens(110, 3), "b": rig.tokens(70, 22), "c": rig.tokens(9, 23), "d": rig.tokens(40, 24)}
  plan = [[("a", 50), ("b", 2)], [("a", 1), ("b", 30), ("c", 9)], [("a", 1), ("d", 17)], [("a", 40), ("b", 1), ("d", 1)],
          [("b", 37), ("d", 22)], [("a", 18)]]
  at = {k: 0 for k in seqs}
  got = {k: [] for k in seqs}
  for stepplan in plan:
    entries = [(r, seqs[r][at[r]:at[r] + n]) for r, n in stepplan]
    for (r, n), o in zip(stepplan, rig.step(entries)):
      got[r].append(o)
      at[r] += n
      if at[r] == len(seqs[r]):
        rig.runner.free(r)
  for r, toks in seqs.items():
    assert at[r] == len(toks)
    rig.check(torch.cat(got[r]), toks, f"request {r} in mixed batches")


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_pages_and_slots_are_reused(dev, dtype):
  """Four pages and two state slots serve six requests in turn, two at a time: every page and slot is handed out again with
  another request's keys, states and convolution inputs in it."""
  rig = Rig(SMALL, dev, dtype, pages=4, slots=2)
  for rnd in range(3):
    seqs = {f"r{rnd}x": rig.tokens(100 + rnd, 30 + rnd), f"r{rnd}y": rig.tokens(90 - rnd, 40 + rnd)}
    got = {k: [] for k in seqs}
    for lo in range(0, 128, 16):
      entries = [(r, t[lo:lo + 16]) for r, t in seqs.items() if t[lo:lo + 16]]
      if not entries:
        break
      for (r, _), o in zip(entries, rig.step(entries)):
        got[r].append(o)
    for r, toks in seqs.items():
      rig.runner.free(r)
      rig.check(torch.cat(got[r]), toks, f"round {rnd} request {r}")
  assert rig.runner.bm.num_free == 4 and rig.runner.sm.num_free == 2


# ------------------------------------------------------------------ other sizes
SIZES = [
  # one of everything: heads, groups, taps, a window and a chunk of one token, no kept tokens, no rotation, no cap, rank 1
  config([layer("channel_delta", delta(1, 1, 8, 8, conv=1, rank=1, gate_rank=1), dense(16)), layer("attention", attention(1, 1, 8, 8, window=1, keep=0, r={})),
          layer("parallel", pair(1, 1, 8, 8, conv=1, chunk=1, cap=0, r={}, rheads=1, rvdim=8, state=1, groups=1, rconv=1, norm_groups=1))],
         width=40, vocab=50, scale=1.0),
  # sizes that are no multiples of 8 or 16, filters of five and six taps, the left one longer, key sizes above 64, odd ranks
  config([layer("channel_delta", delta(6, 3, 12, 20, conv=6, rank=7, gate_rank=33), dense(50)),
          layer("parallel", pair(6, 3, 72, 12, conv=5, chunk=70, cap=3.0, r=rot(40, 1e6, None), rheads=5, rvdim=6, state=9, groups=5, rconv=2, norm_groups=3), dense(24)),
          layer("attention", attention(5, 5, 76, 20, window=70, keep=66, r=rot(6)), dense(8, 0.3)),
          layer("parallel", pair(6, 3, 72, 12, conv=5, chunk=70, cap=3.0, r=rot(40, 1e6, None), rheads=5, rvdim=6, state=9, groups=5, rconv=2, norm_groups=3), dense(24), of=1)],
         width=72, vocab=130, scale=9.0),
  # many heads on one, value sizes above and below the keys', everything causal, norm groups across heads
  config([layer("channel_delta", delta(8, 1, 40, 8, conv=2)), layer("attention", attention(8, 1, 32, 40, window=0, keep=0)),
          layer("parallel", pair(8, 2, 16, 48, conv=3, chunk=0, cap=20.0, rheads=8, rvdim=16, state=64, groups=1, rconv=3, norm_groups=4), dense(130, 7.0))],
         width=32, vocab=40, scale=5.5),
  # heads as in larger models: 128 wide, ranks of 128, several kv heads, the matrix-core attention kernels
  config([layer("channel_delta", delta(2, 2, 128, 128, conv=4, rank=128, gate_rank=64), dense(256)),
          layer("attention", attention(4, 2, 128, 128, window=50, keep=4, r=rot(64), scale=0.09)),
          layer("parallel", pair(2, 1, 64, 64, conv=4, chunk=48, cap=10.0, r=rot(64), rheads=4, rvdim=64, state=128, groups=2, rconv=4, norm_groups=2))],
         width=128, vocab=64, scale=11.0),
  # shared tensors in a chain and ahead of their owner, layers in another order
  config([layer("parallel", pair(), None, of=3), layer("channel_delta", delta(), None), layer("channel_delta", delta(), None, of=1),
          layer("parallel", pair(), None), layer("channel_delta", delta(), None, of=2)], width=56, vocab=70),
]


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("n", range(len(SIZES)))
def test_other_sizes(dev, dtype, n):
  rig = Rig(SIZES[n], dev, dtype, seed=50 + n)
  toks = rig.tokens(150 if n == 1 else 90, 60 + n)
  rig.check(rig.run_alone("a", toks, [33, 2, 1, 1, 29, 1]), toks, f"sizes {n}")


# ------------------------------------------------------------------ faults that random weights would hide
def _marked_window(window, keep):
  """One attention layer whose keys measure how much a token's normed input points along token B's and whose queries do
  so times a large negative factor; token C's embedding is minus token B's, so C's query stands far above all others on
  B's key: whether a B is visible moves C's logits."""
  d = 8
  cfg = config([layer("attention", attention(2, 1, d, 16, window=window, keep=keep, scale=1.0, r={}))], width=32, vocab=24, scale=1.0)

  def tweak(t):
    t["embed"][2] = -t["embed"][1]
    e = t["embed"][1] - t["embed"][1].mean()
    e = e / e.pow(2).mean().sqrt() * t["l0.norm1"]
    w = (torch.ones(d, 1) * e[None, :] / e.pow(2).sum()).bfloat16().float()
    t["l0.mix.k"], t["l0.mix.q"] = w, torch.cat([-w, -w]) * 1.25
  return cfg, tweak


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("window,keep", [(16, 4), (64, 1), (65, 64), (9, 70), (100, 0), (44, 130)])
def test_window_and_kept_token_edges(dev, dtype, window, keep):
  """B as the last kept token and as the first that is not kept, B just inside and just outside the window: in a prompt, in
  portions that end on and straddle the edges, and decoded one by one."""
  cfg, tweak = _marked_window(window, keep)
  rig = Rig(cfg, dev, dtype, tweak=tweak, pages=16)
  n = keep + 3 * window + 8
  base = [3 + (i % 5) for i in range(n)]
  for b, c in ((keep - 1, keep + 2 * window), (keep, keep + 2 * window), (keep + 5, keep + 5 + window - 1), (keep + 5, keep + 5 + window)):
    if b < 0:
      continue
    toks = list(base)
    toks[b], toks[c] = 1, 2
    rig.check(rig.run_alone("a", toks, [n]), toks, f"B at {b}, C at {c}: prompt")
    rig.check(rig.run_alone("a", toks, [c - 1, 2, 2]), toks, f"B at {b}, C at {c}: portions")
    rig.check(rig.run_alone("a", toks, [max(c - 2, 1), 1]), toks, f"B at {b}, C at {c}: decoded")
    other = list(toks)
    other[b] = 3
    seen = oracle.sees_window(c, b, window, keep)
    assert moves(rig.want(other)[c], rig.want(toks)[c]) == seen, "the test must bite"


def _marked_chunk(chunk):
  """One parallel layer without rotation whose left filters pass only the current token and whose left keys measure token B's
  direction in half of their dims and every token's common direction in the other half (the head norms leave the ratio);
  C's queries stand far above all others on B's key."""
  d = 8
  cfg = config([layer("parallel", pair(2, 1, d, 16, conv=2, chunk=chunk, cap=30.0, scale=1.2, r={}, rheads=2, rvdim=8, state=4, groups=1, rconv=2, norm_groups=1))],
               width=32, vocab=24, scale=1.0)

  def tweak(t):
    common = torch.randn(32, generator=torch.Generator().manual_seed(3))
    common -= common.mean()
    b = torch.randn(32, generator=torch.Generator().manual_seed(4))
    b -= b.mean()
    b -= common * (b @ common) / common.pow(2).sum()
    t["embed"] = t["embed"] * 0.3 + common
    t["embed"][1], t["embed"][2] = common + 2.0 * b, common - 2.0 * b
    t["l0.norm1"] = torch.ones(32)
    wb, wc = b / b.pow(2).sum(), common / common.pow(2).sum()
    t["l0.mix.left.k"] = torch.cat([wb.repeat(d // 2, 1), wc.repeat(d // 2, 1)]).bfloat16().float()
    q = torch.cat([-wb.repeat(d // 2, 1), 0.5 * wc.repeat(d // 2, 1)])
    t["l0.mix.left.q"] = torch.cat([q, q]).bfloat16().float()
    for n in ("q", "k"):
      t[f"l0.mix.left.{n}.conv"] = torch.zeros_like(t[f"l0.mix.left.{n}.conv"])
      t[f"l0.mix.left.{n}.conv"][:, -1] = 1.0
      t[f"l0.mix.left.{n}.norm"] = torch.ones(d)
    t["l0.mix.right.out"] = t["l0.mix.right.out"] * 0.1
  return cfg, tweak


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("chunk", [16, 64, 65, 9])
def test_chunk_edges(dev, dtype, chunk):
  """A token B as the last of a chunk and as the first of the next, each followed by a C at the chunk's last and at the
  next chunk's first place: in a prompt, in portions that end on and straddle the edges, and decoded one by one."""
  cfg, tweak = _marked_chunk(chunk)
  rig = Rig(cfg, dev, dtype, tweak=tweak, pages=16)
  n = 4 * chunk + 3
  toks = [3 + (i % 5) for i in range(n)]
  for at, tok in ((chunk - 1, 1), (chunk, 2), (2 * chunk, 1), (3 * chunk - 1, 2), (3 * chunk, 2), (3 * chunk + 2, 1), (4 * chunk - 1, 2), (4 * chunk, 2)):
    toks[at] = tok
  rig.check(rig.run_alone("a", toks, [n]), toks, "prompt")
  rig.check(rig.run_alone("a", toks, [chunk, 2, chunk - 3, 2, 2, chunk, 3, 1]), toks, "portions over the edges")
  rig.check(rig.run_alone("a", toks, [max(chunk - 3, 1), 1]), toks, "decoding over the edges")
  for c2 in (chunk + 1, chunk - 1):
    cfg2 = json.loads(json.dumps(cfg))
    cfg2["layers"][0]["mixer"]["left"]["mask"]["size"] = c2
    assert moves(oracle.forward(cfg2, rig.tensors, toks), rig.want(toks)), "the test must bite"


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_far_kept_key(dev, dtype):
  """The last kept token, a thousand tokens and many pages before the query, and the first one that is not kept."""
  cfg, tweak = _marked_window(33, 66)
  rig = Rig(cfg, dev, dtype, tweak=tweak, pages=18)
  for b, seen in ((65, True), (66, False)):
    toks = [3 + (i % 7) for i in range(1100)]
    toks[b], toks[1090] = 1, 2
    got = rig.run_alone("a", toks, [900, 180, 8, 1])
    rig.check(got, toks, f"B at {b}")
    assert moves(rig.want(toks[:b] + [3] + toks[b + 1:])[1090], rig.want(toks)[1090]) == seen, "the test must bite"


@pytest.mark.parametrize("dev,dtype", RUNS)
@pytest.mark.parametrize("kind", ["channel_delta", "parallel"])
def test_a_first_token_survives_in_the_state(dev, dtype, kind):
  """Slow decays and a text of three words: what the first token wrote is still in the recurrent state 260 single-token steps
  later (a lost or restarted state shows)."""
  mixer = delta(2, 2, 32, 16, conv=2) if kind == "channel_delta" else pair(1, 1, 8, 8, chunk=2, r={}, rheads=4, rvdim=16, state=24, groups=2, norm_groups=1)
  cfg = config([layer(kind, mixer)], width=48, vocab=40)

  def tweak(t):
    p = "l0.mix." if kind == "channel_delta" else "l0.mix.right."
    t[p + "A_log"] = torch.full_like(t[p + "A_log"], -7.0)
    if kind == "parallel":
      t["l0.mix.left.out"] = t["l0.mix.left.out"] * 0.1
      # step sizes: large for the first token alone
      e = t["embed"][1] - t["embed"][1].mean()
      e = e / e.pow(2).mean().sqrt() * t["l0.norm1"]
      t[p + "dt_bias"] = torch.full_like(t[p + "dt_bias"], -4.0)
      t[p + "in"][-4:] = (10.0 * e / e.pow(2).sum()).bfloat16().float()
      t[p + "D"] = t[p + "D"] * 0.1
  rig = Rig(cfg, dev, dtype, tweak=tweak)
  toks = [1] + [3 + i % 3 for i in range(280)] + [9]
  got = rig.run_alone("a", toks, [20, 1])
  rig.check(got, toks, "decoded")
  rig.check(rig.run_alone("a", toks, [150, 2, 100, 1]), toks, "portions")
  assert moves(rig.want([2] + toks[1:])[-1], rig.want(toks)[-1]), "the first token must matter"


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_channel_decays_differ_within_a_head(dev, dtype):
  """Half of the key channels forget at once, the others hardly: one decay per head, whichever, would show."""
  cfg = config([layer("channel_delta", delta(2, 1, 16, 16))], width=48, vocab=40)

  def tweak(t):
    t["l0.mix.A_log"] = torch.zeros(2)
    b = torch.full((2, 16), -6.0)
    b[:, ::2] = 3.0
    t["l0.mix.dt_bias"] = b.reshape(-1)
  rig = Rig(cfg, dev, dtype, tweak=tweak)
  toks = rig.tokens(60, 2)
  rig.check(rig.run_alone("a", toks, [40, 1]), toks)
  flat = dict(rig.tensors)
  flat["l0.mix.dt_bias"] = torch.full((32,), -1.5)
  assert moves(oracle.forward(cfg, flat, toks), rig.want(toks))


@pytest.mark.parametrize("dev,dtype", RUNS)
def test_limit_of_the_feed_forward_shows(dev, dtype):
  cfg = config([layer("attention", attention(1, 1, 8, 8, window=4, keep=0), dense(40, 0.5))], 48, 60)

  def tweak(t):
    t["l0.mlp.gate"], t["l0.mlp.up"] = t["l0.mlp.gate"] * 6.0, t["l0.mlp.up"] * 6.0
  rig = Rig(cfg, dev, dtype, tweak=tweak)
  toks = rig.tokens(50, 2)
  rig.check(rig.run_alone("a", toks, [40, 1]), toks)
  c2 = json.loads(json.dumps(cfg))
  c2["layers"][0]["mlp"]["limit"] = 1.0
  assert moves(oracle.forward(c2, rig.tensors, toks), rig.want(toks))


# ------------------------------------------------------------------ configuration, shards
def test_configuration_is_read_from_the_json():
  c = from_hf_config(SIZES[1])
  r, p, a = (c.layer_specs[i] for i in range(3))
  assert (r.rec.rule, r.rec.heads, r.rec.kv_heads, r.rec.conv, r.rec.rank, r.rec.gate_rank) == ("channel_delta", 6, 3, 6, 7, 33)
  assert (p.wattn.chunk, p.wattn.conv, p.wattn.softcap, p.wattn.head_norm, p.wattn.rot_interleaved, p.wattn.rot_scaling) == (70, 5, 3.0, True, True, None)
  assert p.state_dims == (5, 6, 9, 5, 6 * 72 + 3 * 84 + 5 * 6 + 2 * 5 * 9, 0) and p.kv_dims == (3, 72, 12)
  assert (a.wattn.window, a.wattn.keep_first, a.wattn.rot_scaling) == (70, 66, ("yarn", 4.0, 128.0, 16.0, 1.0)) and a.state_dims is None
  assert c.embed_scale == 9.0 and c.norm_kind == "layer" and not c.norm_bias and c.tie_word_embeddings and c.has_state
  assert [c.weights_owner(i) for i in range(4)] == [0, 1, 2, 1]
  for cfg in (SMALL, *SIZES):
    cc = from_hf_config(cfg)
    assert cc.num_params() == sum(t.numel() for t in random_mixed_tensors(cc).values())
  short = json.loads(json.dumps(SMALL))  # a sharing layer may leave its entry to the owner
  short["layers"][2] = {"weights_of": 0}
  assert from_hf_config(short).layer_specs == from_hf_config(SMALL).layer_specs
  for bad in (layer("channel_delta", delta(3, 2)), layer("attention", attention(r=rot(7))), layer("attention", attention(5, 2)),
              layer("parallel", pair(groups=4)), layer("parallel", pair(norm_groups=5)), layer("mystery", delta())):
    with pytest.raises(ValueError):
      from_hf_config(config([bad]))
  for of in (5, 0):  # nobody, oneself
    with pytest.raises(ValueError, match="weights_of"):
      from_hf_config(config([layer("channel_delta", delta(), of=of)]))
  with pytest.raises(ValueError, match="weights_of"):  # another size
    from_hf_config(config([layer("channel_delta", delta()), layer("channel_delta", delta(dim=8), of=0)]))


def test_layers_that_share_tensors_share_them_on_the_device():
  c = from_hf_config(SMALL)
  w = mixed_weights(c, Shard("t", 0, 5, 6), random_mixed_tensors(c).__getitem__, torch.device("cpu"), torch.float32)
  assert w.layers[0] is w.layers[2] and w.layers[1] is w.layers[4] and w.layers[3] is w.layers[5]


@pytest.mark.parametrize("cut", [1, 3, 4])
def test_shards_in_a_row(cut):
  """Two shards give the whole model's logits, also where a layer's tensors belong to a layer of the other shard."""
  c = from_hf_config(SMALL)
  tensors = random_mixed_tensors(c, 3)
  runners = []
  for lo, hi in ((0, cut - 1), (cut, 5)):
    s = Shard("t", lo, hi, 6)
    w = mixed_weights(c, s, tensors.__getitem__, torch.device("cpu"), torch.float32)
    runners.append(ShardRunner(c, s, "cpu", weights=w, num_pages=8, max_batch=2, max_ctx=256, dtype=torch.float32))
  toks = torch.randint(0, 96, (50,), generator=torch.Generator().manual_seed(1)).tolist()
  got = []
  for lo, hi in ((0, 31), (31, 33), (33, 34), (34, 50)):
    h = runners[0].forward(["a"], [hi - lo], torch.tensor(toks[lo:hi], dtype=torch.int32))
    assert h.shape == (hi - lo, c.hidden_size) and h.dtype == torch.float32
    got.append(runners[1].forward(["a"], [hi - lo], h, logit_rows=list(range(hi - lo))))
  want = oracle.forward(SMALL, tensors, toks)
  assert (torch.cat(got).double() - want).abs().max() < 2e-4 * want.abs().max()


# ------------------------------------------------------------------ the engine's own entry point
@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)])
def test_greedy_generation_through_the_engine(dev):
  """Three prompts of unequal length at once through ShardedInferenceEngine (queue, batched steps, sampler at
  temperature 0): every token drawn is the oracle's greedy token for the text so far (ties within rounding
  aside), and all pages and slots are free at the end."""
  from xotorch_support_jetson_amd.download.shard_download import NoopShardDownloader
  from xotorch_support_jetson_amd.inference.sharded_engine import ShardedInferenceEngine
  from xotorch_support_jetson_amd.models.config import preset
  c = preset("tiny-zepalorn")
  tensors = random_mixed_tensors(c, 0)
  shard = Shard("tiny-zepalorn", 0, c.num_layers - 1, c.num_layers)
  prompts = {"p0": [7, 3, 99, 42, 5, 17], "p1": [11] * 53, "p2": [200, 1]}
  steps = 24

  async def one(e, rid, ids):
    out, st = await e.infer_tensor(rid, shard, np.array([ids]), {"temperature": 0.0})
    seq = list(ids)
    for _ in range(steps):
      tok = int(np.asarray(await e.sample(out, temp=0.0)).reshape(-1)[0])
      seq.append(tok)
      out, st = await e.infer_tensor(rid, shard, np.array([[tok]]), dict(st, temperature=0.0))
    await e.finish_request(rid)
    return seq

  async def main():
    e = ShardedInferenceEngine(NoopShardDownloader(), device=torch.device(dev))
    seqs = await asyncio.gather(*[one(e, r, p) for r, p in prompts.items()])
    return e, seqs
  e, seqs = asyncio.run(main())
  assert e.runner.bm.num_free == e.runner.bm.num_blocks and e.runner.sm.num_free == e.runner.max_batch
  slack = 0.05 if dev == "cpu" else 0.25  # (the GPU serves in bfloat16)
  for (rid, p), seq in zip(prompts.items(), seqs):
    lg = oracle.forward(TINY_ZEPALORN, tensors, seq[:-1])
    for t in range(len(p) - 1, len(seq) - 1):
      best = float(lg[t].max())
      assert float(lg[t][seq[t + 1]]) >= best - slack * float(lg[t].std()), f"{rid}: token {t + 1} is not the greedy one"


def _save(tmp_path, cfg, seed):
  from safetensors.torch import save_file
  tensors = random_mixed_tensors(from_hf_config(cfg), seed)
  plain = json.loads(json.dumps(cfg))
  for L in plain["layers"]:  # (a checkpoint's config names no ranks: the tensors' shapes give them)
    L["mixer"].pop("rank", None)
    L["mixer"].pop("gate_rank", None)
  (tmp_path / "config.json").write_text(json.dumps(plain))
  save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()}, str(tmp_path / "model.safetensors"))
  return tensors


def test_checkpoint_directory_through_registry_and_engine(tmp_path):
  """config.json + model.safetensors (bf16) in a folder: registered as a local model, loaded by the engine's own
  build path, and the prompt's last-token logits match the oracle run on the same tensors."""
  from xotorch_support_jetson_amd.download.shard_download import NoopShardDownloader
  from xotorch_support_jetson_amd.inference.sharded_engine import ShardedInferenceEngine
  from xotorch_support_jetson_amd.models import registry
  cfg = SIZES[1]
  tensors = _save(tmp_path, cfg, 5)
  mid = registry.register_local_model(str(tmp_path))
  assert mid is not None and registry.model_cards[mid]["layers"] == len(cfg["layers"])
  shard = registry.build_full_shard(mid, "ShardedInferenceEngine")
  toks = [3, 99, 7, 7, 120, 64, 1, 0, 55]

  async def main():
    e = ShardedInferenceEngine(NoopShardDownloader(), device=torch.device("cpu"))
    out, _ = await e.infer_tensor("r", shard, np.array([toks]), {})
    return e, out
  e, out = asyncio.run(main())
  assert e.config.model_type == "zepalorn" and e.config.layer_specs[2].wattn.keep_first == 66
  want = oracle.forward(cfg, tensors, toks)[-1]
  assert (out.double().reshape(-1) - want).abs().max() < 0.05 * want.abs().max()  # bf16 activations on the serving path
  assert needed_files(tmp_path, e.config, Shard("t", 3, 3, 4)) == {"model.safetensors"}


def test_wrong_shapes_are_refused(tmp_path):
  from safetensors.torch import save_file
  from xotorch_support_jetson_amd.models.weights import load_hf_weights
  tensors = _save(tmp_path, SIZES[0], 5)
  tensors["l0.mix.o"] = tensors["l0.mix.o"][:, :-1]
  save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()}, str(tmp_path / "model.safetensors"))
  with pytest.raises(ValueError, match="l0.mix.o"):
    load_hf_weights(tmp_path, from_hf_config(SIZES[0]), Shard("t", 0, 2, 3), "cpu", torch.float32)


def test_trace_replay(tmp_path):
  """The replay program on a checkpoint folder: two requests in portions and single tokens, logits at the asked places."""
  import io
  import sys
  from xotorch_support_jetson_amd import trace_run
  cfg = SIZES[4]
  tensors = _save(tmp_path, cfg, 6)
  a, b = [1, 2, 3, 4, 5, 6, 7, 8, 9], [30, 31, 32]
  steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:5], "want": [0, 4]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
           {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [0]}, {"id": "a", "tokens": a[5:], "want": [3]}], "end": ["a", "b"]}]
  keep = sys.stdin
  sys.stdin = io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n")
  try:
    assert trace_run.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path / "o"), "--max-tokens", "128",
                           "--device", "cpu"]) == 0
  finally:
    sys.stdin = keep
  wa, wb = oracle.forward(cfg, tensors, a), oracle.forward(cfg, tensors, b)
  for n, want in ((0, torch.stack([wa[0], wa[4]])), (1, torch.stack([wb[2], wa[8]]))):
    got = np.fromfile(tmp_path / "o" / f"{n}.f32", dtype="<f4").reshape(want.shape)
    assert np.abs(got - want.numpy()).max() < 2e-4 * float(want.abs().max())
