"""Plain float64 implementation of the Torinex design: whole sequences, one function per mechanism, one query at a time
where a mask decides what it sees.  Written from the design's equations only; it shares no code with the package and is
slow on purpose.  `tensors` maps checkpoint names to torch tensors, `cfg` is the parsed config.json."""
import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
  """x / sqrt(mean(x^2) + eps) * w over the last axis."""
  return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
  return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rope_interleaved(x, base, dims):
  """x [n, heads, d]: dims (2i, 2i + 1), i < dims / 2, of the token at position p turn by p * base^(-2i / dims)."""
  if not dims:
    return x
  out = x.clone()
  for p in range(x.shape[0]):
    for i in range(dims // 2):
      a = p * base ** (-2.0 * i / dims)
      u, v = x[p, :, 2 * i], x[p, :, 2 * i + 1]
      out[p, :, 2 * i] = u * math.cos(a) - v * math.sin(a)
      out[p, :, 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
  return out


def sees(i, j, chunk):
  """Token i attends to token j: not later, and in the same block of `chunk` positions (0: no blocks)."""
  return j <= i and (not chunk or i // chunk == j // chunk)


def softmax_plus_one(s):
  """exp(s) / (1 + sum exp(s)), as a softmax beside a logit of zero."""
  top = max(0.0, float(s.max()))
  e = torch.exp(s - top)
  return e / (math.exp(-top) + e.sum())


def chunk_attention(q, k, v, scale, chunk):
  """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]."""
  n, H, _ = q.shape
  G = k.shape[1]
  out = torch.zeros(n, H, v.shape[2], dtype=F64)
  for i in range(n):
    js = [j for j in range(n) if sees(i, j, chunk)]
    for h in range(H):
      g = h // (H // G)
      out[i, h] = softmax_plus_one((k[js, g] @ q[i, h]) * scale) @ v[js, g]
  return out


def project(h, t, name):
  return h @ t[name].T + t[name + ".b"]


def queries(h, m, t, p, eps):
  n, rot = h.shape[0], m.get("rot") or {}
  q = rms_norm(project(h, t, p + "q"), t[p + "q.norm"], eps)  # (one norm over all heads together)
  return rope_interleaved(q.reshape(n, m["heads"], m["dim"]), float(rot.get("base", 1.0)), int(rot.get("dims", 0)))


def keys_values(h, m, t, p, eps):
  n, rot = h.shape[0], m.get("rot") or {}
  k = rms_norm(project(h, t, p + "k"), t[p + "k.norm"], eps)
  k = rope_interleaved(k.reshape(n, m["kv_heads"], m["dim"]), float(rot.get("base", 1.0)), int(rot.get("dims", 0)))
  return k, project(h, t, p + "v").reshape(n, m["kv_heads"], m["vdim"])


def attention(h, m, t, p, eps, kept):
  """kept: {layer: (keys, values)} of the layers so far; a layer with kv_from reads another layer's."""
  k, v = kept
  o = chunk_attention(queries(h, m, t, p, eps), k, v, m["scale"], int((m.get("mask") or {}).get("size", 0)))
  return project(o.reshape(h.shape[0], -1), t, p + "o")


def relu2_mlp(h, t, p):
  return torch.relu(h @ t[p + "up"].T) ** 2 @ t[p + "down"].T


def clamped_expert(h, t, p, limit):
  g = (h @ t[p + "gate"].T).clamp(max=limit)
  u = (h @ t[p + "up"].T).clamp(-limit, limit)
  return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


def route(z, r):
  """Router logits z [E] -> (chosen experts, weights): softmax scores over all experts; the choice among the groups whose
  largest score is best; the scores themselves as weights."""
  E, top = r["experts"], r["top"]
  s = torch.softmax(z, -1)
  gr = r.get("groups") or {"count": 1, "keep": 1}
  cnt, keep = int(gr["count"]), int(gr["keep"])
  per = E // cnt
  best = sorted(range(cnt), key=lambda g: -float(s[g * per:(g + 1) * per].max()))[:keep]
  allowed = [e for e in range(E) if e // per in best]
  idx = sorted(allowed, key=lambda e: -float(s[e]))[:top]
  return idx, [float(s[e]) for e in idx]


def moe(h, f, t, p):
  out = torch.zeros(h.shape[0], t[p + "e0.down"].shape[0], dtype=F64)
  z = h @ t[p + "router"].T
  for i in range(h.shape[0]):
    for e, w in zip(*route(z[i], f["router"])):
      out[i] += w * clamped_expert(h[i], t, f"{p}e{e}.", f["expert"]["limit"])
  if f.get("shared"):
    out = out + clamped_expert(h, t, p + "shared.", f["shared"]["limit"])
  return out


def side_input(x, ids, i, dim, t, p, eps):
  """The layer's slice of the per-layer token table, gated by the stream: -> what is added to it."""
  e = t["side.embed"][ids, i * dim:(i + 1) * dim]
  y = (gelu_tanh(x @ t[p + "side.gate"].T) * e) @ t[p + "side.proj"].T
  return rms_norm(y, t[p + "side.norm"], eps)


def forward(cfg, tensors, tokens, collect=None):
  """Logits [n, vocab] of one sequence; collect: a list that receives the residual stream after every layer."""
  t = {k: v.to(F64) for k, v in tensors.items()}
  eps = cfg["norm"]["eps"]
  ids = torch.as_tensor(tokens, dtype=torch.long)
  x = t["embed"][ids]
  kept = {}
  for i, lay in enumerate(cfg["layers"]):
    p, m = f"l{i}.", lay["mixer"]
    if m.get("kv_from") is None:
      kept[i] = keys_values(x, m, t, p + "mix.", eps)
    y = attention(x, m, t, p + "mix.", eps, kept[i if m.get("kv_from") is None else m["kv_from"]])
    x = x + rms_norm(y, t[p + "norm1"], eps)
    f = lay.get("mlp")
    if f:
      y = relu2_mlp(x, t, p + "mlp.") if f["kind"] == "dense" else moe(x, f, t, p + "mlp.")
      x = x + rms_norm(y, t[p + "norm2"], eps)
    side = cfg.get("token_side")
    if side:
      x = x + side_input(x, ids, i, int(side["dim"]), t, p, eps)
    if collect is not None:
      collect.append(x.clone())
  return rms_norm(x, t["final.norm"], eps) @ t["embed"].T
