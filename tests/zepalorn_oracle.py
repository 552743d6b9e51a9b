"""Plain float64 implementation of the Zepalorn design: whole sequences, token by token where a state is carried, one
function per mechanism.  Written from the design's equations only; it shares no code with the package and is slow on
purpose.  `tensors` maps checkpoint names to torch tensors, `cfg` is the parsed config.json."""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, eps):
  c = x - x.mean(-1, keepdim=True)
  return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def rms(x, eps):
  return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
  return x * torch.sigmoid(x)


def short_conv(u, w, b=None):
  """u [n, C] over time, w [C, taps] (last column: the current token), zeros before the start."""
  n, taps = u.shape[0], w.shape[1]
  y = torch.zeros_like(u)
  for t in range(n):
    for j in range(taps):
      s = t - (taps - 1) + j
      if s >= 0:
        y[t] += w[:, j] * u[s]
  return y if b is None else y + b


def frequencies(rot):
  """(frequencies [dims / 2], factor on cos and sin) of a rotation, with YaRN scaling when the config has it."""
  R, base = int(rot["dims"]), float(rot["base"])
  f = [base ** (-2.0 * i / R) for i in range(R // 2)]
  sc = rot.get("scaling")
  if not sc:
    return torch.tensor(f, dtype=F64), 1.0

  def dim(turns):
    return R * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
  lo = max(math.floor(dim(sc["fast"])), 0)
  hi = min(math.ceil(dim(sc["slow"])), R - 1)
  out = []
  for i, fi in enumerate(f):
    r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
    out.append(fi / sc["factor"] * r + fi * (1.0 - r))
  return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot, interleaved):
  """x [n, heads, d]: the pairs (2i, 2i + 1) (interleaved) or (i, i + dims / 2) of the token at position p turn by p f_i."""
  if not rot or not rot.get("dims"):
    return x
  R = int(rot["dims"])
  f, m = frequencies(rot)
  ang = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
  c, s = (m * torch.cos(ang))[:, None, :], (m * torch.sin(ang))[:, None, :]
  out = x.clone()
  if interleaved:
    u, v = x[..., 0:R:2].clone(), x[..., 1:R:2].clone()
    out[..., 0:R:2] = u * c - v * s
    out[..., 1:R:2] = v * c + u * s
  else:
    u, v = x[..., :R // 2].clone(), x[..., R // 2:R].clone()
    out[..., :R // 2] = u * c - v * s
    out[..., R // 2:R] = v * c + u * s
  return out


def sees_window(i, j, size, keep):
  return j <= i and (not size or i - j < size or j < keep)


def sees_chunk(i, j, size):
  return j <= i and (not size or i // size == j // size)


def attend(q, k, v, scale, sees, softcap=0.0):
  """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]: softmax over the keys j for which sees(i, j)."""
  n, H, _ = q.shape
  G = k.shape[1]
  mask = torch.tensor([[sees(i, j) for j in range(n)] for i in range(n)])
  out = torch.zeros(n, H, v.shape[2], dtype=F64)
  for h in range(H):
    g = h // (H // G)
    s = (q[:, h] @ k[:, g].T) * scale
    if softcap:
      s = softcap * torch.tanh(s / softcap)
    out[:, h] = torch.softmax(s.masked_fill(~mask, -math.inf), -1) @ v[:, g]
  return out


def window_attention(h, m, t, p):
  n = h.shape[0]
  H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  mask = m.get("mask") or {}
  q = rotate((h @ t[p + "q"].T).reshape(n, H, d), m.get("rot"), False)
  k = rotate((h @ t[p + "k"].T).reshape(n, G, d), m.get("rot"), False)
  v = (h @ t[p + "v"].T).reshape(n, G, dv)
  size, keep = int(mask.get("size", 0)), int(mask.get("keep_first", 0))
  o = attend(q, k, v, m["scale"], lambda i, j: sees_window(i, j, size, keep))
  return o.reshape(n, H * dv) @ t[p + "o"].T


def conv_attention(h, m, t, p, eps):
  """Chunk-local attention on convolved projections, per-head query / key norms, capped scores."""
  n = h.shape[0]
  H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q = short_conv(h @ t[p + "q"].T, t[p + "q.conv"]).reshape(n, H, d)
  k = short_conv(h @ t[p + "k"].T, t[p + "k.conv"]).reshape(n, G, d)
  v = short_conv(h @ t[p + "v"].T, t[p + "v.conv"]).reshape(n, G, dv)
  q = rotate(rms(q, eps) * t[p + "q.norm"], m.get("rot"), True)
  k = rotate(rms(k, eps) * t[p + "k.norm"], m.get("rot"), True)
  size = int((m.get("mask") or {}).get("size", 0))
  o = attend(q, k, v, m["scale"], lambda i, j: sees_chunk(i, j, size), float(m.get("softcap") or 0.0))
  return o.reshape(n, H * dv) @ t[p + "o"].T


def channel_delta_state(q, k, v, g, beta):
  """q, k [n, H, d], v [n, H, dv], g [n, H, d], beta [n, H] -> o [n, H, dv]; the state's key rows decay one by one."""
  n, H, d = q.shape
  out = torch.zeros(n, H, v.shape[2], dtype=F64)
  for h in range(H):
    S = torch.zeros(d, v.shape[2], dtype=F64)
    for i in range(n):
      S = g[i, h][:, None] * S
      u = beta[i, h] * (v[i, h] - S.T @ k[i, h])
      S = S + torch.outer(k[i, h], u)
      out[i, h] = S.T @ q[i, h]
  return out


def channel_delta(h, m, t, p, eps):
  n = h.shape[0]
  H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q = silu(short_conv(h @ t[p + "q"].T, t[p + "q.conv"])).reshape(n, G, d)
  k = silu(short_conv(h @ t[p + "k"].T, t[p + "k.conv"])).reshape(n, G, d)
  v = silu(short_conv(h @ t[p + "v"].T, t[p + "v.conv"])).reshape(n, H, dv)
  q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * d ** -0.5
  k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
  beta = torch.sigmoid(h @ t[p + "b"].T)
  z = (h @ t[p + "a1"].T) @ t[p + "a2"].T + t[p + "dt_bias"]
  rate = torch.exp(t[p + "A_log"])[None, :, None]
  g = torch.exp(-rate * torch.nn.functional.softplus(z).reshape(n, H, d))
  src = [hd // (H // G) for hd in range(H)]
  o = channel_delta_state(q[:, src], k[:, src], v, g, beta)
  o = rms(o, eps) * t[p + "norm"] * torch.sigmoid((h @ t[p + "g1"].T) @ t[p + "g2"].T).reshape(n, H, dv)
  return o.reshape(n, H * dv) @ t[p + "o"].T


def mamba2(h, m, t, p, eps):
  n = h.shape[0]
  H, dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
  inner = H * dv
  z, x, B, C, dt = torch.split(h @ t[p + "in"].T, [inner, inner, G * N, G * N, H], dim=1)
  xbc = silu(short_conv(torch.cat([x, B, C], 1), t[p + "conv"], t[p + "conv.b"]))
  x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=1)
  x, B, C = x.reshape(n, H, dv), B.reshape(n, G, N), C.reshape(n, G, N)
  dt = torch.nn.functional.softplus(dt + t[p + "dt_bias"])
  a = torch.exp(-torch.exp(t[p + "A_log"]) * dt)
  y = torch.zeros(n, H, dv, dtype=F64)
  for hd in range(H):
    g = hd // (H // G)
    S = torch.zeros(N, dv, dtype=F64)
    for i in range(n):
      S = a[i, hd] * S + dt[i, hd] * torch.outer(B[i, g], x[i, hd])
      y[i, hd] = S.T @ C[i, g] + t[p + "D"][hd] * x[i, hd]
  y = (y.reshape(n, inner) * silu(z)).reshape(n, m["norm_groups"], -1)
  return (rms(y, eps).reshape(n, inner) * t[p + "norm"]) @ t[p + "o"].T


def parallel_mixer(h, m, t, p, eps):
  a = conv_attention(h, m["left"], t, p + "left.", eps)
  b = mamba2(h, m["right"], t, p + "right.", eps)
  return 0.5 * (rms(a, eps) * t[p + "left.out"] + rms(b, eps) * t[p + "right.out"])


def clamped_glu(h, f, t, p):
  lim = float(f["limit"])
  g = torch.clamp(h @ t[p + "gate"].T, max=lim)
  u = torch.clamp(h @ t[p + "up"].T, -lim, lim)
  return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


def owner(cfg, i):
  """The layer whose tensors layer i uses."""
  while cfg["layers"][i].get("weights_of") is not None:
    i = int(cfg["layers"][i]["weights_of"])
  return i


def forward(cfg, tensors, tokens, collect=None):
  """Logits [n, vocab] of one sequence; collect: a list that receives the residual stream after every layer."""
  t = {k: v.to(F64) for k, v in tensors.items()}
  eps = cfg["norm"]["eps"]
  x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
  for i, lay in enumerate(cfg["layers"]):
    p = f"l{owner(cfg, i)}."
    h = layer_norm(x, t[p + "norm1"], eps)
    kind = lay["type"]
    if kind == "channel_delta":
      y = channel_delta(h, lay["mixer"], t, p + "mix.", eps)
    elif kind == "attention":
      y = window_attention(h, lay["mixer"], t, p + "mix.")
    elif kind == "parallel":
      y = parallel_mixer(h, lay["mixer"], t, p + "mix.", eps)
    else:
      raise ValueError(kind)
    x = x + layer_norm(y, t[p + "norm1b"], eps)
    if lay.get("mlp"):
      y = clamped_glu(layer_norm(x, t[p + "norm2"], eps), lay["mlp"], t, p + "mlp.")
      x = x + layer_norm(y, t[p + "norm2b"], eps)
    if collect is not None:
      collect.append(x.clone())
  return layer_norm(x, t["final.norm"], eps) @ t["embed"].T
