"""Plain, slow implementation of the decoder with chunked grouped-query attention and norms behind the sublayers (design
"Feduzen"), one function per mechanism: numpy, whole sequences, no cache, no batching.

TEST INFRASTRUCTURE ONLY.  It is written from the equations and shares no code with the product:

  start     x = scale * embed[token]
  layer     x <- x + N_1(A(x)),  x <- x + N_2(F(x));   N(y) = y / sqrt(mean y^2 + eps) * w;   the sublayers read x itself
  A         q, k, v = W x + b;  per head q, k <- N(q), N(k) (one weight for all heads), then rotated in the first d
            dimensions: pairs (i, i + d/2), angle p f_i, f_i = base^(-2 i / d), slow waves slowed down further
            score = q . k * scale over j <= p of p's own chunk (floor(j / size) = floor(p / size)), softmax with exp(sink)
            in the denominator;  query head h reads key / value head floor(h / (H / G))
  F         W_d relu(W_u x)^2
  output    logits = W_head N(x)

`rnd` is applied where the product in bf16 rounds a value to bf16 (identity for the exact result).
"""
import math

import numpy as np


def rms_norm(x, w, eps):
  return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def rotary_frequencies(rot):
  """f [dims / 2] of a rotation {'dims', 'base', optional 'scaling': {'factor', 'low', 'high', 'original'}}."""
  d, s = rot['dims'], rot.get('scaling')
  out = []
  for i in range(d // 2):
    f = rot['base'] ** (-2.0 * i / d)
    if s:
      wave = 2.0 * math.pi / f
      if wave > s['original'] / s['low']:
        f = f / s['factor']
      elif wave >= s['original'] / s['high']:
        t = (s['original'] / wave - s['low']) / (s['high'] - s['low'])
        f = (1.0 - t) * f / s['factor'] + t * f
    out.append(f)
  return np.array(out)


def rotate(x, positions, rot):
  """x [T, D] with its first rot['dims'] columns rotated at positions [T]."""
  h = rot['dims'] // 2
  ang = positions[:, None].astype(np.float64) * rotary_frequencies(rot)
  c, s = np.cos(ang), np.sin(ang)
  u, v = x[:, :h], x[:, h:2 * h]
  return np.concatenate([u * c - v * s, v * c + u * s, x[:, 2 * h:]], -1)


def visible(t, mask):
  """bool [T, T]: position i sees position j."""
  i, j = np.arange(t)[:, None], np.arange(t)[None]
  ok = j <= i
  if mask:
    ok &= i // mask['size'] == j // mask['size']
  return ok


def attend(q, k, v, scale, sink, ok):
  """One head: q [T, D], k [T, D], v [T, E]; sink: a logit without a value, or None."""
  s = np.where(ok, (q @ k.T) * scale, -np.inf)
  top = s.max(-1, keepdims=True)
  if sink is not None:
    top = np.maximum(top, sink)
  e = np.exp(s - top)
  den = e.sum(-1, keepdims=True)
  if sink is not None:
    den = den + np.exp(sink - top)
  return (e / den) @ v


def mixer(w, p, m, h, eps, rnd):
  t, H, G = h.shape[0], m['heads'], m['kv_heads']
  pos = np.arange(t)
  q, k, v = (rnd(h @ w[f'{p}.{n}'].T + w[f'{p}.{n}.b']).reshape(t, c, -1) for n, c in (('q', H), ('k', G), ('v', G)))
  head = lambda x, n: rnd(rotate(rms_norm(x, w[f'{p}.{n}.norm'], eps), pos, m['rot']))
  keys = [head(k[:, g], 'k') for g in range(G)]
  ok = visible(t, m.get('mask'))
  out = []
  for a in range(H):
    g = a // (H // G)
    out.append(rnd(attend(head(q[:, a], 'q'), keys[g], v[:, g], m['scale'], float(w[f'{p}.sink'][a]), ok)))
  return rnd(np.concatenate(out, -1) @ w[f'{p}.o'].T)


def feed_forward(w, p, h, rnd):
  return rnd(rnd(np.maximum(h @ w[f'{p}.up'].T, 0.0) ** 2) @ w[f'{p}.down'].T)


def forward(cfg, w, tokens, rnd=None, dtype=np.float64, layers_out=None):
  """Logits [T, V] of one sequence.  cfg: the model's configuration as a mapping; w: name -> array.
  layers_out: list that receives the residual after every layer."""
  rnd = rnd or (lambda x: x)
  w = {k: np.asarray(v, dtype) for k, v in w.items()}
  eps = cfg['norm']['eps']
  x = w['embed'][np.asarray(tokens)] * cfg['embedding']['scale']
  for i, layer in enumerate(cfg['layers']):
    src = i
    while cfg['layers'][src].get('weights_of') is not None:
      src = cfg['layers'][src]['weights_of']
    l = f'l{src}'
    x = x + rms_norm(mixer(w, f'{l}.mix', layer['mixer'], rnd(x), eps, rnd), w[f'{l}.norm1'], eps)
    if layer.get('mlp'):
      x = x + rms_norm(feed_forward(w, f'{l}.mlp', rnd(x), rnd), w[f'{l}.norm2'], eps)
    if layers_out is not None:
      layers_out.append(x)
  return rnd(rms_norm(x, w['final.norm'], eps)) @ w['head'].T
