"""Plain, slow implementation of the decoder with latent attention and several residual streams (design
"Kagapel"), one function per mechanism: numpy, whole sequences, no cache, no batching.

TEST INFRASTRUCTURE ONLY.  It is written from the equations and shares no code with the product:

  streams   x_1 .. x_S, all equal to embed[token] + pos[p] at the start; per sublayer
            u = sum_s a_s x_s,  y = f(norm(u)),  x_t <- sum_s M_{s t} x_s + b_t y   (all t from the old x)
  mixer     q = W_q h per head [n | r];  (c', k_r) = W_dkv h;  c = norm(c');  k_n = W_uk c, v = W_uv c per head
            score = (q_n . k_n + R_p q_r . R_j k_r) * scale over j <= p, softmax (optionally with a sink term in
            the denominator), out = W_o (concat of the heads, optionally * sigmoid(W_g h))
  rotation  pairs (i, i + d/2), angle p f_i, f_i = base^(-2 i / d), optionally rescaled (YaRN)
  ff        W_d (silu(W_g h + b_g) * (W_u h + b_u)) + b_d
  output    logits = logit_scale * W_head norm(sum_s x_s)

`rnd` is applied where the product in bf16 rounds a value to bf16 (identity for the exact result).
"""
import math

import numpy as np

MIXERS = {'latent_attention': {'gate': True, 'sink': False}, 'latent_attention_2': {'gate': False, 'sink': True}}


def rms_norm(x, w, eps):
  return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def rotary_frequencies(rot):
  """(f [dims / 2], factor on cos and sin) of a rotation {'dims', 'base', optional 'scaling'}."""
  d, base = rot['dims'], rot['base']
  f = np.array([base ** (-2.0 * i / d) for i in range(d // 2)])
  s = rot.get('scaling')
  if not s:
    return f, 1.0
  dim_of = lambda turns: d * math.log(s['original'] / (2 * math.pi * turns)) / (2 * math.log(base))
  lo, hi = max(math.floor(dim_of(s['fast'])), 0), min(math.ceil(dim_of(s['slow'])), d - 1)
  out = np.empty_like(f)
  for i in range(d // 2):
    ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
    out[i] = f[i] / s['factor'] * ramp + f[i] * (1 - ramp)
  return out, 0.1 * math.log(s['factor']) + 1.0


def rotate(x, positions, rot):
  """x [..., T, dims] rotated at positions [T]."""
  f, mult = rotary_frequencies(rot)
  ang = positions[:, None].astype(np.float64) * f
  c, s = np.cos(ang) * mult, np.sin(ang) * mult
  h = rot['dims'] // 2
  u, v = x[..., :h], x[..., h:]
  return np.concatenate([u * c - v * s, v * c + u * s], -1)


def sigmoid(z):
  return 1.0 / (1.0 + np.exp(-z))


def latent_keys(w, p, m, h, eps, rnd):
  """(c [T, kv_rank], rotated shared key part [T, rot_dim]): what a layer's cache holds."""
  y = rnd(h @ w[f'{p}.dkv'].T)
  c = rnd(rms_norm(y[:, :m['kv_rank']], w[f'{p}.dkv.norm'], eps))
  kr = rnd(rotate(y[:, m['kv_rank']:], np.arange(h.shape[0]), m['rot']))
  return c, kr


def latent_attention(w, p, m, kind, h, c, kr, rnd):
  """Mixer output [T, D] from the normed input h and the layer's (or another layer's) latents."""
  t, H, n, r, vd = h.shape[0], m['heads'], m['dim'], m['rot_dim'], m['vdim']
  q = rnd(h @ w[f'{p}.q'].T).reshape(t, H, n + r)
  k = (c @ w[f'{p}.uk'].T).reshape(t, H, n)
  v = (c @ w[f'{p}.uv'].T).reshape(t, H, vd)
  out = np.zeros((t, H, vd), h.dtype)
  mask = np.tril(np.ones((t, t), bool))
  for a in range(H):
    qr = rnd(rotate(q[:, a, n:], np.arange(t), m['rot']))
    s = (q[:, a, :n] @ k[:, a].T + qr @ kr.T) * m['scale']
    s = np.where(mask, s, -np.inf)
    top = s.max(-1, keepdims=True)
    sink = None
    if MIXERS[kind]['sink']:
      sink = float(w[f'{p}.sink'][a])
      top = np.maximum(top, sink)
    e = np.exp(s - top)
    den = e.sum(-1, keepdims=True)
    if sink is not None:
      den = den + np.exp(sink - top)
    out[:, a] = (e / den) @ v[:, a]
  o = out.reshape(t, H * vd)
  if MIXERS[kind]['gate']:
    o = o * sigmoid(rnd(h @ w[f'{p}.g'].T))
  return rnd(rnd(o) @ w[f'{p}.o'].T)


def feed_forward(w, p, h, rnd):
  g = h @ w[f'{p}.gate'].T + w[f'{p}.gate.b']
  u = h @ w[f'{p}.up'].T + w[f'{p}.up.b']
  return rnd(rnd(g * sigmoid(g) * u) @ w[f'{p}.down'].T + w[f'{p}.down.b'])


def mix_streams(xs, hc, y):
  """xs [S, T, D] -> the streams after a sublayer that returned y [T, D]; hc['mix'] is [from, to]."""
  return np.einsum('st,snd->tnd', hc['mix'], xs) + hc['out'][:, None, None] * y[None]


def forward(cfg, w, tokens, rnd=None, dtype=np.float64, layers_out=None):
  """Logits [T, V] of one sequence.  cfg: the model's configuration as a mapping; w: name -> array.
  layers_out: list that receives the sum of the streams after every layer."""
  rnd = rnd or (lambda x: x)
  w = {k: np.asarray(v, dtype) for k, v in w.items()}
  tokens = np.asarray(tokens)
  eps = cfg['norm']['eps']
  x = w['embed'][tokens] + w['pos'][:len(tokens)]
  xs = np.repeat(x[None], cfg['streams'], 0)
  cache = {}
  for i, layer in enumerate(cfg['layers']):
    l, m = f'l{i}', layer['mixer']

    def sublayer(q, fn):
      hc = {k: w[f'{l}.hc{q}.{k}'] for k in ('in', 'out', 'mix')}
      u = np.einsum('s,snd->nd', hc['in'], xs)
      return mix_streams(xs, hc, fn(rnd(rms_norm(u, w[f'{l}.norm{q}'], eps))))

    def mixer(h):
      if m.get('kv_from') is None:
        cache[i] = latent_keys(w, f'{l}.mix', m, h, eps, rnd)
      src = i if m.get('kv_from') is None else m['kv_from']
      return latent_attention(w, f'{l}.mix', m, layer['type'], h, *cache[src], rnd)

    xs = sublayer(1, mixer)
    if layer.get('mlp'):
      xs = sublayer(2, lambda h: feed_forward(w, f'{l}.mlp', h, rnd))
    if layers_out is not None:
      layers_out.append(xs.sum(0))
  return rnd(rms_norm(xs.sum(0), w['final.norm'], eps)) @ w['head'].T * cfg['logit_scale']
