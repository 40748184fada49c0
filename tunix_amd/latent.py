"""Decoders with dense weights, latent attention and several residual streams (TMX_FAMILY_LATENT).

The mechanisms are parameters of a layer, so that another design made of them needs a row in MIXERS and a reader of
its configuration:

* mixer: latent attention (one cached latent vector and one rotated key part per token, shared by all heads), with an
  optional output gate, an optional softmax sink, its own latents or those of an earlier layer (``kv_from``);
* rotation: pairs (i, i + d / 2), optionally with YaRN-scaled frequencies;
* feed-forward: SwiGLU with biases, or none;
* residual: ``streams`` copies mixed at every sublayer (hyper-connections), plus a learned position vector.

``LatentModel`` has the surface the Sampler expects of a transformer (config, desc, init_cache, lora_state).
"""
import ctypes
import dataclasses
import math
from typing import Optional

import numpy as np
import torch

from tunix_amd.model import (DenseDesc, FAMILY_LATENT, LatentLayerDesc, ModelDesc, StreamsDesc)

ACT_BF16, ACT_F32 = 0, 1
MAX_STREAMS = 8
# what a mixer type has besides latent attention itself
MIXERS = {
    'latent_attention': {'gate': True, 'sink': False},
    'latent_attention_2': {'gate': False, 'sink': True},
}


def _up(v, k):
  return -(-v // k) * k


@dataclasses.dataclass(frozen=True)
class YarnScaling:
  factor: float
  original: float
  fast: float
  slow: float


@dataclasses.dataclass(frozen=True)
class Rotation:
  dims: int
  base: float
  scaling: Optional[YarnScaling] = None

  def frequencies(self):
    """(frequencies f64 [dims / 2], factor on cos and sin)."""
    i = np.arange(self.dims // 2, dtype=np.float64)
    f = np.power(float(self.base), -2.0 * i / self.dims)
    if self.scaling is None:
      return f, 1.0
    s = self.scaling

    def turning(t):  # the dimension whose wave turns t times over the original length
      return self.dims * math.log(s.original / (2.0 * math.pi * t)) / (2.0 * math.log(self.base))

    lo = max(math.floor(turning(s.fast)), 0)
    hi = min(math.ceil(turning(s.slow)), self.dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f * (1.0 - ramp) + f / s.factor * ramp, 0.1 * math.log(s.factor) + 1.0

  def table(self, positions):
    """f32 [positions, dims / 2, 2]: cos, sin of every position, with the factor applied."""
    f, mult = self.frequencies()
    ang = np.arange(positions, dtype=np.float64)[:, None] * f[None]
    return torch.from_numpy((np.stack([np.cos(ang), np.sin(ang)], axis=-1) * mult).astype(np.float32))


@dataclasses.dataclass(frozen=True)
class LatentLayer:
  kind: str
  heads: int
  dim: int
  rot_dim: int
  vdim: int
  kv_rank: int
  scale: float
  rot: Rotation
  kv_from: Optional[int] = None
  ff: Optional[int] = None  # None: no feed-forward

  @property
  def gate(self):
    return MIXERS[self.kind]['gate']

  @property
  def sink(self):
    return MIXERS[self.kind]['sink']

  # widths the kernels work with
  @property
  def dim_p(self):
    return _up(self.dim, 64)

  @property
  def vdim_p(self):
    return _up(self.vdim, 64)

  @property
  def rank_p(self):
    return next(p for p in (64, 128, 256, 512) if self.kv_rank <= p)

  @property
  def rot_p(self):
    return 64 if self.rot_dim <= 64 else 128

  @property
  def cache_width(self):
    return self.rank_p + self.rot_p

  def columns(self):
    """Column offsets of the fused projection: (query rotated, latent or -1, gate or -1, total)."""
    off = off_qr = self.heads * self.dim_p
    off += _up(self.heads * self.rot_dim, 32)
    off_kv = off_gate = -1
    if self.kv_from is None:
      off_kv = off
      off += _up(self.kv_rank + self.rot_dim, 32)
    if self.gate:
      off_gate = off
      off += self.heads * self.vdim_p
    return off_qr, off_kv, off_gate, off


@dataclasses.dataclass(frozen=True)
class LatentConfig:
  vocab_size: int
  embed_dim: int
  max_positions: int
  streams: int
  norm_eps: float
  logit_scale: float
  layers: tuple
  dtype: str = 'bfloat16'  # 'bfloat16' or 'float32': activations, cache and matrix products

  def __post_init__(self):
    if self.dtype not in ('bfloat16', 'float32'):
      raise ValueError(f'dtype must be bfloat16 or float32, not {self.dtype!r}')
    if not 1 <= self.streams <= MAX_STREAMS:
      raise ValueError(f'{self.streams} residual streams: 1 to {MAX_STREAMS} are supported')
    for i, l in enumerate(self.layers):
      if l.kind not in MIXERS:
        raise ValueError(f'layer {i}: unknown mixer {l.kind!r} (known: {sorted(MIXERS)})')
      if l.kv_rank > 512 or l.rot_dim > 128 or l.rot_dim % 2:
        raise ValueError(f'layer {i}: latents of up to 512 and an even rotated part of up to 128 are supported, '
                         f'got {l.kv_rank} and {l.rot_dim}')
      if l.rot.dims != l.rot_dim:
        raise ValueError(f'layer {i}: the rotation covers {l.rot.dims} dimensions of a rotated part of {l.rot_dim}')
      if l.kv_from is not None:
        if not 0 <= l.kv_from < i:
          raise ValueError(f'layer {i}: kv_from {l.kv_from} is not an earlier layer')
        src = self.layers[l.kv_from]
        if src.kv_from is not None or (src.kv_rank, src.rot_dim, src.rot) != (l.kv_rank, l.rot_dim, l.rot):
          raise ValueError(f'layer {i}: layer {l.kv_from} has no latents of its own of the same sizes and rotation')

  @classmethod
  def from_dict(cls, cfg, dtype='bfloat16'):
    """From the mapping a config.json of the design holds."""
    layers = []
    for e in cfg['layers']:
      m = e['mixer']
      rot = m['rot']
      sc = rot.get('scaling')
      mlp = e.get('mlp')
      if mlp is not None and mlp.get('kind', 'dense') != 'dense':
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
      layers.append(LatentLayer(
          e['type'], int(m['heads']), int(m['dim']), int(m['rot_dim']), int(m['vdim']), int(m['kv_rank']),
          float(m['scale']),
          Rotation(int(rot['dims']), float(rot['base']),
                   YarnScaling(*(float(sc[k]) for k in ('factor', 'original', 'fast', 'slow'))) if sc else None),
          None if m.get('kv_from') is None else int(m['kv_from']), int(mlp['ff']) if mlp is not None else None))
    return cls(int(cfg['vocab']), int(cfg['width']), int(cfg['max_positions']), int(cfg['streams']),
               float(cfg['norm']['eps']), float(cfg['logit_scale']), tuple(layers), dtype)

  @classmethod
  def uniform(cls, num_layers, vocab_size, embed_dim, ff, heads, dim, rot_dim, vdim, kv_rank, streams=4,
              max_positions=4096, base=500_000.0, dtype='bfloat16'):
    """Equal layers of alternating mixer types (benchmarks)."""
    rot = Rotation(rot_dim, base)
    kinds = sorted(MIXERS)
    return cls(vocab_size, embed_dim, max_positions, streams, 1e-5, 1.0,
               tuple(LatentLayer(kinds[i % 2], heads, dim, rot_dim, vdim, kv_rank, (dim + rot_dim) ** -0.5, rot, None, ff)
                     for i in range(num_layers)), dtype)

  # -- what the Sampler and the rollout ask of a configuration ----------------
  @property
  def num_layers(self):
    return len(self.layers)

  num_kv_heads = 1  # every head reads the same cache row

  @property
  def head_dim(self):
    return max(l.cache_width for l in self.layers)

  @property
  def torch_dtype(self):
    return torch.float32 if self.dtype == 'float32' else torch.bfloat16

  @property
  def logits_width(self):
    return _up(self.vocab_size, 32)

  max_rows_rule = 'sequences x tokens of one pass'

  def max_rows(self):
    return 4096

  def cache_shape(self, batch, cache_size):
    """One flat tensor: the layers with latents of their own, each [B][C][width]."""
    return (batch * cache_size * sum(l.cache_width for l in self.layers if l.kv_from is None),)

  def cache_rows(self, cache, batch, cache_size):
    out, off = [], 0
    for l in self.layers:
      if l.kv_from is None:
        n = batch * cache_size * l.cache_width
        out.append(cache[off:off + n].view(batch, cache_size, l.cache_width))
        off += n
    return out

  def cache_bytes_per_token(self):
    return sum(l.cache_width for l in self.layers if l.kv_from is None) * (4 if self.dtype == 'float32' else 2)


def tensor_shapes(c):
  """name -> shape of every tensor of a model."""
  d = c.embed_dim
  out = {'embed': (c.vocab_size, d), 'pos': (c.max_positions, d), 'final.norm': (d,), 'head': (c.vocab_size, d)}
  for i, l in enumerate(c.layers):
    p = f'l{i}'
    h = l.heads
    out[f'{p}.norm1'] = (d,)
    out[f'{p}.mix.q'] = (h * (l.dim + l.rot_dim), d)
    if l.kv_from is None:
      out[f'{p}.mix.dkv'] = (l.kv_rank + l.rot_dim, d)
      out[f'{p}.mix.dkv.norm'] = (l.kv_rank,)
    out[f'{p}.mix.uk'] = (h * l.dim, l.kv_rank)
    out[f'{p}.mix.uv'] = (h * l.vdim, l.kv_rank)
    if l.gate:
      out[f'{p}.mix.g'] = (h * l.vdim, d)
    if l.sink:
      out[f'{p}.mix.sink'] = (h,)
    out[f'{p}.mix.o'] = (d, h * l.vdim)
    subs = ['1']
    if l.ff is not None:
      subs.append('2')
      out[f'{p}.norm2'] = (d,)
      for n in ('gate', 'up'):
        out[f'{p}.mlp.{n}'], out[f'{p}.mlp.{n}.b'] = (l.ff, d), (l.ff,)
      out[f'{p}.mlp.down'], out[f'{p}.mlp.down.b'] = (d, l.ff), (d,)
    for q in subs:
      out[f'{p}.hc{q}.in'], out[f'{p}.hc{q}.out'] = (c.streams,), (c.streams,)
      out[f'{p}.hc{q}.mix'] = (c.streams, c.streams)
  return out


def pack_tiles(w):
  """bf16 [V, D] (V % 32 == 0, D % 64 == 0) -> the same elements in the tile layout of tmx_head_tiles_pack."""
  v, d = w.shape
  t = w.reshape(v // 32, 32, d // 64, 2, 4, 8)       # [tile, row, k-tile, half, step, 8]
  return t.permute(0, 2, 4, 3, 1, 5).contiguous().reshape(v, d)


class DenseMatrix:
  """`heads` matrices [N, K] in the layout the projections read, with an optional f32 bias [N]."""

  def __init__(self, w, bias, act):
    heads, n, k = w.shape
    self.heads, self.n, self.k, self.bias = heads, n, k, bias
    w2 = w.reshape(heads * n, k)
    self.w = w2.float().contiguous() if act == ACT_F32 else pack_tiles(w2.to(torch.bfloat16))

  def desc(self):
    return DenseDesc(self.w.data_ptr(), self.bias.data_ptr() if self.bias is not None else None, self.k, self.n,
                     self.heads)

  @property
  def bytes(self):
    return self.w.numel() * self.w.element_size()


class LatentModel:
  """Device-resident weights of a LatentConfig model; built with ``from_state`` or ``random_init``."""

  def __init__(self, config, device='cuda'):
    self.config = config
    self.device = torch.device(device)
    self.act = ACT_F32 if config.dtype == 'float32' else ACT_BF16
    self.layers = []
    self._tables = {}
    self._desc = None
    self._keep = None

  # -- construction -----------------------------------------------------------
  def _padded(self, w, *shape):
    """w in the leading corner of a zero tensor of `shape`."""
    w = w.to(self.device)
    if tuple(w.shape) == shape:
      return w
    out = torch.zeros(*shape, dtype=w.dtype, device=self.device)
    out[tuple(slice(0, s) for s in w.shape)] = w
    return out

  def _f32(self, w, n=None):
    return self._padded(w.to(self.device).float(), *(w.shape if n is None else (n,))).contiguous()

  def _layer(self, l, get, streams):
    """get(name): tensor of this layer ('mix.q', 'mlp.gate', ...)."""
    c, h, dp = self.config, l.heads, _up(self.config.embed_dim, 64)
    d = c.embed_dim
    dense = lambda w, bias=None: DenseMatrix(w, bias, self.act)
    q = get('mix.q').to(self.device).reshape(h, l.dim + l.rot_dim, d)
    off_qr, off_kv, off_gate, total = l.columns()
    fused = torch.zeros(total, dp, dtype=q.dtype, device=self.device)
    fused[:h * l.dim_p].view(h, l.dim_p, dp)[:, :l.dim, :d] = q[:, :l.dim]
    fused[off_qr:off_qr + h * l.rot_dim].view(h, l.rot_dim, dp)[:, :, :d] = q[:, l.dim:]
    layer = {'norm1': self._f32(get('norm1'), dp), 'hc1': streams('hc1')}
    if off_kv >= 0:
      fused[off_kv:off_kv + l.kv_rank + l.rot_dim, :d] = get('mix.dkv').to(self.device)
      layer['kv_norm'] = self._f32(get('mix.dkv.norm'))
    if off_gate >= 0:
      fused[off_gate:].view(h, l.vdim_p, dp)[:, :l.vdim, :d] = get('mix.g').to(self.device).reshape(h, l.vdim, d)
    layer['in'] = dense(fused[None])
    del fused
    uk = get('mix.uk').to(self.device).reshape(h, l.dim, l.kv_rank).transpose(1, 2)
    layer['uk'] = dense(self._padded(uk, h, l.rank_p, l.dim_p))
    uv = get('mix.uv').to(self.device).reshape(h, l.vdim, l.kv_rank)
    layer['uv'] = dense(self._padded(uv, h, l.vdim_p, l.rank_p))
    o = get('mix.o').to(self.device).reshape(d, h, l.vdim)
    layer['o'] = dense(self._padded(o, dp, h, l.vdim_p).reshape(1, dp, h * l.vdim_p))
    if l.sink:
      layer['sink'] = self._f32(get('mix.sink'))
    if l.rot not in self._tables:
      self._tables[l.rot] = l.rot.table(c.max_positions).to(self.device)
    layer['table'] = self._tables[l.rot]
    if l.ff is not None:
      fp = _up(l.ff, 64)
      layer['norm2'], layer['hc2'] = self._f32(get('norm2'), dp), streams('hc2')
      gu = torch.stack([self._padded(get(f'mlp.{n}'), fp, dp) for n in ('gate', 'up')])
      bias = torch.cat([self._f32(get(f'mlp.{n}.b'), fp) for n in ('gate', 'up')])
      layer['gate_up'] = dense(gu.reshape(1, 2 * fp, dp), bias)
      layer['down'] = dense(self._padded(get('mlp.down'), dp, fp)[None], self._f32(get('mlp.down.b'), dp))
    return layer

  def _outer(self, embed, pos, final_norm, head):
    c, dp = self.config, _up(self.config.embed_dim, 64)
    bf = torch.bfloat16
    self.embed = self._padded(embed.to(bf), c.vocab_size, dp).contiguous()
    self.pos = self._padded(pos.to(bf), c.max_positions, dp).contiguous()
    self.final_norm = self._f32(final_norm, dp)
    head = self._padded(head, c.logits_width, dp)
    self.head = head.float().contiguous() if self.act == ACT_F32 else head.to(bf).contiguous()
    self.head_tiles = None if self.act == ACT_F32 else pack_tiles(self.head)
    self.final_in = torch.ones(c.streams, dtype=torch.float32, device=self.device)

  @classmethod
  def from_state(cls, config, state, device='cuda'):
    """state: name -> tensor, exactly the names and shapes of tensor_shapes(config)."""
    want = tensor_shapes(config)
    # a layer without a feed-forward has no use for the norm and the stream coefficients in front of one
    idle = tuple(f'l{i}.{n}' for i, l in enumerate(config.layers) if l.ff is None for n in ('norm2', 'hc2.'))
    missing = sorted(set(want) - set(state))
    extra = sorted(k for k in set(state) - set(want) if not (idle and k.startswith(idle)))
    if missing or extra:
      raise KeyError(f'checkpoint does not fit the configuration: missing {missing[:4]}, unexpected {extra[:4]}')
    for k, shape in want.items():
      if tuple(state[k].shape) != shape:
        raise ValueError(f'{k}: shape {tuple(state[k].shape)}, the configuration asks for {shape}')
    m = cls(config, device)
    m._outer(state['embed'], state['pos'], state['final.norm'], state['head'])
    for i, l in enumerate(config.layers):
      streams = lambda q, i=i: {k: m._f32(state[f'l{i}.{q}.{k}']) for k in ('in', 'out', 'mix')}
      m.layers.append(m._layer(l, lambda n, i=i: state[f'l{i}.{n}'], streams))
    return m

  @classmethod
  def random_init(cls, config, seed=0, device='cuda', std=0.02):
    """Synthetic weights generated layer by layer on the device: matrices std * N(0, 1), norms 1, stream
    coefficients that average the streams and add a sublayer's result to each."""
    g = torch.Generator(device=device).manual_seed(seed)
    rnd = lambda *s: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(torch.bfloat16)
    shapes = tensor_shapes(config)

    def make(name):
      s = shapes[name]
      return torch.ones(s, dtype=torch.bfloat16, device=device) if name.endswith(('norm', 'norm1', 'norm2')) else rnd(*s)

    m = cls(config, device)
    m._outer(*(make(n) for n in ('embed', 'pos', 'final.norm', 'head')))
    n = config.streams
    hc = {'in': torch.full((n,), 1.0 / n), 'out': torch.ones(n), 'mix': torch.eye(n) * 0.5 + 0.5 / n}
    for i, l in enumerate(config.layers):
      m.layers.append(m._layer(l, lambda name, i=i: make(f'l{i}.{name}'), lambda q: {k: m._f32(v) for k, v in hc.items()}))
    return m

  # -- the surface of a policy --------------------------------------------------
  @property
  def num_embed(self):
    return self.config.vocab_size

  @property
  def dtype(self):
    return self.config.torch_dtype

  def init_cache(self, batch_size, cache_size, dtype=None):
    return torch.zeros(self.config.cache_shape(batch_size, cache_size), dtype=dtype or self.dtype, device=self.device)

  def lora_state(self):
    return {}  # dense weights carry no adapters

  def update_lora(self, state):
    if state:
      raise ValueError('New state must have the same structure as the old state: this model has no LoRA parameters')

  def expert_fraction(self, batch):
    del batch
    return 1.0

  def weight_bytes(self, batch=1):
    """(bytes one step streams from the layers, bytes of the head)."""
    del batch
    total = sum(layer[k].bytes for layer in self.layers for k in ('in', 'uk', 'uv', 'o', 'gate_up', 'down') if k in layer)
    return total, self.head.numel() * self.head.element_size()

  # -- C ABI descriptor -----------------------------------------------------------
  def desc(self):
    """ctypes tmx_model_desc (cached)."""
    if self._desc is not None:
      return self._desc
    c = self.config
    ptr = lambda t: t.data_ptr() if t is not None else None
    hc = lambda s: StreamsDesc(ptr(s['in']), ptr(s['out']), ptr(s['mix']))
    arr = (LatentLayerDesc * c.num_layers)()
    for i, (l, w) in enumerate(zip(c.layers, self.layers)):
      a = arr[i]
      a.norm1_w, a.hc1 = ptr(w['norm1']), hc(w['hc1'])
      a.heads, a.rot_dim, a.kv_rank = l.heads, l.rot_dim, l.kv_rank
      a.dim_p, a.rot_p, a.rank_p, a.vdim_p = l.dim_p, l.rot_p, l.rank_p, l.vdim_p
      a.off_qr, a.off_kv, a.off_gate, _ = l.columns()
      a.kv_layer = i if l.kv_from is None else l.kv_from
      a.scale = l.scale
      a.in_, a.uk, a.uv, a.o = (w[k].desc() for k in ('in', 'uk', 'uv', 'o'))
      a.kv_norm_w, a.table, a.sink = ptr(w.get('kv_norm')), ptr(w['table']), ptr(w.get('sink'))
      if l.ff is not None:
        a.norm2_w, a.hc2 = ptr(w['norm2']), hc(w['hc2'])
        a.gate_up, a.down = w['gate_up'].desc(), w['down'].desc()
    d = ModelDesc()
    d.family, d.num_layers, d.vocab_size, d.embed_dim = FAMILY_LATENT, c.num_layers, c.vocab_size, c.embed_dim
    d.norm_eps = c.norm_eps
    d.embed, d.pos_embed, d.final_norm_w, d.head = ptr(self.embed), ptr(self.pos), ptr(self.final_norm), ptr(self.head)
    d.head_tiles = ptr(self.head_tiles)
    d.latent_layers = ctypes.cast(arr, ctypes.POINTER(LatentLayerDesc))
    d.act, d.streams, d.max_positions = self.act, c.streams, c.max_positions
    d.final_in, d.logit_scale = ptr(self.final_in), c.logit_scale
    self._desc, self._keep = d, arr
    return d
