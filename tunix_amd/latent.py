"""Decoders with dense weights, latent attention and several residual streams (design "Kagapel").

The mechanisms are parameters of a layer, so that another design made of them needs a row in MIXERS and a reader of
its configuration:

* mixer: latent attention (one cached latent vector and one rotated key part per token, shared by all heads), with an
  optional output gate, an optional softmax sink, its own latents or those of an earlier layer (``kv_from``);
* rotation: pairs (i, i + d / 2), optionally with YaRN-scaled frequencies;
* feed-forward: SwiGLU with biases, or none;
* residual: ``streams`` copies mixed at every sublayer (hyper-connections), plus a learned position vector.
"""
import dataclasses
from typing import Optional

import torch

from tunix_amd.dense import (ACT_F32, DenseConfig, DenseMatrix, DenseModel, MIXER_LATENT, Rotation, SWIGLU, YarnScaling,  # noqa: F401
                             pack_tiles, ptr, up as _up)
from tunix_amd.model import StreamsDesc

MAX_STREAMS = 8
# what a mixer type has besides latent attention itself
MIXERS = {
    'latent_attention': {'gate': True, 'sink': False},
    'latent_attention_2': {'gate': False, 'sink': True},
}


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

  @property
  def cache_parts(self):
    return ((1, self.cache_width),) if self.kv_from is None else ()

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
class LatentConfig(DenseConfig):
  vocab_size: int
  embed_dim: int
  max_positions: int
  streams: int
  norm_eps: float
  logit_scale: float
  layers: tuple
  dtype: str = 'bfloat16'  # 'bfloat16' or 'float32': activations, cache and matrix products

  def __post_init__(self):
    self.check_dtype()
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

  def tensor_shapes(self):
    c = self
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

  def idle_tensors(self):
    # a layer without a feed-forward has no use for the norm and the stream coefficients in front of one
    return tuple(f'l{i}.{n}' for i, l in enumerate(self.layers) if l.ff is None for n in ('norm2', 'hc2.'))


def tensor_shapes(config):
  return config.tensor_shapes()


class LatentModel(DenseModel):
  """Device-resident weights of a LatentConfig model."""

  def _build(self, tensor):
    c = self.config
    self.pos = self._padded(tensor('pos').to(torch.bfloat16), c.max_positions, _up(c.embed_dim, 64)).contiguous()
    self.final_in = torch.ones(c.streams, dtype=torch.float32, device=self.device)
    super()._build(tensor)

  def _random(self, name, shape, draw):
    """Stream coefficients that average the streams and add a sublayer's result to each."""
    n = self.config.streams
    if '.hc' not in name:
      return draw()
    return {'in': torch.full((n,), 1.0 / n), 'out': torch.ones(n), 'mix': torch.eye(n) * 0.5 + 0.5 / n}[name.rsplit('.', 1)[1]]

  def _layer(self, l, get):
    h, d = l.heads, self.config.embed_dim
    dp = _up(d, 64)
    dense = self._dense
    streams = lambda q: {k: self._f32(get(f'{q}.{k}')) for k in ('in', 'out', 'mix')}
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
    self._table(l.rot)
    if l.ff is not None:
      fp = _up(l.ff, 64)
      layer['norm2'], layer['hc2'] = self._f32(get('norm2'), dp), streams('hc2')
      gu = torch.stack([self._padded(get(f'mlp.{n}'), fp, dp) for n in ('gate', 'up')])
      bias = torch.cat([self._f32(get(f'mlp.{n}.b'), fp) for n in ('gate', 'up')])
      layer['gate_up'] = dense(gu.reshape(1, 2 * fp, dp), bias)
      layer['down'] = dense(self._padded(get('mlp.down'), dp, fp)[None], self._f32(get('mlp.down.b'), dp))
    return layer

  def _fill(self, a, i, l, w):
    hc = lambda s: StreamsDesc(ptr(s['in']), ptr(s['out']), ptr(s['mix']))
    a.mixer, a.ff, a.hc1 = MIXER_LATENT, SWIGLU, hc(w['hc1'])
    a.heads, a.rot_dim, a.kv_rank = l.heads, l.rot_dim, l.kv_rank
    a.dim_p, a.rot_p, a.rank_p, a.vdim_p = l.dim_p, l.rot_p, l.rank_p, l.vdim_p
    a.off_qr, a.off_kv, a.off_gate, _ = l.columns()
    a.kv_layer = i if l.kv_from is None else l.kv_from
    a.scale = l.scale
    a.uk, a.uv = w['uk'].desc(), w['uv'].desc()
    a.kv_norm_w, a.table, a.sink = ptr(w.get('kv_norm')), ptr(self._table(l.rot)), ptr(w.get('sink'))
    if l.ff is not None:
      a.hc2 = hc(w['hc2'])

  def _fill_model(self, d):
    c = self.config
    d.pos_embed, d.streams, d.final_in, d.logit_scale = ptr(self.pos), c.streams, ptr(self.final_in), c.logit_scale
