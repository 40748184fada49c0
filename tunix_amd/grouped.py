"""Decoders with dense weights, grouped-query attention in chunks and norms behind the sublayers (design "Feduzen").

The mechanisms are parameters of a layer:

* mixer: grouped-query attention, query / key and value heads of their own widths, biases on the three projections, a norm
  per query and key head, a rotation of the first ``rot.dims`` dimensions (pairs (i, i + dims / 2), optionally with
  band-scaled frequencies), chunks of positions that do not see each other, a softmax sink per head;
* feed-forward: squared relu, or none;
* residual: one stream that the sublayers read as it is; the norm lies on a sublayer's result;
* a layer may use the tensors of another one (``weights_of``), with a cache of its own.
"""
import dataclasses
from typing import Optional

import torch

from tunix_amd.dense import BandScaling, DenseConfig, DenseModel, MIXER_HEADS, RELU2, Rotation, ptr, up

HEAD_WIDTHS = (64, 128, 256)  # padded widths the attention kernels take


def _head_width(d):
  return next(p for p in HEAD_WIDTHS if d <= p)


@dataclasses.dataclass(frozen=True)
class GroupedLayer:
  heads: int
  kv_heads: int
  dim: int
  vdim: int
  scale: float
  rot: Rotation
  chunk: Optional[int] = None       # positions of a chunk (None: every earlier token is seen)
  ff: Optional[int] = None          # None: no feed-forward
  weights_of: Optional[int] = None  # the layer whose tensors this one uses

  # widths the kernels work with
  @property
  def dim_p(self):
    return _head_width(self.dim)

  @property
  def vdim_p(self):
    return _head_width(self.vdim)

  @property
  def cache_parts(self):
    return (self.kv_heads, self.dim_p), (self.kv_heads, self.vdim_p)


@dataclasses.dataclass(frozen=True)
class GroupedConfig(DenseConfig):
  vocab_size: int
  embed_dim: int
  embed_scale: float
  norm_eps: float
  layers: tuple
  dtype: str = 'bfloat16'

  max_positions = None  # the rotation tables grow with the sequences

  def __post_init__(self):
    self.check_dtype()
    for i, l in enumerate(self.layers):
      if min(l.heads, l.kv_heads, l.dim, l.vdim) < 1 or max(l.dim, l.vdim) > HEAD_WIDTHS[-1]:
        raise ValueError(f'layer {i}: heads of 1 to {HEAD_WIDTHS[-1]} dimensions are supported, got {l.dim} and {l.vdim}')
      if l.heads % l.kv_heads:
        raise ValueError(f'layer {i}: {l.heads} query heads do not divide into {l.kv_heads} key heads')
      if l.rot.dims % 2 or not 0 <= l.rot.dims <= l.dim:
        raise ValueError(f'layer {i}: a rotation of {l.rot.dims} dimensions does not fit heads of {l.dim}')
      if l.chunk is not None and l.chunk < 1:
        raise ValueError(f'layer {i}: chunks of {l.chunk} positions')
      if l.weights_of is not None:
        src = self.layers[l.weights_of] if 0 <= l.weights_of < len(self.layers) else None
        if src is None or src.weights_of is not None or dataclasses.replace(l, weights_of=None) != src:
          raise ValueError(f'layer {i}: layer {l.weights_of} has no tensors of its own of the same sizes and constants')

  @classmethod
  def from_dict(cls, cfg, dtype='bfloat16'):
    """From the mapping a config.json of the design holds."""
    layers = []
    for i, e in enumerate(cfg['layers']):
      if e['type'] != 'attention':
        raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
      m, mlp = e['mixer'], e.get('mlp')
      if mlp is not None and mlp.get('kind', 'dense') != 'dense':
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
      rot, mask = m['rot'], m.get('mask')
      sc = rot.get('scaling')
      layers.append(GroupedLayer(
          int(m['heads']), int(m['kv_heads']), int(m['dim']), int(m['vdim']), float(m['scale']),
          Rotation(int(rot['dims']), float(rot['base']),
                   BandScaling(*(float(sc[k]) for k in ('factor', 'low', 'high', 'original'))) if sc else None),
          int(mask['size']) if mask else None, int(mlp['ff']) if mlp is not None else None, e.get('weights_of')))
    # (a layer may name one that itself borrows: both use the tensors of the same layer)
    for i, l in enumerate(layers):
      src, hops = l.weights_of, 0
      while src is not None and 0 <= src < len(layers) and layers[src].weights_of is not None and hops < len(layers):
        src, hops = layers[src].weights_of, hops + 1
      layers[i] = dataclasses.replace(l, weights_of=src)
    return cls(int(cfg['vocab']), int(cfg['width']), float(cfg['embedding']['scale']), float(cfg['norm']['eps']),
               tuple(layers), dtype)

  @classmethod
  def uniform(cls, num_layers, vocab_size, embed_dim, ff, heads, kv_heads, dim, vdim, chunk, rot_dims=None, base=500_000.0,
              dtype='bfloat16'):
    """Equal layers (benchmarks)."""
    layer = GroupedLayer(heads, kv_heads, dim, vdim, dim ** -0.5,
                         Rotation(rot_dims or dim, base, BandScaling(8.0, 1.0, 4.0, 8192.0)), chunk, ff)
    return cls(vocab_size, embed_dim, 1.0, 1e-5, (layer,) * num_layers, dtype)

  def tensor_shapes(self):
    d = self.embed_dim
    out = {'embed': (self.vocab_size, d), 'final.norm': (d,), 'head': (self.vocab_size, d)}
    for i, l in enumerate(self.layers):
      if l.weights_of is not None:
        continue
      out[f'l{i}.norm1'] = (d,)
      for n, heads, width in (('q', l.heads, l.dim), ('k', l.kv_heads, l.dim), ('v', l.kv_heads, l.vdim)):
        out[f'l{i}.mix.{n}'], out[f'l{i}.mix.{n}.b'] = (heads * width, d), (heads * width,)
      out[f'l{i}.mix.q.norm'] = out[f'l{i}.mix.k.norm'] = (l.dim,)
      out[f'l{i}.mix.sink'] = (l.heads,)
      out[f'l{i}.mix.o'] = (d, l.heads * l.vdim)
      if l.ff is not None:
        out[f'l{i}.norm2'] = (d,)
        out[f'l{i}.mlp.up'], out[f'l{i}.mlp.down'] = (l.ff, d), (d, l.ff)
    return out

  def idle_tensors(self):
    return tuple(f'l{i}.norm2' for i, l in enumerate(self.layers) if l.ff is None)  # the norm behind no feed-forward


class GroupedModel(DenseModel):
  """Device-resident weights of a GroupedConfig model."""

  def _layer(self, l, get):
    d = self.config.embed_dim
    dp = up(d, 64)
    rows, biases = [], []
    for n, heads, width, padded in (('q', l.heads, l.dim, l.dim_p), ('k', l.kv_heads, l.dim, l.dim_p),
                                    ('v', l.kv_heads, l.vdim, l.vdim_p)):
      w = get(f'mix.{n}').reshape(heads, width, d)
      rows.append(self._padded(w, heads, padded, dp).reshape(heads * padded, dp))
      b = get(f'mix.{n}.b').reshape(heads, width)
      biases.append(self._padded(b.float(), heads, padded).reshape(-1))
    o = get('mix.o').reshape(d, l.heads, l.vdim)
    layer = {
        'norm1': self._f32(get('norm1'), dp),
        'in': self._dense(torch.cat(rows)[None], torch.cat(biases).contiguous()),
        'q_norm': self._f32(get('mix.q.norm'), l.dim_p), 'k_norm': self._f32(get('mix.k.norm'), l.dim_p),
        'sink': self._f32(get('mix.sink')),
        'o': self._dense(self._padded(o, dp, l.heads, l.vdim_p).reshape(1, dp, l.heads * l.vdim_p)),
    }
    self._table(l.rot)
    if l.ff is not None:
      fp = up(l.ff, 64)
      layer['norm2'] = self._f32(get('norm2'), dp)
      layer['gate_up'] = self._dense(self._padded(get('mlp.up'), fp, dp)[None])
      layer['down'] = self._dense(self._padded(get('mlp.down'), dp, fp)[None])
    return layer

  def _fill(self, a, i, l, w):
    a.mixer, a.ff = MIXER_HEADS, RELU2
    a.heads, a.kv_heads, a.dim, a.dim_p, a.vdim_p, a.rot_dim = l.heads, l.kv_heads, l.dim, l.dim_p, l.vdim_p, l.rot.dims
    a.scale, a.chunk = l.scale, l.chunk or 0
    a.q_norm_w, a.k_norm_w, a.sink, a.table = ptr(w['q_norm']), ptr(w['k_norm']), ptr(w['sink']), ptr(self._table(l.rot))

  def _fill_model(self, d):
    d.embed_scale, d.norm_after = self.config.embed_scale, 1
