"""What decoders with dense weights (TMX_FAMILY_DENSE) have in common: rotations, the layout of the weights, the cache,
construction from named tensors, and the surface the Sampler expects of a configuration and of a transformer.

A design is a subclass of DenseConfig (its layers, its reader of config.json, the names and shapes of its tensors) and of
DenseModel (how a layer's tensors become the operands of the kernels)."""
import ctypes
import dataclasses
import math
from typing import Any, Optional

import numpy as np
import torch

from tunix_amd.model import DenseDesc, DenseLayerDesc, FAMILY_DENSE, ModelDesc

ACT_BF16, ACT_F32 = 0, 1
PLAIN, SWIGLU, GATED, RELU2 = 0, 1, 2, 3       # TMX_DENSE_*
MIXER_LATENT, MIXER_HEADS = 0, 1               # TMX_MIXER_*


def up(v, k):
  return -(-v // k) * k


# -- rotations -------------------------------------------------------------------
@dataclasses.dataclass(frozen=True)
class YarnScaling:
  """Fast waves stay, slow ones are stretched by `factor`, a ramp over the dimensions in between; cos and sin grow."""
  factor: float
  original: float
  fast: float
  slow: float

  def apply(self, f, rot):
    def turning(t):  # the dimension whose wave turns t times over the original length
      return rot.dims * math.log(self.original / (2.0 * math.pi * t)) / (2.0 * math.log(rot.base))

    lo = max(math.floor(turning(self.fast)), 0)
    hi = min(math.ceil(turning(self.slow)), rot.dims - 1)
    ramp = np.clip((np.arange(rot.dims // 2, dtype=np.float64) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f * (1.0 - ramp) + f / self.factor * ramp, 0.1 * math.log(self.factor) + 1.0


@dataclasses.dataclass(frozen=True)
class BandScaling:
  """Waves that turn more than `high` times over the original length stay, those that turn less than `low` times are
  stretched by `factor`, a ramp over the number of turns in between (the Llama 3.1 rule)."""
  factor: float
  low: float
  high: float
  original: float

  def apply(self, f, rot):
    del rot
    turns = self.original * f / (2.0 * math.pi)
    keep = np.clip((turns - self.low) / (self.high - self.low), 0.0, 1.0) if self.high > self.low else (turns >= self.low) * 1.0
    return f * keep + f / self.factor * (1.0 - keep), 1.0


@dataclasses.dataclass(frozen=True)
class Rotation:
  dims: int
  base: float
  scaling: Optional[Any] = None

  def frequencies(self):
    """(frequencies f64 [dims / 2], factor on cos and sin)."""
    f = np.power(float(self.base), -2.0 * np.arange(self.dims // 2, dtype=np.float64) / self.dims)
    return (f, 1.0) if self.scaling is None else self.scaling.apply(f, self)

  def table(self, positions):
    """f32 [positions, dims / 2, 2]: cos, sin of every position, with the factor applied."""
    f, mult = self.frequencies()
    ang = np.arange(positions, dtype=np.float64)[:, None] * f[None]
    return torch.from_numpy((np.stack([np.cos(ang), np.sin(ang)], axis=-1) * mult).astype(np.float32))


# -- weights ---------------------------------------------------------------------
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


class DenseConfig:
  """Base of the configurations: vocab_size, embed_dim, norm_eps, layers, dtype ('bfloat16' or 'float32': activations,
  cache and matrix products), max_positions (None: not bounded).  A layer answers `cache_parts`: (heads, width) of every
  row it caches per token."""

  max_rows_rule = 'sequences x tokens of one pass'

  def check_dtype(self):
    if self.dtype not in ('bfloat16', 'float32'):
      raise ValueError(f'dtype must be bfloat16 or float32, not {self.dtype!r}')

  def tensor_shapes(self):
    """name -> shape of every tensor of a model."""
    raise NotImplementedError

  def idle_tensors(self):
    """Prefixes of tensors a checkpoint may hold that no layer uses."""
    return ()

  @property
  def num_layers(self):
    return len(self.layers)

  @property
  def num_kv_heads(self):
    return max(h for l in self.layers for h, _ in l.cache_parts)

  @property
  def head_dim(self):
    return max(w for l in self.layers for _, w in l.cache_parts)

  @property
  def torch_dtype(self):
    return torch.float32 if self.dtype == 'float32' else torch.bfloat16

  @property
  def logits_width(self):
    return up(self.vocab_size, 32)

  def max_rows(self):
    return 4096

  def _slot_width(self):
    return sum(h * w for l in self.layers for h, w in l.cache_parts)

  def cache_shape(self, batch, cache_size):
    """One flat tensor: every part of every layer in order, each [B][heads][C][width]."""
    return (batch * cache_size * self._slot_width(),)

  def cache_rows(self, cache, batch, cache_size):
    """Views [B, C, heads, width] of a cache tensor, together all of it."""
    out, off = [], 0
    for l in self.layers:
      for h, w in l.cache_parts:
        n = batch * cache_size * h * w
        out.append(cache[off:off + n].view(batch, h, cache_size, w).transpose(1, 2))
        off += n
    return out

  def cache_bytes_per_token(self):
    return self._slot_width() * (4 if self.dtype == 'float32' else 2)


class DenseModel:
  """Device-resident weights of a DenseConfig model; built with ``from_state`` or ``random_init``."""

  ONES = ('norm', 'norm1', 'norm2')  # endings of the names that random_init sets to one
  INITIAL_POSITIONS = 1024           # rows of the rotation tables before a longer sequence asks for more

  def __init__(self, config, device='cuda'):
    self.config = config
    self.device = torch.device(device)
    self.act = ACT_F32 if config.dtype == 'float32' else ACT_BF16
    self.layers = []
    self._tables = {}
    self._positions = config.max_positions or self.INITIAL_POSITIONS
    self._desc = None
    self._keep = None

  # -- construction -----------------------------------------------------------
  def _layer(self, l, get):
    """Operands of layer `l`: name -> DenseMatrix or f32 tensor; get(name): its tensor 'mix.q', 'mlp.up', ..."""
    raise NotImplementedError

  def _fill(self, a, i, l, w):
    """The design's part of tmx_dense_layer_desc `a` of layer i from its operands w."""
    raise NotImplementedError

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

  def _dense(self, w, bias=None):
    return DenseMatrix(w, bias, self.act)

  def _table(self, rot):
    if rot not in self._tables:
      self._tables[rot] = rot.table(self._positions).to(self.device)
    return self._tables[rot]

  def _outer(self, embed, final_norm, head):
    c, dp = self.config, up(self.config.embed_dim, 64)
    bf = torch.bfloat16
    self.embed = self._padded(embed.to(bf), c.vocab_size, dp).contiguous()
    self.final_norm = self._f32(final_norm, dp)
    head = self._padded(head, c.logits_width, dp)
    self.head = head.float().contiguous() if self.act == ACT_F32 else head.to(bf).contiguous()
    self.head_tiles = None if self.act == ACT_F32 else pack_tiles(self.head)

  def _build(self, tensor):
    """Everything from tensor(name)."""
    self._outer(tensor('embed'), tensor('final.norm'), tensor('head'))
    layers = self.config.layers
    owner = [i if getattr(l, 'weights_of', None) is None else l.weights_of for i, l in enumerate(layers)]
    own = {i: self._layer(l, lambda n, i=i: tensor(f'l{i}.{n}')) for i, l in enumerate(layers) if owner[i] == i}
    self.layers = [own[i] for i in owner]  # a layer without tensors of its own shares the operands of another one

  @classmethod
  def from_state(cls, config, state, device='cuda'):
    """state: name -> tensor, exactly the names and shapes of config.tensor_shapes()."""
    want, idle = config.tensor_shapes(), config.idle_tensors()
    missing = sorted(set(want) - set(state))
    extra = sorted(k for k in set(state) - set(want) if not (idle and k.startswith(idle)))
    if missing or extra:
      raise KeyError(f'checkpoint does not fit the configuration: missing {missing[:4]}, unexpected {extra[:4]}')
    for k, shape in want.items():
      if tuple(state[k].shape) != shape:
        raise ValueError(f'{k}: shape {tuple(state[k].shape)}, the configuration asks for {shape}')
    m = cls(config, device)
    m._build(lambda name: state[name])
    return m

  @classmethod
  def random_init(cls, config, seed=0, device='cuda', std=0.02):
    """Synthetic weights generated layer by layer on the device: matrices std * N(0, 1), norms 1."""
    m = cls(config, device)
    g = torch.Generator(device=device).manual_seed(seed)
    shapes = config.tensor_shapes()

    def make(name):
      s = shapes[name]
      if name.endswith(cls.ONES):
        return torch.ones(s, dtype=torch.bfloat16, device=device)
      return m._random(name, s, lambda: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(torch.bfloat16))

    m._build(make)
    return m

  def _random(self, name, shape, draw):
    """A tensor of random_init that is not a norm."""
    del name, shape
    return draw()

  # -- the surface of a policy --------------------------------------------------
  @property
  def num_embed(self):
    return self.config.vocab_size

  @property
  def dtype(self):
    return self.config.torch_dtype

  def init_cache(self, batch_size, cache_size, dtype=None):
    return torch.zeros(self.config.cache_shape(batch_size, cache_size), dtype=dtype or self.dtype, device=self.device)

  def reserve_positions(self, n):
    """Makes the rotation tables cover n positions (a bounded model's do from the start)."""
    if self.config.max_positions is not None or n <= self._positions:
      return
    while self._positions < n:
      self._positions *= 2
    self._tables = {rot: rot.table(self._positions).to(self.device) for rot in self._tables}
    self._desc = None

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
    total = sum(w.bytes for layer in self.layers for w in layer.values() if isinstance(w, DenseMatrix))
    return total, self.head.numel() * self.head.element_size()

  # -- C ABI descriptor -----------------------------------------------------------
  def desc(self):
    """ctypes tmx_model_desc (cached)."""
    if self._desc is not None:
      return self._desc
    c = self.config
    arr = (DenseLayerDesc * c.num_layers)()
    for i, (l, w) in enumerate(zip(c.layers, self.layers)):
      a = arr[i]
      a.norm1_w = ptr(w['norm1'])
      a.in_, a.o = w['in'].desc(), w['o'].desc()
      if 'down' in w:
        a.norm2_w, a.gate_up, a.down = ptr(w['norm2']), w['gate_up'].desc(), w['down'].desc()
      self._fill(a, i, l, w)
    d = ModelDesc()
    d.family, d.num_layers, d.vocab_size, d.embed_dim = FAMILY_DENSE, c.num_layers, c.vocab_size, c.embed_dim
    d.norm_eps = c.norm_eps
    d.embed, d.final_norm_w, d.head, d.head_tiles = ptr(self.embed), ptr(self.final_norm), ptr(self.head), ptr(self.head_tiles)
    d.dense_layers = ctypes.cast(arr, ctypes.POINTER(DenseLayerDesc))
    d.act, d.max_positions = self.act, self._positions
    d.streams, d.logit_scale, d.embed_scale = 1, 1.0, 1.0
    self._fill_model(d)
    self._desc, self._keep = d, arr
    return d

  def _fill_model(self, d):
    """The design's part of tmx_model_desc."""


def ptr(t):
  return t.data_ptr() if t is not None else None
