"""Small random models of the chunked grouped-attention design for the tests: configuration mappings, weights, product
models and the plain implementation's logits."""
import numpy as np
import torch

from latent_common import error, LIMIT  # noqa: F401
from oracle import grouped as OG
from oracle.bf16 import bf16_round

BANDS = {'factor': 4.0, 'low': 1.0, 'high': 3.0, 'original': 64}


def rot(dims, base=10_000.0, scaling=None):
  r = {'dims': dims, 'base': base}
  if scaling:
    r['scaling'] = scaling
  return r


def layer(heads, kv_heads, dim, vdim, r, chunk, ff, scale=None, weights_of=None):
  m = {'heads': heads, 'kv_heads': kv_heads, 'dim': dim, 'vdim': vdim, 'rot': r, 'scale': dim ** -0.5 if scale is None else scale}
  if chunk is not None:
    m['mask'] = {'size': chunk}
  out = {'type': 'attention', 'mixer': m, 'mlp': None if ff is None else {'kind': 'dense', 'ff': ff}}
  if weights_of is not None:
    out['weights_of'] = weights_of
  return out


def config(layers, vocab=101, width=80, eps=1e-5, scale=1.0):
  return {'architecture': 'Feduzen', 'layers': layers, 'vocab': vocab, 'width': width, 'norm': {'eps': eps},
          'embedding': {'scale': scale}}


_A = (6, 2, 24, 40, rot(16, 5_000.0, BANDS), 32, 144)
_B = (5, 5, 40, 24, rot(40, 700.0), 20, None)
# sizes off every padding, groups of 1, 3 and more than 32 query heads, chunks of one token, off and on blocks of 32 slots,
# no chunks, rotations of few, some and all dimensions, layers without a feed-forward, borrowed weights
CONFIGS = {
    'mixed': config([layer(*_A), layer(*_B), layer(3, 1, 72, 136, rot(6, 50.0, BANDS), 7, 96), layer(*_A, weights_of=0),
                     layer(*_B, weights_of=1)], scale=3.0),
    'one': config([layer(1, 1, 8, 8, rot(2, 100.0), 1, 24), layer(1, 1, 10, 16, rot(10, 20_000.0, BANDS), 64, 24)], vocab=64,
                  width=36, eps=1e-3, scale=0.5),
    'wide': config([layer(40, 1, 96, 160, rot(32, 1e4, BANDS), 100, 272), layer(16, 4, 200, 64, rot(50, 1e5), 64, 320, scale=0.11),
                    layer(8, 8, 64, 130, rot(64), None, 128)], vocab=160, width=224, scale=2.0),
}


def make_state(cfg, seed=0, gain=1.0):
  """name -> f32 array holding bf16 values.  Head norms scale queries and keys so that softmax weights are far from equal;
  the sinks take a visible share."""
  from tunix_amd.grouped import GroupedConfig
  rng = np.random.default_rng(seed)
  out = {}
  for name, shape in GroupedConfig.from_dict(cfg).tensor_shapes().items():
    w = rng.standard_normal(shape)
    if name.endswith(('q.norm', 'k.norm')):
      w = (1.3 + 0.3 * w) * gain
    elif name.endswith(('norm', 'norm1', 'norm2')):
      w = 1.0 + 0.2 * w
    elif name.endswith('.sink'):
      w = 1.0 + w
    elif name.endswith('.b'):
      w = 0.5 * w
    elif name != 'embed':
      w = w * shape[1] ** -0.5
    out[name] = bf16_round(w.astype(np.float32))
  return out


def product(cfg, state, dtype='float32', device='cuda'):
  from tunix_amd.grouped import GroupedConfig, GroupedModel
  st = {k: torch.from_numpy(v).to(torch.bfloat16) for k, v in state.items()}
  return GroupedModel.from_state(GroupedConfig.from_dict(cfg, dtype), st, device=device)


def plain(cfg, state, tokens, dtype='float32', layers_out=None):
  """Logits [T, V] of the plain implementation: exact, or with the product's bf16 roundings."""
  return OG.forward(cfg, state, tokens, bf16_round if dtype == 'bfloat16' else None,
                    np.float32 if dtype == 'bfloat16' else np.float64, layers_out)
