"""Small random models of the latent-attention design for the tests: configuration mappings, weights, product models
and the plain implementation's logits."""
import numpy as np
import torch

from oracle import latent as OL
from oracle.bf16 import bf16_round


def rot(dims, base=10_000.0, scaling=None):
  r = {'dims': dims, 'base': base}
  if scaling:
    r['scaling'] = scaling
  return r


def layer(kind, heads, dim, rot_dim, vdim, kv_rank, ff, r=None, kv_from=None, scale=None):
  m = {'heads': heads, 'dim': dim, 'rot_dim': rot_dim, 'vdim': vdim, 'kv_rank': kv_rank, 'rot': r or rot(rot_dim),
       'scale': scale if scale is not None else (dim + rot_dim) ** -0.5}
  if kv_from is not None:
    m['kv_from'] = kv_from
  return {'type': kind, 'mixer': m, 'mlp': None if ff is None else {'kind': 'dense', 'ff': ff}}


def config(layers, vocab=101, width=80, streams=2, max_positions=300, eps=1e-5, logit_scale=1.0):
  return {'architecture': 'Kagapel', 'layers': layers, 'vocab': vocab, 'width': width, 'streams': streams,
          'max_positions': max_positions, 'norm': {'eps': eps}, 'logit_scale': logit_scale}


YARN = {'factor': 4.0, 'original': 64, 'fast': 4.0, 'slow': 1.0}

# sizes off every padding, equal and unequal pairs, one head, one stream, layers without a feed-forward, latents shared
# over a distance and by several layers, both rotations
CONFIGS = {
    'mixed': config([
        layer('latent_attention', 3, 24, 16, 40, 72, 144, rot(16, 5_000.0, YARN)),
        layer('latent_attention_2', 5, 40, 8, 24, 48, None),
        layer('latent_attention_2', 2, 16, 8, 56, 48, 200, kv_from=1),
        layer('latent_attention', 3, 24, 16, 40, 72, 96, rot(16, 5_000.0)),
    ], logit_scale=0.7),
    'one': config([
        layer('latent_attention_2', 1, 8, 4, 8, 12, 24, rot(4, 100.0)),
        layer('latent_attention', 1, 72, 66, 8, 12, 24, rot(66, 20_000.0, YARN)),
    ], vocab=64, width=36, streams=1, eps=1e-3),
    'wide': config([
        layer('latent_attention_2', 7, 56, 32, 48, 300, 272),
        layer('latent_attention', 34, 32, 32, 16, 200, 320, scale=0.3),
        layer('latent_attention_2', 9, 96, 32, 32, 300, 128, kv_from=0),
        layer('latent_attention_2', 4, 32, 32, 128, 300, 128, kv_from=0),
    ], vocab=160, width=224, streams=5, max_positions=600, logit_scale=1.5),
}


def make_state(cfg, seed=0, gain=1.0):
  """name -> f32 array holding bf16 values.  Matrices keep the scale of what they multiply; queries are `gain` times
  larger, so that softmax weights are far from equal."""
  from tunix_amd.latent import LatentConfig, tensor_shapes
  rng = np.random.default_rng(seed)
  out = {}
  n = cfg['streams']
  for name, shape in tensor_shapes(LatentConfig.from_dict(cfg)).items():
    w = rng.standard_normal(shape)
    if name.endswith(('norm', 'norm1', 'norm2')):
      w = 1.0 + 0.2 * w
    elif name.endswith('.b') or name.endswith('.sink'):
      w = 0.5 * w
    elif '.hc' in name:
      w = {'in': 0.3 * w + 1.0 / n, 'out': 0.3 * w + 1.0, 'mix': 0.2 * w + (np.eye(n) if w.ndim == 2 else 0)}[name.rsplit('.', 1)[1]]
    elif name in ('embed', 'pos'):
      w = w * (1.0 if name == 'embed' else 0.5)
    else:
      w = w * shape[1] ** -0.5 * (2.0 * gain if name.endswith('mix.q') else 1.0)
    out[name] = bf16_round(w.astype(np.float32))
  return out


def product(cfg, state, dtype='float32', device='cuda'):
  from tunix_amd.latent import LatentConfig, LatentModel
  st = {k: torch.from_numpy(v).to(torch.bfloat16) for k, v in state.items()}
  return LatentModel.from_state(LatentConfig.from_dict(cfg, dtype), st, device=device)


def plain(cfg, state, tokens, dtype='float32', layers_out=None):
  """Logits [T, V] of the plain implementation: exact, or with the product's bf16 roundings."""
  return OL.forward(cfg, state, tokens, bf16_round if dtype == 'bfloat16' else None,
                    np.float32 if dtype == 'bfloat16' else np.float64, layers_out)


def error(got, want):
  """Root mean square of the difference over that of the expected logits (means taken off), worst position."""
  d = np.asarray(got, np.float64) - want
  d -= d.mean(-1, keepdims=True)
  w = want - want.mean(-1, keepdims=True)
  return float(np.sqrt((d * d).mean(-1)).max() / np.sqrt((w * w).mean()))


LIMIT = {'float32': 3e-5, 'bfloat16': 3e-2}
