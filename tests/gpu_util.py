"""Helpers for the GPU parity tests: numpy <-> device tensors and thin C-ABI callers."""
import ctypes

import numpy as np
import torch

import common as C
from oracle.bf16 import bf16_round
from tunix_amd import _lib

DEV = 'cuda'


def bf(x):
  """numpy f32 holding bf16 values -> device bf16 tensor."""
  return torch.from_numpy(np.ascontiguousarray(x, dtype=np.float32)).to(torch.bfloat16).to(DEV)


def f32(x):
  return torch.from_numpy(np.ascontiguousarray(x, dtype=np.float32)).to(DEV)


def i32(x):
  return torch.from_numpy(np.ascontiguousarray(x, dtype=np.int32)).to(DEV)


def u8(x):
  return torch.from_numpy(np.ascontiguousarray(x, dtype=np.uint8)).to(DEV)


def host(t):
  return t.float().cpu().numpy()


def p(t):
  return None if t is None else t.data_ptr()


def ulp_bf16(ref):
  """One bf16 ulp at the magnitude of ref (elementwise)."""
  a = np.maximum(np.abs(ref), 2.0 ** -120).astype(np.float32)
  return np.exp2(np.floor(np.log2(a)) - 7).astype(np.float32)


def assert_bf16_close(got, ref, ulps=1.0, extra=0.0, min_exact=0.0, what='', stragglers=0):
  """|got - ref| <= ulps bf16 ulp + extra everywhere; `stragglers` elements (coincidences of several
  rounding flips in samples of millions) may reach three times that bound."""
  d = np.abs(got - ref)
  bound = ulps * ulp_bf16(np.maximum(np.abs(ref), np.abs(got))) + extra
  bad = d > bound
  if stragglers and 0 < bad.sum() <= stragglers:
    bad = d > 3.0 * bound
  assert not bad.any(), f'{what}: {bad.sum()} of {bad.size} beyond {ulps} bf16 ulp; worst {d.max()} at ref {ref.flat[d.argmax()]}'
  if min_exact:
    assert (d == 0).mean() >= min_exact, f'{what}: only {(d == 0).mean():.5f} exact'


def call(name, *args):
  lib = _lib.lib()
  rc = getattr(lib, name)(*args)
  _lib.check(rc, name)


def sync():
  torch.cuda.synchronize()


class Keep:
  """Creates device tensors and keeps them alive until the arena is dropped, returning raw
  pointers (a temporary tensor would be recycled by the caching allocator before the launch)."""

  def __init__(self):
    self.t = []

  def _k(self, t):
    self.t.append(t)
    return t.data_ptr()

  def bf(self, x):
    return self._k(bf(x))

  def f32(self, x):
    return self._k(f32(x))

  def i32(self, x):
    return self._k(i32(x))

  def u8(self, x):
    return self._k(u8(x))


# -- dense decoders: number formats, and whole models through the Sampler ------------------
def dev(x, dtype):
  return f32(x) if dtype == 'float32' else bf(x)


def act(dtype):
  return 1 if dtype == 'float32' else 0


def rounded(x, dtype):
  return x if dtype == 'float32' else bf16_round(x)


def up(v, k):
  return -(-v // k) * k


def sampler(m, size):
  from tunix_amd.configs import CacheConfig
  from tunix_amd.sampler import Sampler
  c = m.config
  s = Sampler(m, C.ToyTokenizer(), CacheConfig(size, c.num_layers, c.num_kv_heads, c.head_dim))
  s.eos_ids = np.array([-1])
  return s


def batch_state(s, rows, total):
  width = max(len(r) for r in rows)
  ids = np.zeros((len(rows), width), np.int32)
  for i, r in enumerate(rows):
    ids[i, width - len(r):] = r
  st = s.init_sample_state(ids, total, False, None, 1.0, None, None, 0, prompt_lengths=np.array([len(r) for r in rows]))
  st['fresh'] = False
  return st, width


def all_logits(s, rows, total, cuts=None):
  """Logits of every token of every row; the columns in portions of `cuts` (None: as the walk likes)."""
  st, width = batch_state(s, rows, total)
  got = [np.zeros((len(r), s.transformer.config.vocab_size)) for r in rows]
  beg = 0
  for n in (cuts or [width]):
    wanted = [(i, c - beg) for i, r in enumerate(rows) for c in range(beg, beg + n) if c >= width - len(r)]
    lg = s.walk_logits(st, n, wanted).cpu().numpy()
    for (i, off), v in zip(wanted, lg):
      got[i][beg + off - (width - len(rows[i]))] = v
    beg += n
  assert beg == width
  s.check_device_status(st)
  return got
