"""Chunked grouped-attention decoders without a GPU: configuration, weight layout, cache views, rotation tables, registry,
argument checks of the C ABI, and the plain implementation's own checks (that a fault of a mechanism would show)."""
import copy
import ctypes
import json

import numpy as np
import pytest
import torch

import grouped_common as GC
from oracle import grouped as OG
from test_latent import unpack
from tunix_amd import _lib, registry
from tunix_amd.dense import BandScaling, Rotation
from tunix_amd.grouped import GroupedConfig, GroupedModel


def tokens(cfg, n, seed=1):
  return np.random.default_rng(seed).integers(0, cfg['vocab'], n)


# -- configuration -------------------------------------------------------------
def test_configuration_reads_every_size_and_constant():
  c = GroupedConfig.from_dict(GC.CONFIGS['mixed'])
  assert (c.vocab_size, c.embed_dim, c.embed_scale, c.norm_eps, c.num_layers, c.max_positions) == (101, 80, 3.0, 1e-5, 5, None)
  l = c.layers[0]
  assert (l.heads, l.kv_heads, l.dim, l.vdim, l.chunk, l.ff, l.weights_of) == (6, 2, 24, 40, 32, 144, None)
  assert l.scale == 24 ** -0.5 and l.rot == Rotation(16, 5000.0, BandScaling(4.0, 1.0, 3.0, 64.0))
  assert c.layers[1].ff is None and c.layers[1].rot.scaling is None and c.layers[3].weights_of == 0
  assert GroupedConfig.from_dict(GC.CONFIGS['wide']).layers[2].chunk is None
  assert (c.num_kv_heads, c.head_dim, c.logits_width) == (5, 256, 128)


def test_a_layer_may_borrow_from_one_that_borrows():
  raw = copy.deepcopy(GC.CONFIGS['mixed'])
  raw['layers'].append(copy.deepcopy(raw['layers'][3]))
  raw['layers'][5]['weights_of'] = 3
  assert GroupedConfig.from_dict(raw).layers[5].weights_of == 0


def test_a_layer_may_borrow_from_a_later_one():
  layers = [GC.layer(*GC._A, weights_of=1), GC.layer(*GC._A), GC.layer(*GC._B)]
  cfg = GC.config(layers)
  st = GC.make_state(cfg)
  assert not any(k.startswith('l0.') for k in st)
  m = GC.product(cfg, st, device='cpu')
  assert m.layers[0] is m.layers[1] and m.desc().num_layers == 3
  assert np.isfinite(GC.plain(cfg, st, tokens(cfg, 5))).all()


@pytest.mark.parametrize('edit, text', [
    (lambda c: c['layers'][0].update(type='other'), 'unknown mixer'),
    (lambda c: c['layers'][0]['mlp'].update(kind='sparse'), 'feed-forward kind'),
    (lambda c: c['layers'][0]['mixer'].update(kv_heads=4), 'do not divide'),
    (lambda c: c['layers'][0]['mixer'].update(dim=300), '1 to 256 dimensions'),
    (lambda c: c['layers'][0]['mixer'].update(vdim=257), '1 to 256 dimensions'),
    (lambda c: c['layers'][1]['mixer']['rot'].update(dims=42), 'does not fit'),
    (lambda c: c['layers'][1]['mixer']['rot'].update(dims=5), 'does not fit'),
    (lambda c: c['layers'][0]['mixer'].update(mask={'size': -2}), 'chunks of'),
    (lambda c: c['layers'][3].update(weights_of=2), 'no tensors of its own of the same'),
    (lambda c: c['layers'][3].update(weights_of=3), 'no tensors of its own'),
    (lambda c: c['layers'][3].update(weights_of=9), 'no tensors of its own'),
])
def test_configurations_outside_the_design_are_refused(edit, text):
  raw = copy.deepcopy(GC.CONFIGS['mixed'])
  edit(raw)
  with pytest.raises(ValueError, match=text):
    GroupedConfig.from_dict(raw)


@pytest.mark.parametrize('r', [GC.rot(16, 5000.0), GC.rot(2, 7.0, GC.BANDS), GC.rot(64, 1e6, GC.BANDS),
                               GC.rot(128, 5e5, {'factor': 8.0, 'low': 1.0, 'high': 4.0, 'original': 8192}),
                               GC.rot(32, 1e4, {'factor': 2.5, 'low': 2.0, 'high': 32.0, 'original': 100})])
def test_rotation_table_is_the_plain_rotation(r):
  s = r.get('scaling')
  product = Rotation(r['dims'], r['base'], BandScaling(**s) if s else None)
  f, mult = product.frequencies()
  np.testing.assert_allclose(f, OG.rotary_frequencies(r), rtol=1e-13)
  assert mult == 1.0
  t = product.table(70).numpy()
  x = np.random.default_rng(0).standard_normal((70, r['dims'] + 3))
  h = r['dims'] // 2
  u, v = x[:, :h], x[:, h:2 * h]
  got = np.concatenate([u * t[..., 0] - v * t[..., 1], v * t[..., 0] + u * t[..., 1], x[:, 2 * h:]], -1)
  np.testing.assert_allclose(got, OG.rotate(x, np.arange(70), r), atol=1e-5)


def test_frequency_bands_have_all_three_parts():
  r = GC.rot(64, 1e4, GC.BANDS)
  ratio = OG.rotary_frequencies(GC.rot(64, 1e4)) / OG.rotary_frequencies(r)
  assert (ratio == 1).any() and (np.abs(ratio - 4) < 1e-12).any() and ((ratio > 1.01) & (ratio < 3.99)).any()


def test_rotation_tables_grow_with_the_sequences():
  cfg = GC.CONFIGS['one']
  m = GC.product(cfg, GC.make_state(cfg), device='cpu')
  n = m._positions
  d = m.desc()
  m.reserve_positions(n)
  assert m.desc() is d and d.max_positions == n
  m.reserve_positions(3 * n)
  assert m._positions >= 3 * n and m.desc().max_positions == m._positions
  for l, a in zip(m.config.layers, m._keep):
    t = m._table(l.rot)
    assert t.shape == (m._positions, l.rot.dims // 2, 2) and a.table == t.data_ptr()


# -- weights --------------------------------------------------------------------
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', sorted(GC.CONFIGS))
def test_weights_sit_where_the_kernels_read_them_and_padding_is_zero(name, dtype):
  cfg = GC.CONFIGS[name]
  st = GC.make_state(cfg, 3)
  m = GC.product(cfg, st, dtype, device='cpu')
  d = cfg['width']
  for i, (l, w) in enumerate(zip(m.config.layers, m.layers)):
    src = i if l.weights_of is None else l.weights_of
    assert w is m.layers[src]
    z, bias = unpack(w['in'])[0].numpy(), w['in'].bias.numpy()
    want, wb = np.zeros_like(z), np.zeros_like(bias)
    off = 0
    for n, heads, width, padded in (('q', l.heads, l.dim, l.dim_p), ('k', l.kv_heads, l.dim, l.dim_p), ('v', l.kv_heads, l.vdim, l.vdim_p)):
      for h in range(heads):
        want[off:off + width, :d] = st[f'l{src}.mix.{n}'][h * width:(h + 1) * width]
        wb[off:off + width] = st[f'l{src}.mix.{n}.b'][h * width:(h + 1) * width]
        off += padded
    assert off == z.shape[0]
    np.testing.assert_array_equal(z, want)
    np.testing.assert_array_equal(bias, wb)
    o = unpack(w['o'])[0].numpy().reshape(-1, l.heads, l.vdim_p)
    for h in range(l.heads):
      np.testing.assert_array_equal(o[:d, h, :l.vdim], st[f'l{src}.mix.o'][:, h * l.vdim:(h + 1) * l.vdim])
    assert not o[d:].any() and not o[:, :, l.vdim:].any()
    for n in ('q', 'k'):
      np.testing.assert_array_equal(w[f'{n}_norm'].numpy(), np.pad(st[f'l{src}.mix.{n}.norm'], (0, l.dim_p - l.dim)))
    if l.ff is not None:
      g = unpack(w['gate_up'])[0].numpy()
      np.testing.assert_array_equal(g[:l.ff, :d], st[f'l{src}.mlp.up'])
      assert not g[l.ff:].any() and not g[:, d:].any()
      np.testing.assert_array_equal(unpack(w['down'])[0].numpy()[:d, :l.ff], st[f'l{src}.mlp.down'])


def test_state_must_fit_the_configuration():
  cfg = GC.CONFIGS['mixed']
  st = {k: torch.from_numpy(v) for k, v in GC.make_state(cfg).items()}
  c = GroupedConfig.from_dict(cfg)
  with pytest.raises(KeyError, match='missing'):
    GroupedModel.from_state(c, {k: v for k, v in st.items() if k != 'l0.mix.sink'}, device='cpu')
  with pytest.raises(KeyError, match='unexpected'):
    GroupedModel.from_state(c, {**st, 'l3.mix.q': st['l0.mix.q']}, device='cpu')  # a layer that borrows has none
  with pytest.raises(ValueError, match='shape'):
    GroupedModel.from_state(c, {**st, 'l0.mix.q.b': st['l0.mix.q.b'][:3]}, device='cpu')
  GroupedModel.from_state(c, {**st, 'l1.norm2': st['l0.norm2']}, device='cpu')    # the norm behind no feed-forward is idle


def test_cache_views_tile_the_cache_and_every_layer_has_its_own():
  c = GroupedConfig.from_dict(GC.CONFIGS['mixed'])
  b, size = 3, 40
  cache = torch.zeros(c.cache_shape(b, size))
  views = c.cache_rows(cache, b, size)
  assert [tuple(v.shape) for v in views[:4]] == [(b, size, 2, 64), (b, size, 2, 64), (b, size, 5, 64), (b, size, 5, 64)]
  assert [v.shape[-1] for v in views[4:6]] == [128, 256] and len(views) == 10
  for v in views:
    v += 1
  assert bool((cache == 1).all())


# -- registry ---------------------------------------------------------------------
def test_registry_builds_the_model_config_json_names(tmp_path):
  from test_latent import save_model
  cfg = GC.CONFIGS['mixed']
  save_model(tmp_path / 'm', cfg, GC.make_state(cfg))
  m = registry.load_model(str(tmp_path / 'm'), 'float32', device='cpu')
  assert isinstance(m, GroupedModel) and m.dtype == torch.float32 and m.config == GroupedConfig.from_dict(cfg, 'float32')
  (tmp_path / 'm' / 'config.json').write_text(json.dumps(dict(cfg, architecture=None, architectures=['Feduzen'])))
  assert registry.load_config(str(tmp_path / 'm')).dtype == 'bfloat16'


# -- C ABI without a device ------------------------------------------------------------
def test_argument_checks_of_the_entry_points():
  lib = _lib.lib()
  p = 0x1000
  assert lib.tmx_residual_rows(None, 0, None, p, p, p, p, 4, 64, 64, 1e-5, 1) == -1
  assert lib.tmx_residual_rows(None, 0, p, p, p, p, p, 4, 65, 64, 1e-5, 1) == -2
  assert lib.tmx_residual_rows(None, 0, p, p, p, p, p, 4, 20000, 20032, 1e-5, 1) == -2
  assert lib.tmx_row_places(None, p, p, p, 8, None, 4, 1, 8, 3) == -1
  assert lib.tmx_row_places(None, p, p, p, 8, p, 5, 2, 8, 3) == -2
  rows = lambda H=4, Kh=2, dim=50, dk=64, dv=64, rot=8, ldz=512, table=p: lib.tmx_head_rows(
      None, 0, p, ldz, p, p, 1e-5, table, 8, p, p, 8, p, p, p, 1, 1, H, Kh, dim, dk, dv, rot, 8)
  assert rows(table=None) == -1
  assert [rows(H=3), rows(dim=65), rows(dk=96), rows(dv=32), rows(rot=7), rows(rot=52), rows(ldz=508)] == [-2] * 7
  att = lambda H=4, Kh=2, dk=64, dv=64, T=1, C=8, place=p: lib.tmx_head_attention(
      None, 0, p, p, p, None, place, p, p, 8, p, None, 1, T, H, Kh, dk, dv, C, 0, 1.0)
  assert att(place=None) == -1
  assert [att(H=5), att(dk=192), att(dv=0), att(T=9)] == [-2] * 4
  assert att(C=4096) == -1                                # several splits need a workspace
  dec = lambda H=4, Kh=2: lib.tmx_head_decode(None, p, 8192, p, p, 1e-5, p, 8, p, p, p, p, p, p, 8, p, None, 1, H, Kh, 64, 64, 64, 8, 8, 4, 1.0)
  assert dec(H=33, Kh=1) == -1                            # more query heads per key head than one tile holds
  size = lib.tmx_head_attention_workspace_bytes
  assert size(300, 1, 8, 8, 64, 64, 0) == 0 and size(1, 1, 8, 2, 64, 4096, 0) > size(1, 1, 8, 2, 64, 4096, 300) > 0
  assert size(1, 1, 8, 3, 64, 4096, 0) == 0


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_step_descriptor_is_accepted_and_its_faults_are_not(dtype):
  lib = _lib.lib()
  m = GC.product(GC.CONFIGS['mixed'], GC.make_state(GC.CONFIGS['mixed']), dtype, device='cpu')
  d = m.desc()
  n = lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64)
  assert 0 < n < lib.tmx_decode_workspace_bytes(ctypes.byref(d), 400, 64)
  for field, bad in (('streams', 2), ('act', 7), ('max_positions', 0), ('norm_after', 0)):
    good = getattr(d, field)
    setattr(d, field, bad)
    assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == 0, field
    setattr(d, field, good)
  a = m._keep[2]
  for field, bad in (('mixer', 5), ('ff', 0), ('kv_heads', 2), ('dim', 200), ('dim_p', 192), ('rot_dim', 3), ('chunk', -1), ('table', None)):
    good = getattr(a, field)
    setattr(a, field, bad)
    assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == 0, field
    setattr(a, field, good)
  assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == n


# -- the plain implementation -----------------------------------------------------------
def _faults():
  """name -> (configuration, state) -> the same with one mechanism left out or changed."""
  def cfg_edit(fn):
    def go(cfg, st):
      cfg = copy.deepcopy(cfg)
      fn(cfg)
      return cfg, st
    return go

  def st_edit(fn):
    def go(cfg, st):
      st = dict(st)
      fn(st)
      return cfg, st
    return go

  def every(key, fn):
    return st_edit(lambda s: s.update({k: fn(v) for k, v in s.items() if k.endswith(key)}))

  mix = lambda c, i: c['layers'][i]['mixer']
  return {
      'no sink': every('.sink', lambda v: np.full_like(v, -1e4)),
      'no bias of q': every('mix.q.b', np.zeros_like),
      'no bias of k': every('mix.k.b', np.zeros_like),
      'no bias of v': every('mix.v.b', np.zeros_like),
      'q norm weights in another order': every('q.norm', lambda v: v[::-1].copy()),
      'no norm weight behind the mixer': every('norm1', np.ones_like),
      'no bands': cfg_edit(lambda c: mix(c, 0)['rot'].pop('scaling')),
      'fewer rotated dimensions': cfg_edit(lambda c: [mix(c, i)['rot'].update(dims=8) for i in (0, 3)]),
      'chunk one longer': cfg_edit(lambda c: [mix(c, i)['mask'].update(size=33) for i in (0, 3)]),
      'chunk one shorter': cfg_edit(lambda c: mix(c, 2)['mask'].update(size=6)),
      'a window instead of chunks': cfg_edit(lambda c: [mix(c, i).pop('mask') for i in (1, 4)]),
      'other scale': cfg_edit(lambda c: mix(c, 2).update(scale=mix(c, 2)['scale'] * 1.05)),
      'other embedding scale': cfg_edit(lambda c: c['embedding'].update(scale=3.2)),
      'other eps': cfg_edit(lambda c: c['norm'].update(eps=1e-2)),
      'other borrowed layer': st_edit(lambda s: s.update({'l1.mix.o': s['l1.mix.o'][:, ::-1].copy()})),
  }


@pytest.mark.parametrize('fault', sorted(_faults()))
def test_a_fault_of_one_mechanism_shows_in_the_logits(fault):
  """The tolerances of the device tests are far below what leaving a mechanism out changes."""
  cfg = GC.CONFIGS['mixed']
  st = GC.make_state(cfg, 5)
  t = tokens(cfg, 80)
  want = GC.plain(cfg, st, t)
  bad_cfg, bad_st = _faults()[fault](cfg, st)
  assert GC.error(GC.plain(bad_cfg, bad_st, t), want) > 30 * GC.LIMIT['float32']
  if fault not in ('other eps', 'other scale'):
    assert GC.error(GC.plain(bad_cfg, bad_st, t), want) > 1.5 * GC.LIMIT['bfloat16']


def test_heads_read_the_key_head_of_their_group():
  cfg = GC.CONFIGS['mixed']
  st = GC.make_state(cfg, 5)
  w = {k: v.astype(np.float64) for k, v in st.items()}
  m = cfg['layers'][0]['mixer']
  h = np.random.default_rng(0).standard_normal((20, 80))
  base = OG.mixer(w, 'l0.mix', m, h, 1e-5, lambda x: x)
  w['l0.mix.o'] = np.where(np.arange(240) // 40 < 3, 0.0, w['l0.mix.o'])          # only query heads 3, 4, 5 reach the output
  one = OG.mixer(w, 'l0.mix', m, h, 1e-5, lambda x: x)
  w['l0.mix.v.b'] = w['l0.mix.v.b'] + np.where(np.arange(80) < 40, 1.0, 0.0)      # value head 0 changes
  np.testing.assert_array_equal(OG.mixer(w, 'l0.mix', m, h, 1e-5, lambda x: x), one)
  assert np.abs(base - one).max() > 0.1


def test_the_roundings_of_the_bf16_form_stay_within_its_tolerance():
  for name, cfg in GC.CONFIGS.items():
    st = GC.make_state(cfg, 6)
    t = tokens(cfg, 33)
    assert 0 < GC.error(GC.plain(cfg, st, t, 'bfloat16'), GC.plain(cfg, st, t)) < GC.LIMIT['bfloat16'], name


def test_plain_attention_is_causal_and_chunks_do_not_see_each_other():
  cfg = GC.config([GC.layer(4, 2, 16, 16, GC.rot(8), 12, 64)] * 2)
  st = GC.make_state(cfg, 7)
  t = tokens(cfg, 40)
  other = t.copy()
  other[20] = (other[20] + 1) % cfg['vocab']
  a, b = GC.plain(cfg, st, t), GC.plain(cfg, st, other)
  same = np.r_[0:20, 24:40]
  np.testing.assert_array_equal(a[same], b[same])
  assert (np.abs(a[20:24] - b[20:24]).max(-1) > 1e-3).all()
