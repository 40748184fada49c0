"""Chunked grouped-attention decoders on the GPU: every mechanism alone against the plain implementation's function, then
whole models (both number formats) through the Sampler: prompts, decoding, portions, mixed batches, chunk edges, reused
caches, long sequences, generation and the trace command."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import common as C
import gpu_util as G
import grouped_common as GC
from gpu_util import act, all_logits, dev, rounded, sampler, up
from oracle import grouped as OG
from tunix_amd import _lib
from tunix_amd.configs import RolloutConfig
from tunix_amd.dense import BandScaling, Rotation

pytestmark = pytest.mark.gpu
S = _lib.stream
FORMATS = ['float32', 'bfloat16']


def widths(d):
  return next(p for p in (64, 128, 256) if d <= p)


# -- mechanisms alone -------------------------------------------------------------
@pytest.mark.parametrize('dtype', FORMATS)
def test_residual_rows(dtype):
  """A norm behind the sublayer, in front of the next one, both or none; every row width class."""
  rng = np.random.default_rng(1)
  for m, d in [(3, 36), (65, 192), (5, 1100), (7, 2304), (2, 4100), (2, 9000)]:
    dp = up(d, 64)
    pad = lambda a: np.pad(a, [(0, 0)] * (a.ndim - 1) + [(0, dp - d)])
    x = pad(rng.standard_normal((m, d)).astype(np.float32))
    y = pad(rounded((3.0 * rng.standard_normal((m, d))).astype(np.float32), dtype))
    pw, nw = (pad(rng.standard_normal(d).astype(np.float32)) for _ in range(2))
    eps = 0.02
    for update in (True, False):
      for post in (True, False):
        for norm in (True, False):
          store = int(not norm)
          add = 0.0 if not update else (OG.rms_norm(y[:, :d].astype(np.float64), pw[:d], eps) if post else y[:, :d])
          new = x[:, :d] + add
          want = OG.rms_norm(new, nw[:d], eps) if norm else new
          xt, yt = G.f32(x), dev(y, dtype) if update else None
          k = [G.f32(pw) if post else None, G.f32(nw) if norm else None]
          xn = dev(np.full((m, dp), np.nan, np.float32), dtype)
          G.call('tmx_residual_rows', S(), act(dtype), G.p(xt), G.p(yt), G.p(k[0]), G.p(k[1]), G.p(xn), m, d, dp, eps, store)
          G.sync()
          got = G.host(xn)
          assert not got[:, d:].any()
          tol = dict(atol=5e-6, rtol=1e-5) if dtype == 'float32' else dict(atol=2e-2, rtol=8e-3)
          np.testing.assert_allclose(got[:, :d], want, **tol)
          np.testing.assert_allclose(G.host(xt)[:, :d], new if (store and update) else x[:, :d], atol=5e-6, rtol=1e-5)


def places(positions, mask, step, T, chunk):
  """Brute force of tmx_row_places for rows that hold tokens: the oldest slot with a token of the same chunk."""
  out = []
  for s in range(positions.shape[0]):
    for t in range(T):
      c = step + t
      p = positions[s, c]
      same = [j for j in range(c + 1) if mask[s, j] and (not chunk or positions[s, j] // chunk == p // chunk)]
      out.append((min(same) if same else c, p))
  return np.array(out)


@pytest.mark.parametrize('chunk', [0, 1, 2, 7, 16, 33, 500])
def test_row_places(chunk):
  """Padding on the left, unused slots inside a sequence, every place within a chunk."""
  rng = np.random.default_rng(chunk)
  buf, T, n = 90, 5, 6
  mask = np.ones((n, buf), bool)
  for s in range(n):
    mask[s, :s * 5] = False
    if s >= 3:
      mask[s, rng.integers(s * 5 + 1, buf, 12)] = False
  pos = np.maximum(np.cumsum(mask, 1) - 1, 0).astype(np.int32)
  for step in (0, 1, 29, 31, 64, 85):
    k = [G.i32(pos), G.u8(mask), G.i32([step])]
    out = torch.full((n * T, 2), -7, dtype=torch.int32, device=G.DEV)
    G.call('tmx_row_places', S(), *(G.p(t) for t in k), buf, out.data_ptr(), n * T, T, 88 + T, chunk)
    G.sync()
    got = out.cpu().numpy()
    np.testing.assert_array_equal(got[:, 1], pos[:, step:step + T].reshape(-1))
    want = places(pos, mask, step, T, chunk)
    for i in range(n * T):
      if not mask[i // T, step + i % T]:
        continue
      first = got[i, 0]
      # a slot without a token in front of the chunk may be named: it is masked anyway
      assert first <= want[i, 0] and not mask[i // T, first:want[i, 0]].any() if chunk else first == 0, (step, i)


def row_case(rng, dtype, H, Kh, dim, vdim, r, m, nseq, cs, buf, maxpos):
  dk, dv = widths(dim), widths(vdim)
  head = lambda n, d, p: np.pad(rng.standard_normal((m, n, d)), [(0, 0), (0, 0), (0, p - d)]).reshape(m, -1)
  z = rounded(np.concatenate([head(H, dim, dk), head(Kh, dim, dk), head(Kh, vdim, dv)], 1).astype(np.float32), dtype)
  nw = [np.pad(1.0 + 0.3 * rng.standard_normal(dim), (0, dk - dim)).astype(np.float32) for _ in range(2)]
  s = r.get('scaling')
  table = Rotation(r['dims'], r['base'], BandScaling(**s) if s else None).table(maxpos).to(G.DEV)
  return dk, dv, z, nw, table


def plain_heads(z, nw, H, Kh, dim, vdim, dk, dv, r, eps, pos):
  """Rows z [m, ...] -> (q [m, H, dim], k [m, Kh, dim], v [m, Kh, vdim]) normed and rotated at pos [m]."""
  m = z.shape[0]
  z = z.astype(np.float64)
  q, k = z[:, :H * dk].reshape(m, H, dk)[..., :dim], z[:, H * dk:(H + Kh) * dk].reshape(m, Kh, dk)[..., :dim]
  v = z[:, (H + Kh) * dk:].reshape(m, Kh, dv)[..., :vdim]
  turn = lambda x, w: np.stack([OG.rotate(OG.rms_norm(x[:, h], w[:dim], eps), pos, r) for h in range(x.shape[1])], 1)
  return turn(q, nw[0]), turn(k, nw[1]), v


SIZES = [(3, 1, 12, 24, GC.rot(12, 50.0)), (6, 2, 64, 100, GC.rot(10, 500.0, GC.BANDS)), (5, 5, 100, 64, GC.rot(100, 1e4)),
         (17, 1, 128, 128, GC.rot(128, 1e4, GC.BANDS)), (4, 2, 200, 256, GC.rot(6, 90.0)), (2, 2, 256, 30, GC.rot(250, 1e4, GC.BANDS)),
         (40, 20, 33, 7, GC.rot(2, 10.0))]


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('size', range(len(SIZES)))
def test_head_rows(dtype, size):
  """Norm per head, rotation at the row's position, cache rows at the row's slot; one and several tokens per pass, a
  position past the table (clamped)."""
  H, Kh, dim, vdim, r = SIZES[size]
  rng = np.random.default_rng(size)
  cs, buf, maxpos, step, eps = 40, 50, 30, 6, 1e-3
  for T, nseq in [(1, 5), (3, 2), (7, 3)]:
    m = nseq * T
    dk, dv, z, nw, table = row_case(rng, dtype, H, Kh, dim, vdim, r, m, nseq, cs, buf, maxpos)
    pos = rng.integers(0, maxpos, m)
    place = np.stack([np.zeros(m), pos], 1).astype(np.int32)
    place[-1, 1] = maxpos + 4
    pos[-1] = maxpos - 1
    zt, qt = dev(z, dtype), dev(np.full((m, H, dk), np.nan, np.float32), dtype)
    kc, vc = (dev(np.full((nseq, Kh, cs, w), 9.0, np.float32), dtype) for w in (dk, dv))
    k = [G.f32(nw[0]), G.f32(nw[1]), G.i32(place), G.i32([step])]
    G.call('tmx_head_rows', S(), act(dtype), G.p(zt), z.shape[1], G.p(k[0]), G.p(k[1]), eps, table.data_ptr(), maxpos,
           G.p(k[2]), G.p(k[3]), buf, G.p(qt), G.p(kc), G.p(vc), m, T, H, Kh, dim, dk, dv, r['dims'], cs)
    G.sync()
    q, kr, vr = plain_heads(z, nw, H, Kh, dim, vdim, dk, dv, r, eps, pos)
    tol = dict(atol=5e-6, rtol=2e-5) if dtype == 'float32' else dict(atol=2e-2, rtol=8e-3)
    got = G.host(qt)
    np.testing.assert_allclose(got[..., :dim], q, **tol)
    assert not got[..., dim:].any()
    kh, vh = G.host(kc), G.host(vc)
    for i in range(m):
      np.testing.assert_allclose(kh[i // T, :, step + i % T, :dim], kr[i], **tol)
      np.testing.assert_array_equal(vh[i // T, :, step + i % T, :vdim], vr[i])
      assert not kh[i // T, :, step + i % T, dim:].any() and not vh[i // T, :, step + i % T, vdim:].any()
    assert (np.delete(kh, np.s_[step:step + T], 2) == 9).all() and (np.delete(vh, np.s_[step:step + T], 2) == 9).all()


def attention_case(dtype, dk, dv, H, Kh, T, nseq, step, cs, sink, seed, chunk=0, far=None, pad=0):
  """Runs tmx_head_attention and returns (got, want) [m, H, dv]; far: (query row, slot) whose score stands out;
  pad: slots without a token in front of sequence s: pad * s."""
  rng = np.random.default_rng(seed)
  m, buf, g = nseq * T, cs + 3, H // Kh
  q = rng.standard_normal((m, H, dk)).astype(np.float32)
  kc = rng.standard_normal((nseq, Kh, cs, dk)).astype(np.float32)
  vc = rng.standard_normal((nseq, Kh, cs, dv)).astype(np.float32)
  if far:
    row, slot = far
    q[row] *= 0.3
    q[row] = q[row, :1]
    kc[row // T, :, slot] = np.sign(q[row, 0]) * 3.0     # one score far above the rest
    vc[row // T, :, slot] = 3.0
  q, kc, vc = (rounded(x, dtype) for x in (q, kc, vc))
  scale = dk ** -0.5
  mask = np.ones((nseq, buf), bool)
  for s in range(nseq):
    mask[s, :min(pad * s, step)] = False
  pos = np.maximum(np.cumsum(mask, 1) - 1, 0).astype(np.int32)
  snk = (2.0 * rng.standard_normal(H)).astype(np.float32) if sink else None
  want = np.zeros((m, H, dv))
  for i in range(m):
    s, c = i // T, step + i % T
    ok = mask[s, :c + 1].copy()
    if chunk:
      ok &= pos[s, :c + 1] // chunk == pos[s, c] // chunk
    for h in range(H):
      want[i, h] = OG.attend(q[i, h:h + 1].astype(np.float64), kc[s, h // g, :c + 1].astype(np.float64), vc[s, h // g, :c + 1].astype(np.float64),
                             scale, None if snk is None else float(snk[h]), ok[None])[0]
  # slots behind the newest one hold large garbage
  jk, jv = kc.copy(), vc.copy()
  jk[:, :, step + T:], jv[:, :, step + T:] = 50.0, 50.0
  out = dev(np.full((m, H, dv), np.nan, np.float32), dtype)
  nb = _lib.lib().tmx_head_attention_workspace_bytes(nseq, T, H, Kh, dv, cs, chunk)
  ws = torch.empty(max(nb, 4), dtype=torch.uint8, device=G.DEV)
  place = torch.zeros(m, 2, dtype=torch.int32, device=G.DEV)
  k = [dev(q, dtype), dev(jk, dtype), dev(jv, dtype), None if snk is None else G.f32(snk), G.u8(mask), G.i32([step]), G.i32(pos)]
  G.call('tmx_row_places', S(), G.p(k[6]), G.p(k[4]), G.p(k[5]), buf, place.data_ptr(), m, T, cs, chunk)
  G.call('tmx_head_attention', S(), act(dtype), *(G.p(t) for t in k[:4]), place.data_ptr(), G.p(k[4]), G.p(k[5]), buf, G.p(out),
         G.p(ws), nseq, T, H, Kh, dk, dv, cs, chunk, scale)
  G.sync()
  return G.host(out), want


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('dk, dv', [(a, b) for a in (64, 128, 256) for b in (64, 128, 256)])
def test_head_attention(dtype, dk, dv):
  """One and many tokens per pass, groups of 1 to 40 query heads (both forms of the walk), every remainder of a block of 32
  slots, one and several splits, padding on the left, chunks on and off block borders, with and without a sink."""
  seed = 0
  for H, Kh, T, nseq, step, cs, chunk in [(1, 1, 1, 2, 0, 40, 0), (6, 2, 1, 3, 31, 64, 32), (16, 4, 1, 1, 700, 800, 0),
                                          (8, 1, 1, 2, 500, 512, 150), (40, 1, 1, 2, 95, 96, 33), (6, 3, 2, 2, 30, 64, 7),
                                          (8, 2, 16, 1, 100, 300, 0), (3, 3, 37, 2, 5, 60, 20), (4, 2, 128, 1, 130, 258, 64),
                                          (4, 4, 1, 140, 40, 64, 16), (3, 1, 128, 1, 0, 128, 1)]:
    for sink in (False, True):
      seed += 1
      print('head attention', dtype, dk, dv, H, Kh, T, nseq, step, cs, chunk, sink, flush=True)
      got, want = attention_case(dtype, dk, dv, H, Kh, T, nseq, step, cs, sink, seed, chunk, pad=3)
      tol = 2e-5 if dtype == 'float32' else 1.2e-2
      assert np.abs(got - want).max() <= tol * max(1.0, np.abs(want).max()), (H, Kh, T, nseq, step, cs, chunk, sink)


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('chunk', [0, 50, 64, 97])
def test_a_single_far_key_decides_the_output(dtype, chunk):
  """A key whose score stands out, around the ends of blocks, of the chunk and of the visible range: a visible one decides
  the output, one slot further it does not exist."""
  for T, step in ((1, 300), (16, 284)):
    border = (step + T - 1) // chunk * chunk if chunk else 0
    for slot in sorted({max(s, 0) for s in (0, 1, 31, 32, border - 2, border - 1, border, border + 1, 255, 256, 287, 288, 298, 299, 300)}):
      row = T - 1
      got, want = attention_case(dtype, 128, 64, 4, 2, T, 1, step, 320, True, slot, chunk, far=(row, slot))
      assert np.abs(got - want).max() <= (3e-5 if dtype == 'float32' else 3e-2) * np.abs(want).max(), (T, slot)
      visible = border <= slot <= step + T - 1
      assert (float(want[row, 0].mean()) > 1.5) == visible, (T, slot)   # the key's value (3) is there, or not at all


@pytest.mark.parametrize('size', range(len(SIZES)))
def test_rows_and_attention_of_one_token_in_one_launch(size):
  """The queries and the new cache row made inside the attention launch: the new token counts, its row is stored, also
  where it opens a block or a chunk; one and several splits."""
  H, Kh, dim, vdim, r = SIZES[size]
  rng = np.random.default_rng(40 + size)
  eps, maxpos, scale = 1e-3, 700, 1.5 * dim ** -0.5
  for nseq, step, cs, chunk in [(3, 0, 40, 0), (3, 32, 64, 32), (2, 63, 100, 20), (1, 600, 700, 0), (1, 640, 700, 300), (70, 33, 50, 17)]:
    print('one launch', size, nseq, step, cs, chunk, flush=True)
    buf = cs + 2
    dk, dv, z, nw, table = row_case(rng, 'bfloat16', H, Kh, dim, vdim, r, nseq, nseq, cs, buf, maxpos)
    mask = np.ones((nseq, buf), bool)
    for s in range(nseq):
      mask[s, :min(2 * s, step)] = False
    pos = np.maximum(np.cumsum(mask, 1) - 1, 0).astype(np.int32)
    pad = lambda x, p: np.pad(x, [(0, 0)] * 3 + [(0, p - x.shape[-1])])
    kc = rounded(pad(rng.standard_normal((nseq, Kh, cs, dim)), dk).astype(np.float32), 'bfloat16')
    vc = rounded(pad(rng.standard_normal((nseq, Kh, cs, vdim)), dv).astype(np.float32), 'bfloat16')
    snk = rng.standard_normal(H).astype(np.float32)
    kc[:, :, step:], vc[:, :, step:] = 20.0, 20.0      # what the slot held before must not be seen
    q, kr, vr = plain_heads(z, nw, H, Kh, dim, vdim, dk, dv, r, eps, pos[:, step])
    q, kr = (rounded(x.astype(np.float32), 'bfloat16').astype(np.float64) for x in (q, kr))
    want = np.zeros((nseq, H, vdim))
    for s in range(nseq):
      ok = mask[s, :step + 1] & ((pos[s, :step + 1] // chunk == pos[s, step] // chunk) if chunk else True)
      for h in range(H):
        g = h // (H // Kh)
        ks = np.concatenate([kc[s, g, :step, :dim], kr[s, g][None]])
        vs = np.concatenate([vc[s, g, :step, :vdim], vr[s, g][None]])
        want[s, h] = OG.attend(q[s, h][None], ks, vs, scale, float(snk[h]), ok[None])[0]
    out = G.bf(np.full((nseq, H, dv), np.nan, np.float32))
    ws = torch.empty(max(_lib.lib().tmx_head_attention_workspace_bytes(nseq, 1, H, Kh, dv, cs, chunk), 4), dtype=torch.uint8, device=G.DEV)
    place = torch.zeros(nseq, 2, dtype=torch.int32, device=G.DEV)
    zt, kt, vt = G.bf(z), G.bf(kc), G.bf(vc)
    k = [G.f32(nw[0]), G.f32(nw[1]), G.f32(snk), G.u8(mask), G.i32([step]), G.i32(pos)]
    G.call('tmx_row_places', S(), G.p(k[5]), G.p(k[3]), G.p(k[4]), buf, place.data_ptr(), nseq, 1, cs, chunk)
    G.call('tmx_head_decode', S(), G.p(zt), z.shape[1], G.p(k[0]), G.p(k[1]), eps, table.data_ptr(), maxpos, place.data_ptr(), G.p(kt),
           G.p(vt), G.p(k[2]), G.p(k[3]), G.p(k[4]), buf, G.p(out), G.p(ws), nseq, H, Kh, dim, dk, dv, r['dims'], cs, chunk, scale)
    G.sync()
    got = G.host(out)
    assert np.abs(got[..., :vdim] - want).max() <= 2e-2 * max(1.0, np.abs(want).max()) and not got[..., vdim:].any()
    kh, vh = G.host(kt), G.host(vt)
    np.testing.assert_allclose(kh[:, :, step, :dim], kr, atol=2e-2, rtol=8e-3)
    np.testing.assert_array_equal(vh[:, :, step, :vdim], vr)
    for new, old in ((kh, kc), (vh, vc)):
      np.testing.assert_array_equal(np.delete(new, step, 2), np.delete(old, step, 2))


# -- whole models -------------------------------------------------------------------
_built, _plain = {}, {}


def model(name, dtype, seed=11):
  if (name, dtype, seed) not in _built:
    st = GC.make_state(GC.CONFIGS[name], seed)
    _built[name, dtype, seed] = GC.product(GC.CONFIGS[name], st, dtype), st
  return _built[name, dtype, seed]


def plain(name, st, t, dtype):
  key = (name, dtype, tuple(int(x) for x in t))
  if key not in _plain:
    _plain[key] = GC.plain(GC.CONFIGS[name], st, t, dtype)
  return _plain[key]


def toks(name, n, seed):
  return np.random.default_rng(seed).integers(0, GC.CONFIGS[name]['vocab'], n)


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(GC.CONFIGS))
def test_prompt_logits(name, dtype):
  m, st = model(name, dtype)
  for n in (1, 2, 33, 200):
    t = toks(name, n, n)
    got = all_logits(sampler(m, 256), [t], 256)[0]
    assert GC.error(got, plain(name, st, t, dtype)) < GC.LIMIT[dtype], n


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(GC.CONFIGS))
def test_portions_and_token_by_token_decoding(name, dtype):
  """However the tokens are cut, down to two and one at a time, the logits are those of the whole prompt."""
  m, st = model(name, dtype)
  t = toks(name, 137, 5)
  want = plain(name, st, t, dtype)
  for cuts in ([1] * 137, [2] * 68 + [1], [3] * 45 + [2], [64, 73], [31, 1, 1, 32, 35, 36, 1], [136, 1], [7] * 19 + [4], [100, 1, 36]):
    got = all_logits(sampler(m, 160), [t], 160, cuts)[0]
    assert GC.error(got, want) < GC.LIMIT[dtype], cuts[:4]


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(GC.CONFIGS))
def test_unequal_requests_in_one_batch(name, dtype):
  """Rows of different lengths (padding on the left, so that their chunks begin at different slots), each as if it were
  alone; more rows than one kernel form takes."""
  m, st = model(name, dtype)
  for lens in ((1, 50, 23, 2), (110, 69, 1), tuple(range(1, 41))):
    rows = [toks(name, n, 100 + n) for n in lens]
    got = all_logits(sampler(m, 128), rows, 128, [max(lens) - 13] + [1] * 11 + [2] if max(lens) > 40 else None)
    for r, g in zip(rows, got):
      assert GC.error(g, plain(name, st, r, dtype)) < GC.LIMIT[dtype], len(r)


@pytest.mark.parametrize('dtype', FORMATS)
def test_a_cache_that_is_used_again(dtype):
  """Batches of other shapes on one sampler, the cache kept or given back in between."""
  m, st = model('mixed', dtype)
  s = sampler(m, 128)
  for i, lens in enumerate([(90, 40), (3, 60), (90, 1), (5,), (2, 2, 2), (100,)]):
    rows = [toks('mixed', n, 200 + 10 * i + n) for n in lens]
    for r, g in zip(rows, all_logits(s, rows, 128, [max(lens) - 1, 1] if max(lens) > 3 else None)):
      assert GC.error(g, plain('mixed', st, r, dtype)) < GC.LIMIT[dtype], lens
    if i % 2:
      s.delete_cache()


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', ['mixed', 'one'])
def test_long_decoding_past_the_first_rotation_table(name, dtype):
  m, st = model(name, dtype)
  m._positions, m._tables, m._desc = 128, {}, None    # a table of 128 positions to begin with
  t = toks(name, 290, 9)
  got = all_logits(sampler(m, 300), [t], 300, [4] + [1] * 286)[0]
  assert m._positions >= 300
  want = plain(name, st, t, dtype)
  assert GC.error(got, want) < GC.LIMIT[dtype]
  assert GC.error(got[:4], want[:4]) < GC.LIMIT[dtype] and GC.error(got[-20:], want[-20:]) < GC.LIMIT[dtype]


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('chunk', [24, 32, 45])
def test_edges_of_chunks_in_prompts_and_in_decoding(dtype, chunk):
  """A token replaced by another just inside or just outside the chunk: the later logits move as the plain model says, or
  not at all, whether they are made in a prompt's portion or one by one."""
  cfg = GC.config([GC.layer(4, 2, 32, 48, GC.rot(16), chunk, 96), GC.layer(4, 1, 64, 32, GC.rot(32, 500.0), chunk, 64)], width=96)
  st = GC.make_state(cfg, 3, gain=1.5)
  m = GC.product(cfg, st, dtype)
  n = 3 * chunk + 5
  t = np.random.default_rng(4).integers(0, 101, n)
  want, edge = GC.plain(cfg, st, t), 2 * chunk
  for cuts in ([n], [edge - 1] + [1] * (n - edge + 1), [edge + 1, n - edge - 1], [chunk, chunk, n - 2 * chunk]):
    s = sampler(m, n + 3)
    base = all_logits(s, [t], n + 3, cuts)[0]
    for at in (0, chunk - 1, chunk, edge - 1, edge, edge + 1):
      o = t.copy()
      o[at] = (o[at] + 7) % 101
      got, w2 = all_logits(s, [o], n + 3, cuts)[0], GC.plain(cfg, st, o)
      assert GC.error(got, w2) < GC.LIMIT[dtype], (cuts[:2], at)
      inside = np.arange(n) // chunk == at // chunk
      inside &= np.arange(n) >= at
      np.testing.assert_array_equal(got[~inside], base[~inside])
      last = np.flatnonzero(inside)[-1]
      if last > at:
        move, expected = got[last] - base[last], w2[last] - want[last]
        assert np.abs(expected).max() > 0 and (dtype == 'bfloat16' or np.abs(move - expected).max() < 0.05 * np.abs(expected).max())


def test_more_rows_than_the_streaming_kernels_take():
  """Passes of more than 128 rows (the 256-row blocks, planes of split projections) and the head in both forms."""
  cfg = GC.config([GC.layer(8, 2, 48, 100, GC.rot(16), 25, 1100), GC.layer(6, 3, 130, 64, GC.rot(64, 1e5, GC.BANDS), 64, 1024)],
                  vocab=300, width=1088)
  st = GC.make_state(cfg, 2)
  rows = [np.random.default_rng(i).integers(0, 300, 40) for i in range(20)]
  want = [GC.plain(cfg, st, r, 'bfloat16') for r in rows[:3]]
  m = GC.product(cfg, st, 'bfloat16')
  for n in (3, 20):
    got = all_logits(sampler(m, 64), rows[:n], 64, [38, 1, 1])
    for g, w in zip(got, want):
      assert GC.error(g, w) < GC.LIMIT['bfloat16']
  # scoring passes take the wide head (width a multiple of 128): compare its log-probs with the logits'
  cfg = dict(cfg, width=1152)
  st = GC.make_state(cfg, 2)
  m = GC.product(cfg, st, 'bfloat16')
  s = sampler(m, 64)
  lp = s.per_token_logps(np.stack([r[:10] for r in rows]), np.stack([r[10:] for r in rows]), pad_id=0, token_mask=np.ones((20, 40), bool))
  z = GC.plain(cfg, st, rows[0])
  z = z - np.log(np.exp(z - z.max(-1, keepdims=True)).sum(-1, keepdims=True)) - z.max(-1, keepdims=True)
  ref = np.array([z[c - 1, rows[0][c]] for c in range(10, 40)])
  assert np.abs(lp[0] - ref).max() < 0.1


def test_scoring_with_unused_slots_between_prompt_and_completion():
  """Prompts padded on the right: the slots of a chunk are not consecutive."""
  m, st = model('mixed', 'float32')
  rng = np.random.default_rng(8)
  p, c = [23, 9, 30], 45
  prompts, comps = np.zeros((3, 30), int), rng.integers(1, 101, (3, c))
  for i, n in enumerate(p):
    prompts[i, :n] = rng.integers(1, 101, n)
  lp = sampler(m, 96).per_token_logps(prompts, comps, pad_id=0)
  for i, n in enumerate(p):
    seq = np.concatenate([prompts[i, :n], comps[i]])
    z = plain('mixed', st, seq, 'float32')
    z = z - z.max(-1, keepdims=True)
    z = z - np.log(np.exp(z).sum(-1, keepdims=True))
    # the first completion token is scored by the logits of the slot before it, which holds no token in padded rows
    ref = np.array([z[k - 1, seq[k]] for k in range(n, n + c)])
    np.testing.assert_allclose(lp[i][1:], ref[1:], atol=2e-4)


@pytest.mark.parametrize('dtype', FORMATS)
def test_projections_whose_k_is_split(dtype):
  """Long K behind the mixer and the feed-forward: the slices' planes are added by the row kernel, in both kernel forms."""
  cfg = GC.config([GC.layer(32, 4, 20, 60, GC.rot(8), 16, 4050), GC.layer(17, 17, 20, 130, GC.rot(20), 9, 2100)], vocab=96, width=250)
  st = GC.make_state(cfg, 4)
  m = GC.product(cfg, st, dtype)
  rows = [np.random.default_rng(i).integers(0, 96, 24) for i in range(12)]
  want = [GC.plain(cfg, st, r, dtype) for r in rows[:2]]
  for n, cuts in ((1, [20, 1, 1, 2]), (2, [24]), (12, [22, 1, 1]), (12, [24])):
    got = all_logits(sampler(m, 32), rows[:n], 32, cuts)
    for g, w in zip(got, want):
      assert GC.error(g, w) < GC.LIMIT[dtype], (n, cuts)


# -- generation through the framework's entry points ------------------------------------
@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', ['mixed', 'wide'])
def test_greedy_generation(name, dtype):
  m, st = model(name, dtype)
  s = sampler(m, 96)
  prompts = [toks(name, n, 300 + n) for n in (5, 31, 12)]
  out = s(prompt_token_ids=prompts, max_generation_steps=24, eos_tokens=[-1], return_logprobs=True)
  checked = 0
  for p, got, lps in zip(prompts, out.tokens, out.logprobs):
    seq = np.concatenate([p, got])
    lg = plain(name, st, seq, 'float32')[len(p) - 1:-1]
    lp = lg - lg.max(-1, keepdims=True)
    lp -= np.log(np.exp(lp).sum(-1, keepdims=True))
    top = np.sort(lg, axis=-1)
    for i, (t, l) in enumerate(zip(got, lps)):
      slack = 1e-3 if dtype == 'float32' else 0.15
      assert lg[i].max() - lg[i, t] <= slack and abs(lp[i, t] - l) <= slack
      checked += top[i, -1] - top[i, -2] > slack and t == lg[i].argmax()
  assert checked > 30
  assert max(int(t.max()) for t in out.tokens) < GC.CONFIGS[name]['vocab']


@pytest.mark.parametrize('dtype', FORMATS)
def test_sampling_modes_logits_and_forbidden_ids(dtype):
  m, st = model('mixed', dtype)       # 101 ids: the head's padding rows must never be drawn
  s = sampler(m, 64)
  prompts = [toks('mixed', 9, i) for i in range(6)]
  for kw in (dict(temperature=3.0, top_p=1.0), dict(temperature=3.0, top_p=0.9), dict(temperature=5.0, top_p=1.0, top_k=40)):
    a = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=3, return_logprobs=True, **kw)
    b = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=3, return_logprobs=True, **kw)
    c = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=4, return_logprobs=True, **kw)
    assert all((x == y).all() for x, y in zip(a.tokens, b.tokens)) and any((x != y).any() for x, y in zip(a.tokens, c.tokens))
    assert all(0 <= int(t) < 101 for r in a.tokens for t in r)
  free = s(prompt_token_ids=prompts, max_generation_steps=8, eos_tokens=[-1])
  banned = sorted({int(t) for r in free.tokens for t in r})[:20]
  held = s(prompt_token_ids=prompts, max_generation_steps=8, eos_tokens=[-1], forbidden_tokens=banned, return_logits=True)
  assert not {int(t) for r in held.tokens for t in r} & set(banned)
  assert held.logits[0].shape == (8, 101)
  want = plain('mixed', st, np.concatenate([prompts[0], held.tokens[0]]), dtype)[8:-1]
  assert GC.error(held.logits[0], want) < GC.LIMIT[dtype]


def test_samples_of_one_prompt_and_graph_replay_agree_with_plain_decoding():
  """The cache fill shared by samples of one prompt, and recorded steps replayed, give the tokens of the plain run."""
  m, _ = model('wide', 'bfloat16')
  base = [toks('wide', 70, i) for i in range(2)]
  prompts = [p for p in base for _ in range(4)]
  s = sampler(m, 128)
  s.share_prompt_kv = False
  want = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
  s.share_prompt_kv = True
  got = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
  assert all((a == b).all() for a, b in zip(want.tokens, got.tokens))
  s.use_graph = True
  for _ in range(3):
    again = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
    assert all((a == b).all() for a, b in zip(got.tokens, again.tokens))
    torch.cuda.synchronize()
    s.use_graph = not s.use_graph


def test_rollout_and_scoring():
  from tunix_amd.rollout import TmxRollout
  m, st = model('mixed', 'float32')
  r = TmxRollout(rollout_actor=m, tokenizer=C.ToyTokenizer(), rollout_config=RolloutConfig(kv_cache_size=64))
  prompts = [toks('mixed', 8, i + 40) for i in range(3)]
  out = r.generate(None, RolloutConfig(max_tokens_to_generate=10, temperature=1.0, top_p=1.0, seed=1, max_prompt_length=8,
                                       kv_cache_size=64, eos_tokens=[-1], return_logprobs=True), prompt_token_ids=prompts)
  lp = r.get_per_token_logps(np.stack(prompts), np.stack(out.tokens))
  ids = np.concatenate([np.stack(prompts), np.stack(out.tokens)], 1)
  if (ids != 0).all():                      # id 0 pads, and would be masked out of the scored sequence
    np.testing.assert_allclose(lp, np.stack([np.array(x) for x in out.logprobs]), atol=2e-4)
  assert r.model() is m and np.isfinite(lp).all()


@pytest.mark.parametrize('dtype', FORMATS)
def test_trace_command(dtype, tmp_path):
  from test_latent import save_model
  cfg = GC.CONFIGS['mixed']
  _, st = model('mixed', dtype)
  save_model(tmp_path / 'model', cfg, st)
  (tmp_path / 'out').mkdir()
  a, b = toks('mixed', 50, 1), toks('mixed', 20, 2)
  steps = [{'step': 0, 'entries': [{'id': 'a', 'tokens': a[:40].tolist(), 'want': [0, 31, 39]}, {'id': 'b', 'tokens': b[:18].tolist(), 'want': [17]}], 'end': []}]
  for i in range(10):
    ent = [{'id': 'a', 'tokens': [int(a[40 + i])], 'want': [0] if i % 3 == 0 else []}]
    if i < 2:
      ent.insert(0, {'id': 'b', 'tokens': [int(b[18 + i])], 'want': [0]})
    steps.append({'step': i + 1, 'entries': ent, 'end': (['b'] if i == 1 else []) + (['a'] if i == 9 else [])})
  steps.append({'step': 11, 'entries': [{'id': 'b', 'tokens': b.tolist(), 'want': [3]}], 'end': ['b']})
  root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
  p = subprocess.run([sys.executable, os.path.join(root, 'bin', 'trace_run'), '--model', str(tmp_path / 'model'), '--dtype', dtype,
                      '--out', str(tmp_path / 'out'), '--max-tokens', '80'], input='\n'.join(json.dumps(s) for s in steps) + '\n',
                     capture_output=True, text=True, timeout=100)
  assert p.returncode == 0, p.stderr[-2000:]
  assert [l for l in p.stdout.splitlines() if l.startswith('done')] == [f'done {i}' for i in range(12)]
  read = lambda n: np.fromfile(tmp_path / 'out' / f'{n}.f32', '<f4').reshape(-1, 101)
  pa, pb = plain('mixed', st, a, dtype), plain('mixed', st, b, dtype)
  assert GC.error(read(0), np.stack([pa[0], pa[31], pa[39], pb[17]])) < GC.LIMIT[dtype]
  assert GC.error(read(1), np.stack([pb[18], pa[40]])) < GC.LIMIT[dtype]
  assert GC.error(read(10), pa[49:50]) < GC.LIMIT[dtype] and GC.error(read(11), pb[3:4]) < GC.LIMIT[dtype]
  assert not (tmp_path / 'out' / '3.f32').exists()
