"""The mechanisms of the decoder-only models with latent attention on the GPU, each
alone through the C ABI, against the plain float64 oracle.  (Whole models of this
kind run through the tests of test_gpu_hybrid.py.)"""

import numpy as np
import pytest
import torch

from oracle import latent_lm as oracle
from oracle.hybrid_lm import rms
from oracle.hybrid_lm import sigmoid
from tests import hybrid_cases as cases
from tests.test_gpu_hybrid import DTYPES
from tests.test_gpu_hybrid import Ragged
from tests.test_gpu_hybrid import dev
from tests.test_gpu_hybrid import host
from tests.test_gpu_hybrid import rel

pytestmark = pytest.mark.gpu


def tol(dt):
  return 2e-6 if dt == torch.float32 else 6e-3


# ---- experts ------------------------------------------------------------------------


@pytest.mark.parametrize('M,E,top,skew', [(1, 3, 1, False), (37, 5, 2, False),
                                          (300, 4, 3, False), (700, 40, 4, False),
                                          (90, 7, 1, True), (2000, 3, 2, False)])
@pytest.mark.parametrize('dt', DTYPES)
def test_experts_by_table(dt, M, E, top, skew):
  """Every tile height; experts without tokens and one with all of them."""
  from t5x_amd import ops
  rs = np.random.RandomState(M)
  V, K, F, N = 50, 96, 64, 128
  table = np.argsort(rs.rand(V, E), axis=1)[:, :top]
  if skew:
    table[:] = np.arange(top) + E - top
  ids = rs.randint(0, V, M)
  tiles, token_of, entry_of, rows = ops.route_tokens(
      dev(ids, torch.int32), dev(table, torch.int32), E, dt)
  t, tok, ent = (x.cpu().numpy() for x in (tiles, token_of, entry_of))
  expert = np.full(M * top, -1)
  for e, first, n, _ in t:
    if e >= 0:
      assert 0 < n <= rows and (expert[first:first + n] == -1).all()
      expert[first:first + n] = e
  assert sorted(ent.ravel()) == list(range(M * top))
  np.testing.assert_array_equal(expert[ent], table[ids])
  np.testing.assert_array_equal(tok[ent], np.repeat(np.arange(M)[:, None], top, 1))

  a = dev(2 * rs.randn(M, K), dt)
  gate, up = (dev(rs.randn(E, K, F) / np.sqrt(K)) for _ in range(2))
  down = dev(rs.randn(E, F, N) / np.sqrt(F))
  hidden = torch.full((M * top, F), 7.0, dtype=dt, device='cuda')
  ops.grouped_dense(a, [ops.pack_weight(g, dt, gate_kernel=u)
                        for g, u in zip(gate, up)], hidden, tiles, token_of, rows,
                    glu=(0.8, 1.702, 1.0))
  out = torch.full((M * top, N), 7.0, dtype=dt, device='cuda')
  ops.grouped_dense(hidden, [ops.pack_weight(d, dt) for d in down], out, tiles,
                    None, rows)
  w = lambda x, e: host(x[e].to(dt)).T
  got = host(out)
  for e in range(E):
    at = np.flatnonzero(expert == e)
    if len(at) == 0:
      continue
    g = np.minimum(host(a)[tok[at]] @ w(gate, e).T, 0.8)
    u = np.clip(host(a)[tok[at]] @ w(up, e).T, -0.8, 0.8)
    want = g * sigmoid(1.702 * g) * (u + 1)
    assert rel(host(hidden)[at], want) < tol(dt)
    assert rel(got[at], host(hidden)[at] @ w(down, e).T) < tol(dt)


@pytest.mark.parametrize('M', [1, 16, 17, 200])
@pytest.mark.parametrize('dt', DTYPES)
def test_groups_of_columns(dt, M):
  """A kernel per head; the last columns of a group's kernel are not stored."""
  from t5x_amd import ops
  rs = np.random.RandomState(M)
  H, K, N, keep = 5, 64, 48, 36
  a = dev(rs.randn(M, H * K + 8), dt)
  w = dev(rs.randn(H, K, N) / 8)
  out = torch.full((M, H * keep + 4), 7.0, dtype=dt, device='cuda')
  ops.grouped_dense(a, [ops.pack_weight(x, dt) for x in w], out, groups=H,
                    a_step=K, c_step=keep, n_store=keep)
  got = host(out)
  assert (got[:, H * keep:] == 7.0).all()
  for h in range(H):
    want = host(a)[:, h * K:(h + 1) * K] @ host(w[h].to(dt))[:, :keep]
    assert rel(got[:, h * keep:(h + 1) * keep], want) < tol(dt)


@pytest.mark.parametrize('dt', DTYPES)
def test_silu_unit(dt):
  from t5x_amd import ops
  rs = np.random.RandomState(0)
  for M in (5, 300):
    a = dev(4 * rs.randn(M, 64), dt)
    gate, up = (dev(rs.randn(64, 40) / 8) for _ in range(2))
    got = ops.dense(a, ops.pack_weight(gate, dt, gate_kernel=up),
                    glu=(float('inf'), 1.0, 0.0))
    g = host(a) @ host(gate.to(dt))
    want = g * sigmoid(g) * (host(a) @ host(up.to(dt)))
    assert rel(host(got), want) < tol(dt)


# ---- streams ------------------------------------------------------------------------


@pytest.mark.parametrize('dt', DTYPES)
def test_embed_streams(dt):
  from t5x_amd import ops
  rs = np.random.RandomState(3)
  table = np.zeros((20, 64))
  table[:, :40] = rs.randn(20, 40)
  t = dev(table, dt)
  ids = [0, 19, 7, 7]
  got = host(ops.embed_streams(t, dev(ids, torch.int32), 2.5, 40, 3))
  np.testing.assert_allclose(got, np.repeat(2.5 * host(t)[ids][:, None], 3, 1),
                             rtol=1e-6)


@pytest.mark.parametrize('M,n,width,ld', [(1, 1, 40, 64), (5, 3, 90, 128),
                                          (3, 4, 1100, 1152), (4, 6, 37, 64),
                                          (2, 16, 64, 64), (2, 2, 5000, 5056)])
@pytest.mark.parametrize('dt', DTYPES)
def test_hyper_norm(dt, M, n, width, ld):
  from t5x_amd import ops
  rs = np.random.RandomState(M * n)
  eps, top = 1e-4, 2

  def rows(*shape):
    x = np.zeros(shape + (ld,))
    x[..., :width] = 2 * rs.randn(*shape, width)
    return x

  x = dev(rows(M, n))
  y, parts = dev(rows(M), dt), dev(rows(3 * M), dt)
  part_row = dev(rs.randint(0, 3 * M, (M, top)), torch.int32)
  gate = dev(rs.rand(M))
  mix, spread, collect = (dev(rs.randn(n, n)), dev(rs.randn(n)), dev(rs.randn(n)))
  norm, gate_w = dev(rs.randn(width)), dev(rs.randn(width) / np.sqrt(width))
  old = host(x).transpose(1, 0, 2)
  out, total, gate_out = ops.hyper_norm(
      x, width, dt, y=y, y_gate=gate, parts=parts, part_row=part_row,
      part_weight=1 / 3, mix=mix, spread=spread, collect=collect, norm=norm,
      want_sum=True, gate_w=gate_w, eps=eps)
  b = host(gate)[:, None] * host(y) + host(parts)[part_row.cpu().numpy()].sum(1) / 3
  new = oracle.spread(old, host(mix), host(spread), b)
  np.testing.assert_allclose(host(x).transpose(1, 0, 2), new, rtol=1e-5, atol=2e-5)
  u = oracle.collect(new, host(collect))
  np.testing.assert_allclose(host(total), u, rtol=1e-5, atol=1e-4)
  h = rms(u[:, :width], eps) * host(norm)
  assert rel(host(out)[:, :width], h) < tol(dt)
  assert not host(out)[:, width:].any()
  np.testing.assert_allclose(host(gate_out), sigmoid(h @ host(gate_w)), atol=1e-5)
  # picked rows of the plain sum; streams stay
  pick = dev(rs.permutation(M)[:(M + 1) // 2], torch.int32)
  before = host(x)
  out, total, _ = ops.hyper_norm(x, width, dt, norm=norm, rows=pick, want_sum=True,
                                 eps=eps)
  np.testing.assert_array_equal(host(x), before)
  u = before[pick.cpu().numpy()].sum(1)
  np.testing.assert_allclose(host(total), u, rtol=1e-5, atol=1e-4)
  assert rel(host(out)[:, :width], rms(u[:, :width], eps) * host(norm)) < tol(dt)
  # without a mix matrix the branch is added to every stream
  ops.hyper_norm(x, width, dt, y=y)
  np.testing.assert_allclose(host(x), before + host(y)[:, None], rtol=1e-5,
                             atol=1e-5)


# ---- latent attention ------------------------------------------------------------------


class Latent:
  """A latent attention mixer's kernels over random latent inputs."""

  def __init__(self, dt, H, D, Dv, q_rank, rank, window, slots, portion, max_len,
               scale=0.2, eps=1e-5, own=True, ring=None, weights=None, seed=0):
    from t5x_amd import _lib, hybrid
    self.dt, self.dims, self.own = dt, (H, D, Dv, q_rank, rank), own
    self.window, self.scale, self.eps = window, scale, eps
    rs = self.rs = np.random.RandomState(seed)
    m = hybrid.MixerConfig(
        type='latent_attention', heads=H, kv_heads=H, dim=D, vdim=Dv,
        window=window, scale=scale, q_rank=q_rank, kv_rank=rank,
        kv_from=None if own else 0)
    mixer = hybrid.MIXERS[m.type]
    self.w = {}
    for name, shape in mixer.shapes(m, 64).items():
      x = rs.randn(*shape)
      x = (1 + 0.3 * x if 'norm' in name else x if name == 'sink'
           else x / np.sqrt(shape[1]))
      self.w[name] = cases.bf16(x)
    self.w.update(weights or {})
    self.kept = []

    def keep(t, dtype=torch.float32):
      self.kept.append(t.to(device='cuda', dtype=dtype).contiguous())
      return self.kept[-1].data_ptr()

    layer = _lib.HybridLayer()
    mixer.fill(layer, m, lambda name: dev(self.w[name]), keep, eps, 64,
               hybrid.Packer(dt, self.kept))
    a = self.a = layer.latent
    self.cols = layer.proj_n
    self.hp, self.rp, self.qp = mixer.pads(m)
    if ring is None:
      n = window - 1 + portion if window else max_len
      ring = torch.full((slots, (n + 63) // 64 * 64, self.rp), 3.0, dtype=dt,
                        device='cuda')
    self.ring = ring
    a.dtype, a.ring, a.ld_proj = _lib.dtype_code(dt), ring.shape[1], self.cols
    a.latent_ring = ring.data_ptr()

  def sequence(self, T):
    x = torch.zeros((T, self.cols), dtype=self.dt, device='cuda')
    H, D, Dv, q_rank, rank = self.dims
    x[:, :q_rank] = dev(self.rs.randn(T, q_rank), self.dt)
    if self.own:
      x[:, self.a.off_kv:self.a.off_kv + rank] = dev(self.rs.randn(T, rank), self.dt)
    return x

  def run(self, portions, proj, variant=0, workspace=True):
    """portions [(slot, start)], proj their rows -> [M, H * Dv]."""
    from t5x_amd import _lib, hybrid, ops
    H, _, Dv, _, rank = self.dims
    x = torch.cat(proj).contiguous()
    p = hybrid.Portions([(s, at, np.zeros(len(t), np.int32))
                         for (s, at), t in zip(portions, proj)], [], 'cuda',
                        [self.window])
    if variant == 2 and p.ragged.n_spans == 0:
      variant = 0
    M = len(x)
    ld = (H * Dv + 3) // 4 * 4 + 4
    out = torch.full((M, ld), 5.0, dtype=self.dt, device='cuda')
    make = lambda n, c: torch.empty((n, c), dtype=self.dt, device='cuda')
    a, rows = self.a, 2 * M
    bufs = dict(cq=make(M, self.qp), q=make(M, H * self.hp), ql=make(M, H * self.rp),
                ol=make(M, H * self.rp), lat=make(rows, self.rp),
                kv=make(rows, 2 * H * self.hp))
    for name, t in bufs.items():
      setattr(a, name, t.data_ptr())
    ws = torch.empty((_lib.load().t5d_latent_workspace_bytes(rank),),
                     dtype=torch.uint8, device='cuda')
    a.span_rows, a.proj, a.out, a.ld_out = rows, x.data_ptr(), out.data_ptr(), ld
    a.workspace = ws.data_ptr() if workspace else None
    ops.latent_attention(a, p.ragged, variant)
    got = host(out)
    assert (got[:, H * Dv:] == 5.0).all()
    return got[:, :H * Dv]

  def oracle(self, proj, latents=None):
    H, D, Dv, q_rank, rank = self.dims
    x, T = host(proj), len(proj)
    rounded = (lambda v: cases.bf16(v).astype(float)
               ) if self.dt == torch.bfloat16 else (lambda v: v)
    cq = rounded(rms(x[:, :q_rank], self.eps) * self.w['dq.norm'])
    if latents is None:
      latents = self.latents(proj)
    part = lambda v, n: (v.astype(float)).reshape(T, H, n)
    o = oracle.sink_window_attention(
        part(rounded(cq @ self.w['uq'].T), D), part(latents @ self.w['uk'].T, D),
        part(latents @ self.w['uv'].T, Dv), self.scale, self.window or None,
        self.w['sink'])
    return o.reshape(T, H * Dv)

  def latents(self, proj):
    x = host(proj)[:, self.a.off_kv:self.a.off_kv + self.dims[4]]
    c = rms(x, self.eps) * self.w['dkv.norm']
    return cases.bf16(c).astype(float) if self.dt == torch.bfloat16 else c

  @property
  def tol(self):
    return 3e-6 if self.dt == torch.float32 else 1.5e-2


SHAPES = [(4, 32, 32, 64, 64), (5, 24, 40, 20, 72), (16, 64, 48, 100, 128),
          (17, 20, 10, 40, 200), (40, 16, 16, 30, 64), (2, 128, 128, 64, 512),
          (33, 40, 24, 16, 300), (1, 10, 200, 8, 9)]
WAVE_SHAPES = SHAPES[:4] + [(3, 300, 12, 40, 600)]


@pytest.mark.parametrize('dt,variant,H,D,Dv,q_rank,rank', [
    (dt, v, *shape) for dt, v, shapes in (
        (torch.float32, 0, WAVE_SHAPES), (torch.bfloat16, 1, SHAPES),
        (torch.bfloat16, 2, SHAPES), (torch.bfloat16, 3, WAVE_SHAPES))
    for shape in shapes])
@pytest.mark.parametrize('window', [0, 1, 9, 64, 65])
def test_prompts_and_portions(dt, variant, H, D, Dv, q_rank, rank, window):
  a = Latent(dt, H, D, Dv, q_rank, rank, window, 2, 100, 160, seed=H + window)
  x = a.sequence(150)
  want = a.oracle(x)
  at = 0
  for n in (97, 2, 1, 3, 47):
    got = a.run([(1, at)], [x[at:at + n]], variant)
    assert rel(got, want[at:at + n]) < a.tol, at
    at += n


@pytest.mark.parametrize('window', [0, 7, 600])
@pytest.mark.parametrize('H', [3, 16, 40])
def test_decoding_with_the_keys_split_over_workgroups(window, H):
  """Long windows, few sequences: parts and their merge; and without scratch."""
  a = Latent(torch.bfloat16, H, 32, 24, 40, 96, window, 2, 300, 900, seed=H)
  x = a.sequence(900)
  want = a.oracle(x)
  for at in (0, 300, 600):
    a.run([(0, at)], [x[at:at + 290 if at == 600 else at + 300]])
  for i in range(890, 900):
    got = a.run([(0, i)], [x[i:i + 1]], 1, workspace=i % 2 == 0)
    assert rel(got, want[i:i + 1]) < a.tol, i


@pytest.mark.parametrize('dt', DTYPES)
def test_batches_match_each_alone(dt):
  a = Latent(dt, 6, 24, 40, 32, 100, 20, 5, 130, 400)
  lens = [130, 1, 2, 65, 64]
  seqs = [a.sequence(300) for _ in lens]
  want = [a.oracle(s) for s in seqs]
  at = [0] * 5
  for take in (lens, lens, [1] * 5, [1, 2, 1, 3, 1]):
    got = a.run([(s, at[s]) for s in range(5)],
                [seqs[s][at[s]:at[s] + take[s]] for s in range(5)])
    row = 0
    for s, n in enumerate(take):
      assert rel(got[row:row + n], want[s][at[s]:at[s] + n]) < a.tol
      row += n
      at[s] += n
  # slot 0 again, from position 0, with another sequence
  again = a.sequence(40)
  assert rel(a.run([(0, 0)], [again]), a.oracle(again)) < a.tol


@pytest.mark.parametrize('dt', DTYPES)
def test_another_layers_latents(dt):
  """A reader with sizes and a window of its own over an earlier layer's ring."""
  src = Latent(dt, 4, 32, 32, 40, 72, 30, 2, 60, 200, seed=1)
  ring = torch.full((2, 192, src.rp), 3.0, dtype=dt, device='cuda')
  src = Latent(dt, 4, 32, 32, 40, 72, 30, 2, 60, 200, seed=1, ring=ring)
  reader = Latent(dt, 7, 16, 48, 24, 72, 100, 2, 60, 200, own=False, ring=ring,
                  seed=2)
  x, z = src.sequence(150), reader.sequence(150)
  c = src.latents(x)
  want, swant = reader.oracle(z, c), src.oracle(x)
  at = 0
  for n in (60, 2, 50, 1, 1, 36):
    got = src.run([(1, at)], [x[at:at + n]])
    assert rel(got, swant[at:at + n]) < src.tol
    got = reader.run([(1, at)], [z[at:at + n]])
    assert rel(got, want[at:at + n]) < reader.tol, at
    at += n


def pointed(window, dt, sink=-30.0):
  """A mixer in which latent direction 0 is the one key that queries look for, with
  a value of ones; direction 1 has neither."""
  H, D, Dv, r = 3, 32, 20, 32
  uk, uv, uq = np.zeros((H * D, r)), np.zeros((H * Dv, r)), np.zeros((H * D, r))
  uk[::D, 0] = uq[::D, 0] = 1.0
  uv[:, 0] = r ** -0.5           # (a latent has root mean square 1)
  ones = np.ones(r)
  return Latent(dt, H, D, Dv, r, r, window, 1, 200, 400, scale=1.0, weights={
      'uk': uk, 'uv': uv, 'uq': uq, 'dq.norm': ones, 'dkv.norm': ones,
      'sink': np.full(H, sink)})


@pytest.mark.parametrize('dt,variants', [(torch.float32, (0, 0)),
                                         (torch.bfloat16, (2, 1)),
                                         (torch.bfloat16, (1, 1)),
                                         (torch.bfloat16, (3, 3))])
@pytest.mark.parametrize('window', [5, 64, 100])
def test_a_key_just_inside_and_just_outside_the_window(dt, variants, window):
  """The key at distance window - 1 is found, at distance window it is not: in a
  prompt, across portions, and decoded."""
  a = pointed(window, dt)
  kv = a.a.off_kv
  for dist, seen in ((window - 1, 1.0), (window, 0.0)):
    for i in (window, 127, 128, 191, 229):
      x = torch.zeros((230, a.cols), dtype=dt, device='cuda')
      x[:, 0] = 1.0
      x[:, kv + 1] = 1.0
      x[i - dist, kv:kv + 2] = torch.tensor([1.0, 0.0]).to(dt).cuda()
      whole = a.run([(0, 0)], [x[:200]], variants[0])
      if i >= 200:
        for at in range(200, i, 3):
          a.run([(0, at)], [x[at:min(i, at + 3)]], variants[0])
        got = a.run([(0, i)], [x[i:i + 1]], variants[1])[0]
      else:
        got = whole[i]
      np.testing.assert_allclose(got, seen, atol=5e-3, err_msg=f'{i} {dist}')
      if i < 200:  # the same query decoded alone
        a.run([(0, 0)], [x[:i]], variants[0])
        got = a.run([(0, i)], [x[i:i + 1]], variants[1])[0]
        np.testing.assert_allclose(got, seen, atol=5e-3)


@pytest.mark.parametrize('dt,variant', [(torch.float32, 0), (torch.bfloat16, 1),
                                        (torch.bfloat16, 2), (torch.bfloat16, 3)])
def test_a_sink_shows_and_is_not_scaled(dt, variant):
  """Equal scores of zero: n seen keys share the weight with exp(sink)."""
  window, sink = 50, 1.7
  a = pointed(window, dt, sink=sink)
  x = torch.zeros((90, a.cols), dtype=dt, device='cuda')
  x[:, 1] = 1.0                # queries look for nothing
  x[:, a.a.off_kv] = 64.0      # every key has the value of ones (eps is nothing)
  got = a.run([(0, 0)], [x], variant)
  n = np.minimum(np.arange(90) + 1, window)
  want = n / (n + np.exp(sink))
  np.testing.assert_allclose(got, np.repeat(want[:, None], got.shape[1], 1),
                             rtol=1e-5 if dt == torch.float32 else 5e-3)


@pytest.mark.parametrize('dt', DTYPES)
def test_a_far_key_without_a_window(dt):
  """One key among hundreds, found from every distance."""
  a = pointed(0, dt)
  x = torch.zeros((330, a.cols), dtype=dt, device='cuda')
  x[:, 0] = 1.0
  x[:, a.a.off_kv + 1] = 1.0
  x[2, a.a.off_kv:a.a.off_kv + 2] = torch.tensor([1.0, 0.0]).to(dt).cuda()
  got = np.concatenate([a.run([(0, at)], [x[at:end]]) for at, end in
                        ((0, 200), (200, 202), (202, 329), (329, 330))])
  np.testing.assert_allclose(got[2:], 1.0, atol=5e-3)
  assert abs(got[:2]).max() < 1e-3


def test_a_table_beyond_the_experts_is_refused():
  from t5x_amd import registry
  cfg = cases.CONFIGS['latent']
  params = cases.random_params(cfg)
  params['l0.mlp.table'] = params['l0.mlp.table'] + 1
  with pytest.raises(ValueError, match='experts'):
    registry.module_from_config(cfg, 'float32').decoder_weights(params)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_token_ids_choose_the_experts(dtype):
  """Two tokens with the same embedding and different experts give different
  logits, a third with the first one's experts gives the first one's."""
  from t5x_amd import registry, sequences
  cfg = cases.CONFIGS['latent']
  params = cases.random_params(cfg)
  params['embed'][[5, 6]] = params['embed'][4]
  for i in (0, 2):
    t = params[f'l{i}.mlp.table']
    t[6] = t[4]
    t[5] = (t[4] + 1) % cfg['layers'][i]['mlp']['router']['experts']
  live = sequences.Sequences(registry.module_from_config(cfg, dtype), params, 3, 8)
  got = host(live.step([(t, [3, t], [1]) for t in (4, 5, 6)]))
  np.testing.assert_array_equal(got[0], got[2])
  assert abs(got[0] - got[1]).max() > 0.1
