"""Hybrid decoder-only models on the GPU against the plain float64 oracle:
mechanisms alone through the C ABI, then whole models in every way a sequence can
be fed."""

import functools
import io
import json

import numpy as np
import pytest
import torch

from oracle import decoding as odec
from oracle import hybrid_lm as oracle
from tests import hybrid_cases as cases

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
NAMES = {torch.float32: 'float32', torch.bfloat16: 'bfloat16'}


def dev(x, dtype=torch.float32):
  return torch.as_tensor(np.ascontiguousarray(x), device='cuda').to(dtype)


def host(t):
  return t.detach().double().cpu().numpy()


def rel(got, want):
  """Root mean square error over the root mean square of what is wanted."""
  return np.sqrt(np.mean((got - want) ** 2) / np.mean(want ** 2))


# ---- dense layers, embedding, row kernel ------------------------------------------


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('M', [1, 5, 128, 129, 300])
def test_dense_row_strides_and_partial_stores(dt, M):
  from t5x_amd import ops
  rs = np.random.RandomState(M)
  K, N, keep = 96, 208, 201
  wide = dev(rs.randn(M, 160), dt)
  a = wide[:, 64:]
  w = dev(rs.randn(K, N) / np.sqrt(K))
  packed = ops.pack_weight(w, dt)
  want = host(a) @ host(w.to(dt))
  got = ops.dense(a, packed, out_dtype=torch.float32)
  assert rel(host(got), want) < (1e-6 if dt == torch.float32 else 2e-6)
  if dt == torch.bfloat16:
    part = ops.dense(a, packed, out_dtype=torch.float32, n_store=keep)
    np.testing.assert_array_equal(part.cpu().numpy(),
                                  got[:, :keep].cpu().numpy())
    assert rel(host(ops.dense(a, packed)), want) < 4e-3


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('M,K,F', [(3, 64, 40), (128, 96, 72), (200, 64, 136),
                                   (400, 32, 200), (520, 128, 512)])
def test_clamped_glu(dt, M, K, F):
  from t5x_amd import ops
  rs = np.random.RandomState(M)
  limit, alpha = 0.8, 1.702
  a = dev(2 * rs.randn(M, K), dt)
  gate, up = (dev(rs.randn(K, F) / np.sqrt(K)) for _ in range(2))
  got = ops.dense(a, ops.pack_weight(gate, dt, gate_kernel=up),
                  glu=(limit, alpha, 1.0))
  g = np.minimum(host(a) @ host(gate.to(dt)), limit)
  u = np.clip(host(a) @ host(up.to(dt)), -limit, limit)
  want = g * oracle.sigmoid(alpha * g) * (u + 1)
  assert rel(host(got), want) < (1e-6 if dt == torch.float32 else 4e-3)


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('width,ld', [(40, 64), (64, 64), (90, 128), (37, 64)])
def test_embed_sinusoid(dt, width, ld):
  from t5x_amd import ops
  rs = np.random.RandomState(width)
  table = np.zeros((30, ld))
  table[:, :width] = rs.randn(30, width)
  table = dev(table, dt)
  ids = rs.randint(0, 30, 9)
  pos = np.array([0, 1, 2, 63, 64, 999, 4097, 100000, 12])
  got = host(ops.embed_sinusoid(table, dev(ids, torch.int32),
                                dev(pos, torch.int32), width))
  want = host(table)[ids]
  want[:, :width] += oracle.sinusoid(pos, width)
  np.testing.assert_allclose(got, want, atol=1e-6)


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('M,width,ld', [(1, 40, 64), (7, 1100, 1152),
                                        (33, 37, 64), (2, 5000, 5056)])
def test_stream_norm(dt, M, width, ld):
  from t5x_amd import ops
  rs = np.random.RandomState(M + width)
  eps = 1e-5

  def stream():
    x = np.zeros((M, ld))
    x[:, :width] = 3 * rs.randn(M, width)
    return x

  x, x0 = dev(stream()), dev(stream())
  y = dev(stream(), dt)
  wy, add, w = (dev(rs.randn(width)) for _ in range(3))
  before = host(x)[:, :width]
  out = ops.stream_norm(x, width, dt, y=y, y_norm=wy, add=add, norm=w, eps=eps)
  want = before + oracle.rms(host(y)[:, :width], eps) * host(wy) + host(add)
  np.testing.assert_allclose(host(x)[:, :width], want, rtol=2e-6, atol=2e-6)
  tol = 1e-6 if dt == torch.float32 else 4e-3
  assert rel(host(out)[:, :width], oracle.rms(want, eps) * host(w)) < tol
  assert not host(x)[:, width:].any() and not host(out)[:, width:].any()
  cat = ops.stream_norm(x, width, dt, x0=x0)
  assert rel(host(cat)[:, :ld], host(x)) < tol
  assert rel(host(cat)[:, ld:], host(x0)) < tol
  rows = dev(rs.permutation(M)[:(M + 1) // 2], torch.int32)
  picked = ops.stream_norm(x, width, dt, norm=w, rows=rows, eps=eps)
  assert rel(host(picked)[:, :width],
             (oracle.rms(want, eps) * host(w))[rows.cpu().numpy()]) < tol
  before = host(x)
  assert ops.stream_norm(x, width, dt, y=y) is None
  np.testing.assert_allclose(host(x), before + host(y), rtol=2e-6, atol=1e-5)


# ---- windowed attention ---------------------------------------------------------------


class Ragged:
  """t5d_ragged of portions [(slot, start, length)]."""

  def __init__(self, portions):
    from t5x_amd import hybrid
    self.p = hybrid.Portions([(s, at, np.zeros(n, np.int32))
                              for s, at, n in portions], [], 'cuda')
    self.ragged = self.p.ragged


class Attention:
  """An attention mixer's kernels over sequences of random projections."""

  def __init__(self, dt, H, G, D, Dv, window, slots, portion, max_len, seed=0,
               scale=0.3, eps=1e-5, bias=True, sink=True, norms=True):
    from t5x_amd import _lib
    self.dt, self.dims = dt, (H, G, D, Dv)
    self.window, self.scale, self.eps = window, scale, eps
    rs = self.rs = np.random.RandomState(seed)
    # the columns before and between the three blocks are not theirs
    self.off = (16, 16 + H * D + 5, 16 + H * D + 5 + G * D + 3)
    self.cols = self.off[2] + G * Dv + 7
    self.qn, self.kn = (dev(1 + 0.3 * rs.randn(D)) if norms else None
                        for _ in range(2))
    self.sink = dev(rs.randn(H)) if sink else None
    slopes = [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]
    self.slopes = dev(np.array(slopes)) if bias else None
    hp = _lib.load().t5d_window_head_pad(D, Dv)
    ring = (window - 1 + portion if window else max_len)
    ring = (ring + 63) // 64 * 64
    self.rings = [torch.full((slots, G, ring, hp), 7.0, dtype=dt, device='cuda')
                  for _ in range(2)]
    a = self.a = _lib.WindowAttention()
    a.dtype = _lib.dtype_code(dt)
    a.H, a.G, a.D, a.Dv, a.ring, a.window = H, G, D, Dv, ring, window
    a.scale, a.eps, a.ld_proj = scale, eps, self.cols
    a.off_q, a.off_k, a.off_v = self.off
    P = _lib.ptr
    a.q_norm, a.k_norm, a.slopes, a.sink = (P(self.qn), P(self.kn),
                                            P(self.slopes), P(self.sink))
    a.key_ring, a.value_ring = P(self.rings[0]), P(self.rings[1])
    self.hp = hp

  def sequence(self, T):
    """Random projections [T, cols] of one sequence."""
    return dev(self.rs.randn(T, self.cols), self.dt)

  def run(self, portions, proj, variant=0):
    """portions [(slot, start, rows of proj)] -> [M, H * Dv]."""
    from t5x_amd import _lib, ops
    H, G, D, Dv = self.dims
    x = torch.cat(proj).contiguous()
    r = Ragged([(s, at, len(p)) for (s, at), p in zip(portions, proj)])
    M, S = len(x), len(proj)
    ld = (H * Dv + 3) // 4 * 4 + 4
    out = torch.full((M, ld), 3.0, dtype=self.dt, device='cuda')
    q = torch.empty((M, H, self.hp), dtype=self.dt, device='cuda')
    ws = torch.empty((_lib.load().t5d_window_workspace_bytes(S, H, D, Dv),),
                     dtype=torch.uint8, device='cuda')
    a = self.a
    a.proj, a.q_rows, a.out, a.ld_out = (x.data_ptr(), q.data_ptr(),
                                         out.data_ptr(), ld)
    a.workspace = ws.data_ptr()
    ops.window_attention(a, r.ragged, variant)
    got = host(out)
    assert (got[:, H * Dv:] == 3.0).all()
    return got[:, :H * Dv]

  def oracle(self, proj):
    H, G, D, Dv = self.dims
    x, T = host(proj), len(proj)
    cut = lambda at, n, d: x[:, at:at + n * d].reshape(T, n, d)
    q, k, v = (cut(self.off[0], H, D), cut(self.off[1], G, D),
               cut(self.off[2], G, Dv))
    if self.qn is not None:
      q = oracle.rms(q, self.eps) * host(self.qn)
      k = oracle.rms(k, self.eps) * host(self.kn)
    if self.dt == torch.bfloat16:  # as the cache and the products hold them
      q, k = cases.bf16(q).astype(float), cases.bf16(k).astype(float)
    out = np.zeros((T, H, Dv))
    slopes = None if self.slopes is None else host(self.slopes)
    for h in range(H):
      g = h // (H // G)
      for i in range(T):
        lo = max(0, i - self.window + 1) if self.window else 0
        s = self.scale * k[lo:i + 1, g] @ q[i, h]
        if slopes is not None:
          s = s - slopes[h] * (i - np.arange(lo, i + 1))
        e = np.exp(s - s.max())
        den = e.sum()
        if self.sink is not None:
          den += np.exp(float(self.sink[h]) - s.max())
        out[i, h] = e @ v[lo:i + 1, g] / den
    return out.reshape(T, H * Dv)

  @property
  def tol(self):
    return 2e-6 if self.dt == torch.float32 else 6e-3


SHAPES = [(6, 3, 48, 48), (3, 1, 20, 70), (8, 8, 64, 64), (2, 1, 100, 128),
          (16, 1, 32, 24), (6, 2, 200, 36), (5, 5, 16, 10), (20, 1, 40, 40)]
WAVE_SHAPES = SHAPES + [(2, 1, 300, 40), (1, 1, 24, 520)]


@pytest.mark.parametrize('dt,variant,H,G,D,Dv', [
    (dt, v, *shape) for dt, v, shapes in (
        (torch.float32, 0, WAVE_SHAPES), (torch.bfloat16, 2, SHAPES),
        (torch.bfloat16, 3, WAVE_SHAPES)) for shape in shapes])
@pytest.mark.parametrize('window', [0, 1, 9, 64, 65])
def test_window_attention_prompts_and_portions(dt, variant, H, G, D, Dv, window):
  T, portion = 150, 70
  a = Attention(dt, H, G, D, Dv, window, 3, portion, T, seed=H + D + window)
  x = a.sequence(T)
  want = a.oracle(x)
  for cuts in ([70, 140], [1, 3, 60, 64, 66, 128]):
    got, at = [], 0
    for end in cuts + [T]:
      got.append(a.run([(2, at)], [x[at:end]], variant))
      at = end
    assert rel(np.concatenate(got), want) < a.tol, cuts


@pytest.mark.parametrize('H,G,D,Dv', SHAPES[:-1])  # up to 16 heads per group
@pytest.mark.parametrize('window', [0, 1, 9, 64, 65, 600])
def test_window_attention_step_kernel(H, G, D, Dv, window):
  """One token per sequence for sequences of unequal lengths, ring wrapping."""
  T = 190
  a = Attention(torch.bfloat16, H, G, D, Dv, window, 4, 8, T + 8,
                seed=H + D + window)
  starts = [0, 3, 61, 130]
  seqs = [a.sequence(T) for _ in starts]
  for slot, (n, x) in enumerate(zip(starts, seqs)):
    for at in range(0, n, 8):
      a.run([(slot, at)], [x[at:min(n, at + 8)]])
  wants = [a.oracle(x) for x in seqs]
  order = [2, 0, 3, 1]
  for step in range(40):
    got = a.run([(s, starts[s] + step) for s in order],
                [seqs[s][starts[s] + step:starts[s] + step + 1] for s in order],
                variant=1)
    for row, s in zip(got, order):
      assert rel(row, wants[s][starts[s] + step]) < 1e-2, (step, s)


@pytest.mark.parametrize('bias,sink,norms', [(False, True, True),
                                             (True, False, True),
                                             (True, True, False)])
@pytest.mark.parametrize('dt', DTYPES)
def test_window_attention_without_optional_parts(dt, bias, sink, norms):
  a = Attention(dt, 4, 2, 40, 24, 12, 1, 40, 40, bias=bias, sink=sink,
                norms=norms)
  x = a.sequence(41)
  want = a.oracle(x)
  assert rel(a.run([(0, 0)], [x[:40]]), want[:40]) < a.tol
  assert rel(a.run([(0, 40)], [x[40:]]), want[40:]) < 1e-2


@pytest.mark.parametrize('dt,variants', [(torch.float32, (0, 0)),
                                         (torch.bfloat16, (2, 1)),
                                         (torch.bfloat16, (3, 3))])
@pytest.mark.parametrize('window', [5, 64, 100])
def test_a_key_just_inside_and_just_outside_the_window(dt, variants, window):
  """Key j alone matches query i (score far above all others), and only its
  value is not zero: the output is that value at distance window - 1 and zero at
  distance window — in a prompt, across portions, and decoded."""
  H, G, D, Dv, T = 2, 1, 32, 32, 230
  a = Attention(dt, H, G, D, Dv, window, 1, 200, T, scale=20.0, bias=False,
                sink=False, norms=False)
  for dist, seen in ((window - 1, 1.0), (window, 0.0)):
    for i in (window, 127, 128, 191, 229):
      j = i - dist
      x = torch.zeros((T, a.cols), dtype=dt, device='cuda')
      x[:, a.off[1] + 1] = 1.0                       # every key: direction 1
      x[j, a.off[1]:a.off[1] + 2] = torch.tensor([1.0, 0.0]).to(dt).cuda()
      x[i, a.off[0]:a.off[0] + H * D:D] = 1.0        # query i: direction 0
      x[j, a.off[2]:a.off[2] + Dv] = 1.0
      whole = a.run([(0, 0)], [x[:200]], variants[0])
      if i >= 200:
        for at in range(200, i):
          a.run([(0, at)], [x[at:at + 1]], variants[1])
        got = a.run([(0, i)], [x[i:i + 1]], variants[1])[0]
      else:
        got = whole[i]
      np.testing.assert_allclose(got, seen, atol=1e-3, err_msg=f'{i} {dist}')
      if i < 200:  # the same query decoded alone
        a.run([(0, 0)], [x[:i]], variants[0])
        got = a.run([(0, i)], [x[i:i + 1]], variants[1])[0]
        np.testing.assert_allclose(got, seen, atol=1e-3)


@pytest.mark.parametrize('dt', DTYPES)
def test_a_sink_and_the_distance_bias_show(dt):
  """Equal scores: the weights are those of the bias and the sink alone."""
  H, D = 4, 16
  a = Attention(dt, H, 2, D, D, 0, 1, 70, 70)
  x = torch.zeros((70, a.cols), dtype=dt, device='cuda')
  x[:, a.off[2]:a.off[2] + 2 * D] = 1.0
  got = a.run([(0, 0)], [x])
  i = np.arange(70)
  for h in range(H):
    slope, sink = 2.0 ** (-2.0 * (h + 1)), float(a.sink[h])
    mass = np.cumsum(np.exp(-slope * i))
    np.testing.assert_allclose(got[:, h * D], mass / (mass + np.exp(sink)),
                               rtol=1e-5 if dt == torch.float32 else 5e-3)


@pytest.mark.parametrize('dt', DTYPES)
def test_window_attention_batches_match_each_alone(dt):
  a = Attention(dt, 6, 2, 24, 40, 20, 5, 130, 400)
  lens = [130, 1, 2, 65, 64]
  seqs = [a.sequence(300) for _ in lens]
  at = [0] * 5
  for _ in range(2):
    got = a.run([(s, at[s]) for s in range(5)],
                [seqs[s][at[s]:at[s] + lens[s]] for s in range(5)])
    row = 0
    for s in range(5):
      want = a.oracle(seqs[s][:at[s] + lens[s]])[at[s]:]
      assert rel(got[row:row + lens[s]], want) < (a.tol if lens[s] > 2 else 1e-2)
      row += lens[s]
      at[s] += lens[s]


# ---- recurrences ----------------------------------------------------------------------


class Recurrence:
  """A recurrent mixer's kernels over sequences of random projections."""

  def __init__(self, dt, delta, H, G, D, Dv, taps, slots, seed=0, strong=False):
    from t5x_amd import _lib
    self.dt, self.delta, self.taps = dt, delta, taps
    self.dims = (H, G, D, Dv)
    rs = self.rs = np.random.RandomState(seed)
    sizes = [G * D, G * D, H * Dv, H, H * Dv]      # q, k, v, beta, gate
    self.off, n = [], 8
    for s in sizes:
      self.off.append(n)
      n += s + 3
    self.cols = n
    self.low_off = (4, 4 + H * D + 4)
    self.low_cols = self.low_off[1] + H * Dv + 4
    C = 2 * G * D + H * Dv
    self.bias = dev((-4.0 if strong else 2.0) + 2 * rs.randn(H * D) if not delta
                    else (1.0 if strong else -3.0) + 2 * rs.randn(H * D))
    self.A = dev((2.0 if strong else 0.0) + rs.randn(H))
    self.conv = dev(rs.randn(C, taps)) if taps else None
    self.norm = dev(1 + 0.3 * rs.randn(Dv))
    # what another sequence may have left behind
    self.state = torch.full((slots, H, D, Dv), float('nan'), device='cuda')
    self.ring = torch.full((slots, max(1, taps), C), float('nan'), dtype=dt,
                           device='cuda')
    r = self.r = _lib.Recurrence()
    P = _lib.ptr
    r.dtype = _lib.dtype_code(dt)
    r.H, r.G, r.D, r.Dv, r.taps = H, G, D, Dv, taps
    r.delta = r.unit = r.decay = r.gate = int(delta)
    self.tau, self.eps = 6.0, 1e-5
    r.q_scale, r.decay_power, r.unit_eps, r.eps = (D ** -0.5, 1 / self.tau, 1e-6,
                                                   self.eps)
    r.ld_proj, r.ld_low = self.cols, self.low_cols
    r.off_q, r.off_k, r.off_v, r.off_beta, r.off_gate = self.off
    r.off_z, r.off_low_gate = self.low_off
    r.decay_bias, r.A_log, r.conv, r.norm = (P(self.bias), P(self.A),
                                             P(self.conv), P(self.norm))
    r.conv_ring, r.state = P(self.ring), P(self.state)

  def sequence(self, T):
    return (dev(self.rs.randn(T, self.cols), self.dt),
            dev(2 * self.rs.randn(T, self.low_cols)))

  def run(self, portions, seqs, variant=0):
    """portions [(slot, start, end)] of seqs -> [M, H * Dv]."""
    from t5x_amd import _lib, ops
    H, G, D, Dv = self.dims
    proj = torch.cat([p[a:b] for (_, a, b), (p, _) in zip(portions, seqs)])
    low = torch.cat([z[a:b] for (_, a, b), (_, z) in zip(portions, seqs)])
    x = Ragged([(s, a, b - a) for s, a, b in portions])
    M = len(proj)
    out = torch.full((M, H * Dv + 6), 3.0, dtype=self.dt, device='cuda')
    ws = torch.empty(
        (_lib.load().t5d_recurrence_workspace_bytes(
            M, len(portions), H, G, D, Dv),), dtype=torch.uint8, device='cuda')
    r = self.r
    r.proj, r.low, r.out, r.ld_out = (proj.data_ptr(), low.data_ptr(),
                                      out.data_ptr(), H * Dv + 6)
    r.workspace, r.workspace_bytes = ws.data_ptr(), ws.numel()
    ops.recurrence(r, x.ragged, variant)
    got = host(out)
    assert (got[:, H * Dv:] == 3.0).all()
    return got[:, :H * Dv]

  def oracle(self, seq):
    H, G, D, Dv = self.dims
    x, z, T = host(seq[0]), host(seq[1]), len(seq[0])
    q, k, v = (x[:, o:o + n] for o, n in zip(self.off, (G * D, G * D, H * Dv)))
    if self.taps:
      w = host(self.conv)
      q, k, v = (oracle.silu(oracle.causal_conv(y, t)) for y, t in (
          (q, w[:G * D]), (k, w[G * D:2 * G * D]), (v, w[2 * G * D:])))
    q, k, v = (q.reshape(T, G, D), k.reshape(T, G, D), v.reshape(T, H, Dv))
    z = (z[:, self.low_off[0]:self.low_off[0] + H * D] + host(self.bias)
         ).reshape(T, H, D)
    if self.delta:
      q, k = oracle.unit(q), oracle.unit(k)
    q = np.repeat(q * D ** -0.5, H // G, axis=1)
    k = np.repeat(k, H // G, axis=1)
    if self.delta:
      g = np.exp(-np.exp(host(self.A))[None, :, None] * oracle.softplus(z))
      beta = oracle.sigmoid(x[:, self.off[3]:self.off[3] + H])
      o = oracle.delta_rule(q, k, v, g, beta)
      gate = oracle.sigmoid(
          seq_cols(host(seq[1]), self.low_off[1], H * Dv))
    else:
      alpha = oracle.sigmoid(z) ** (1 / self.tau)
      o = oracle.gated_linear_attention(q, k, v, alpha)
      gate = oracle.silu(seq_cols(x, self.off[4], H * Dv))
    return (oracle.rms(o, self.eps) * host(self.norm)).reshape(T, H * Dv) * gate

  @property
  def tol(self):
    return 1e-5 if self.dt == torch.float32 else 4e-3


def seq_cols(x, at, n):
  return x[:, at:at + n]


REC = [(True, 2, 2, 64, 64, 4), (True, 6, 2, 24, 40, 4), (True, 2, 1, 130, 20, 5),
       (True, 2, 2, 200, 256, 2), (True, 3, 1, 8, 6, 1), (True, 1, 1, 40, 33, 0),
       (True, 2, 1, 300, 24, 3), (True, 1, 1, 16, 260, 9),
       (False, 5, 5, 32, 32, 0), (False, 3, 3, 20, 36, 0),
       (False, 2, 2, 256, 100, 0), (False, 5, 5, 72, 10, 0)]


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('strong', [False, True])
@pytest.mark.parametrize('delta,H,G,D,Dv,taps', REC)
def test_recurrence_portions_and_steps(dt, strong, delta, H, G, D, Dv, taps):
  """Whole, in portions down to one token, and token by token on both paths, in
  slots that hold garbage."""
  T = 83
  r = Recurrence(dt, delta, H, G, D, Dv, taps, 2, seed=D + Dv, strong=strong)
  seq = r.sequence(T)
  want = r.oracle(seq)
  assert rel(r.run([(1, 0, T)], [seq]), want) < r.tol
  for variant in (2, 3) if taps <= 8 else (2,):  # token by token, in chunks
    assert rel(r.run([(1, 0, T)], [seq], variant), want) < r.tol, variant
    for cuts in ([1, 2, 3, 5, 8, 24, 25, 41, 57], [16, 32, 64], [2, 4, 6, 70]):
      got, at = [], 0
      for end in cuts + [T]:
        got.append(r.run([(0, at, end)], [seq], variant))
        at = end
      assert rel(np.concatenate(got), want) < r.tol, (variant, cuts)
  got = [r.run([(1, 0, 40)], [seq])]
  got += [r.run([(1, t, t + 1)], [seq]) for t in range(40, T)]
  assert rel(np.concatenate(got), want) < r.tol
  got = [r.run([(0, t, t + 1)], [seq]) for t in range(20)]
  assert rel(np.concatenate(got), want[:20]) < r.tol


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('delta', [True, False])
def test_recurrence_batches_match_each_alone(dt, delta):
  r = Recurrence(dt, delta, 4, 2 if delta else 4, 48, 32, 3 if delta else 0, 6)
  lens = [40, 1, 17, 2, 64]
  slots = [3, 0, 5, 1, 4]
  seqs = [r.sequence(100) for _ in lens]
  wants = [r.oracle(s) for s in seqs]
  at = [0] * 5
  for step in range(4):
    n = lens if step == 0 else [1] * 5 if step > 1 else [3, 2, 1, 9, 20]
    got = r.run([(slots[i], at[i], at[i] + n[i]) for i in range(5)], seqs)
    row = 0
    for i in range(5):
      assert rel(got[row:row + n[i]], wants[i][at[i]:at[i] + n[i]]) < 2 * r.tol
      row += n[i]
      at[i] += n[i]


@pytest.mark.parametrize('dt', DTYPES)
@pytest.mark.parametrize('delta', [True, False])
def test_a_memory_from_far_back_survives(dt, delta):
  """Channel 0 of the first key never decays and nothing else uses it: its value
  is read back after hundreds of tokens and several portions."""
  H, D, Dv, T = 1, 32, 16, 400
  r = Recurrence(dt, delta, H, H, D, Dv, 0, 1)
  bias = np.zeros(D)
  bias[0] = -40.0 if delta else 60.0     # decay 1
  r.bias.copy_(dev(bias))
  proj = torch.zeros((T, r.cols), dtype=dt, device='cuda')
  low = torch.zeros((T, r.low_cols), device='cuda')
  oq, ok, ov, ob, og = r.off
  proj[:, ok + 1] = 1.0
  proj[0, ok:ok + 2] = torch.tensor([1.0, 0.0]).to(dt).cuda()
  proj[0, ov:ov + Dv] = dev(1.0 + np.arange(Dv), dt)
  proj[:, ob] = 9.0
  proj[:, og:og + Dv] = 1.0
  proj[T - 1, oq] = 1.0
  seq = (proj, low)
  want = r.oracle(seq)[-1]
  assert np.abs(want).max() > 0.1
  for cuts in ([], [1, 100, 164, 399], [63, 64, 65, 300]):
    at = 0
    for end in cuts + [T]:
      got = r.run([(0, at, end)], [seq])
      at = end
    np.testing.assert_allclose(got[-1], want, rtol=1e-2, atol=1e-4)


# ---- whole models -----------------------------------------------------------------------


def build(name, dtype, seed=0, **attrs):
  from t5x_amd import models, registry
  cfg = cases.CONFIGS[name]
  module = registry.module_from_config(cfg, dtype)
  for k, v in attrs.items():
    setattr(module, k, v)
  return cfg, cases.random_params(cfg, seed), module


def err(got, want):
  """Error of logits rows, their means taken off, over the logits' size."""
  d = got - want
  d = d - d.mean(-1, keepdims=True)
  w = want - want.mean(-1, keepdims=True)
  return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean())


def close(got, want, dtype):
  """Logits as near as rounding allows.  In bfloat16 a read-out that happens to
  be nearly zero is all rounding once its head is normed, so a few positions are
  far off; a wrong key, tap or state shows in most of them."""
  e = err(got, want)
  if dtype == 'float32':
    return e.max() < 1e-4
  return (np.median(e) < 2e-2 and np.mean(e > 6e-2) <= max(0.03, 1 / len(e)) and
          e.max() < 0.4)


def feed(live, name, tokens, cuts):
  """All logits of a request fed in the given pieces."""
  out, at = [], 0
  for end in list(cuts) + [len(tokens)]:
    if end > at:
      out.append(host(live.step([(name, tokens[at:end],
                                  list(range(end - at)))])))
      at = end
  live.end(name)
  return np.concatenate(out)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', sorted(cases.CONFIGS))
def test_logits_whole_in_portions_and_token_by_token(name, dtype):
  from t5x_amd import sequences
  cfg, params, module = build(name, dtype)
  rs = np.random.RandomState(5)
  tokens = rs.randint(0, cfg['vocab'], 150).tolist()
  want = cases.forward(cfg, params, tokens)
  live = sequences.Sequences(module, params, 2, 200)
  whole = feed(live, 'a', tokens, [])
  assert close(whole, want, dtype)
  for cuts in ([2, 4, 6, 9, 64, 66, 128], [65, 130, 132],
               [100] + list(range(101, 150)), range(1, 40)):
    got = feed(live, str(cuts), tokens, cuts)
    assert close(got, want, dtype), cuts
    assert close(got, whole, dtype), cuts


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', ['all', 'latent', 'latent_plain'])
def test_residual_stream_after_every_layer_run(name, dtype):
  from t5x_amd import sequences
  cfg, params, module = build(name, dtype)
  tokens = np.random.RandomState(6).randint(0, cfg['vocab'], 20).tolist()
  want, got = [], []
  cases.forward(cfg, params, tokens, want)
  live = sequences.Sequences(module, params, 1, 32)
  live.step([('a', tokens, [])], trace=got)
  assert got[0].shape == (len(want), 20, cfg['width'])
  for r, w in enumerate(want):
    assert rel(host(got[0][r]), w) < (2e-6 if dtype == 'float32' else 2e-2), r


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', ['all', 'all_looped', 'odd_values'] + cases.LATENT)
def test_small_rings_wrap_in_long_requests(name, dtype):
  """Rings as small as the windows allow, reused slots, a request far longer than
  every ring."""
  from t5x_amd import sequences
  cfg, params, module = build(name, dtype, max_portion=5)
  rs = np.random.RandomState(7)
  live = sequences.Sequences(module, params, 1, 700)
  for n, cuts in ((700, [300, 302, 304]), (31, [30]), (260, range(60, 260))):
    tokens = rs.randint(0, cfg['vocab'], n).tolist()
    want = cases.forward(cfg, params, tokens)
    assert close(feed(live, n, tokens, cuts), want, dtype), n


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', ['all', 'latent', 'latent_one_stream'])
def test_mixed_batches_match_each_alone(name, dtype):
  """Prompts, portions and single tokens of unequal requests in one step, slots
  given back and taken again in between."""
  from t5x_amd import sequences
  cfg, params, module = build(name, dtype, max_tokens=90)
  rs = np.random.RandomState(8)
  live = sequences.Sequences(module, params, 3, 128)
  req = {n: rs.randint(0, cfg['vocab'], l).tolist() for n, l in
         (('a', 100), ('b', 41), ('c', 1), ('d', 77), ('e', 23))}
  want = {n: cases.forward(cfg, params, t) for n, t in req.items()}
  at = dict.fromkeys(req, 0)
  plan = [{'a': 60, 'b': 1, 'c': 1}, {'a': 1, 'b': 2, 'd': 70}, {'d': 7, 'b': 37},
          {'b': 1, 'a': 2}, {'e': 20, 'a': 30}, {'e': 1, 'a': 1}, {'a': 6, 'e': 2}]
  for step in plan:
    entries = [(n, req[n][at[n]:at[n] + k], list(range(k)))
               for n, k in step.items()]
    got = host(live.step(entries))
    row = 0
    for n, k in step.items():
      assert close(got[row:row + k], want[n][at[n]:at[n] + k], dtype), (n, at[n])
      row += k
      at[n] += k
      if at[n] == len(req[n]):
        live.end(n)
  assert len(live) == 0


def test_wanted_places_come_in_the_order_asked_for():
  from t5x_amd import sequences
  cfg, params, module = build('one_kind', 'float32', max_tokens=8)
  tokens = list(range(20))
  live = sequences.Sequences(module, params, 2, 32)
  got = host(live.step([('a', tokens, [19, 0, 7, 7]), ('b', tokens[:3], [1])]))
  want = cases.forward(cfg, params, tokens)
  assert err(got, want[[19, 0, 7, 7, 1]]).max() < 2e-5


# ---- generation through the model object -------------------------------------------------


def greedy(cfg, params, prompt, n):
  tokens = list(prompt)
  for _ in range(n):
    tokens.append(int(np.argmax(cases.forward(cfg, params, tokens)[-1])))
  return tokens[len(prompt):]


def model_for(name, dtype='float32', eos=-1, **kw):
  from t5x_amd import decoding, models
  cfg, params, module = build(name, dtype)
  fn = functools.partial(decoding.temperature_sample, temperature=0.0, topk=0)
  return cfg, params, models.DecoderOnlyModel(
      module, models.Vocabulary(eos), decode_fn=kw.pop('decode_fn', fn))


@pytest.mark.parametrize('name', ['all', 'no_loop'] + cases.LATENT)
def test_greedy_generation_equals_the_oracle(name):
  """Unequal prompts in batches, several in flight, float32: exact tokens."""
  cfg, params, model = model_for(name)
  rs = np.random.RandomState(9)
  prompts = [rs.randint(1, cfg['vocab'], n).tolist() for n in (5, 1, 30, 12, 2)]
  want = [greedy(cfg, params, p, 12) for p in prompts]
  got = list(model.generate(params, prompts, 12, batch_size=2))
  assert got == want
  # the same contexts again, one batch at a time
  assert list(model.generate(params, prompts[:2], 12, batch_size=2)) == want[:2]


def test_the_host_loop_over_a_dataset():
  """get_infer_fn pads the last batch, keeps several decoding, restores order."""
  from t5x_amd import infer
  cfg, params, model = model_for('all')
  rs = np.random.RandomState(13)
  L, n = 16, [4, 7, 1, 9, 2]
  tokens = rs.randint(1, cfg['vocab'], (5, L)).astype(np.int32)
  mask = (np.arange(L)[None, :] < np.array(n)[:, None]).astype(np.int32)
  ds = [(i, {'decoder_input_tokens': tokens[i],
             'decoder_causal_attention': mask[i]}) for i in range(5)]
  out = infer.get_infer_fn(model.predict_batch, batch_size=2)(ds, params)
  assert [i for i, _ in out] == list(range(5))
  for i, row in out:
    want = tokens[i, 1:n[i]].tolist() + greedy(cfg, params, tokens[i, :n[i]],
                                               L - n[i])
    assert row[:L - 1] == want


def test_generation_stops_at_the_end_token():
  cfg, params, model = model_for('all')
  prompt = [3, 1, 4, 1, 5]
  plain = list(model.generate(params, [prompt], 14))[0]
  eos = plain[6]
  _, _, stopping = model_for('all', eos=eos)
  cut = plain[:plain.index(eos) + 1]
  assert list(stopping.generate(params, [prompt], 14))[0] == cut


@pytest.mark.parametrize('name', ['all', 'latent'])
def test_replayed_graph_equals_the_step_by_step_loop(name):
  """The captured loop against the loop that calls the step function every
  iteration (a state callback keeps it off the graph), bit for bit, twice."""
  from t5x_amd import decoding, models
  for dtype in ('float32', 'bfloat16'):
    cfg, params, model = model_for(name, dtype)
    rs = np.random.RandomState(10)
    L, lens = 40, [7, 20, 1]
    batch = {'decoder_input_tokens': rs.randint(1, cfg['vocab'], (3, L)),
             'decoder_causal_attention': (np.arange(L)[None, :] <
                                          np.array(lens)[:, None]).astype(int)}
    slow = models.DecoderOnlyModel(
        model.module, models.Vocabulary(-1),
        decode_fn=functools.partial(decoding.temperature_sample,
                                    temperature=0.7, topk=5,
                                    state_callback_fn=lambda s: s))
    fast = models.DecoderOnlyModel(
        model.module, models.Vocabulary(-1),
        decode_fn=functools.partial(decoding.temperature_sample,
                                    temperature=0.7, topk=5))
    want, aux = slow.predict_batch_with_aux(params, batch, rng=3, num_decodes=2,
                                            return_all_decodes=True)
    for _ in range(2):
      got, gaux = fast.predict_batch_with_aux(params, batch, rng=3,
                                              num_decodes=2,
                                              return_all_decodes=True)
      np.testing.assert_array_equal(got.cpu().numpy(), want.cpu().numpy())
      np.testing.assert_array_equal(gaux['scores'].cpu().numpy(),
                                    aux['scores'].cpu().numpy())
    for r, n in enumerate(lens):
      np.testing.assert_array_equal(
          got[r, :, :n - 1].cpu().numpy(),
          np.broadcast_to(batch['decoder_input_tokens'][r, 1:n], (2, n - 1)))


@pytest.mark.parametrize('name', ['no_loop', 'latent'])
def test_beam_search_equals_the_oracle(name):
  from t5x_amd import decoding
  cfg, params, model = model_for(name, eos=1,
                                 decode_fn=decoding.beam_search)
  rs = np.random.RandomState(11)
  B, K, L, lens = 2, 3, 12, np.array([6, 3])
  tokens = rs.randint(2, cfg['vocab'], (B, L)).astype(np.int32)
  mask = (np.arange(L)[None, :] < lens[:, None]).astype(np.int32)
  got, aux = model.predict_batch_with_aux(
      params, {'decoder_input_tokens': tokens, 'decoder_causal_attention': mask},
      num_decodes=K, return_all_decodes=True)

  room = 2 * L + 4
  history = np.zeros((B, 1, room), np.int32)
  history[:, 0, :L] = tokens * mask

  def step(state):
    h = state.cache['history'].copy()
    at = state.cache['cache_index'].reshape(-1)
    logits = np.zeros((len(h), cfg['vocab']), np.float32)
    for r in range(len(h)):
      h[r, 0, at[r]] = state.cur_token[r, 0]
      logits[r] = cases.forward(cfg, params, h[r, 0, :at[r] + 1])[-1]
    return logits, {'history': h,
                    'cache_index': state.cache['cache_index'] + 1}

  want, scores = odec.beam_search(
      tokens * mask, {'history': history, 'cache_index': lens - 1}, step,
      eos_id=1, num_decodes=K, initial_index=lens - 1)
  np.testing.assert_array_equal(got.cpu().numpy(), want)
  np.testing.assert_allclose(aux['scores'].cpu().numpy(), scores, atol=1e-3)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', ['all', 'latent'])
def test_saved_model_through_the_commands(tmp_path, monkeypatch, capsys, name,
                                          dtype):
  from t5x_amd import generate, trace_replay
  cfg = cases.CONFIGS[name]
  params = cases.random_params(cfg, seed=3)
  cases.save_model(tmp_path, cfg, params)
  tokens = np.random.RandomState(12).randint(0, cfg['vocab'], 30).tolist()
  want = cases.forward(cfg, params, tokens)
  steps = [{'step': 0, 'entries': [{'id': 'a', 'tokens': tokens[:21],
                                    'want': [0, 20]}], 'end': []},
           {'step': 1, 'entries': [{'id': 'a', 'tokens': tokens[21:22],
                                    'want': []}], 'end': []},
           {'step': 2, 'entries': [{'id': 'a', 'tokens': tokens[22:],
                                    'want': [7]}], 'end': ['a']},
           {'step': 3, 'entries': [{'id': 'b', 'tokens': tokens[:2],
                                    'want': [1]}], 'end': ['b']}]
  monkeypatch.setattr('sys.stdin',
                      io.StringIO('\n'.join(json.dumps(s) for s in steps)))
  out = tmp_path / 'out'
  assert trace_replay.main(['--model', str(tmp_path), '--dtype', dtype, '--out',
                            str(out), '--max-tokens', '32', '--slots',
                            '1']) == 0
  assert capsys.readouterr().out.split('\n')[:4] == [
      f'done {n}' for n in range(4)]
  read = lambda n: np.fromfile(out / f'{n}.f32', '<f4').reshape(-1, cfg['vocab'])
  assert not (out / '1.f32').exists()
  for n, places in ((0, [0, 20]), (2, [29]), (3, [1])):
    assert close(read(n), want[places], dtype)
  if dtype == 'float32':
    monkeypatch.setattr('sys.stdin', io.StringIO(
        f'{json.dumps(tokens[:5])}\n{json.dumps(tokens[:9])}\n'))
    assert generate.main(['--model', str(tmp_path), '--dtype', dtype,
                          '--tokens', '6', '--eos', '-1']) == 0
    lines = [json.loads(x) for x in capsys.readouterr().out.split('\n') if x]
    assert lines == [greedy(cfg, params, tokens[:n], 6) for n in (5, 9)]
