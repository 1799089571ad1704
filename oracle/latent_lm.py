"""Plain float64 NumPy forward of the decoder-only latent-attention language
models (queries, keys and values through low-rank latents, sliding windows with
sinks, latents shared between layers, hyper-connected residual streams, experts
chosen by a table of token ids), one function per mechanism and no cache:
`forward` runs a whole sequence from its start.  The tests compare the product
with it; nothing here is shared with the product.

`cfg` is the parsed config.json (a dict), `w` a dict of NumPy arrays by tensor
name.
"""

import numpy as np

from oracle.hybrid_lm import rms
from oracle.hybrid_lm import sigmoid


def silu_glu(h, t):
  g = h @ t('gate').T
  return (g * sigmoid(g) * (h @ t('up').T)) @ t('down').T


def clamped_glu(h, limit, t):
  g = np.minimum(h @ t('gate').T, limit)
  u = np.clip(h @ t('up').T, -limit, limit)
  return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t('down').T


def table_experts(h, tokens, m, t):
  """Mean of the experts that the table lists for each token, plus the shared
  expert behind a sigmoid gate of one number per token."""
  table = np.asarray(t('table')).astype(np.int64)
  out = np.zeros_like(h)
  for n, token in enumerate(tokens):
    for e in table[token]:
      out[n] += clamped_glu(h[n], m['expert']['limit'],
                            lambda k, e=e: t(f'e{e}.{k}')) / table.shape[1]
  if m.get('shared'):
    gate = sigmoid(h @ t('shared.sg').T)
    out = out + gate * clamped_glu(h, m['shared']['limit'],
                                   lambda k: t('shared.' + k))
  return out


def latent(h, t, eps):
  """What a layer caches of every position: [T, kv_rank]."""
  return rms(h @ t('dkv').T, eps) * t('dkv.norm')


def sink_window_attention(q, k, v, scale, window, sink):
  """q [T, H, D], k [T, H, D], v [T, H, Dv] -> [T, H, Dv].  Query i weighs the
  keys i - window < j <= i (window None: all j <= i) by exp(scale q.k) over
  their sum plus exp(sink_h)."""
  T, H, _ = q.shape
  out = np.zeros((T, H, v.shape[2]))
  for h in range(H):
    for i in range(T):
      lo = 0 if window is None else max(0, i - window + 1)
      s = k[lo:i + 1, h] @ q[i, h] * scale
      top = max(s.max(), sink[h])
      e = np.exp(s - top)
      out[i, h] = (e @ v[lo:i + 1, h]) / (e.sum() + np.exp(sink[h] - top))
  return out


def latent_attention(h, c, m, t, eps):
  """h: the mixer's input, c: the latents it attends to."""
  T, H, D, Dv = len(h), m['heads'], m['dim'], m['vdim']
  cq = rms(h @ t('dq').T, eps) * t('dq.norm')
  q = (cq @ t('uq').T).reshape(T, H, D)
  k = (c @ t('uk').T).reshape(T, H, D)
  v = (c @ t('uv').T).reshape(T, H, Dv)
  window = (m.get('mask') or {}).get('size')
  o = sink_window_attention(q, k, v, m['scale'], window, t('sink'))
  return o.reshape(T, H * Dv) @ t('o').T


def collect(streams, weights):
  """sum_s weights[s] streams[s], streams [n, T, width]."""
  return np.einsum('s,stw->tw', weights, streams)


def spread(streams, mix, out, y):
  """All streams at once: stream t is sum_s mix[s, t] streams[s] + out[t] y."""
  return np.einsum('st,snw->tnw', mix, streams) + out[:, None, None] * y


def connections(w, n, q):
  """Hyper-connections (in, mix, out) of branch q of the layer named n; without
  any a branch takes the one stream and adds to it."""
  if n + f'hc{q}.in' not in w:
    return np.ones(1), np.eye(1), np.ones(1)
  return tuple(w[n + f'hc{q}.{k}'] for k in ('in', 'mix', 'out'))


def forward(cfg, w, tokens, trace=None):
  """Logits [T, vocab] of one sequence; `trace` (a list) receives the sum of the
  residual streams after every layer."""
  w = {k: np.asarray(v, np.float64) for k, v in w.items()}
  eps, tokens = cfg['norm']['eps'], np.asarray(tokens)
  x = w['embed'][tokens] * cfg['embedding']['scale']
  x = np.repeat(x[None], cfg.get('streams') or 1, axis=0)
  latents = {}
  for i, layer in enumerate(cfg['layers']):
    n, m, mlp = f'l{i}.', layer['mixer'], layer.get('mlp')
    mix = lambda name, n=n: w[n + 'mix.' + name]
    ff = lambda name, n=n: w[n + 'mlp.' + name]
    h_in, h_mix, h_out = connections(w, n, 1)
    h = rms(collect(x, h_in), eps) * w[n + 'norm1']
    src = m.get('kv_from')
    latents[i] = latent(h, mix, eps) if src is None else latents[src]
    y = latent_attention(h, latents[i], m, mix, eps)
    x = spread(x, h_mix, h_out, y)
    if mlp is not None:
      h_in, h_mix, h_out = connections(w, n, 2)
      h = rms(collect(x, h_in), eps) * w[n + 'norm2']
      if mlp['kind'] == 'dense':
        y = silu_glu(h, ff)
      else:
        y = table_experts(h, tokens, mlp, ff)
      x = spread(x, h_mix, h_out, y)
    if trace is not None:
      trace.append(x.sum(axis=0))
  return rms(x.sum(axis=0), eps) * w['final.norm'] @ w['head'].T
