"""Plain float64 NumPy forward of the decoder-only hybrid language models
(gated linear attention, delta-rule recurrences with a decay per key channel,
sliding-window softmax attention with distance bias and sinks), one function
per mechanism and no cache: `forward` runs a whole sequence from its start.
The tests compare the product with it; nothing here is shared with the product.

`cfg` is the parsed config.json (a dict), `w` a dict of NumPy arrays by tensor
name.
"""

import numpy as np


def rms(x, eps):
  """x over its root mean square along the last axis."""
  return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def sigmoid(z):
  return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z)))


def silu(z):
  return z * sigmoid(z)


def softplus(z):
  return np.logaddexp(0.0, z)


def sinusoid(positions, width):
  """[T, width]: sine in the even entries, cosine in the odd ones."""
  i = np.arange((width + 1) // 2)
  angle = np.asarray(positions, np.float64)[:, None] * np.power(
      10000.0, -2.0 * i / width)[None, :]
  out = np.zeros((len(positions), width))
  out[:, 0::2] = np.sin(angle)
  out[:, 1::2] = np.cos(angle)[:, :width // 2]
  return out


def causal_conv(x, taps):
  """Per-channel convolution over time, x [T, C], taps [C, n]; the last tap
  multiplies the current row, rows before the start are zero."""
  T, C = x.shape
  n = taps.shape[1]
  padded = np.concatenate([np.zeros((n - 1, C)), x])
  out = np.zeros((T, C))
  for j in range(n):
    out += padded[j:j + T] * taps[:, j]
  return out


def window_attention(q, k, v, scale, window, sink):
  """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv].  Query i weighs the
  keys i - window < j <= i (window None: all j <= i) by
  exp(scale q.k - slope_h (i - j)) over their sum plus exp(sink_h)."""
  T, H, _ = q.shape
  G = k.shape[1]
  out = np.zeros((T, H, v.shape[2]))
  for h in range(H):
    g = h // (H // G)
    slope = 2.0 ** (-8.0 * (h + 1) / H)
    for i in range(T):
      lo = 0 if window is None else max(0, i - window + 1)
      dist = i - np.arange(lo, i + 1)
      s = k[lo:i + 1, g] @ q[i, h] * scale - slope * dist
      top = max(s.max(), sink[h])
      e = np.exp(s - top)
      out[i, h] = (e @ v[lo:i + 1, g]) / (e.sum() + np.exp(sink[h] - top))
  return out


def gated_linear_attention(q, k, v, alpha):
  """S <- diag(alpha) S + k v^T, o = S^T q; q, k, alpha [T, H, D], v
  [T, H, Dv] -> o [T, H, Dv]."""
  T, H, D = q.shape
  S = np.zeros((H, D, v.shape[2]))
  out = np.zeros((T, H, v.shape[2]))
  for t in range(T):
    S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
    out[t] = np.einsum('hdv,hd->hv', S, q[t])
  return out


def delta_rule(q, k, v, g, beta):
  """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k, g
  [T, H, D], v [T, H, Dv], beta [T, H] -> o [T, H, Dv]."""
  T, H, D = q.shape
  S = np.zeros((H, D, v.shape[2]))
  out = np.zeros((T, H, v.shape[2]))
  for t in range(T):
    S = g[t][:, :, None] * S
    u = beta[t][:, None] * (v[t] - np.einsum('hdv,hd->hv', S, k[t]))
    S = S + k[t][:, :, None] * u[:, None, :]
    out[t] = np.einsum('hdv,hd->hv', S, q[t])
  return out


def attention_mixer(h, m, t, eps):
  T = len(h)
  H, G, D, Dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
  q = rms((h @ t('q').T).reshape(T, H, D), eps) * t('q.norm')
  k = rms((h @ t('k').T).reshape(T, G, D), eps) * t('k.norm')
  v = (h @ t('v').T).reshape(T, G, Dv)
  window = (m.get('mask') or {}).get('size')
  o = window_attention(q, k, v, m['scale'], window, t('sink'))
  return o.reshape(T, H * Dv) @ t('o').T


def gla_mixer(h, m, t, eps):
  T = len(h)
  H, D, Dv = m['heads'], m['dim'], m['vdim']
  q = (h @ t('q').T).reshape(T, H, D) * D ** -0.5
  k = (h @ t('k').T).reshape(T, H, D)
  v = (h @ t('v').T).reshape(T, H, Dv)
  z = h @ t('a1').T @ t('a2').T + t('a2.b')
  alpha = np.power(sigmoid(z), 1.0 / m['tau']).reshape(T, H, D)
  o = rms(gated_linear_attention(q, k, v, alpha), eps) * t('norm')
  return (o.reshape(T, H * Dv) * silu(h @ t('g').T)) @ t('o').T


def unit(x):
  return x / np.sqrt(np.sum(np.square(x), axis=-1, keepdims=True) + 1e-6)


def channel_delta_mixer(h, m, t, eps):
  T = len(h)
  H, G, D, Dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
  proj = lambda n: silu(causal_conv(h @ t(n).T, t(n + '.conv')))
  q = np.repeat(unit(proj('q').reshape(T, G, D)) * D ** -0.5, H // G, axis=1)
  k = np.repeat(unit(proj('k').reshape(T, G, D)), H // G, axis=1)
  v = proj('v').reshape(T, H, Dv)
  beta = sigmoid(h @ t('b').T)
  step = softplus(h @ t('a1').T @ t('a2').T + t('dt_bias')).reshape(T, H, D)
  g = np.exp(-np.exp(t('A_log'))[None, :, None] * step)
  o = rms(delta_rule(q, k, v, g, beta), eps) * t('norm')
  gate = sigmoid(h @ t('g1').T @ t('g2').T)
  return (o.reshape(T, H * Dv) * gate) @ t('o').T


MIXERS = {'attention': attention_mixer, 'gla': gla_mixer,
          'channel_delta': channel_delta_mixer}


def clamped_glu(h, m, t):
  g = np.minimum(h @ t('gate').T, m['limit'])
  u = np.clip(h @ t('up').T, -m['limit'], m['limit'])
  return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t('down').T


def layer_runs(cfg):
  """The layers in the order they run, as (layer, pass of the loop or None)."""
  n, loop = len(cfg['layers']), cfg.get('loop')
  if not loop:
    return [(i, None) for i in range(n)]
  start, stop, times = loop['start'], loop['stop'], loop['times']
  return ([(i, None) for i in range(start)] +
          [(i, t) for t in range(times) for i in range(start, stop)] +
          [(i, None) for i in range(stop, n)])


def forward(cfg, w, tokens, trace=None):
  """Logits [T, vocab] of one sequence; `trace` (a list) receives the residual
  stream after every layer run."""
  w = {k: np.asarray(v, np.float64) for k, v in w.items()}
  eps, tokens = cfg['norm']['eps'], np.asarray(tokens)
  x0 = w['embed'][tokens] + sinusoid(np.arange(len(tokens)), cfg['width'])
  x = x0
  for i, t in layer_runs(cfg):
    if t is not None and i == cfg['loop']['start']:
      x = np.concatenate([x, x0], axis=-1) @ w['loop.in'].T
      x = x + w['loop.step'][t]
    layer, n = cfg['layers'][i], f'l{i}.'
    mix = lambda name, n=n: w[n + 'mix.' + name]
    mlp = lambda name, n=n: w[n + 'mlp.' + name]
    h = rms(x, eps) * w[n + 'norm1']
    y = MIXERS[layer['type']](h, layer['mixer'], mix, eps)
    x = x + rms(y, eps) * w[n + 'norm1b']
    if layer['mlp'] is not None:
      h = rms(x, eps) * w[n + 'norm2']
      y = clamped_glu(h, layer['mlp'], mlp)
      x = x + rms(y, eps) * w[n + 'norm2b']
    if trace is not None:
      trace.append(x)
  return rms(x, eps) * w['final.norm'] @ w['head'].T
