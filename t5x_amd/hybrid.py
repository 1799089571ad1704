"""Decoder-only models whose layers mix windowed softmax attention, latent
attention and linear recurrences, on the HIP kernels behind t5d_hybrid_step.

A model is a list of layers, each a mixer from MIXERS (with sizes of its own) and
an optional feed-forward — one gated unit, or a mixture of them chosen by token id
— over a float32 residual stream, or several that hyper-connections mix.  A range of
layers may run several times in a row (a loop), every pass with caches of its own.
What a family of models fixes beside that is its Design.
Sequences are fed in portions of any length: what a sequence carries from one
portion to the next — a ring of keys and values (or of the latents they come from)
per attention pass, a matrix state and the convolution's last inputs per recurrent
pass — lives in its slot of the cache tree, and a portion that starts at position 0
starts from nothing whatever the slot held before.

Weights are packed once per parameter set.  All widths are padded to the tiles of
the matrix-core kernels with zero weights, so the padding columns of every
activation are zero.
"""

import ctypes
import dataclasses
from typing import Any, Mapping, Optional, Tuple, Union

import numpy as np
import torch

from t5x_amd import _lib
from t5x_amd import network
from t5x_amd import ops

_ACT = {'float32': torch.float32, 'bfloat16': torch.bfloat16}
UNIT_EPS = 1e-6       # inside the root of the unit norms
# A call expands the latents its windows show into keys and values where they are
# at most this many per new token.
SPAN_ROWS = 2


@dataclasses.dataclass(frozen=True)
class Design:
  """What every model of an architecture has in common.
  streams: one residual stream with hyper-connections between as many as the
  configuration says, a scaled embedding and a norm before every branch; else one
  stream, the embedding plus a sinusoid of the position, a norm before and after.
  dense: the gated unit of a feed-forward that is not a mixture; every unit is
  min(g, limit) sigmoid(alpha g) (clamp(u, limit) + add), as (alpha, add), and
  dense_limit None reads the limit from the configuration."""
  streams: bool
  dense: Tuple[float, float]
  dense_limit: Optional[float] = None


CLAMPED_UNIT = (1.702, 1.0)
SILU_UNIT = (1.0, 0.0)

DESIGNS = {
    'Mokivik': Design(streams=False, dense=CLAMPED_UNIT),
    'Nutizen': Design(streams=True, dense=SILU_UNIT, dense_limit=float('inf')),
}


@dataclasses.dataclass(frozen=True)
class MixerConfig:
  """Sizes and constants of one mixer; a type reads the ones it has."""
  type: str
  heads: int
  kv_heads: int
  dim: int
  vdim: int
  window: int = 0        # attention: keys a query sees, 0 = all before it
  scale: float = 1.0     # attention: factor of q . k
  taps: int = 0          # convolution length, 0 = none
  tau: float = 1.0       # decay = sigmoid(z)^(1 / tau)
  q_rank: int = 0        # latent attention: sizes of the queries' latent and
  kv_rank: int = 0       # of the cached one
  kv_from: Optional[int] = None  # the layer whose cached latents it reads
  reach: int = 0         # window that the ring serves: the widest of its readers


@dataclasses.dataclass(frozen=True)
class FeedForwardConfig:
  ff: int
  limit: float
  alpha: float = CLAMPED_UNIT[0]
  add: float = CLAMPED_UNIT[1]


@dataclasses.dataclass(frozen=True)
class ExpertsConfig:
  """A mixture: a table gives each token id `top` of `experts` units, each with
  weight 1 / top; a shared one runs for every token behind a sigmoid gate."""
  experts: int
  top: int
  expert: FeedForwardConfig
  shared: Optional[FeedForwardConfig] = None


@dataclasses.dataclass(frozen=True)
class LayerConfig:
  mixer: MixerConfig
  mlp: Union[None, FeedForwardConfig, ExpertsConfig] = None

  @property
  def experts(self) -> Optional[ExpertsConfig]:
    return self.mlp if isinstance(self.mlp, ExpertsConfig) else None

  @property
  def dense(self) -> Optional[FeedForwardConfig]:
    return self.mlp if isinstance(self.mlp, FeedForwardConfig) else None


@dataclasses.dataclass(frozen=True)
class LoopConfig:
  """Layers start .. stop - 1 run `times` times in a row."""
  start: int
  stop: int
  times: int


@dataclasses.dataclass(frozen=True)
class HybridConfig:
  vocab_size: int
  width: int
  eps: float
  layers: Tuple[LayerConfig, ...]
  loop: Optional[LoopConfig] = None
  dtype: str = 'bfloat16'
  streams: int = 0           # 0: one residual stream, see Design
  hyper: bool = False        # hyper-connections between the streams
  embed_scale: float = 1.0

  @classmethod
  def from_dict(cls, c: Mapping[str, Any], dtype: str = 'bfloat16'):
    """From a parsed config.json; raises on what these kernels do not compute."""
    design = DESIGNS[c.get('architecture', 'Mokivik')]
    layers = []
    for i, entry in enumerate(c['layers']):
      kind, m, mlp = entry['type'], entry['mixer'], entry.get('mlp')
      if kind not in MIXERS:
        raise ValueError(f'layer {i}: unknown mixer {kind!r}')
      heads = int(m['heads'])
      mixer = MixerConfig(
          type=kind, heads=heads, kv_heads=int(m.get('kv_heads', heads)),
          dim=int(m['dim']), vdim=int(m['vdim']),
          window=int((m.get('mask') or {}).get('size', 0)),
          scale=float(m.get('scale', 1.0)), taps=int(m.get('conv', 0)),
          tau=float(m.get('tau', 1.0)), q_rank=int(m.get('q_rank', 0)),
          kv_rank=int(m.get('kv_rank', 0)), kv_from=m.get('kv_from'))
      if mixer.heads % mixer.kv_heads:
        raise ValueError(f'layer {i}: {mixer.heads} heads over '
                         f'{mixer.kv_heads} key/value heads')
      if mixer.kv_from is not None:
        j = mixer.kv_from
        src = layers[j].mixer if 0 <= j < i else None
        if (src is None or src.type != kind or src.kv_from is not None or
            src.kv_rank != mixer.kv_rank):
          raise ValueError(f'layer {i}: no latents of size {mixer.kv_rank} '
                           f'in layer {j}')
      layers.append(LayerConfig(mixer, _feed_forward(mlp, design, i)))
    for i, layer in enumerate(layers):
      windows = [l.mixer.window for j, l in enumerate(layers)
                 if i in (j, l.mixer.kv_from)]
      reach = 0 if 0 in windows else max(windows)
      layers[i] = dataclasses.replace(
          layer, mixer=dataclasses.replace(layer.mixer, reach=reach))
    loop = c.get('loop')
    if design.streams and loop is not None:
      raise ValueError('a loop over layers with several residual streams')
    if not design.streams and any(
        l.experts or l.mixer.kv_from is not None for l in layers):
      raise ValueError('experts and shared latents need a design with streams')
    if loop is not None:
      loop = LoopConfig(int(loop['start']), int(loop['stop']),
                        int(loop['times']))
      if not (0 <= loop.start < loop.stop <= len(layers) and loop.times > 0):
        raise ValueError(f'loop {loop} over {len(layers)} layers')
    if dtype not in _ACT:
      raise ValueError(f'unsupported dtype {dtype!r}')
    return cls(vocab_size=int(c['vocab']), width=int(c['width']),
               eps=float(c['norm']['eps']), layers=tuple(layers), loop=loop,
               dtype=dtype,
               streams=int(c.get('streams', 1)) if design.streams else 0,
               hyper=design.streams and 'streams' in c,
               embed_scale=float((c.get('embedding') or {}).get('scale', 1.0)))

  def runs(self):
    """The layers in the order they run: (layer, pass that starts here or
    None)."""
    n, loop = len(self.layers), self.loop
    if loop is None:
      return [(i, None) for i in range(n)]
    body = [(i, t if i == loop.start else None) for t in range(loop.times)
            for i in range(loop.start, loop.stop)]
    return ([(i, None) for i in range(loop.start)] + body +
            [(i, None) for i in range(loop.stop, n)])

  def span_windows(self):
    """Windows of the layers that attend to expanded latents."""
    return sorted({l.mixer.window for l in self.layers
                   if l.mixer.type == 'latent_attention'})

  def param_shapes(self):
    """name -> shape of every tensor."""
    W, V = self.width, self.vocab_size
    out = {'embed': (V, W), 'final.norm': (W,), 'head': (V, W)}
    if self.loop is not None:
      out['loop.in'] = (W, 2 * W)
      out['loop.step'] = (self.loop.times, W)
    n = self.streams

    def unit(prefix, F):
      out[prefix + 'gate'] = out[prefix + 'up'] = (F, W)
      out[prefix + 'down'] = (W, F)

    def around(p, q):  # what stands before and after branch q of a layer
      out[f'{p}norm{q}'] = (W,)
      if not n:
        out[f'{p}norm{q}b'] = (W,)
      if self.hyper:
        out.update({f'{p}hc{q}.in': (n,), f'{p}hc{q}.out': (n,),
                    f'{p}hc{q}.mix': (n, n)})

    for i, layer in enumerate(self.layers):
      p = f'l{i}.'
      around(p, 1)
      out.update({p + 'mix.' + k: v for k, v in
                  MIXERS[layer.mixer.type].shapes(layer.mixer, W).items()})
      if layer.mlp is not None:
        around(p, 2)
      if layer.dense:
        unit(p + 'mlp.', layer.dense.ff)
      elif layer.experts:
        x = layer.experts
        out[p + 'mlp.table'] = (V, x.top)
        for e in range(x.experts):
          unit(f'{p}mlp.e{e}.', x.expert.ff)
        if x.shared:
          unit(p + 'mlp.shared.', x.shared.ff)
          out[p + 'mlp.shared.sg'] = (1, W)
    return out


def _feed_forward(c, design: Design, i: int):
  """The feed-forward that layer i's configuration names."""
  if c is None:
    return None
  kind = c.get('kind', 'dense')
  if kind == 'dense':
    limit = design.dense_limit
    return FeedForwardConfig(int(c['ff']), float(c['limit'] if limit is None
                                                 else limit), *design.dense)
  if kind != 'moe':
    raise ValueError(f'layer {i}: unknown feed-forward {kind!r}')
  unit = lambda u: FeedForwardConfig(int(u['ff']), float(u['limit']))
  experts, top = int(c['router']['experts']), int(c['router']['top'])
  if not 0 < top <= experts:
    raise ValueError(f'layer {i}: {top} of {experts} experts')
  return ExpertsConfig(experts, top, unit(c['expert']),
                       unit(c['shared']) if c.get('shared') else None)


def _pad(n: int, to: int) -> int:
  return (n + to - 1) // to * to


# ------------------------------------------------------------------------------
# Mixers: how a type's tensors become one packed projection, an optional packed
# low-rank second stage, and the constants its kernels take.
# ------------------------------------------------------------------------------


class _Columns:
  """Output columns of a fused projection: pieces side by side, each starting
  at a multiple of 16 unless it is glued to the one before."""

  def __init__(self):
    self.pieces, self.at, self.n = [], {}, 0

  def add(self, name, weight, glue=False):
    if not glue:
      self.n = _pad(self.n, 16)
    self.at[name] = self.n
    self.pieces.append((self.n, weight))
    self.n += weight.shape[0]

  def matrix(self, k_pad, n=None):
    """float32 [k_pad, n] kernel (input-major), zero where no piece is."""
    n = _pad(self.n, 16) if n is None else n
    first = self.pieces[0][1]
    out = torch.zeros((k_pad, n), dtype=torch.float32, device=first.device)
    for at, w in self.pieces:
      out[:w.shape[1], at:at + w.shape[0]] = w.t()
    return out


class _AttentionMixer:
  """Grouped-query attention over a sliding window with per-head query / key
  norms, a linear distance bias per head and a sink in the denominator."""

  @staticmethod
  def shapes(m, width):
    return {'q': (m.heads * m.dim, width), 'k': (m.kv_heads * m.dim, width),
            'v': (m.kv_heads * m.vdim, width), 'q.norm': (m.dim,),
            'k.norm': (m.dim,), 'sink': (m.heads,),
            'o': (width, m.heads * m.vdim)}

  @staticmethod
  def fill(layer, m, get, keep, eps, ld, pack):
    cols = _Columns()
    for name in ('q', 'k', 'v'):
      cols.add(name, get(name))
    layer.mix = _lib.MIX_WINDOW_ATTENTION
    layer.proj_n = _pad(cols.n, 16)
    layer.proj = pack(cols.matrix(ld))
    a = layer.attention
    a.H, a.G, a.D, a.Dv = m.heads, m.kv_heads, m.dim, m.vdim
    a.window, a.scale, a.eps = m.window, m.scale, eps
    a.off_q, a.off_k, a.off_v = (cols.at[n] for n in ('q', 'k', 'v'))
    a.q_norm, a.k_norm = keep(get('q.norm')), keep(get('k.norm'))
    a.sink = keep(get('sink'))
    slopes = [2.0 ** (-8.0 * (h + 1) / m.heads) for h in range(m.heads)]
    a.slopes = keep(torch.tensor(slopes, dtype=torch.float32))

  @staticmethod
  def cache(m, rows, ring_len, act, dev):
    hp = _lib.load().t5d_window_head_pad(m.dim, m.vdim)
    if hp < 0:
      raise ValueError(f'head size {m.dim} / {m.vdim} is not supported')
    ring = ring_len(m.window)
    make = lambda: torch.zeros((rows, m.kv_heads, ring, hp), dtype=act,
                               device=dev)
    return {'key_ring': make(), 'value_ring': make()}

  leaves = ('key_ring', 'value_ring')

  @staticmethod
  def bytes_per_row(m, ring_len, el):
    return 2 * m.kv_heads * ring_len(m.window) * el * _lib.load(
    ).t5d_window_head_pad(m.dim, m.vdim)

  @staticmethod
  def ring(tensors):
    return tensors[0].shape[2]

  @staticmethod
  def set_ring(layer, ring):
    layer.attention.ring = ring


class _LatentAttentionMixer:
  """Sliding-window attention with a sink whose keys and values are linear maps of
  a cached latent, the layer's own or an earlier layer's, and whose queries come
  through a latent too."""

  @staticmethod
  def shapes(m, width):
    out = {'dq': (m.q_rank, width), 'dq.norm': (m.q_rank,),
           'uq': (m.heads * m.dim, m.q_rank),
           'uk': (m.heads * m.dim, m.kv_rank),
           'uv': (m.heads * m.vdim, m.kv_rank), 'sink': (m.heads,),
           'o': (width, m.heads * m.vdim)}
    if m.kv_from is None:
      out.update({'dkv': (m.kv_rank, width), 'dkv.norm': (m.kv_rank,)})
    return out

  @staticmethod
  def pads(m):
    """(columns per head of queries, keys and values; of the cached latent; of
    the queries' latent)."""
    lib = _lib.load()
    hp, rp = lib.t5d_window_head_pad(m.dim, m.vdim), lib.t5d_latent_pad(m.kv_rank)
    if hp < 0 or rp < 0:
      raise ValueError(f'head size {m.dim} / {m.vdim} or latent size {m.kv_rank} '
                       'is not supported')
    return hp, rp, _pad(m.q_rank, 64)

  @classmethod
  def fill(cls, layer, m, get, keep, eps, ld, pack):
    H, D, Dv, rank = m.heads, m.dim, m.vdim, m.kv_rank
    hp, rp, qp = cls.pads(m)
    cols = _Columns()
    own = m.kv_from is None
    for name in ('dq', 'dkv') if own else ('dq',):
      cols.add(name, get(name))
    layer.mix = _lib.MIX_LATENT_ATTENTION
    layer.proj_n = _pad(cols.n, 16)
    layer.proj = pack(cols.matrix(ld))
    a = layer.latent
    a.H, a.D, a.Dv, a.rank, a.q_rank = H, D, Dv, rank, m.q_rank
    a.window, a.scale, a.eps = m.window, m.scale, eps
    a.off_q, a.off_kv = cols.at['dq'], cols.at['dkv'] if own else -1

    def padded(w, *shape):
      out = torch.zeros(shape, dtype=torch.float32, device=w.device)
      out[tuple(slice(n) for n in w.shape)] = w
      return out

    a.q_norm = keep(padded(get('dq.norm'), qp))
    if own:
      a.kv_norm = keep(padded(get('dkv.norm'), rp))
    a.sink = keep(get('sink'))
    uq = padded(get('uq').reshape(H, D, m.q_rank), H, hp, qp)
    uk = padded(get('uk').reshape(H, D, rank), H, hp, rp)
    uv = padded(get('uv').reshape(H, Dv, rank), H, hp, rp)
    a.uq = pack(uq.reshape(H * hp, qp).t().contiguous())
    a.ukv = pack(torch.cat([uk, uv]).reshape(2 * H * hp, rp).t().contiguous())
    a.absorb = pack.many(list(uk))[0]
    vp = _pad(Dv, 16)
    uv = padded(get('uv').reshape(H, Dv, rank), H, vp, rp)
    a.expand = pack.many([w.t().contiguous() for w in uv])[0]

  @classmethod
  def cache(cls, m, rows, ring_len, act, dev):
    if m.kv_from is not None:
      return {}
    return {'latent_ring': torch.zeros((rows, ring_len(m.reach), cls.pads(m)[1]),
                                       dtype=act, device=dev)}

  leaves = ('latent_ring', None)

  @classmethod
  def bytes_per_row(cls, m, ring_len, el):
    return 0 if m.kv_from is not None else (
        ring_len(m.reach) * cls.pads(m)[1] * el)

  @staticmethod
  def ring(tensors):
    return tensors[0].shape[1]

  @staticmethod
  def set_ring(layer, ring):
    layer.latent.ring = ring


class _RecurrentMixer:
  """What the linear recurrences share."""
  leaves = ('state', 'conv_ring')

  @staticmethod
  def bytes_per_row(m, ring_len, el):
    del ring_len
    return 4 * m.heads * m.dim * m.vdim + el * m.taps * (
        2 * m.kv_heads * m.dim + m.heads * m.vdim)

  @staticmethod
  def ring(tensors):
    del tensors  # a state of fixed size

  @staticmethod
  def set_ring(layer, ring):
    pass

  @staticmethod
  def cache(m, rows, ring_len, act, dev):
    del ring_len
    out = {'state': torch.zeros((rows, m.heads, m.dim, m.vdim),
                                dtype=torch.float32, device=dev)}
    if m.taps:
      c = 2 * m.kv_heads * m.dim + m.heads * m.vdim
      out['conv_ring'] = torch.zeros((rows, m.taps, c), dtype=act, device=dev)
    return out

  @staticmethod
  def common(layer, m, get, keep, eps, cols, low, ld, pack):
    """cols: the projection, its last pieces (glued) the inputs of the low-rank
    stage, whose own pieces are `low`: (name, weight, first input column)."""
    r = layer.recurrence
    layer.mix = _lib.MIX_RECURRENCE
    layer.off_low = cols.at['a1']
    rank = cols.n - layer.off_low
    layer.low_k = _pad(rank, 64)
    # the low-rank stage reads low_k columns: the projection has them all
    layer.proj_n = layer.off_low + layer.low_k
    layer.proj = pack(cols.matrix(ld, layer.proj_n))
    at, n = {}, 0
    for name, w, _ in low:
      at[name] = n
      n = _pad(n + w.shape[0], 16)
    layer.low_n = n
    second = torch.zeros((layer.low_k, n), dtype=torch.float32,
                         device=low[0][1].device)
    for name, w, row in low:
      second[row:row + w.shape[1], at[name]:at[name] + w.shape[0]] = w.t()
    layer.low = pack(second)
    r.H, r.G, r.D, r.Dv = m.heads, m.kv_heads, m.dim, m.vdim
    r.taps, r.eps, r.unit_eps = m.taps, eps, UNIT_EPS
    r.q_scale = m.dim ** -0.5
    r.off_q, r.off_k, r.off_v = (cols.at[n] for n in ('q', 'k', 'v'))
    r.off_z = at['z']
    r.norm = keep(get('norm'))
    return r, at


class _GatedLinearMixer(_RecurrentMixer):
  """Linear attention with a decay sigmoid(z)^(1 / tau) per key channel and a
  silu gate on the normed read-out."""

  @staticmethod
  def shapes(m, width):
    kd, vd, rank = m.heads * m.dim, m.heads * m.vdim, None
    return {'q': (kd, width), 'k': (kd, width), 'v': (vd, width),
            'g': (vd, width), 'o': (width, vd), 'norm': (m.vdim,),
            'a1': (rank, width), 'a2': (kd, rank), 'a2.b': (kd,)}

  @staticmethod
  def fill(layer, m, get, keep, eps, ld, pack):
    cols = _Columns()
    for name in ('q', 'k', 'v', 'g', 'a1'):
      cols.add(name, get(name))
    r, _ = _RecurrentMixer.common(layer, m, get, keep, eps, cols,
                                  [('z', get('a2'), 0)], ld, pack)
    r.delta, r.unit, r.taps = 0, 0, 0
    r.decay, r.decay_power = _lib.DECAY_SIGMOID_POWER, 1.0 / m.tau
    r.decay_bias = keep(get('a2.b'))
    r.gate, r.off_gate = _lib.GATE_SILU, cols.at['g']


class _ChannelDeltaMixer(_RecurrentMixer):
  """Delta rule with a decay exp(-exp(A) softplus(z)) per head and key channel,
  short convolutions and unit norms in front, a low-rank sigmoid gate behind."""

  @staticmethod
  def shapes(m, width):
    qk, v, kd = m.kv_heads * m.dim, m.heads * m.vdim, m.heads * m.dim
    rank = None
    out = {'b': (m.heads, width), 'A_log': (m.heads,), 'norm': (m.vdim,),
           'a1': (rank, width), 'a2': (kd, rank), 'dt_bias': (kd,),
           'g1': (rank, width), 'g2': (v, rank), 'o': (width, v)}
    for name, n in (('q', qk), ('k', qk), ('v', v)):
      out[name], out[name + '.conv'] = (n, width), (n, m.taps)
    return out

  @staticmethod
  def fill(layer, m, get, keep, eps, ld, pack):
    cols = _Columns()
    for name in ('q', 'k', 'v', 'b', 'a1'):
      cols.add(name, get(name))
    cols.add('g1', get('g1'), glue=True)
    r, at = _RecurrentMixer.common(
        layer, m, get, keep, eps, cols,
        [('z', get('a2'), 0), ('gate', get('g2'), get('a1').shape[0])], ld, pack)
    r.delta, r.unit = 1, 1
    r.decay = _lib.DECAY_EXP_SOFTPLUS
    r.decay_bias, r.A_log = keep(get('dt_bias')), keep(get('A_log'))
    r.off_beta = cols.at['b']
    r.gate, r.off_low_gate = _lib.GATE_SIGMOID_LOW, at['gate']
    r.conv = keep(torch.cat([get(n + '.conv') for n in ('q', 'k', 'v')]))


MIXERS = {'attention': _AttentionMixer, 'gla': _GatedLinearMixer,
          'channel_delta': _ChannelDeltaMixer,
          'latent_attention': _LatentAttentionMixer}


# ------------------------------------------------------------------------------
# Weights
# ------------------------------------------------------------------------------


class Packer:
  """Packs input-major float32 kernels for the dense layers and keeps the packed
  tensors in the list `kept`."""

  def __init__(self, act_dtype, kept):
    self.act_dtype, self.kept = act_dtype, kept

  def _data(self, kernel, gate):
    act = self.act_dtype
    return ops.pack_weight(kernel, act, act, gate_kernel=gate).data

  def __call__(self, kernel, gate=None):
    self.kept.append(self._data(kernel, gate))
    return self.kept[-1].data_ptr()

  def many(self, kernels, gates=None):
    """Kernels of one shape one after the other -> (address, bytes of each)."""
    gates = gates or [None] * len(kernels)
    out = None
    for i, (kernel, gate) in enumerate(zip(kernels, gates)):
      data = self._data(kernel, gate)
      if out is None:
        out = data.new_empty((len(kernels),) + tuple(data.shape))
      out[i] = data
    self.kept.append(out)
    return out.data_ptr(), out[0].numel() * out.element_size()


class HybridWeights:
  """The parameters of a model, cast and packed once on the device, and the
  t5d_hybrid_layer descriptions that name them."""

  def __init__(self, cfg: HybridConfig, params: Mapping[str, Any], device):
    self.cfg, self.act_dtype = cfg, _ACT[cfg.dtype]
    act = self.act_dtype
    self.ld = ld = _pad(cfg.width, 64)
    self._kept = []
    shapes = cfg.param_shapes()
    for name, shape in shapes.items():
      if name not in params:
        raise ValueError(f'parameter {name!r} is missing')
      have = tuple(np.shape(params[name]))
      if len(have) != len(shape) or any(
          s is not None and s != h for s, h in zip(shape, have)):
        raise ValueError(f'parameter {name!r} has shape {have}, expected '
                         f'{shape}')
    get = lambda name: network._f32(params[name], device)

    def keep(t, dtype=torch.float32):
      t = t.to(device=device, dtype=dtype).contiguous()
      self._kept.append(t)
      return t.data_ptr()

    pack = Packer(act, self._kept)

    def padded(name, k, n):
      """Transposed to input-major and padded to [k, n]."""
      w = get(name)
      out = torch.zeros((k, n), dtype=torch.float32, device=device)
      out[:w.shape[1], :w.shape[0]] = w.t()
      return out

    table = torch.zeros((cfg.vocab_size, ld), dtype=torch.float32, device=device)
    table[:, :cfg.width] = get('embed')
    self.embedding = keep(table, act)
    self.final_norm = keep(get('final.norm'))
    self.head_n = (cfg.vocab_size if act == torch.float32 else
                   _pad(cfg.vocab_size, 16))
    self.head = pack(padded('head', ld, self.head_n))
    self.loop_in, self.loop_steps = None, []
    if cfg.loop is not None:
      w = get('loop.in')
      both = torch.zeros((2 * ld, ld), dtype=torch.float32, device=device)
      both[:cfg.width, :cfg.width] = w[:, :cfg.width].t()
      both[ld:ld + cfg.width, :cfg.width] = w[:, cfg.width:].t()
      self.loop_in = pack(both)
      steps = get('loop.step')
      self.loop_steps = [keep(steps[t]) for t in range(cfg.loop.times)]
    self.layers = (_lib.HybridLayer * len(cfg.layers))()
    for i, lc in enumerate(cfg.layers):
      layer, m = self.layers[i], lc.mixer
      mix = lambda name, i=i: get(f'l{i}.mix.{name}')
      around = [('norm1', 'norm1'), ('norm1b', 'norm1b')]
      around += [(f'{leaf}1', f'hc1.{leaf}') for leaf in ('in', 'mix', 'out')]
      if lc.mlp is not None:
        around += [(field.replace('1', '2'), name.replace('1', '2'))
                   for field, name in around]
      for field, name in around:
        if f'l{i}.{name}' in shapes:
          setattr(layer, field, keep(get(f'l{i}.{name}')))
      MIXERS[m.type].fill(layer, m, mix, keep, cfg.eps, ld, pack)
      layer.out_k = _pad(m.heads * m.vdim, 64)
      layer.out = pack(padded(f'l{i}.mix.o', layer.out_k, ld))

      def unit(prefix, ff):
        F = _pad(ff, 64)
        return (F, pack(padded(prefix + 'gate', ld, F),
                        padded(prefix + 'up', ld, F)),
                pack(padded(prefix + 'down', F, ld)))

      if lc.dense:
        layer.F, layer.glu, layer.down = unit(f'l{i}.mlp.', lc.dense.ff)
        layer.glu_limit, layer.glu_alpha, layer.glu_add = (
            lc.dense.limit, lc.dense.alpha, lc.dense.add)
      elif lc.experts:
        x, e, p = lc.experts, layer.experts, f'l{i}.mlp.'
        table = torch.as_tensor(np.asarray(
            params[p + 'table'].cpu() if isinstance(params[p + 'table'],
                                                    torch.Tensor)
            else params[p + 'table']).astype(np.int64))
        if int(table.min()) < 0 or int(table.max()) >= x.experts:
          raise ValueError(f'parameter {p}table names experts beyond the '
                           f'{x.experts} there are')
        e.table = keep(table, torch.int32)
        e.n, e.top, e.F = x.experts, x.top, _pad(x.expert.ff, 64)
        each = lambda leaf, *shape, p=p, n=x.experts: [
            padded(f'{p}e{k}.{leaf}', *shape) for k in range(n)]
        e.glu, e.glu_stride = pack.many(each('gate', ld, e.F),
                                        each('up', ld, e.F))
        e.down, e.down_stride = pack.many(each('down', e.F, ld))
        e.limit, e.alpha, e.add = x.expert.limit, x.expert.alpha, x.expert.add
        if x.shared:
          e.shared_F, e.shared_glu, e.shared_down = unit(p + 'shared.',
                                                         x.shared.ff)
          e.shared_limit = x.shared.limit
          e.shared_gate = keep(get(p + 'shared.sg').reshape(-1))

  def nbytes(self):
    return sum(t.numel() * t.element_size() for t in self._kept)


class _Buffers:
  """Activations of a call of up to `tokens` tokens of up to `seqs` sequences,
  and this call's copies of the layer descriptions, which name them."""

  def __init__(self, w: HybridWeights, tokens: int, seqs: int, device):
    cfg, act, ld = w.cfg, w.act_dtype, w.ld
    self.tokens, self.seqs = tokens, seqs
    self.layers = (_lib.HybridLayer * len(cfg.layers))()
    self._kept = kept = []

    def rows(n, dtype=act, zero=False, per=1):
      t = (torch.zeros if zero else torch.empty)((tokens * per, n), dtype=dtype,
                                                 device=device)
      kept.append(t)
      return t

    lib = _lib.load()
    f32 = torch.float32
    self.x = rows(ld * max(1, cfg.streams), f32)
    self.h, self.y = rows(ld), rows(ld)
    self.x0, self.cat = ((rows(ld, f32), rows(2 * ld)) if cfg.loop else
                         (None, None))
    self.proj = rows(max(l.proj_n for l in w.layers))
    low_n = max(l.low_n for l in w.layers)
    self.low = rows(low_n, f32) if low_n else None
    pools = {}

    def pooled(valid, n):
      # the padding columns are zero once and never written, so buffers are
      # shared only between layers with the same ones
      if (valid, n) not in pools:
        pools[valid, n] = rows(n, zero=True)
      return pools[valid, n].data_ptr()

    q_cols, ws = 0, 0
    for i, lc in enumerate(cfg.layers):
      self.layers[i] = w.layers[i]
      layer, m = self.layers[i], lc.mixer
      layer.mix_rows = pooled(m.heads * m.vdim, layer.out_k)
      if lc.dense:
        layer.ff_rows = pooled(lc.dense.ff, layer.F)
      if layer.mix == _lib.MIX_LATENT_ATTENTION:
        ws = max(ws, lib.t5d_latent_workspace_bytes(m.kv_rank))
      elif layer.mix == _lib.MIX_WINDOW_ATTENTION:
        hp = lib.t5d_window_head_pad(m.dim, m.vdim)
        q_cols = max(q_cols, m.heads * hp)
        ws = max(ws, lib.t5d_window_workspace_bytes(seqs, m.heads, m.dim,
                                                    m.vdim))
      else:
        # (one token per sequence: no scratch for chunks)
        ws = max(ws, lib.t5d_recurrence_workspace_bytes(
            tokens, seqs if tokens > seqs else 0, m.heads, m.kv_heads, m.dim,
            m.vdim))
    self.q_rows = rows(q_cols) if q_cols else None
    self.workspace = torch.empty((ws,), dtype=torch.uint8, device=device)
    self._latent_buffers(cfg, act, rows)
    self._expert_buffers(cfg, ld, act, rows, device)

  def _latent_buffers(self, cfg, act, rows):
    """Scratch of the latent attention layers, which run one after the other."""
    layers = [(l.latent, cfg.layers[i].mixer) for i, l in enumerate(self.layers)
              if l.mix == _lib.MIX_LATENT_ATTENTION]
    if not layers:
      return
    pads = [(m.heads,) + _LatentAttentionMixer.pads(m) for _, m in layers]
    cq, q = rows(max(p[3] for p in pads)), rows(max(p[0] * p[1] for p in pads))
    ql, ol = (rows(max(p[0] * p[2] for p in pads)) for _ in range(2))
    # keys and values expanded from the latents of a span: where portions can
    # be longer than a token, and for bfloat16 only
    spans = act == torch.bfloat16 and self.tokens > self.seqs
    if spans:
      lat = rows(max(p[2] for p in pads), per=SPAN_ROWS)
      kv = rows(max(2 * p[0] * p[1] for p in pads), per=SPAN_ROWS)
    for a, _ in layers:
      a.cq, a.q, a.ql, a.ol = (t.data_ptr() for t in (cq, q, ql, ol))
      if spans:
        a.lat, a.kv = lat.data_ptr(), kv.data_ptr()
        a.span_rows = SPAN_ROWS * self.tokens

  def _expert_buffers(self, cfg, ld, act, rows, device):
    """What the mixtures share, and each one's sorted tokens (found for all of
    them at the start of a call)."""
    layers = [l.experts for l in self.layers if l.experts.n]
    if not layers:
      return
    lib = _lib.load()
    top = max(e.top for e in layers)
    hidden = rows(max(e.F * e.top for e in layers))
    out, gate = rows(ld * top), rows(1, torch.float32)
    shared = max(e.shared_F for e in layers)
    shared = rows(shared) if shared else None
    least = 8 if act == torch.float32 else 16  # rows of the smallest tiles

    def ints(n):
      t = torch.full((n,), -1, dtype=torch.int32, device=device)
      self._kept.append(t)
      return t.data_ptr()

    for e in layers:
      n = self.tokens * e.top
      e.max_tiles = lib.t5d_route_max_tiles(n, e.n, least)
      e.tiles, e.token_of, e.entry_of = ints(4 * e.max_tiles), ints(n), ints(n)
      e.rows, e.out, e.gate = (t.data_ptr() for t in (hidden, out, gate))
      e.shared_rows = _lib.ptr(shared)


class Portions:
  """The token arrays of one call (t5d_ragged), uploaded as one int32 array.
  portions: (slot, position of the first token, token ids) per sequence.
  windows: of the layers that expand latents (t5d_span)."""

  def __init__(self, portions, want_rows, device, windows=()):
    lens = np.array([len(t) for _, _, t in portions], np.int32)
    self.M, self.S = int(lens.sum()), len(portions)
    self.max_len = int(lens.max())
    start = np.array([s for _, s, _ in portions], np.int32)
    slot = np.array([s for s, _, _ in portions], np.int32)
    off = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
    seq = np.repeat(np.arange(self.S, dtype=np.int32), lens)
    pos = np.arange(self.M, dtype=np.int32) - off[seq] + start[seq]
    tokens = np.concatenate([np.asarray(t, np.int32) for _, _, t in portions])
    want = np.asarray(want_rows, np.int32)
    parts = [tokens, pos, seq, off, start, slot, want]
    spans = []
    if self.max_len > 1:
      end = (start + lens + 63) // 64 * 64
      for window in windows:
        first = start * 0
        if window:
          first = np.maximum(0, start - window + 1) // 64 * 64
        rows = np.concatenate([[0], np.cumsum(end - first)])
        if rows[-1] <= SPAN_ROWS * self.M:
          spans.append((window, int(rows[-1]), len(parts)))
          parts += [rows.astype(np.int32), first.astype(np.int32)]
    self.data = torch.from_numpy(np.concatenate(parts)).to(device)
    r = self.ragged = _lib.Ragged()
    r.M, r.S, r.max_len = self.M, self.S, self.max_len
    at = self.data.data_ptr()
    addresses = []
    for part in parts:
      addresses.append(at)
      at += 4 * len(part)
    for name, address in zip(('tokens', 'tok_pos', 'tok_seq', 'seq_off',
                              'seq_start', 'seq_slot'), addresses):
      setattr(r, name, address)
    self.want_ptr, self.n_want = addresses[6], len(want)
    self._spans = (_lib.Span * max(1, len(spans)))()
    for s, (window, rows, n) in zip(self._spans, spans):
      s.window, s.rows = window, rows
      s.off, s.first = addresses[n], addresses[n + 1]
    r.spans = ctypes.cast(self._spans, ctypes.c_void_p)
    r.n_spans = len(spans)


class StepRows:
  """The token arrays of a step of one token per row, all on the device: row r
  has slot r, its token in tokens[r] and its position in positions[r]."""

  def __init__(self, tokens, positions):
    R, dev = tokens.numel(), tokens.device
    self.rows = torch.arange(R + 1, dtype=torch.int32, device=dev)
    if not (tokens.is_contiguous() and positions.is_contiguous()):
      raise ValueError('tokens and positions must be contiguous')
    self.tokens, self.positions = tokens, positions
    r = self.ragged = _lib.Ragged()
    r.M = r.S = R
    r.max_len = 1
    r.tokens, r.tok_pos = tokens.data_ptr(), positions.data_ptr()
    r.seq_start = positions.data_ptr()
    r.tok_seq = r.seq_off = r.seq_slot = self.rows.data_ptr()


# ------------------------------------------------------------------------------
# The module
# ------------------------------------------------------------------------------


class HybridDecoder(network.DecodeContexts):
  """A decoder-only model: packed weights, cache trees, the step function."""

  # Longest portion of one sequence that runs at once; longer ones are cut.  The
  # rings of windowed layers hold window - 1 + max_portion positions.
  max_portion = 2048
  # Tokens of one call over all its sequences.
  max_tokens = 16384

  def __init__(self, config: HybridConfig, device=None):
    self.config, self.dtype, self.device = config, config.dtype, device
    self._weights = {}
    self._bufs = None
    self._step = None
    self._beam_ctx = {}

  def decoder_weights(self, params) -> HybridWeights:
    key = id(params)
    if key not in self._weights:
      self._weights[key] = (params, HybridWeights(self.config, params,
                                                  self._dev()))
    return self._weights[key][1]

  # -- caches -----------------------------------------------------------------
  def init_cache(self, rows: int, max_len: int, portion: Optional[int] = None):
    """A cache tree for `rows` slots of up to `max_len` positions: one scope per
    layer run that keeps something, and cache_index [rows] = positions each slot
    holds.  portion: the longest portion it will be fed (max_portion)."""
    cfg, dev = self.config, self._dev()
    ring_len = self._ring_len(max_len, portion)
    act = _ACT[cfg.dtype]
    tree = {}
    for r, (i, _) in enumerate(cfg.runs()):
      m = cfg.layers[i].mixer
      leaves = MIXERS[m.type].cache(m, rows, ring_len, act, dev)
      if leaves:  # (nothing where another layer's are read)
        tree[f'run_{r}'] = leaves
    return {'decoder': tree,
            'cache_index': torch.zeros((rows,), dtype=torch.int32, device=dev)}

  def _ring_len(self, max_len, portion):
    """window -> positions in a ring (window 0: all)."""
    portion = min(portion or self.max_portion, self.max_portion, max_len)
    return lambda window: _pad(
        max_len if window == 0 else window - 1 + portion, 64)

  def cache_bytes(self, rows: int, max_len: int, portion=None) -> int:
    cfg, ring_len = self.config, self._ring_len(max_len, portion)
    el = 2 if cfg.dtype == 'bfloat16' else 4
    mixers = [cfg.layers[i].mixer for i, _ in cfg.runs()]
    return rows * sum(MIXERS[m.type].bytes_per_row(m, ring_len, el)
                      for m in mixers)

  def _run_cache(self, cache, run, layer):
    """The cache leaf that a run of a layer reads and writes."""
    src = self.config.layers[layer].mixer.kv_from
    # (layers with shared latents run once each: run = layer)
    return cache['decoder'][f'run_{run if src is None else src}']

  # -- the step function --------------------------------------------------------
  def _buffers(self, w, tokens, seqs):
    """Shared activation buffers of at least this size (calls on one stream)."""
    b = self._bufs
    have = (b[1].tokens, b[1].seqs) if b is not None and b[0] is w else (0, 0)
    if tokens > have[0] or seqs > have[1]:
      grow = lambda n, h: max(1 << (n - 1).bit_length(), h)
      self._bufs = self._step = b = None
      seqs = grow(seqs, have[1])
      tokens = max(grow(tokens, have[0]), 2 * seqs)
      b = self._bufs = (w, _Buffers(w, tokens, seqs, self._dev()))
    return b[1]

  def _model(self, w: HybridWeights, bufs: _Buffers, cache, gate=None):
    """Fills a t5d_hybrid_model over this cache tree."""
    cfg, P = self.config, _lib.ptr
    runs = cfg.runs()
    layers = (_lib.HybridLayer * len(cfg.layers))()
    for i in range(len(cfg.layers)):
      layers[i] = bufs.layers[i]
    cruns = (_lib.HybridRun * len(runs))()
    kept = []
    for r, (i, start) in enumerate(runs):
      m, leaf = cfg.layers[i].mixer, self._run_cache(cache, r, i)
      c = [leaf.get(n) for n in MIXERS[m.type].leaves]
      for t in c:
        if t is not None and not t.is_contiguous():
          raise ValueError(f'cache leaf of run {r} is not contiguous')
      kept.append(c)
      cruns[r].layer, cruns[r].enter = i, int(start is not None)
      cruns[r].enter_add = w.loop_steps[start] if start is not None else None
      cruns[r].cache0, cruns[r].cache1 = P(c[0]), P(c[1])
      MIXERS[m.type].set_ring(layers[i], MIXERS[m.type].ring(c))
    mod = _lib.HybridModel()
    mod.dtype = _lib.dtype_code(w.act_dtype)
    mod.d, mod.ld, mod.V, mod.head_n = (cfg.width, w.ld, cfg.vocab_size,
                                        w.head_n)
    mod.n_layers, mod.n_runs, mod.eps = len(cfg.layers), len(runs), cfg.eps
    mod.streams, mod.embed_scale = cfg.streams, cfg.embed_scale
    mod.embedding, mod.loop_in = w.embedding, w.loop_in
    mod.head, mod.final_norm = w.head, w.final_norm
    mod.layers, mod.runs = layers, cruns
    for name in ('x', 'x0', 'low', 'h', 'cat', 'proj', 'q_rows', 'y',
                 'workspace'):
      setattr(mod, name, P(getattr(bufs, name)))
    mod.workspace_bytes = bufs.workspace.numel()
    mod.gate = P(gate)
    mod._keepalive = (layers, cruns, kept, w, bufs, gate)
    return mod

  def _model_for(self, w, bufs, cache):
    """_model, kept while the cache tree is the same."""
    key = (id(w), id(bufs)) + tuple(
        t.data_ptr() for leaf in cache['decoder'].values()
        for t in leaf.values())
    if self._step is None or self._step[0] != key:
      self._step = (key, self._model(w, bufs, cache))
    return self._step[1]

  def _run(self, w, cache, portions, want_rows, trace=None):
    p = Portions(portions, want_rows, self._dev(), self.config.span_windows())
    bufs = self._buffers(w, p.M, p.S)
    model = self._model_for(w, bufs, cache)
    logits = None
    if p.n_want:
      logits = torch.empty((p.n_want, self.config.vocab_size),
                           dtype=torch.float32, device=self._dev())
    model.trace = _lib.ptr(trace)
    try:
      _lib.call('t5d_hybrid_step', _lib.stream_handle(), model, p.ragged,
                p.want_ptr, p.n_want, _lib.ptr(logits))
    finally:
      model.trace = None
    return logits

  def advance(self, params, cache, portions, want=None, trace=None):
    """Feeds every sequence its next tokens and returns the logits asked for.

    portions: (slot, position of the first token, token ids) per sequence, slots
    distinct; want: per portion the places among its tokens whose logits are
    returned, in this order ([n, vocab] float32, None if there are none).  Portions
    beyond max_portion or calls beyond max_tokens run in pieces.  Positions are
    the caller's: cache_index is not looked at.
    trace: a list that receives the float32 residual stream after every layer run,
    [runs, tokens, width] per piece."""
    cfg, w = self.config, self.decoder_weights(params)
    limit = min(self.max_portion, self._portion_limit(cache, portions))
    want = [[] for _ in portions] if want is None else want
    taken = [0] * len(portions)
    rows = {}  # (portion, place) -> logits row
    while True:
      piece, picks, room = [], [], self.max_tokens
      for n, (slot, start, toks) in enumerate(portions):
        lo = taken[n]
        hi = min(len(toks), lo + limit, lo + room)
        if hi <= lo:
          continue
        base = self.max_tokens - room
        picks += [(base + k - lo, (n, k)) for k in sorted(set(want[n]))
                  if lo <= k < hi]
        piece.append((slot, start + lo, toks[lo:hi]))
        taken[n], room = hi, room - (hi - lo)
      if not piece:
        break
      stream = None
      if trace is not None:
        M = sum(len(t) for _, _, t in piece)
        stream = torch.empty((len(cfg.runs()), M, w.ld), dtype=torch.float32,
                             device=self._dev())
      logits = self._run(w, cache, piece, [r for r, _ in picks], stream)
      for i, (_, key) in enumerate(picks):
        rows[key] = logits[i]
      if trace is not None:
        trace.append(stream[:, :, :cfg.width])
    out = [rows[n, k] for n, places in enumerate(want) for k in places]
    return torch.stack(out) if out else None

  def _portion_limit(self, cache, portions):
    """The longest portion the rings of this cache take at once; raises where
    a sequence would outgrow the ring of a layer without a window."""
    limit = self.max_tokens
    for r, (i, _) in enumerate(self.config.runs()):
      m = self.config.layers[i].mixer
      leaf, mixer = self._run_cache(cache, r, i), MIXERS[m.type]
      ring = mixer.ring([leaf.get(n) for n in mixer.leaves])
      if ring is None:
        continue
      if m.window:
        limit = min(limit, ring - m.window + 1)
      for _, start, toks in portions:
        if not m.window and start + len(toks) > ring:
          raise ValueError(f'{start + len(toks)} positions in a cache of {ring}')
    return limit

  def prefill(self, params, cache, tokens, lengths):
    """Feeds row r of the cache the first lengths[r] entries of tokens[r] and
    sets cache_index."""
    tokens = np.asarray(tokens.cpu() if isinstance(tokens, torch.Tensor)
                        else tokens)
    portions = [(r, 0, tokens[r, :n]) for r, n in enumerate(lengths) if n > 0]
    if portions:
      self.advance(params, cache, portions)
    cache['cache_index'].copy_(torch.as_tensor(
        np.asarray(lengths, np.int32), device=self._dev()))
    return cache

  def decode_step(self, params, cache, ids):
    """One new token per row (device ids [R]), at position cache_index, which
    advances -> logits [R, vocab]."""
    w = self.decoder_weights(params)
    ids = ids.reshape(-1).to(torch.int32).contiguous()
    R, index = ids.numel(), cache['cache_index']
    if index.numel() != R:  # rows expanded into beams
      index = index.reshape(-1, 1).expand(-1, R // index.numel())
      index = cache['cache_index'] = index.contiguous()
    step = StepRows(ids, index)
    model = self._model_for(w, self._buffers(w, R, R), cache)
    logits = torch.empty((R, self.config.vocab_size), dtype=torch.float32,
                         device=self._dev())
    _lib.call('t5d_hybrid_step', _lib.stream_handle(), model, step.ragged, None,
              R, logits.data_ptr())
    ops.add_i32(index, 1)
    return logits

  # -- fused sampling -------------------------------------------------------------
  def make_fused_sample_step(self, params, cache, owner=None, **kw):
    """A HybridSampleStep that continues from `cache`, kept and re-bound per
    (weights, cache shape, options)."""
    w = self.decoder_weights(params)
    shapes = tuple(tuple(t.shape) for leaf in cache['decoder'].values()
                   for t in leaf.values())
    key = ('sample', id(w), shapes, tuple(kw['sequences'].shape),
           int(kw['eos_id']), int(kw['topk']), float(kw['topp']),
           bool(kw['rescale']), kw.get('noise_source') is not None)
    return self._decode_context(
        key, w, owner,
        make=lambda slot: HybridSampleStep(self, params, cache, slot=slot, **kw),
        rebind=lambda ctx: ctx.rebind(cache, **kw))

  def batches_in_flight(self, batch_size, num_decodes, decode_len) -> int:
    """How many batches of this shape to keep decoding at once: as many as the
    device runs side by side, fewer when their caches would take more than half
    of the free device memory."""
    need = self.cache_bytes(batch_size * num_decodes, decode_len)
    free, _ = torch.cuda.mem_get_info(self._dev())
    return max(1, min(self.streams_side_by_side(), int(free // 4 // max(1, need))))


class HybridSampleStep(network.SampleStepGraph):
  """SampleStepGraph of a HybridDecoder: owns a copy of the prefilled cache and
  activations of its own, so several can run on their own streams."""

  def __init__(self, module, params, cache, *, slot=0, **state):
    self.w = w = module.decoder_weights(params)
    self._init_state(module, module.config.vocab_size, slot, **state)
    R, dev = self.sequences.shape[0], module._dev()
    self.cache = {'decoder': {
        r: {n: t.clone() for n, t in leaf.items()}
        for r, leaf in cache['decoder'].items()}}
    self._check_rows(cache, R)
    self.bufs = _Buffers(w, R, R, dev)
    self.logits = torch.empty((R, module.config.vocab_size),
                              dtype=torch.float32, device=dev)
    self.rows = StepRows(self.cur_token, self.cur_index)
    self.model = module._model(w, self.bufs, self.cache, gate=self.keep_going)
    self._capture()

  @staticmethod
  def _check_rows(cache, R):
    for leaf in cache['decoder'].values():
      for t in leaf.values():
        if t.shape[0] != R:
          raise ValueError(f'a cache of {t.shape[0]} rows for {R} sequences')

  def rebind(self, cache, *, noise_source=None, **state):
    cur = torch.cuda.current_stream()
    cur.wait_stream(self.stream)
    self._rebind_state(noise_source, state)
    for r, leaf in cache['decoder'].items():
      for n, t in leaf.items():
        self.cache['decoder'][r][n].copy_(t)
    self.stream.wait_stream(cur)

  def _enqueue(self):
    self._lib.call('t5d_hybrid_sample_step', self.stream.cuda_stream, self.model,
                   self.rows.ragged, self.logits.data_ptr(), self.sample)


def init_params(cfg: HybridConfig, seed: int = 0, device=None, rank: int = 64):
  """Random parameters by tensor name, generated on the device: linear weights
  normal(0, 1/sqrt(fan_in)), norms 1 + 0.1 normal, low-rank stages of `rank`,
  decay biases spread so that memories last from a few tokens to hundreds,
  hyper-connections near one stream passed on and written to, tables of distinct
  random experts."""
  device = device or torch.device('cuda')
  gen = torch.Generator(device=device)
  gen.manual_seed(seed)
  normal = lambda shape: torch.randn(shape, generator=gen, device=device)
  out = {}
  for name, shape in cfg.param_shapes().items():
    shape = tuple(rank if s is None else s for s in shape)
    leaf = name.rsplit('.', 1)[-1]
    if leaf == 'table':
      experts = cfg.layers[int(name[1:name.index('.')])].experts.experts
      out[name] = torch.rand((shape[0], experts), generator=gen,
                             device=device).argsort(1)[:, :shape[1]].to(torch.int32)
    elif '.hc' in name:
      out[name] = 0.1 * normal(shape) + (
          torch.eye(shape[0], device=device) if leaf == 'mix' else
          1.0 / cfg.streams if leaf == 'in' else 1.0)
    elif 'norm' in leaf:
      out[name] = 1.0 + 0.1 * normal(shape)
    elif leaf == 'conv':
      out[name] = normal(shape) / np.sqrt(shape[1])
    elif name == 'embed' or leaf == 'sink':
      out[name] = normal(shape)
    elif leaf == 'b' and len(shape) == 1:   # a2.b
      out[name] = 2.0 + 1.5 * normal(shape)
    elif leaf == 'A_log':
      out[name] = 0.5 * normal(shape)
    elif leaf == 'dt_bias':
      out[name] = -3.0 + 1.5 * normal(shape)
    elif leaf == 'step':
      out[name] = 0.1 * normal(shape)
    else:
      out[name] = normal(shape) / np.sqrt(shape[1])
  return out
