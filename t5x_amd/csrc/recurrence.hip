// Linear recurrences over a matrix state per head, with one decay per key
// channel, for sequences that are fed in portions of any length:
//
//   S <- diag(g_t) S;  u = v_t  or, with the delta rule,  u = beta_t (v_t - S^T k_t);
//   S <- S + k_t u^T;  o_t = S^T q_t
//
// S [D, Dv] is float32 and lives in a slot per sequence; a portion that starts at
// position 0 starts from zeros whatever the slot holds.  Around it, in float32:
// an optional short causal convolution with silu on q, k and v (its last inputs
// live in the slot too, a ring by position), optional unit norms of q and k, the
// decay from a low-rank projection, and the norm and gate of the read-out.
//
// A portion runs as prepare (a wavefront per token and head vector), scan and
// finish; a step of one token per sequence is one kernel per (sequence, head)
// that reads and writes the state once.
#include "common.h"

namespace t5d {

struct RecArgs {
  t5d_recurrence a;
  t5d_ragged b;
  // float32 scratch of a portion
  float *wq, *wk, *wv, *wbeta, *wo;
  int C;  // channels of the convolution
  const int32_t* gate;
};

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) {
  return z > 20.f ? z : log1pf(expf(z));
}

// Logarithm of the decay of key channel c of head h from its projection z.
__device__ __forceinline__ float log_decay(const t5d_recurrence& a, float z, int h,
                                           int c) {
  z += a.decay_bias[(size_t)h * a.D + c];
  if (a.decay == T5D_DECAY_SIGMOID_POWER) return -softplus_f(-z) * a.decay_power;
  return -expf(a.A_log[h]) * softplus_f(z);
}

// One channel of q, k or v of the token at row m: the projection itself, or its
// causal convolution and silu.  `first`: row of the portion's first token; cc:
// channel of the convolution; x: value at row m.
template <typename T>
__device__ __forceinline__ float conv_channel(const RecArgs& g, int m, int first,
                                              int pos, int slot, int col, int cc,
                                              float x) {
  const t5d_recurrence& a = g.a;
  const float* w = a.conv + (size_t)cc * a.taps;
  float s = x * w[a.taps - 1];
  const T* ring = reinterpret_cast<const T*>(a.conv_ring) +
                  (size_t)slot * a.taps * g.C + cc;
  for (int j = 1; j < a.taps; ++j) {
    if (pos - j < 0) break;
    const float v = m - j >= first
                        ? to_f32<T>(reinterpret_cast<const T*>(
                              a.proj)[(size_t)(m - j) * a.ld_proj + col])
                        : to_f32<T>(ring[(size_t)((pos - j) % a.taps) * g.C]);
    s = fmaf(v, w[a.taps - 1 - j], s);
  }
  return s / (1.0f + expf(-s));
}

// ---- prepare ----------------------------------------------------------------------
// Vectors of a token: (with a convolution or unit norms) G queries, G keys, H
// values; then H decays.
template <typename T>
__global__ void __launch_bounds__(256)
recurrence_prepare_kernel(RecArgs g) {
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int lane = threadIdx.x & 63;
  const bool qkv = a.taps > 0 || a.unit;
  const int nq = qkv ? 2 * a.G + a.H : 0, nvec = nq + a.H;
  const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (int64_t)g.b.M * nvec) return;
  const int m = unit / nvec, vec = unit % nvec;
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m * a.ld_proj;
  if (vec >= nq) {
    const int h = vec - nq;
    float* z = a.low + (size_t)m * a.ld_low + a.off_z + (size_t)h * a.D;
    for (int c = lane; c < a.D; c += 64) z[c] = log_decay(a, z[c], h, c);
    if (a.delta && lane == 0)
      g.wbeta[(size_t)m * a.H + h] = sigmoid_f(to_f32<T>(p[a.off_beta + h]));
    return;
  }
  const bool query = vec < a.G, key = !query && vec < 2 * a.G;
  const int h = query ? vec : key ? vec - a.G : vec - 2 * a.G;
  const int n = query || key ? a.D : a.Dv;
  const int col0 = query ? a.off_q + h * a.D : key ? a.off_k + h * a.D
                                                   : a.off_v + h * a.Dv;
  const int cc0 = query ? h * a.D : key ? (a.G + h) * a.D : 2 * a.G * a.D + h * a.Dv;
  float* out = query ? g.wq + ((size_t)m * a.G + h) * a.D
               : key ? g.wk + ((size_t)m * a.G + h) * a.D
                     : g.wv + ((size_t)m * a.H + h) * a.Dv;
  const int seq = g.b.tok_seq[m], pos = g.b.tok_pos[m];
  const int first = g.b.seq_off[seq], slot = g.b.seq_slot[seq];
  float ss = 0.f;
  for (int c = lane; c < n; c += 64) {
    float x = to_f32<T>(p[col0 + c]);
    if (a.taps > 0)
      x = conv_channel<T>(g, m, first, pos, slot, col0 + c, cc0 + c, x);
    ss = fmaf(x, x, ss);
    out[c] = x;
  }
  if (!(query || key)) return;
  float f = query ? a.q_scale : 1.f;
  if (a.unit) f /= sqrtf(wave_sum(ss) + a.unit_eps);
  for (int c = lane; c < n; c += 64) out[c] *= f;  // this lane's own stores
}

// ---- scan ---------------------------------------------------------------------------
// A workgroup owns 16 columns of a head's state, a wavefront 4 of them: lane
// (kl, column) holds the rows d = 64 e + 4 kl + j of its column.  Columns never
// interact.  Keys, queries and decays of 8 tokens at a time go through LDS, the
// next 8 are on their way meanwhile.
template <int E4, bool DELTA, typename TQ>
__global__ void __launch_bounds__(256)
recurrence_scan_kernel(RecArgs g, const TQ* q_rows, const TQ* k_rows,
                       const TQ* v_rows, int ldq, int ldk, int ldv, float q_scale) {
  constexpr int DP = 64 * E4, TS = 8, NP = TS * DP / 256;
  __shared__ __align__(16) float s_k[TS][DP];
  __shared__ __align__(16) float s_q[TS][DP];
  __shared__ __align__(16) float s_g[TS][DP];
  __shared__ float s_v[TS][16];
  __shared__ float s_b[TS];
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int h = blockIdx.y, seq = blockIdx.z, hg = h / (a.H / a.G);
  const int off = g.b.seq_off[seq], T = g.b.seq_off[seq + 1] - off;
  const int start = g.b.seq_start[seq], slot = g.b.seq_slot[seq];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int kl = lane & 15, cw = wave * 4 + (lane >> 4);
  const int col = blockIdx.x * 16 + cw;
  const bool col_ok = col < a.Dv;
  if (T <= 0) return;

  float* state = a.state + ((size_t)slot * a.H + h) * a.D * a.Dv + col;
  float st[E4 * 4];
#pragma unroll
  for (int e = 0; e < E4 * 4; ++e) {
    const int d = 64 * (e >> 2) + 4 * kl + (e & 3);
    st[e] = start > 0 && col_ok && d < a.D ? state[(size_t)d * a.Dv] : 0.f;
  }
  const TQ* q = q_rows + (size_t)off * ldq + (size_t)hg * a.D;
  const TQ* k = k_rows + (size_t)off * ldk + (size_t)hg * a.D;
  const TQ* v = v_rows + (size_t)off * ldv + (size_t)h * a.Dv;
  const float* lg = a.low + (size_t)off * a.ld_low + a.off_z + (size_t)h * a.D;
  float* o = g.wo + ((size_t)off * a.H + h) * a.Dv + col;

  float pk[NP], pq[NP], pg[NP], pv = 0.f, pb = 0.f;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int e = threadIdx.x + 256 * i, t = t0 + e / DP, d = e % DP;
      const bool ok = t < T && d < a.D;
      pk[i] = ok ? to_f32<TQ>(k[(size_t)t * ldk + d]) : 0.f;
      pq[i] = ok ? to_f32<TQ>(q[(size_t)t * ldq + d]) * q_scale : 0.f;
      pg[i] = ok ? lg[(size_t)t * a.ld_low + d] : 0.f;
    }
    if (threadIdx.x < TS * 16) {
      const int t = t0 + threadIdx.x / 16, c = blockIdx.x * 16 + threadIdx.x % 16;
      pv = t < T && c < a.Dv ? to_f32<TQ>(v[(size_t)t * ldv + (threadIdx.x % 16) +
                                            blockIdx.x * 16])
                             : 0.f;
    } else if (DELTA && threadIdx.x < TS * 16 + TS) {
      const int t = t0 + threadIdx.x - TS * 16;
      pb = t < T ? g.wbeta[(size_t)(off + t) * a.H + h] : 0.f;
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < T; t0 += TS) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int e = threadIdx.x + 256 * i;
      s_k[e / DP][e % DP] = pk[i];
      s_q[e / DP][e % DP] = pq[i];
      s_g[e / DP][e % DP] = expf(pg[i]);
    }
    if (threadIdx.x < TS * 16) s_v[threadIdx.x / 16][threadIdx.x % 16] = pv;
    else if (DELTA && threadIdx.x < TS * 16 + TS) s_b[threadIdx.x - TS * 16] = pb;
    __syncthreads();
    if (t0 + TS < T) fetch(t0 + TS);
    const int n = min(TS, T - t0);
    for (int t = 0; t < n; ++t) {
      float kk[E4 * 4], qq[E4 * 4];
      float s0 = 0.f, s1 = 0.f, o0 = 0.f, o1 = 0.f;
#pragma unroll
      for (int e = 0; e < E4; ++e) {
        const float4 x = *reinterpret_cast<const float4*>(&s_k[t][64 * e + 4 * kl]);
        const float4 y = *reinterpret_cast<const float4*>(&s_q[t][64 * e + 4 * kl]);
        const float4 w = *reinterpret_cast<const float4*>(&s_g[t][64 * e + 4 * kl]);
        kk[4 * e] = x.x; kk[4 * e + 1] = x.y; kk[4 * e + 2] = x.z; kk[4 * e + 3] = x.w;
        qq[4 * e] = y.x; qq[4 * e + 1] = y.y; qq[4 * e + 2] = y.z; qq[4 * e + 3] = y.w;
        st[4 * e] *= w.x; st[4 * e + 1] *= w.y;
        st[4 * e + 2] *= w.z; st[4 * e + 3] *= w.w;
        if (DELTA) {
          s0 = fmaf(st[4 * e], x.x, s0);
          s1 = fmaf(st[4 * e + 1], x.y, s1);
          s0 = fmaf(st[4 * e + 2], x.z, s0);
          s1 = fmaf(st[4 * e + 3], x.w, s1);
        }
      }
      float u = s_v[t][cw];
      if (DELTA) u = s_b[t] * (u - lanes16_sum(s0 + s1));
#pragma unroll
      for (int e = 0; e < E4 * 4; e += 2) {
        st[e] = fmaf(kk[e], u, st[e]);
        st[e + 1] = fmaf(kk[e + 1], u, st[e + 1]);
        o0 = fmaf(st[e], qq[e], o0);
        o1 = fmaf(st[e + 1], qq[e + 1], o1);
      }
      const float r = lanes16_sum(o0 + o1);
      if (kl == 0 && col_ok) o[(size_t)(t0 + t) * a.H * a.Dv] = r;
    }
  }
#pragma unroll
  for (int e = 0; e < E4 * 4; ++e) {
    const int d = 64 * (e >> 2) + 4 * kl + (e & 3);
    if (col_ok && d < a.D) state[(size_t)d * a.Dv] = st[e];
  }
}

// The convolution's last inputs of a portion, written once nothing of the portion
// reads the ring any more.
template <typename T>
__global__ void __launch_bounds__(256)
recurrence_conv_tail_kernel(RecArgs g) {
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int seq = blockIdx.y;
  const int off = g.b.seq_off[seq], len = g.b.seq_off[seq + 1] - off;
  const int cc = blockIdx.x * 256 + threadIdx.x;
  if (cc >= g.C) return;
  const int qk = a.G * a.D;
  const int col = cc < qk ? a.off_q + cc
                  : cc < 2 * qk ? a.off_k + cc - qk : a.off_v + cc - 2 * qk;
  T* ring = reinterpret_cast<T*>(a.conv_ring) +
            (size_t)g.b.seq_slot[seq] * a.taps * g.C + cc;
  for (int t = max(0, len - (a.taps - 1)); t < len; ++t)
    ring[(size_t)((g.b.seq_start[seq] + t) % a.taps) * g.C] =
        reinterpret_cast<const T*>(a.proj)[(size_t)(off + t) * a.ld_proj + col];
}

// ---- read-out: norm, gate -----------------------------------------------------------
template <typename T>
__device__ __forceinline__ float out_gate(const t5d_recurrence& a, int m, int h,
                                          int c) {
  if (a.gate == T5D_GATE_SIGMOID_LOW)
    return sigmoid_f(a.low[(size_t)m * a.ld_low + a.off_low_gate +
                           (size_t)h * a.Dv + c]);
  const float z = to_f32<T>(reinterpret_cast<const T*>(
      a.proj)[(size_t)m * a.ld_proj + a.off_gate + (size_t)h * a.Dv + c]);
  return z * sigmoid_f(z);
}

template <typename T>
__global__ void __launch_bounds__(256)
recurrence_finish_kernel(RecArgs g) {
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int lane = threadIdx.x & 63;
  const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (int64_t)g.b.M * a.H) return;
  const int m = unit / a.H, h = unit % a.H;
  const float* o = g.wo + (size_t)unit * a.Dv;
  float ss = 0.f;
  for (int c = lane; c < a.Dv; c += 64) ss = fmaf(o[c], o[c], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.Dv + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + (size_t)m * a.ld_out + (size_t)h * a.Dv;
  for (int c = lane; c < a.Dv; c += 64)
    Act<T>::store(out + c, o[c] * inv * a.norm[c] * out_gate<T>(a, m, h, c));
}

// ---- one token per sequence ------------------------------------------------------------
// One workgroup per (sequence, head), a wavefront per 32 columns: lane (quad, dg)
// holds rows dg + 8 i of 4 neighbouring columns, so a load instruction reads 8
// runs of 128 bytes.  The state is requested before q, k, v and the decay are
// formed.
template <int DI, bool DELTA, typename T>
__global__ void __launch_bounds__(512)
recurrence_step_kernel(RecArgs g) {
  constexpr int DP = 8 * DI;
  __shared__ float s_q[DP], s_k[DP], s_g[DP];
  __shared__ __align__(16) float s_v[256];
  __shared__ __align__(16) float s_o[256];
  __shared__ float s_b;
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int h = blockIdx.x % a.H, m = blockIdx.x / a.H, hg = h / (a.H / a.G);
  const int pos = g.b.seq_start[m], slot = g.b.seq_slot[m];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int waves = blockDim.x >> 6;
  const int quad = lane & 7, dg = lane >> 3;
  const int col = 4 * (8 * wave + quad);
  const bool col_ok = col < a.Dv;
  float* state = a.state + ((size_t)slot * a.H + h) * a.D * a.Dv + col;
  float4 st[DI];
#pragma unroll
  for (int i = 0; i < DI; ++i) {
    const int d = dg + 8 * i;
    st[i] = pos > 0 && col_ok && d < a.D
                ? *reinterpret_cast<const float4*>(state + (size_t)d * a.Dv)
                : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m * a.ld_proj;
  for (int role = wave; role < 4; role += waves) {
    if (role == 3) {
      const float* z = a.low + (size_t)m * a.ld_low + a.off_z + (size_t)h * a.D;
      for (int c = lane; c < DP; c += 64)
        s_g[c] = c < a.D ? expf(log_decay(a, z[c], h, c)) : 0.f;
      if (DELTA && lane == 0) s_b = sigmoid_f(to_f32<T>(p[a.off_beta + h]));
      continue;
    }
    const int n = role == 2 ? a.Dv : a.D;
    const int pad = role == 2 ? n : DP;
    const int col0 = role == 0 ? a.off_q + hg * a.D
                     : role == 1 ? a.off_k + hg * a.D : a.off_v + h * a.Dv;
    const int cc0 = role == 0 ? hg * a.D
                    : role == 1 ? (a.G + hg) * a.D : 2 * a.G * a.D + h * a.Dv;
    float x[4];
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = lane + 64 * u;
      x[u] = 0.f;
      if (c < n) {
        x[u] = to_f32<T>(p[col0 + c]);
        if (a.taps > 0) {
          const float raw = x[u];
          x[u] = conv_channel<T>(g, m, m, pos, slot, col0 + c, cc0 + c, raw);
          Act<T>::store(reinterpret_cast<T*>(a.conv_ring) +
                            ((size_t)slot * a.taps + pos % a.taps) * g.C + cc0 + c,
                        raw);
        }
        ss = fmaf(x[u], x[u], ss);
      }
    }
    float f = role == 0 ? a.q_scale : 1.f;
    if (a.unit && role < 2) f /= sqrtf(wave_sum(ss) + a.unit_eps);
    float* dst = role == 0 ? s_q : role == 1 ? s_k : s_v;
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (lane + 64 * u < pad) dst[lane + 64 * u] = x[u] * f;
  }
  __syncthreads();
  float4 r = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int i = 0; i < DI; ++i) {
    const float w = s_g[dg + 8 * i];
    st[i].x *= w; st[i].y *= w; st[i].z *= w; st[i].w *= w;
    if (DELTA) {
      const float k = s_k[dg + 8 * i];
      r.x = fmaf(st[i].x, k, r.x); r.y = fmaf(st[i].y, k, r.y);
      r.z = fmaf(st[i].z, k, r.z); r.w = fmaf(st[i].w, k, r.w);
    }
  }
  // sum over the 8 row groups: lanes ^8, ^16, ^32
  auto over_rows = [](float v) { return rows_sum(v + lane_xor8(v)); };
  float4 u = col_ok ? *reinterpret_cast<const float4*>(s_v + col)
                    : make_float4(0.f, 0.f, 0.f, 0.f);
  if (DELTA) {
    const float beta = s_b;
    u.x = beta * (u.x - over_rows(r.x)); u.y = beta * (u.y - over_rows(r.y));
    u.z = beta * (u.z - over_rows(r.z)); u.w = beta * (u.w - over_rows(r.w));
  }
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int i = 0; i < DI; ++i) {
    const float k = s_k[dg + 8 * i], q = s_q[dg + 8 * i];
    st[i].x = fmaf(k, u.x, st[i].x); st[i].y = fmaf(k, u.y, st[i].y);
    st[i].z = fmaf(k, u.z, st[i].z); st[i].w = fmaf(k, u.w, st[i].w);
    o.x = fmaf(st[i].x, q, o.x); o.y = fmaf(st[i].y, q, o.y);
    o.z = fmaf(st[i].z, q, o.z); o.w = fmaf(st[i].w, q, o.w);
    const int d = dg + 8 * i;
    if (col_ok && d < a.D)
      *reinterpret_cast<float4*>(state + (size_t)d * a.Dv) = st[i];
  }
  o.x = over_rows(o.x); o.y = over_rows(o.y);
  o.z = over_rows(o.z); o.w = over_rows(o.w);
  if (dg == 0 && col_ok) *reinterpret_cast<float4*>(s_o + col) = o;
  __syncthreads();
  if (wave != 0) return;
  float ss = 0.f;
  for (int c = lane; c < a.Dv; c += 64) ss = fmaf(s_o[c], s_o[c], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.Dv + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + (size_t)m * a.ld_out + (size_t)h * a.Dv;
  for (int c = lane; c < a.Dv; c += 64)
    Act<T>::store(out + c, s_o[c] * inv * a.norm[c] * out_gate<T>(a, m, h, c));
}

template <bool DELTA, typename T>
static void launch_step(hipStream_t s, const RecArgs& g) {
  const dim3 grid(g.b.S * g.a.H), block(64 * ((g.a.Dv + 31) / 32));
#define T5D_RS(DI_) \
  hipLaunchKernelGGL((recurrence_step_kernel<DI_, DELTA, T>), grid, block, 0, s, g)
  if (g.a.D <= 32) T5D_RS(4);
  else if (g.a.D <= 64) T5D_RS(8);
  else if (g.a.D <= 128) T5D_RS(16);
  else T5D_RS(32);
#undef T5D_RS
}

template <bool DELTA, typename TQ>
static void launch_scan(hipStream_t s, const RecArgs& g, const TQ* q, const TQ* k,
                        const TQ* v, int ldq, int ldk, int ldv, float q_scale) {
  const dim3 grid((g.a.Dv + 15) / 16, g.a.H, g.b.S), block(256);
#define T5D_SC(E_)                                                               \
  hipLaunchKernelGGL((recurrence_scan_kernel<E_, DELTA, TQ>), grid, block, 0, s, \
                     g, q, k, v, ldq, ldk, ldv, q_scale)
  if (g.a.D <= 64) T5D_SC(1);
  else if (g.a.D <= 128) T5D_SC(2);
  else if (g.a.D <= 256) T5D_SC(4);
  else T5D_SC(8);
#undef T5D_SC
}

template <typename T>
static int run_portions(hipStream_t s, const RecArgs& g) {
  const t5d_recurrence& a = g.a;
  const bool qkv = a.taps > 0 || a.unit;
  const int64_t units = (int64_t)g.b.M * ((qkv ? 2 * a.G + a.H : 0) + a.H);
  hipLaunchKernelGGL(recurrence_prepare_kernel<T>, dim3((unsigned)((units + 3) / 4)),
                     dim3(256), 0, s, g);
  T5D_CHECK_LAUNCH("recurrence (prepare)");
  if (qkv) {
    const int gd = a.G * a.D, hv = a.H * a.Dv;
    if (a.delta)
      launch_scan<true, float>(s, g, g.wq, g.wk, g.wv, gd, gd, hv, 1.f);
    else
      launch_scan<false, float>(s, g, g.wq, g.wk, g.wv, gd, gd, hv, 1.f);
  } else {
    const T* p = reinterpret_cast<const T*>(a.proj);
    if (a.delta)
      launch_scan<true, T>(s, g, p + a.off_q, p + a.off_k, p + a.off_v, a.ld_proj,
                           a.ld_proj, a.ld_proj, a.q_scale);
    else
      launch_scan<false, T>(s, g, p + a.off_q, p + a.off_k, p + a.off_v, a.ld_proj,
                            a.ld_proj, a.ld_proj, a.q_scale);
  }
  T5D_CHECK_LAUNCH("recurrence (scan)");
  if (a.taps > 1) {
    hipLaunchKernelGGL(recurrence_conv_tail_kernel<T>,
                       dim3((g.C + 255) / 256, g.b.S), dim3(256), 0, s, g);
    T5D_CHECK_LAUNCH("recurrence (convolution tail)");
  }
  const int64_t heads = (int64_t)g.b.M * a.H;
  hipLaunchKernelGGL(recurrence_finish_kernel<T>, dim3((unsigned)((heads + 3) / 4)),
                     dim3(256), 0, s, g);
  T5D_CHECK_LAUNCH("recurrence (finish)");
  return T5D_OK;
}

static int64_t round4(int64_t n) { return (n + 3) / 4 * 4; }

}  // namespace t5d

using namespace t5d;

extern "C" int64_t t5d_recurrence_workspace_bytes(int M, int H, int G, int D,
                                                  int Dv) {
  if (M <= 0 || H <= 0 || G <= 0 || D <= 0 || Dv <= 0) return -1;
  return 4 * (2 * round4((int64_t)M * G * D) + 2 * round4((int64_t)M * H * Dv) +
              round4((int64_t)M * H));
}

extern "C" int t5d_recurrence_run(void* stream, const t5d_recurrence* a,
                                  const t5d_ragged* b, int variant) {
  T5D_REQUIRE(a && b, T5D_EINVAL, "t5d_recurrence_run: null arguments");
  T5D_REQUIRE(a->dtype == T5D_F32 || a->dtype == T5D_BF16, T5D_EINVAL,
              "t5d_recurrence_run: dtype %d", a->dtype);
  T5D_REQUIRE(a->H > 0 && a->G > 0 && a->H % a->G == 0 && a->D > 0 && a->Dv > 0 &&
                  a->taps >= 0 && a->H <= 65535,
              T5D_EINVAL, "t5d_recurrence_run: H=%d G=%d D=%d Dv=%d taps=%d", a->H,
              a->G, a->D, a->Dv, a->taps);
  T5D_REQUIRE(a->D <= 512, T5D_ELIMIT, "t5d_recurrence_run: key size %d > 512",
              a->D);
  T5D_REQUIRE(a->proj && a->low && a->decay_bias && a->norm && a->state && a->out &&
                  (a->decay == T5D_DECAY_SIGMOID_POWER || a->A_log) &&
                  (a->taps == 0 || (a->conv && a->conv_ring)) && b->tok_pos &&
                  b->tok_seq && b->seq_off && b->seq_start && b->seq_slot,
              T5D_EINVAL, "t5d_recurrence_run: null buffer");
  T5D_REQUIRE(b->M > 0 && b->S > 0 && b->S <= 65535 && b->max_len > 0 &&
                  b->max_len <= b->M,
              T5D_EINVAL, "t5d_recurrence_run: M=%d S=%d max_len=%d", b->M, b->S,
              b->max_len);
  T5D_REQUIRE(variant >= 0 && variant <= 2, T5D_EINVAL,
              "t5d_recurrence_run: variant %d", variant);
  RecArgs g;
  g.a = *a; g.b = *b; g.gate = tls_gate;
  g.C = 2 * a->G * a->D + a->H * a->Dv;
  const bool can_step = b->max_len == 1 && b->M == b->S && a->D <= 256 &&
                        a->Dv <= 256 && a->Dv % 4 == 0 &&
                        (uintptr_t)a->state % 16 == 0;
  T5D_REQUIRE(variant != 1 || can_step, T5D_EINVAL,
              "t5d_recurrence_run: variant 1 does not cover this call");
  hipStream_t s = as_stream(stream);
  if (variant == 1 || (variant == 0 && can_step)) {
    g.wq = g.wk = g.wv = g.wbeta = g.wo = nullptr;
    const bool bf16 = a->dtype == T5D_BF16;
    if (a->delta) {
      if (bf16) launch_step<true, bf16_t>(s, g);
      else launch_step<true, float>(s, g);
    } else {
      if (bf16) launch_step<false, bf16_t>(s, g);
      else launch_step<false, float>(s, g);
    }
    T5D_CHECK_LAUNCH("recurrence (step)");
    return T5D_OK;
  }
  T5D_REQUIRE(a->workspace && (uintptr_t)a->workspace % 16 == 0, T5D_EINVAL,
              "t5d_recurrence_run: portions need a 16-byte aligned workspace");
  float* w = (float*)a->workspace;
  const int64_t qk = round4((int64_t)b->M * a->G * a->D),
                hv = round4((int64_t)b->M * a->H * a->Dv);
  g.wq = w; g.wk = w + qk; g.wv = w + 2 * qk; g.wo = w + 2 * qk + hv;
  g.wbeta = w + 2 * qk + 2 * hv;
  return a->dtype == T5D_BF16 ? run_portions<bf16_t>(s, g) : run_portions<float>(s, g);
}
