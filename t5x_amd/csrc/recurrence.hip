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
// Short portions run as prepare (a wavefront per token and head vector), a scan
// token by token, and finish.  Long ones are cut into chunks of 16 tokens.  With
// P_t the product of the decays of a chunk up to token t, the state S0 before it
// and X the solution of (I + diag(beta) A) X = diag(beta) R, A[t][s] = sum_d k_t
// (P_t / P_s) k_s for s < t, and B the same with q_t for s <= t,
//   Wk = X(k P), Us = X(v):       u = Us - Wk S0          (no delta rule: u = v)
//   Qs = q P - B Wk, Os = B Us:   o = Os + Qs S0
//   S  = diag(P_16) S0 + Kh^T u,  Kh_t = k_t P_16 / P_t
// Everything but the products with S0 and the state is independent of the other
// chunks: one kernel forms it for all chunks at once, from the projections on
// (quotients of decays as running products, which are at most 1), a second walks
// the chunks with three matrix products each, in float32 on the matrix cores.
// A step of one token per sequence is one kernel per (sequence, head) that reads
// and writes the state once.
#include "common.h"
#include "gemm_tiles.h"

namespace t5d {

struct RecArgs {
  t5d_recurrence a;
  t5d_ragged b;
  // float32 scratch of a portion
  float *wq, *wk, *wv, *wbeta, *wo;
  float* wchunk;  // chunked portions: the chunks' operands (ChunkLayout)
  int chunks;     // of the longest portion: the chunk kernel's grid
  int C;  // channels of the convolution
  const int32_t* gate;
};

__device__ __forceinline__ float exp_f(float z) {
  return __builtin_amdgcn_exp2f(z * 1.4426950408889634f);
}
__device__ __forceinline__ float sigmoid_f(float z) {
  return 1.0f / (1.0f + exp_f(-z));
}
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
  return s * sigmoid_f(s);
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

// ---- chunks ---------------------------------------------------------------------------
constexpr int kChunk = 16;

// A sequence's first chunk in the scratch memory: the sequences before it have
// at most this many chunks together.
__host__ __device__ __forceinline__ size_t chunk_base(int64_t first_token, int seq) {
  return (size_t)(first_token / kChunk + seq);
}

// What the chunk kernel leaves per (chunk, head), in floats, in the
// operand order of v_mfma_f32_16x16x4_f32: lane (x, g) of 16 x 4 holds element
// (row x, k g) of the left operand, (k g, column x) of the right one, and rows
// 4 g + i of column x of the result.  Step i of a product takes k = 4 g + i from
// lane (x, g), so that a result tile is the right operand of the next product as
// it stands; a left operand is then one float4 per lane and tile:
//   wk, qs [tile of 16 channels][lane]: channels 16 tile + 4 g + i of token x
//   kh     [tile][lane]: tokens 4 g + i, channel 16 tile + x
//   us, os [tile of 16 columns][lane]: tokens 4 g + i, column 16 tile + x
//   pc     [channel]: the chunk's whole decay
struct ChunkLayout {
  int dp, vp;
  __host__ __device__ ChunkLayout(int dp_, int vp_) : dp(dp_), vp(vp_) {}
  __host__ __device__ size_t wk() const { return 0; }
  __host__ __device__ size_t qs() const { return (size_t)kChunk * dp; }
  __host__ __device__ size_t kh() const { return (size_t)2 * kChunk * dp; }
  __host__ __device__ size_t us() const { return (size_t)3 * kChunk * dp; }
  __host__ __device__ size_t os() const { return us() + (size_t)kChunk * vp; }
  __host__ __device__ size_t pc() const { return os() + (size_t)kChunk * vp; }
  __host__ __device__ size_t size() const { return pc() + dp; }
};

// 16 tokens of one projection column, through the convolution and silu if there
// is one (TM: at least its taps).  i0: the chunk's first token within the portion.
template <int TM, typename T>
__device__ __forceinline__ void chunk_column(const RecArgs& g, int m0, int n, int i0,
                                             int pos0, int slot, int col, int cc,
                                             float (&y)[kChunk]) {
  const t5d_recurrence& a = g.a;
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m0 * a.ld_proj + col;
  float x[kChunk];
#pragma unroll
  for (int t = 0; t < kChunk; ++t)
    x[t] = t < n ? to_f32<T>(p[(size_t)t * a.ld_proj]) : 0.f;
  if constexpr (TM == 0) {
#pragma unroll
    for (int t = 0; t < kChunk; ++t) y[t] = x[t];
    return;
  }
  constexpr int N = TM > 0 ? TM : 1;
  float w[N], before[N];  // before[j]: the value j tokens before the chunk
  const T* ring = reinterpret_cast<const T*>(a.conv_ring) +
                  (size_t)slot * a.taps * g.C + cc;
#pragma unroll
  for (int j = 0; j < N; ++j) {
    w[j] = j < a.taps ? a.conv[(size_t)cc * a.taps + a.taps - 1 - j] : 0.f;
    before[j] = 0.f;
    if (j > 0 && j < a.taps) {
      if (i0 >= j)
        before[j] = to_f32<T>(p[-(ptrdiff_t)j * a.ld_proj]);
      else if (pos0 >= j)
        before[j] = to_f32<T>(ring[(size_t)((pos0 - j) % a.taps) * g.C]);
    }
  }
#pragma unroll
  for (int t = 0; t < kChunk; ++t) {
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < N; ++j)
      s = fmaf(w[j], t >= j ? x[t >= j ? t - j : 0] : before[t >= j ? 0 : j - t], s);
    y[t] = s * sigmoid_f(s);
  }
}

constexpr int kChunkTaps = 8;  // longest convolution of the chunk kernel

template <int DP, bool DELTA, typename T>
__global__ void __launch_bounds__(256, DP <= 128 ? 4 : DP <= 256 ? 2 : 1)
recurrence_chunk_kernel(RecArgs g) {
  constexpr int LS = DP + 4, C = kChunk;
  __shared__ __align__(16) float s_k[C * LS];
  __shared__ __align__(16) float s_q[C * LS];
  __shared__ __align__(16) float s_g[C * LS];
  __shared__ __align__(16) float s_a[C][C];
  __shared__ __align__(16) float s_b[C][C];
  __shared__ float s_beta[C];
  extern __shared__ float s_v[];  // [C][vp]
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int chunk = blockIdx.x, h = blockIdx.y, seq = blockIdx.z;
  const int hg = h / (a.H / a.G);
  const int off = g.b.seq_off[seq];
  const int n = min(C, g.b.seq_off[seq + 1] - off - chunk * C);
  if (n <= 0) return;
  const int m0 = off + chunk * C;
  const int tid = threadIdx.x;
  const int vp = (a.Dv + 15) / 16 * 16;
  const int slot = g.b.seq_slot[seq], pos0 = g.b.seq_start[seq] + chunk * C;
  // Columns of q, k, v and the decay; tokens past the end have no key, no query,
  // no value and no decay.
  for (int u = tid; u < 3 * DP + vp; u += 256) {
    const int kind = u < DP ? 0 : u < 2 * DP ? 1 : u < 2 * DP + vp ? 2 : 3;
    const int c = kind == 3 ? u - 2 * DP - vp : u - kind * DP;
    float y[C];
    if (c >= (kind == 2 ? a.Dv : a.D)) {
#pragma unroll
      for (int t = 0; t < C; ++t) y[t] = kind == 3 ? 1.f : 0.f;
    } else if (kind == 3) {
      const float* z = a.low + (size_t)m0 * a.ld_low + a.off_z + (size_t)h * a.D + c;
#pragma unroll
      for (int t = 0; t < C; ++t) y[t] = t < n ? z[(size_t)t * a.ld_low] : 0.f;
#pragma unroll
      for (int t = 0; t < C; ++t)
        y[t] = t < n ? exp_f(log_decay(a, y[t], h, c)) : 1.f;
    } else {
      const int col = kind == 0 ? a.off_q + hg * a.D + c
                      : kind == 1 ? a.off_k + hg * a.D + c : a.off_v + h * a.Dv + c;
      const int cc = kind == 0 ? hg * a.D + c
                     : kind == 1 ? (a.G + hg) * a.D + c
                                 : 2 * a.G * a.D + h * a.Dv + c;
      if (a.taps == 0)
        chunk_column<0, T>(g, m0, n, chunk * C, pos0, slot, col, cc, y);
      else if (a.taps <= 4)
        chunk_column<4, T>(g, m0, n, chunk * C, pos0, slot, col, cc, y);
      else
        chunk_column<kChunkTaps, T>(g, m0, n, chunk * C, pos0, slot, col, cc, y);
#pragma unroll
      for (int t = 0; t < C; ++t)  // the convolution reaches past the end
        if (t >= n) y[t] = 0.f;
    }
    float* dst = kind == 0 ? s_q : kind == 1 ? s_k : kind == 2 ? s_v : s_g;
    const int stride = kind == 2 ? vp : LS;
#pragma unroll
    for (int t = 0; t < C; ++t) dst[t * stride + c] = y[t];
  }
  if (tid < C)
    s_beta[tid] =
        DELTA && tid < n
            ? sigmoid_f(to_f32<T>(reinterpret_cast<const T*>(
                  a.proj)[(size_t)(m0 + tid) * a.ld_proj + a.off_beta + h]))
            : 0.f;
  s_a[tid >> 4][tid & 15] = 0.f;
  s_b[tid >> 4][tid & 15] = 0.f;
  __syncthreads();
  {
    // unit norms and the query's factor: 8 lanes per row of q, then of k
    const bool query = tid < 128;
    float* row = (query ? s_q : s_k) + ((tid >> 3) & 15) * LS + 4 * (tid & 7);
    float f = query ? a.q_scale : 1.f;
    if (a.unit) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < DP / 32; ++e) {
        const float4 x = *reinterpret_cast<const float4*>(row + 32 * e);
        ss = fmaf(x.x, x.x, ss); ss = fmaf(x.y, x.y, ss);
        ss = fmaf(x.z, x.z, ss); ss = fmaf(x.w, x.w, ss);
      }
      ss += dpp_move<kDppXor1>(ss);
      ss += dpp_move<kDppXor2>(ss);
      ss += dpp_move<kDppHalfMirror>(ss);
      f /= sqrtf(ss + a.unit_eps);
    }
    if (a.unit || query) {
#pragma unroll
      for (int e = 0; e < DP / 32; ++e) {
        float4 x = *reinterpret_cast<const float4*>(row + 32 * e);
        x.x *= f; x.y *= f; x.z *= f; x.w *= f;
        *reinterpret_cast<float4*>(row + 32 * e) = x;
      }
    }
  }
  __syncthreads();
  {
    // 32 lanes per source token s, which walk t = s .. 15 with k_s decayed on
    // the way; source j then source 15 - j, 17 steps for everyone.
    constexpr int E = (DP + 127) / 128;
    const int j = tid >> 5, c0 = 4 * (tid & 31);
#pragma unroll
    for (int pass = 0; pass < 2; ++pass) {
      const int s = pass == 0 ? j : C - 1 - j;
      float4 x[E];
#pragma unroll
      for (int e = 0; e < E; ++e)
        x[e] = c0 + 128 * e < DP
                   ? *reinterpret_cast<const float4*>(s_k + s * LS + c0 + 128 * e)
                   : make_float4(0.f, 0.f, 0.f, 0.f);
      for (int t = s; t < C; ++t) {
        float ka = 0.f, qa = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
          if (c0 + 128 * e >= DP) continue;
          const int o = t * LS + c0 + 128 * e;
          if (t > s) {
            const float4 w = *reinterpret_cast<const float4*>(s_g + o);
            x[e].x *= w.x; x[e].y *= w.y; x[e].z *= w.z; x[e].w *= w.w;
          }
          const float4 y = *reinterpret_cast<const float4*>(s_q + o);
          qa = fmaf(x[e].x, y.x, qa); qa = fmaf(x[e].y, y.y, qa);
          qa = fmaf(x[e].z, y.z, qa); qa = fmaf(x[e].w, y.w, qa);
          if (DELTA) {
            const float4 z = *reinterpret_cast<const float4*>(s_k + o);
            ka = fmaf(x[e].x, z.x, ka); ka = fmaf(x[e].y, z.y, ka);
            ka = fmaf(x[e].z, z.z, ka); ka = fmaf(x[e].w, z.w, ka);
          }
        }
        auto over32 = [](float f) {
          f = lanes16_sum(f);
          const auto w = __builtin_amdgcn_permlane16_swap(
              __float_as_uint(f), __float_as_uint(f), false, false);
          return __uint_as_float(w[0]) + __uint_as_float(w[1]);
        };
        qa = over32(qa);
        if (DELTA) ka = over32(ka);
        if ((tid & 31) == 0) {
          s_b[t][s] = qa;
          if (DELTA && t > s) s_a[t][s] = ka;
        }
      }
    }
  }
  __syncthreads();

  const ChunkLayout lay(DP, vp);
  float* w = g.wchunk + ((chunk_base(off, seq) + chunk) * a.H + h) * lay.size();
  // A thread per channel, then per value column: the triangular solve and the
  // products with B down the column.
  for (int c = tid; c < DP + vp; c += 256) {
    const bool channel = c < DP;
    const int vc = c - DP;
    // (a zero the compiler cannot see through: it would otherwise read all of A
    // and B into registers ahead of this loop)
    int z = 0;
    asm volatile("" : "+s"(z));
    float x[C], run = 1.f;
    float* sq = s_q + c;
    float* sk = s_k + c;
    float* sg = s_g + c;  // of a channel: read and written by this thread alone
#pragma unroll
    for (int t = 0; t < C; ++t) {
      __builtin_amdgcn_sched_barrier(0);
      float rhs;
      if (channel) {
        run *= sg[t * LS];
        rhs = sk[t * LS] * run;
      } else {
        rhs = s_v[t * vp + vc];
      }
      if (DELTA) {
#pragma unroll
        for (int s = 0; s < t; ++s) rhs = fmaf(-s_a[t + z][s], x[s], rhs);
        rhs *= s_beta[t];
      }
      x[t] = rhs;
      if (channel) {
        float y = sq[t * LS] * run;
        if (DELTA) {
#pragma unroll
          for (int s = 0; s <= t; ++s) y = fmaf(-s_b[t + z][s], x[s], y);
        }
        sq[t * LS] = y;
      }
    }
    if (channel) {
      w[lay.pc() + c] = run;
      float back = 1.f;
#pragma unroll
      for (int t = C - 1; t >= 0; --t) {
        const float gt = sg[t * LS];
        sg[t * LS] = sk[t * LS] * back;
        back *= gt;
        if (DELTA) sk[t * LS] = x[t];
      }
    } else {
      float4* us = reinterpret_cast<float4*>(w + lay.us()) + (vc >> 4) * 64 + (vc & 15);
      float4* os = reinterpret_cast<float4*>(w + lay.os()) + (vc >> 4) * 64 + (vc & 15);
      float y[C];
#pragma unroll
      for (int t = 0; t < C; ++t) {
        __builtin_amdgcn_sched_barrier(0);
        y[t] = 0.f;
#pragma unroll
        for (int s = 0; s <= t; ++s) y[t] = fmaf(s_b[t + z][s], x[s], y[t]);
      }
#pragma unroll
      for (int q4 = 0; q4 < 4; ++q4) {
        us[16 * q4] = make_float4(x[4 * q4], x[4 * q4 + 1], x[4 * q4 + 2], x[4 * q4 + 3]);
        os[16 * q4] = make_float4(y[4 * q4], y[4 * q4 + 1], y[4 * q4 + 2], y[4 * q4 + 3]);
      }
    }
  }
  __syncthreads();
  for (int f = tid; f < DP * 4; f += 256) {
    const int tile = f >> 6, l = f & 63, x = l & 15, g4 = l >> 4;
    const int o = x * LS + 16 * tile + 4 * g4;
    if (DELTA)
      reinterpret_cast<float4*>(w + lay.wk())[f] =
          *reinterpret_cast<const float4*>(s_k + o);
    reinterpret_cast<float4*>(w + lay.qs())[f] =
        *reinterpret_cast<const float4*>(s_q + o);
    const float* kh = s_g + 4 * g4 * LS + 16 * tile + x;
    reinterpret_cast<float4*>(w + lay.kh())[f] =
        make_float4(kh[0], kh[LS], kh[2 * LS], kh[3 * LS]);
  }
}

// Walks the chunks of one (sequence, head) for 16 value columns.  Each of 4
// wavefronts holds NTW tiles of 16 channels x 16 columns of the state.
template <int NTW, bool DELTA>
__global__ void __launch_bounds__(256)
recurrence_chain_kernel(RecArgs g) {
  constexpr int DP = 64 * NTW;
  __shared__ float4 s_u[2][4][64];
  __shared__ float4 s_o[2][4][64];
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  // The workgroups of one (sequence, head) read the same operands: consecutive
  // block ids go round-robin over the 8 XCDs, so theirs are 8 apart.
  const int vp = (a.Dv + 15) / 16 * 16, vts = vp / 16;
  const int pair = (blockIdx.x & 7) + 8 * ((blockIdx.x >> 3) / vts);
  if (pair >= a.H * g.b.S) return;
  const int vt = (blockIdx.x >> 3) % vts, h = pair % a.H, seq = pair / a.H;
  const int off = g.b.seq_off[seq], len = g.b.seq_off[seq + 1] - off;
  if (len <= 0) return;
  const int start = g.b.seq_start[seq], slot = g.b.seq_slot[seq];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int x = lane & 15, g4 = lane >> 4;
  const int col = 16 * vt + x;
  const bool col_ok = col < a.Dv;
  const ChunkLayout lay(DP, vp);
  const int nc = (len + kChunk - 1) / kChunk;
  const size_t stride = (size_t)a.H * lay.size();
  const float* base = g.wchunk + (chunk_base(off, seq) * a.H + h) * lay.size();

  float* state = a.state + ((size_t)slot * a.H + h) * a.D * a.Dv + col;
  f32x4_v st[NTW];
#pragma unroll
  for (int t = 0; t < NTW; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (wave * NTW + t) + 4 * g4 + i;
      st[t][i] = start > 0 && col_ok && d < a.D ? state[(size_t)d * a.Dv] : 0.f;
    }
  float* out = g.wo + ((size_t)off * a.H + h) * a.Dv + col;

  struct Operands {
    float4 wk[NTW], qs[NTW], kh[NTW], pc[NTW], us, os;
  };
  auto load = [&](Operands& o, int c) {
    const float* w = base + (size_t)c * stride;
#pragma unroll
    for (int t = 0; t < NTW; ++t) {
      const int tile = wave * NTW + t;
      if (DELTA)
        o.wk[t] = reinterpret_cast<const float4*>(w + lay.wk())[tile * 64 + lane];
      o.qs[t] = reinterpret_cast<const float4*>(w + lay.qs())[tile * 64 + lane];
      o.kh[t] = reinterpret_cast<const float4*>(w + lay.kh())[tile * 64 + lane];
      o.pc[t] = reinterpret_cast<const float4*>(w + lay.pc())[tile * 4 + g4];
    }
    o.us = reinterpret_cast<const float4*>(w + lay.us())[vt * 64 + lane];
    // (only the row this wavefront stores is used)
    o.os.x = (w + lay.os())[(vt * 64 + lane) * 4 + wave];
  };
  auto step = [&](const Operands& o, int c) {
    const int buf = c & 1;
    f32x4_v u = (f32x4_v){0.f, 0.f, 0.f, 0.f}, r = u;
    if (DELTA) {
#pragma unroll
      for (int t = 0; t < NTW; ++t) {
        const float wk[4] = {o.wk[t].x, o.wk[t].y, o.wk[t].z, o.wk[t].w};
#pragma unroll
        for (int i = 0; i < 4; ++i)
          u = __builtin_amdgcn_mfma_f32_16x16x4f32(wk[i], st[t][i], u, 0, 0, 0);
      }
    }
#pragma unroll
    for (int t = 0; t < NTW; ++t) {
      const float qs[4] = {o.qs[t].x, o.qs[t].y, o.qs[t].z, o.qs[t].w};
#pragma unroll
      for (int i = 0; i < 4; ++i)
        r = __builtin_amdgcn_mfma_f32_16x16x4f32(qs[i], st[t][i], r, 0, 0, 0);
    }
    if (DELTA) s_u[buf][wave][lane] = make_float4(u[0], u[1], u[2], u[3]);
    s_o[buf][wave][lane] = make_float4(r[0], r[1], r[2], r[3]);
    __syncthreads();
    float uu[4] = {o.us.x, o.us.y, o.us.z, o.us.w};
    if (DELTA) {
      const float4 p0 = s_u[buf][0][lane], p1 = s_u[buf][1][lane];
      const float4 p2 = s_u[buf][2][lane], p3 = s_u[buf][3][lane];
      uu[0] -= (p0.x + p1.x) + (p2.x + p3.x);
      uu[1] -= (p0.y + p1.y) + (p2.y + p3.y);
      uu[2] -= (p0.z + p1.z) + (p2.z + p3.z);
      uu[3] -= (p0.w + p1.w) + (p2.w + p3.w);
    }
#pragma unroll
    for (int t = 0; t < NTW; ++t) {
      const float kh[4] = {o.kh[t].x, o.kh[t].y, o.kh[t].z, o.kh[t].w};
      st[t][0] *= o.pc[t].x; st[t][1] *= o.pc[t].y;
      st[t][2] *= o.pc[t].z; st[t][3] *= o.pc[t].w;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        st[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kh[i], uu[i], st[t], 0, 0, 0);
    }
    // the read-out of tokens 4 g + wave
    float y = o.os.x;
#pragma unroll
    for (int p = 0; p < 4; ++p)
      y += reinterpret_cast<const float*>(&s_o[buf][p][lane])[wave];
    const int tok = kChunk * c + 4 * g4 + wave;
    if (tok < len && col_ok) out[(size_t)tok * a.H * a.Dv] = y;
  };
  // The operands of the next chunks are on their way while one is multiplied.
  constexpr int DEPTH = NTW <= 4 ? 4 : 2;
  Operands o[DEPTH];
#pragma unroll
  for (int i = 0; i + 1 < DEPTH; ++i) load(o[i], min(i, nc - 1));
  for (int c0 = 0; c0 < nc; c0 += DEPTH) {
#pragma unroll
    for (int i = 0; i < DEPTH; ++i) {
      if (c0 + i >= nc) break;
      load(o[(i + DEPTH - 1) % DEPTH], min(c0 + i + DEPTH - 1, nc - 1));
      step(o[i], c0 + i);
    }
  }
#pragma unroll
  for (int t = 0; t < NTW; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (wave * NTW + t) + 4 * g4 + i;
      if (col_ok && d < a.D) state[(size_t)d * a.Dv] = st[t][i];
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

// A wavefront per (token, head); with VEC 4 columns per lane, two heads of up to
// 128 columns per wavefront.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
recurrence_finish_kernel(RecArgs g) {
  T5D_GATED(g.gate);
  const t5d_recurrence& a = g.a;
  const int lane = threadIdx.x & 63;
  if constexpr (VEC) {
    const int64_t unit = (int64_t)blockIdx.x * 8 + (threadIdx.x >> 5);
    const bool on = unit < (int64_t)g.b.M * a.H;
    const int m = on ? unit / a.H : 0, h = on ? unit % a.H : 0;
    const int c = 4 * (lane & 31);
    const bool ok = on && c < a.Dv;
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f), z = o;
    if (ok) {
      o = *reinterpret_cast<const float4*>(g.wo + (size_t)unit * a.Dv + c);
      if (a.gate == T5D_GATE_SIGMOID_LOW) {
        z = *reinterpret_cast<const float4*>(a.low + (size_t)m * a.ld_low +
                                             a.off_low_gate + (size_t)h * a.Dv + c);
      } else {
        const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m * a.ld_proj +
                     a.off_gate + (size_t)h * a.Dv + c;
        z = make_float4(to_f32<T>(p[0]), to_f32<T>(p[1]), to_f32<T>(p[2]),
                        to_f32<T>(p[3]));
      }
    }
    float ss = lanes16_sum(o.x * o.x + o.y * o.y + o.z * o.z + o.w * o.w);
    const auto w = __builtin_amdgcn_permlane16_swap(
        __float_as_uint(ss), __float_as_uint(ss), false, false);
    ss = __uint_as_float(w[0]) + __uint_as_float(w[1]);
    if (!ok) return;
    const float inv = 1.0f / sqrtf(ss / (float)a.Dv + a.eps);
    const bool silu = a.gate != T5D_GATE_SIGMOID_LOW;
    auto put = [&](float v, float zz, float nw) {
      return v * inv * nw * (silu ? zz * sigmoid_f(zz) : sigmoid_f(zz));
    };
    const float y0 = put(o.x, z.x, a.norm[c]), y1 = put(o.y, z.y, a.norm[c + 1]);
    const float y2 = put(o.z, z.z, a.norm[c + 2]), y3 = put(o.w, z.w, a.norm[c + 3]);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)m * a.ld_out + (size_t)h * a.Dv + c;
    if constexpr (sizeof(T) == 2) {
      *reinterpret_cast<uint2*>(out) =
          make_uint2(pack_bf16x2(y0, y1), pack_bf16x2(y2, y3));
    } else {
      *reinterpret_cast<float4*>(out) = make_float4(y0, y1, y2, y3);
    }
    return;
  }
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

template <bool DELTA, typename T>
static void launch_chunks(hipStream_t s, const RecArgs& g) {
  const int vts = (g.a.Dv + 15) / 16, pairs = g.a.H * g.b.S;
  const dim3 grid(g.chunks, g.a.H, g.b.S), block(256);
  const dim3 chain((pairs + 7) / 8 * 8 * vts);
  const size_t lds = (size_t)kChunk * vts * 16 * sizeof(float);
#define T5D_CH(E_)                                                               \
  do {                                                                           \
    hipLaunchKernelGGL((recurrence_chunk_kernel<64 * E_, DELTA, T>), grid, block, \
                       lds, s, g);                                               \
    hipLaunchKernelGGL((recurrence_chain_kernel<E_, DELTA>), chain, block, 0, s, \
                       g);                                                       \
  } while (0)
  if (g.a.D <= 64) T5D_CH(1);
  else if (g.a.D <= 128) T5D_CH(2);
  else if (g.a.D <= 256) T5D_CH(4);
  else T5D_CH(8);
#undef T5D_CH
}

// Prepare and scan.
template <bool DELTA, typename T>
static void launch_token_by_token(hipStream_t s, const RecArgs& g) {
  const t5d_recurrence& a = g.a;
  const bool qkv = a.taps > 0 || a.unit;
  const int64_t units = (int64_t)g.b.M * ((qkv ? 2 * a.G + a.H : 0) + a.H);
  hipLaunchKernelGGL(recurrence_prepare_kernel<T>, dim3((unsigned)((units + 3) / 4)),
                     dim3(256), 0, s, g);
  if (qkv) {
    launch_scan<DELTA, float>(s, g, g.wq, g.wk, g.wv, a.G * a.D, a.G * a.D,
                              a.H * a.Dv, 1.f);
  } else {
    const T* p = reinterpret_cast<const T*>(a.proj);
    launch_scan<DELTA, T>(s, g, p + a.off_q, p + a.off_k, p + a.off_v, a.ld_proj,
                          a.ld_proj, a.ld_proj, a.q_scale);
  }
}

template <typename T>
static int run_portions(hipStream_t s, const RecArgs& g) {
  const t5d_recurrence& a = g.a;
  if (g.wchunk != nullptr) {
    if (a.delta) launch_chunks<true, T>(s, g);
    else launch_chunks<false, T>(s, g);
  } else if (a.delta) {
    launch_token_by_token<true, T>(s, g);
  } else {
    launch_token_by_token<false, T>(s, g);
  }
  T5D_CHECK_LAUNCH("recurrence (portions)");
  if (a.taps > 1) {
    hipLaunchKernelGGL(recurrence_conv_tail_kernel<T>,
                       dim3((g.C + 255) / 256, g.b.S), dim3(256), 0, s, g);
    T5D_CHECK_LAUNCH("recurrence (convolution tail)");
  }
  const int64_t heads = (int64_t)g.b.M * a.H;
  const bool vec = a.Dv % 4 == 0 && a.Dv <= 128 && a.ld_out % 4 == 0 &&
                   a.ld_low % 4 == 0 && a.off_low_gate % 4 == 0 &&
                   ((uintptr_t)a.out | (uintptr_t)a.low) % 16 == 0;
  if (vec)
    hipLaunchKernelGGL((recurrence_finish_kernel<T, true>),
                       dim3((unsigned)((heads + 7) / 8)), dim3(256), 0, s, g);
  else
    hipLaunchKernelGGL((recurrence_finish_kernel<T, false>),
                       dim3((unsigned)((heads + 3) / 4)), dim3(256), 0, s, g);
  T5D_CHECK_LAUNCH("recurrence (finish)");
  return T5D_OK;
}

static int64_t round4(int64_t n) { return (n + 3) / 4 * 4; }

// Floats of scratch of the un-chunked kernels.
static int64_t portion_floats(int64_t M, int H, int G, int D, int Dv) {
  return 2 * round4(M * G * D) + 2 * round4(M * H * Dv) + round4(M * H);
}

static int channel_pad(int D) {
  return D <= 64 ? 64 : D <= 128 ? 128 : D <= 256 ? 256 : 512;
}
static int64_t chunk_floats(int64_t M, int S, int H, int D, int Dv) {
  const ChunkLayout lay(channel_pad(D), (Dv + 15) / 16 * 16);
  return (int64_t)chunk_base(M, S) * H * (int64_t)lay.size();
}

// Portions from here on run in chunks.
constexpr int kChunkFrom = 24;

}  // namespace t5d

using namespace t5d;

extern "C" int64_t t5d_recurrence_workspace_bytes(int M, int S, int H, int G, int D,
                                                  int Dv) {
  if (M <= 0 || S < 0 || H <= 0 || G <= 0 || D <= 0 || Dv <= 0) return -1;
  return 4 * (portion_floats(M, H, G, D, Dv) +
              (S > 0 ? chunk_floats(M, S, H, D, Dv) : 0));
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
  T5D_REQUIRE(variant >= 0 && variant <= 3, T5D_EINVAL,
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
    g.wq = g.wk = g.wv = g.wbeta = g.wo = g.wchunk = nullptr;
    g.chunks = 0;
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
  const int64_t plain = portion_floats(b->M, a->H, a->G, a->D, a->Dv);
  g.chunks = (b->max_len + kChunk - 1) / kChunk;
  const bool fits =
      a->taps <= kChunkTaps && a->Dv <= 512 &&
      a->workspace_bytes >=
      4 * (plain + chunk_floats(b->M, b->S, a->H, a->D, a->Dv));
  T5D_REQUIRE(a->workspace_bytes >= 4 * plain && (variant != 3 || fits), T5D_EINVAL,
              "t5d_recurrence_run: a workspace of %lld bytes",
              (long long)a->workspace_bytes);
  g.wchunk = variant == 3 || (variant == 0 && fits && b->max_len >= kChunkFrom)
                 ? w + plain : nullptr;
  return a->dtype == T5D_BF16 ? run_portions<bf16_t>(s, g) : run_portions<float>(s, g);
}
