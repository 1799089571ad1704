// Causal softmax attention over a sliding window (or everything before), with
// grouped key / value heads, per-head norms of queries and keys, a linear
// distance bias and a sink in the denominator — for sequences that are fed in
// portions of any length.
//
// Keys and values live in a ring per (slot, key/value head): position p of the
// slot's sequence is row p % ring.  A launch first writes the new positions,
// then every query reads the ring; the ring holds at least window - 1 + portion
// rows, so nothing a query of the portion needs has been overwritten, and rows
// left by an earlier sequence of the slot lie outside every mask.  Rows are
// padded with zeros to HP (32, 64, 128 or 256 elements), ring is a multiple of
// 64: a tile of 64 keys that starts at a multiple of 64 is consecutive memory.
//
// Three kernels attend:
//   * rows (bfloat16, portions): a tile is 128 (token, head of the group) pairs,
//     so grouped heads share the keys and values that a workgroup stages in LDS.
//     Scores are formed transposed, S^T = K Q^T: a lane then holds 4 consecutive
//     keys of ONE query, which is the operand order of the second product
//     O^T = V^T P^T up to a permutation of the keys that the V^T reads follow —
//     the weights never cross lanes.  They enter that product as two bfloat16
//     terms (value + remainder), which keeps them to 16 bits of mantissa.
//   * step (bfloat16, one new token per sequence): norms, the ring update and the
//     attention in one kernel, a workgroup per (sequence, key/value head, part of
//     the keys); scores on the matrix cores with the group's heads as the columns,
//     weights times values in float32 on the vector ALUs, wavefronts merged
//     through LDS, parts through a small second kernel.
//   * wave (float32, and sizes the other two do not cover): one wavefront per
//     (token, head), all in float32.
#include "common.h"
#include "gemm_tiles.h"

namespace t5d {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNoMax = -1e30f;  // running maximum before the first key

struct WinArgs {
  t5d_window_attention a;
  t5d_ragged b;
  int HP, gs, splits;
  float* parts;  // [S, G, splits, gs, HP + 2]
  const int32_t* gate;
  // window_rows_kernel over a span instead of rings: position first[s] + i of
  // portion s is row off[s] + i, rows ld_kv apart, a head's HP columns side by side
  const int32_t *span_off, *span_first;
  int ld_kv;
};

// ---- norms of the new queries and keys, ring update ------------------------------
// One wavefront per (token, head vector): H queries, G keys, G values.
template <typename T>
__global__ void __launch_bounds__(256)
window_append_kernel(WinArgs g) {
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  const int lane = threadIdx.x & 63;
  const int nvec = a.H + 2 * a.G;
  const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (int64_t)g.b.M * nvec) return;
  const int m = unit / nvec, vec = unit % nvec;
  const int seq = g.b.tok_seq[m];
  const int row = g.b.tok_pos[m] % a.ring;
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m * a.ld_proj;
  T* dst;
  const float* w = nullptr;
  int n = a.D;
  if (vec < a.H) {
    p += a.off_q + vec * a.D;
    w = a.q_norm;
    dst = reinterpret_cast<T*>(a.q_rows) + ((size_t)m * a.H + vec) * g.HP;
  } else {
    const bool key = vec < a.H + a.G;
    const int h = vec - a.H - (key ? 0 : a.G);
    const size_t r =
        ((size_t)g.b.seq_slot[seq] * a.G + h) * a.ring + row;
    dst = reinterpret_cast<T*>(key ? a.key_ring : a.value_ring) + r * g.HP;
    if (key) w = a.k_norm; else n = a.Dv;
    p += key ? a.off_k + h * a.D : a.off_v + h * a.Dv;
  }
  float inv = 1.f;
  if (w != nullptr) {
    float ss = 0.f;
    for (int i = lane; i < n; i += 64) {
      const float v = to_f32<T>(p[i]);
      ss = fmaf(v, v, ss);
    }
    inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps);
  }
  for (int i = lane; i < g.HP; i += 64) {
    float v = 0.f;
    if (i < n) {
      v = to_f32<T>(p[i]);
      if (w != nullptr) v = v * inv * w[i];
    }
    Act<T>::store(dst + i, v);
  }
}

// The same for bfloat16 rows of whole 16-byte pieces: HP / 8 lanes per vector.
__global__ void __launch_bounds__(256)
window_append_vec_kernel(WinArgs g) {
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  const int lpv = g.HP / 8;  // 4, 8, 16 or 32: a power of two
  const int nvec = a.H + 2 * a.G;
  const int64_t unit = (int64_t)blockIdx.x * (256 / lpv) + threadIdx.x / lpv;
  const bool on = unit < (int64_t)g.b.M * nvec;
  const int m = on ? unit / nvec : 0, vec = on ? unit % nvec : 0;
  const int c = 8 * (threadIdx.x % lpv);
  const bool query = vec < a.H, key = !query && vec < a.H + a.G;
  const int h = query ? vec : vec - a.H - (key ? 0 : a.G);
  const int n = query || key ? a.D : a.Dv;
  const bf16_t* p = reinterpret_cast<const bf16_t*>(a.proj) + (size_t)m * a.ld_proj +
                    (query ? a.off_q + h * a.D : key ? a.off_k + h * a.D
                                                     : a.off_v + h * a.Dv);
  const float* w = query ? a.q_norm : key ? a.k_norm : nullptr;
  uint4 v = make_uint4(0, 0, 0, 0);
  if (on && c < n) v = *reinterpret_cast<const uint4*>(p + c);
  if (w != nullptr) {
    float f[8];
    unpack16(v, f);
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(f[e], f[e], ss);
    for (int step = 1; step < lpv; step *= 2) ss += __shfl_xor(ss, step, 64);
    const float inv = 1.0f / sqrtf(ss / (float)n + a.eps);
    if (c < n) {
      const float4 x = *reinterpret_cast<const float4*>(w + c);
      const float4 y = *reinterpret_cast<const float4*>(w + c + 4);
      v.x = pack_bf16x2(f[0] * inv * x.x, f[1] * inv * x.y);
      v.y = pack_bf16x2(f[2] * inv * x.z, f[3] * inv * x.w);
      v.z = pack_bf16x2(f[4] * inv * y.x, f[5] * inv * y.y);
      v.w = pack_bf16x2(f[6] * inv * y.z, f[7] * inv * y.w);
    }
  }
  if (!on) return;
  bf16_t* dst;
  if (query) {
    dst = reinterpret_cast<bf16_t*>(a.q_rows) + ((size_t)m * a.H + h) * g.HP;
  } else {
    const size_t r = ((size_t)g.b.seq_slot[g.b.tok_seq[m]] * a.G + h) * a.ring +
                     g.b.tok_pos[m] % a.ring;
    dst = reinterpret_cast<bf16_t*>(key ? a.key_ring : a.value_ring) + r * g.HP;
  }
  *reinterpret_cast<uint4*>(dst + c) = v;
}

// ---- float32 / any size -----------------------------------------------------------
template <typename T, int NV>
__global__ void __launch_bounds__(64)
window_wave_kernel(WinArgs g) {
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  extern __shared__ float lds[];
  float* s_q = lds;           // [HP]
  float* s_p = lds + g.HP;    // [64]
  const int lane = threadIdx.x;
  const int m = blockIdx.x, h = blockIdx.y, kv = h / g.gs;
  const int seq = g.b.tok_seq[m], i = g.b.tok_pos[m];
  const size_t base = ((size_t)g.b.seq_slot[seq] * a.G + kv) * a.ring;
  const T* K = reinterpret_cast<const T*>(a.key_ring) + base * g.HP;
  const T* V = reinterpret_cast<const T*>(a.value_ring) + base * g.HP;
  const T* q = reinterpret_cast<const T*>(a.q_rows) + ((size_t)m * a.H + h) * g.HP;
  for (int d = lane; d < g.HP; d += 64) s_q[d] = to_f32<T>(q[d]);
  __syncthreads();
  const float slope = a.slopes != nullptr ? a.slopes[h] : 0.f;
  float mx = kNoMax, l = 0.f;
  if (a.sink != nullptr) {
    mx = a.sink[h] * kLog2e;
    l = 1.f;
  }
  float acc[NV];
#pragma unroll
  for (int n = 0; n < NV; ++n) acc[n] = 0.f;
  const int lo = a.window > 0 ? max(0, i - a.window + 1) : 0;
  for (int j0 = lo; j0 <= i; j0 += 64) {
    const int j = j0 + lane;
    float s = -INFINITY;
    if (j <= i) {
      const T* k = K + (size_t)(j % a.ring) * g.HP;
      float dot = 0.f;
      constexpr int E = Act<T>::kElemsPer16B;
      for (int d = 0; d < g.HP; d += E) {
        float f[E];
        unpack16(*reinterpret_cast<const uint4*>(k + d), f);
#pragma unroll
        for (int e = 0; e < E; ++e) dot = fmaf(f[e], s_q[d + e], dot);
      }
      s = (dot * a.scale - slope * (float)(i - j)) * kLog2e;
    }
    const float top = fmaxf(mx, wave_max(s));
    const float alpha = exp2f(mx - top);
    const float p = exp2f(s - top);
    mx = top;
    l = l * alpha + wave_sum(p);
    __syncthreads();
    s_p[lane] = p;
    __syncthreads();
    const int cnt = min(64, i - j0 + 1);
#pragma unroll
    for (int n = 0; n < NV; ++n) acc[n] *= alpha;
    for (int jj = 0; jj < cnt; ++jj) {
      const T* v = V + (size_t)((j0 + jj) % a.ring) * g.HP;
      const float w = s_p[jj];
#pragma unroll
      for (int n = 0; n < NV; ++n)
        if (lane + 64 * n < a.Dv) acc[n] = fmaf(w, to_f32<T>(v[lane + 64 * n]), acc[n]);
    }
  }
  T* o = reinterpret_cast<T*>(a.out) + (size_t)m * a.ld_out + (size_t)h * a.Dv;
#pragma unroll
  for (int n = 0; n < NV; ++n)
    if (lane + 64 * n < a.Dv) Act<T>::store(o + lane + 64 * n, acc[n] / l);
}

// ---- portions, bfloat16 -------------------------------------------------------------
__device__ __forceinline__ f32x4_v mfma(const Frag& x, const Frag& y, f32x4_v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.v, y.v, c, 0, 0, 0);
}

template <int DT, bool SPAN = false>
__global__ void __launch_bounds__(256, DT <= 4 ? 2 : 1)
window_rows_kernel(WinArgs g) {
  constexpr int HP = DT * 32, VT = DT * 2, KB = 64, MT = 2;
  constexpr int KS = HP + 8, VS = KB + 8;        // LDS row strides (elements)
  constexpr int NVP = (VT + 3) / 4;              // V pair pieces per thread
  __shared__ __align__(16) bf16_t s_k[KB * KS];  // [key][dim]
  __shared__ __align__(16) bf16_t s_v[HP * VS];  // [dim][key]
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  const int seq = blockIdx.y, kv = blockIdx.z, gs = g.gs;
  const int off = g.b.seq_off[seq];
  const int rows = (g.b.seq_off[seq + 1] - off) * gs;
  const int r0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * (64 * MT);
  if (r0 >= rows) return;
  const int start = g.b.seq_start[seq];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n16 = lane & 15, gq = lane >> 4;
  const int W = a.window > 0 ? a.window : (1 << 30);
  const size_t base = SPAN ? (size_t)g.span_off[seq] * g.ld_kv + (size_t)kv * HP
                           : ((size_t)g.b.seq_slot[seq] * a.G + kv) * a.ring * HP;
  const bf16_t* K = reinterpret_cast<const bf16_t*>(a.key_ring) + base;
  const bf16_t* V = reinterpret_cast<const bf16_t*>(a.value_ring) + base;
  const int ld_kv = SPAN ? g.ld_kv : HP;
  const int first = SPAN ? g.span_first[seq] : 0;

  const float scale2 = a.scale * kLog2e;
  int pos[MT], tok[MT], head[MT];
  float slope2[MT], mx[MT], l[MT];
  Frag qf[MT][DT];
  const int rw = r0 + wave * 16 * MT;  // the wavefront's first row
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int r = min(rw + 16 * mt + n16, rows - 1);  // past the end: not stored
    const int t = r / gs;
    head[mt] = kv * gs + (r - t * gs);
    tok[mt] = off + t;
    pos[mt] = start + t;
    slope2[mt] = a.slopes != nullptr ? a.slopes[head[mt]] * kLog2e : 0.f;
    mx[mt] = a.sink != nullptr ? a.sink[head[mt]] * kLog2e : kNoMax;
    l[mt] = a.sink != nullptr && gq == 0 ? 1.f : 0.f;
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q_rows) +
                      ((size_t)tok[mt] * a.H + head[mt]) * HP + 8 * gq;
#pragma unroll
    for (int kk = 0; kk < DT; ++kk)
      qf[mt][kk].u = *reinterpret_cast<const uint4*>(q + 32 * kk);
  }
  f32x4_v o[VT][MT];
#pragma unroll
  for (int vt = 0; vt < VT; ++vt)
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) o[vt][mt] = (f32x4_v){0.f, 0.f, 0.f, 0.f};

  const int i_lo = start + r0 / gs;
  const int i_hi = start + min(r0 + 64 * MT - 1, rows - 1) / gs;
  const bool wave_on = rw < rows;
  const int wi_lo = start + min(rw, rows - 1) / gs;
  const int wi_hi = start + min(rw + 16 * MT - 1, rows - 1) / gs;
  const int j_begin = max(0, i_lo - W + 1) & ~(KB - 1);

  uint4 kr[DT], va[NVP], vb[NVP];
  const int kpiece = threadIdx.x % (HP / 8), krow = threadIdx.x / (HP / 8);
  constexpr int KRS = 256 / (HP / 8);            // key rows per pass
  const int vpair = threadIdx.x & 31, vcol = threadIdx.x >> 5;
  auto fetch = [&](int jt) {
    const size_t r = (size_t)(SPAN ? jt - first : jt % a.ring);
#pragma unroll
    for (int i = 0; i < DT; ++i)
      kr[i] = *reinterpret_cast<const uint4*>(K + (r + krow + KRS * i) * ld_kv +
                                              8 * kpiece);
#pragma unroll
    for (int i = 0; i < NVP; ++i)
      if (vcol + 8 * i < HP / 8) {
        const bf16_t* v = V + (r + 2 * vpair) * ld_kv + 8 * (vcol + 8 * i);
        va[i] = *reinterpret_cast<const uint4*>(v);
        vb[i] = *reinterpret_cast<const uint4*>(v + ld_kv);
      }
  };
  fetch(j_begin);
  for (int jt = j_begin; jt <= i_hi; jt += KB) {
    __syncthreads();  // the previous tile has been read
#pragma unroll
    for (int i = 0; i < DT; ++i)
      *reinterpret_cast<uint4*>(s_k + (krow + KRS * i) * KS + 8 * kpiece) = kr[i];
#pragma unroll
    for (int i = 0; i < NVP; ++i)
      if (vcol + 8 * i < HP / 8) {
        // keys 2p and 2p + 1 of 8 dims: one word per dim
        uint32_t* dst = reinterpret_cast<uint32_t*>(
            s_v + (size_t)(8 * (vcol + 8 * i)) * VS + 2 * vpair);
        auto put = [&](int e, uint32_t x, uint32_t y) {
          dst[(2 * e) * (VS / 2)] = (x & 0xFFFFu) | (y << 16);
          dst[(2 * e + 1) * (VS / 2)] = (x >> 16) | (y & 0xFFFF0000u);
        };
        put(0, va[i].x, vb[i].x);
        put(1, va[i].y, vb[i].y);
        put(2, va[i].z, vb[i].z);
        put(3, va[i].w, vb[i].w);
      }
    __syncthreads();
    if (jt + KB <= i_hi) fetch(jt + KB);
    if (!wave_on || jt > wi_hi || jt + KB - 1 <= wi_lo - W) continue;

    f32x4_v s[4][MT];
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) s[t][mt] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < DT; ++kk)
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        Frag kf;
        kf.u = *reinterpret_cast<const uint4*>(s_k + (16 * t + n16) * KS + 32 * kk +
                                               8 * gq);
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) s[t][mt] = mfma(kf, qf[mt][kk], s[t][mt]);
      }
    const bool edge = !(jt + KB - 1 <= wi_lo && jt > wi_hi - W);
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      const int d0 = pos[mt] - jt - 4 * gq;  // distance to this lane's first key
      float top = mx[mt];
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int dist = d0 - 16 * t - i;
          float v = fmaf(s[t][mt][i], scale2, -slope2[mt] * (float)dist);
          if (edge) v = dist >= 0 && dist < W ? v : -INFINITY;
          s[t][mt][i] = v;
          top = fmaxf(top, v);
        }
      top = rows_max(top);
      const float alpha = __builtin_amdgcn_exp2f(mx[mt] - top);
      mx[mt] = top;
      float sum = 0.f;
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = __builtin_amdgcn_exp2f(s[t][mt][i] - top);
          s[t][mt][i] = p;
          sum += p;
        }
      l[mt] = l[mt] * alpha + sum;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
#pragma unroll
        for (int i = 0; i < 4; ++i) o[vt][mt][i] *= alpha;
    }
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      // weights of keys {16 (2 kb) + 4 gq + 0..3, 16 (2 kb + 1) + 4 gq + 0..3}
      Frag hi[MT], lo[MT];
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        uint32_t h[4], r[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float p0 = s[2 * kb + (e >> 1)][mt][2 * (e & 1)];
          const float p1 = s[2 * kb + (e >> 1)][mt][2 * (e & 1) + 1];
          h[e] = pack_bf16x2(p0, p1);
          r[e] = pack_bf16x2(p0 - bf16lo_to_f32(h[e]), p1 - bf16hi_to_f32(h[e]));
        }
        hi[mt].u = make_uint4(h[0], h[1], h[2], h[3]);
        lo[mt].u = make_uint4(r[0], r[1], r[2], r[3]);
      }
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const bf16_t* v = s_v + (16 * vt + n16) * VS + 32 * kb + 4 * gq;
        const uint2 x = *reinterpret_cast<const uint2*>(v);
        const uint2 y = *reinterpret_cast<const uint2*>(v + 16);
        Frag vf;
        vf.u = make_uint4(x.x, x.y, y.x, y.y);
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) {
          o[vt][mt] = mfma(vf, hi[mt], o[vt][mt]);
          o[vt][mt] = mfma(vf, lo[mt], o[vt][mt]);
        }
      }
    }
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const float inv = 1.0f / rows_sum(l[mt]);
    if (rw + 16 * mt + n16 >= rows) continue;
    bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + (size_t)tok[mt] * a.ld_out +
                  (size_t)head[mt] * a.Dv;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int d = 16 * vt + 4 * gq;
      if ((a.Dv & 3) == 0) {
        if (d < a.Dv)
          *reinterpret_cast<uint2*>(out + d) =
              make_uint2(pack_bf16x2(o[vt][mt][0] * inv, o[vt][mt][1] * inv),
                         pack_bf16x2(o[vt][mt][2] * inv, o[vt][mt][3] * inv));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d + i < a.Dv) out[d + i] = f32_to_bf16(o[vt][mt][i] * inv);
      }
    }
  }
}

// ---- one new token per sequence, bfloat16 ----------------------------------------------
__device__ __forceinline__ void wave_lds_fence() {
  // LDS operations of a wavefront complete in order; this only keeps the
  // compiler from moving one lane's read above another lane's write.
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
}

template <int DT, int GS>
__global__ void __launch_bounds__(256)
window_step_kernel(WinArgs g) {
  constexpr int HP = DT * 32;
  constexpr int QS = HP + 8;
  constexpr int LPR = HP / 8;       // lanes on one value row
  constexpr int KPI = 64 / LPR;     // keys per value load
  __shared__ __align__(16) bf16_t s_q[16 * QS];
  __shared__ __align__(16) float s_w[4][64 * GS];  // weights [key][head]
  __shared__ float s_alpha[4][16];
  __shared__ float s_m[4][16], s_l[4][16];
  __shared__ __align__(16) float s_o[4][GS * HP];
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  const int seq = blockIdx.x / a.G, kv = blockIdx.x % a.G, part = blockIdx.y;
  const int gs = g.gs;              // <= GS
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n16 = lane & 15, gq = lane >> 4;
  const int i = g.b.seq_start[seq];
  const int W = a.window > 0 ? a.window : (1 << 30);
  const size_t base = ((size_t)g.b.seq_slot[seq] * a.G + kv) * a.ring;
  bf16_t* K = reinterpret_cast<bf16_t*>(a.key_ring) + base * HP;
  bf16_t* V = reinterpret_cast<bf16_t*>(a.value_ring) + base * HP;

  // The group's queries -> LDS, the new key and value -> ring (every part
  // writes the same bytes there).  Vectors 0 .. gs-1: queries, gs: key, gs + 1:
  // value; rows gs .. 15 of the query tile are zero.
  {
    const bf16_t* p = reinterpret_cast<const bf16_t*>(a.proj) + (size_t)seq * a.ld_proj;
    for (int vec = wave; vec < 18; vec += 4) {
      const bool query = vec < 16, key = vec == 16;
      const bool live = !query || vec < gs;
      const int n = vec == 17 ? a.Dv : a.D;
      const bf16_t* src = p + (query ? a.off_q + (kv * gs + min(vec, gs - 1)) * a.D
                               : key ? a.off_k + kv * a.D
                                     : a.off_v + kv * a.Dv);
      const float* w = query ? a.q_norm : key ? a.k_norm : nullptr;
      float f[(HP + 63) / 64];
      float ss = 0.f;
#pragma unroll
      for (int u = 0; u < (HP + 63) / 64; ++u) {
        const int d = lane + 64 * u;
        f[u] = live && d < n ? bf16_to_f32(src[d]) : 0.f;
        ss = fmaf(f[u], f[u], ss);
      }
      const float inv =
          w != nullptr ? 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps) : 1.f;
      bf16_t* dst = query ? s_q + vec * QS
                          : (key ? K : V) + (size_t)(i % a.ring) * HP;
#pragma unroll
      for (int u = 0; u < (HP + 63) / 64; ++u) {
        const int d = lane + 64 * u;
        if (d < HP)
          dst[d] = f32_to_bf16(w != nullptr && d < n ? f[u] * inv * w[d] : f[u]);
      }
    }
    // the key and value rows are in memory before any wavefront reads the ring
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  }
  __syncthreads();

  Frag qf[DT];
#pragma unroll
  for (int kk = 0; kk < DT; ++kk)
    qf[kk].u = *reinterpret_cast<const uint4*>(s_q + n16 * QS + 32 * kk + 8 * gq);
  const int head = kv * gs + min(n16, gs - 1);
  const float scale2 = a.scale * kLog2e;
  const float slope2 = a.slopes != nullptr ? a.slopes[head] * kLog2e : 0.f;
  float mx = kNoMax, l = 0.f;
  float acc[GS][8];
#pragma unroll
  for (int h = 0; h < GS; ++h)
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[h][e] = 0.f;
  const int j_begin = max(0, i - W + 1) & ~63;
  const int vsub = lane / LPR, vpiece = lane % LPR;

  for (int jt = j_begin + 64 * (part + g.splits * wave); jt <= i;
       jt += 64 * 4 * g.splits) {
    const size_t r = (size_t)(jt % a.ring);
    const bf16_t* kt = K + r * HP;
    const bf16_t* vt = V + r * HP;
    Frag kf[4][DT];
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int kk = 0; kk < DT; ++kk)
        kf[t][kk].u = *reinterpret_cast<const uint4*>(
            kt + (size_t)(16 * t + n16) * HP + 32 * kk + 8 * gq);
    uint4 vr[8];  // the first value rows travel with the keys
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (u * KPI < 64)
        vr[u] = *reinterpret_cast<const uint4*>(
            vt + (size_t)(u * KPI + vsub) * HP + 8 * vpiece);
    f32x4_v s[4];
    float top = mx;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      s[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < DT; ++kk) s[t] = mfma(kf[t][kk], qf[kk], s[t]);
    }
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int dist = i - jt - 16 * t - 4 * gq - e;
        const float v = fmaf(s[t][e], scale2, -slope2 * (float)dist);
        s[t][e] = dist >= 0 && dist < W ? v : -INFINITY;
        top = fmaxf(top, s[t][e]);
      }
    top = rows_max(top);
    const float alpha = __builtin_amdgcn_exp2f(mx - top);
    mx = top;
    float sum = 0.f;
    wave_lds_fence();  // the previous tile's weights have been read
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float p = __builtin_amdgcn_exp2f(s[t][e] - top);
        sum += p;
        if (n16 < GS) s_w[wave][(16 * t + 4 * gq + e) * GS + n16] = p;
      }
    l = l * alpha + sum;
    if (gq == 0) s_alpha[wave][n16] = alpha;
    wave_lds_fence();
#pragma unroll
    for (int h = 0; h < GS; ++h) {
      const float al = s_alpha[wave][h];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[h][e] *= al;
    }
#pragma unroll
    for (int u0 = 0; u0 * KPI < 64; u0 += 8) {
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        if ((u0 + u) * KPI >= 64) continue;
        if (u0 > 0)
          vr[u] = *reinterpret_cast<const uint4*>(
              vt + (size_t)((u0 + u) * KPI + vsub) * HP + 8 * vpiece);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        if ((u0 + u) * KPI >= 64) continue;
        float f[8];
        unpack16(vr[u], f);
        const float* w = &s_w[wave][((u0 + u) * KPI + vsub) * GS];
#pragma unroll
        for (int h = 0; h < GS; ++h) {
          const float p = w[h];
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[h][e] = fmaf(p, f[e], acc[h][e]);
        }
      }
    }
  }
  // Sum over the lanes that took other keys of the same value piece, then the
  // wavefronts' results meet in LDS.
#pragma unroll
  for (int h = 0; h < GS; ++h)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float v = acc[h][e];
#pragma unroll
      for (int step = LPR; step < 64; step *= 2) v += __shfl_xor(v, step, 64);
      acc[h][e] = v;
    }
  if (vsub == 0) {
#pragma unroll
    for (int h = 0; h < GS; ++h)
#pragma unroll
      for (int e = 0; e < 8; ++e) s_o[wave][h * HP + 8 * vpiece + e] = acc[h][e];
  }
  const float lt = rows_sum(l);
  if (gq == 0) {
    s_m[wave][n16] = mx;
    s_l[wave][n16] = lt;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < gs * HP; e += 256) {
    const int h = e / HP, d = e - h * HP;
    if (d >= a.Dv) continue;
    float top = fmaxf(fmaxf(s_m[0][h], s_m[1][h]), fmaxf(s_m[2][h], s_m[3][h]));
    const bool last = g.splits == 1;
    const float sink2 = last && a.sink != nullptr ? a.sink[kv * gs + h] * kLog2e : kNoMax;
    top = fmaxf(top, sink2);
    float num = 0.f, den = last && a.sink != nullptr ? exp2f(sink2 - top) : 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float c = exp2f(s_m[w][h] - top);
      num = fmaf(c, s_o[w][e], num);
      den = fmaf(c, s_l[w][h], den);
    }
    if (last) {
      reinterpret_cast<bf16_t*>(a.out)[(size_t)seq * a.ld_out +
                                       (size_t)(kv * gs + h) * a.Dv + d] =
          f32_to_bf16(num / den);
    } else {
      float* o = g.parts + (((size_t)blockIdx.x * g.splits + part) * gs + h) * (HP + 2);
      o[d] = num;
      if (d == 0) {
        o[HP] = top;
        o[HP + 1] = den;
      }
    }
  }
}

// The parts of window_step_kernel: one wavefront per (sequence, head).
__global__ void __launch_bounds__(64)
window_merge_kernel(WinArgs g) {
  T5D_GATED(g.gate);
  const t5d_window_attention& a = g.a;
  const int seq = blockIdx.x / a.H, h = blockIdx.x % a.H;
  const int kv = h / g.gs, hh = h % g.gs;
  const size_t step = (size_t)g.gs * (g.HP + 2);
  const float* p = g.parts + ((size_t)seq * a.G + kv) * g.splits * step +
                   (size_t)hh * (g.HP + 2);
  const float sink2 = a.sink != nullptr ? a.sink[h] * kLog2e : kNoMax;
  float top = sink2;
  for (int s = 0; s < g.splits; ++s) top = fmaxf(top, p[s * step + g.HP]);
  float den = a.sink != nullptr ? exp2f(sink2 - top) : 0.f;
  for (int s = 0; s < g.splits; ++s)
    den = fmaf(exp2f(p[s * step + g.HP] - top), p[s * step + g.HP + 1], den);
  for (int d = threadIdx.x; d < a.Dv; d += 64) {
    float num = 0.f;
    for (int s = 0; s < g.splits; ++s)
      num = fmaf(exp2f(p[s * step + g.HP] - top), p[s * step + d], num);
    reinterpret_cast<bf16_t*>(a.out)[(size_t)seq * a.ld_out + (size_t)h * a.Dv + d] =
        f32_to_bf16(num / den);
  }
}

constexpr int kMaxSplits = 16;

static int step_splits(const t5d_window_attention& a, int S) {
  const int span = a.window > 0 ? min(a.window, a.ring) : a.ring;
  int n = 1;
  while (n < kMaxSplits && S * a.G * n < 256 && span >= 512 * n) n *= 2;
  return n;
}

// The step kernel's template sizes: heads per group rounded up, 0 if it does
// not cover the shape.
static int step_group(int gs, int HP) {
  if (HP > 256 || gs > 16) return 0;
  int n = 1;
  while (n < gs) n *= 2;
  return n * HP <= 2048 ? n : 0;
}

template <typename T>
static void launch_wave(hipStream_t s, const WinArgs& g) {
  const int nv = (g.a.Dv + 63) / 64;
  const dim3 grid(g.b.M, g.a.H), block(64);
  const size_t lds = (g.HP + 64) * sizeof(float);
#define T5D_WW(N_) \
  hipLaunchKernelGGL((window_wave_kernel<T, N_>), grid, block, lds, s, g)
  if (nv <= 1) T5D_WW(1);
  else if (nv <= 2) T5D_WW(2);
  else if (nv <= 4) T5D_WW(4);
  else T5D_WW(16);
#undef T5D_WW
}

static WinArgs win_args(const t5d_window_attention& a, const t5d_ragged& b, int HP) {
  WinArgs g = {};
  g.a = a; g.b = b;
  g.HP = HP; g.gs = a.H / a.G; g.splits = 1;
  g.parts = (float*)a.workspace;
  g.gate = tls_gate;
  return g;
}

int launch_window_span(hipStream_t s, const t5d_window_attention& a,
                       const t5d_ragged& b, const t5d_span& span, int ld_kv) {
  WinArgs g = win_args(a, b, t5d_window_head_pad(a.D, a.Dv));
  g.span_off = span.off; g.span_first = span.first; g.ld_kv = ld_kv;
  const int64_t tiles = ((int64_t)b.max_len * g.gs + 127) / 128;
  const dim3 grid((unsigned)tiles, b.S, a.G), block(256);
#define T5D_SPAN(DT_) \
  hipLaunchKernelGGL((window_rows_kernel<DT_, true>), grid, block, 0, s, g)
  if (g.HP == 32) T5D_SPAN(1);
  else if (g.HP == 64) T5D_SPAN(2);
  else if (g.HP == 128) T5D_SPAN(4);
  else T5D_SPAN(8);
#undef T5D_SPAN
  T5D_CHECK_LAUNCH("window attention (span)");
  return T5D_OK;
}

int launch_window_wave(hipStream_t s, const t5d_window_attention& a,
                       const t5d_ragged& b, int HP) {
  const WinArgs g = win_args(a, b, HP);
  if (a.dtype == T5D_BF16) launch_wave<bf16_t>(s, g);
  else launch_wave<float>(s, g);
  T5D_CHECK_LAUNCH("window attention (wave)");
  return T5D_OK;
}

}  // namespace t5d

using namespace t5d;

extern "C" int t5d_window_head_pad(int D, int Dv) {
  const int n = D > Dv ? D : Dv;
  if (n <= 0 || n > 1024) return -1;
  for (int p = 32; p <= 256; p *= 2)
    if (n <= p) return p;
  return (n + 63) / 64 * 64;
}

extern "C" int64_t t5d_window_workspace_bytes(int S, int H, int D, int Dv) {
  const int hp = t5d_window_head_pad(D, Dv);
  if (hp < 0 || S <= 0 || H <= 0) return -1;
  return (int64_t)S * H * kMaxSplits * (hp + 2) * 4;
}

extern "C" int t5d_window_attention_run(void* stream, const t5d_window_attention* a,
                                        const t5d_ragged* b, int variant) {
  T5D_REQUIRE(a && b, T5D_EINVAL, "t5d_window_attention_run: null arguments");
  T5D_REQUIRE(a->dtype == T5D_F32 || a->dtype == T5D_BF16, T5D_EINVAL,
              "t5d_window_attention_run: dtype %d", a->dtype);
  T5D_REQUIRE(a->H > 0 && a->G > 0 && a->H % a->G == 0 && a->D > 0 && a->Dv > 0 &&
                  a->window >= 0 && a->H <= 65535 && a->G <= 65535,
              T5D_EINVAL, "t5d_window_attention_run: H=%d G=%d D=%d Dv=%d window=%d",
              a->H, a->G, a->D, a->Dv, a->window);
  T5D_REQUIRE(a->proj && a->key_ring && a->value_ring && a->q_rows && a->out &&
                  b->tok_pos && b->tok_seq && b->seq_off && b->seq_start &&
                  b->seq_slot,
              T5D_EINVAL, "t5d_window_attention_run: null buffer");
  T5D_REQUIRE(b->M > 0 && b->S > 0 && b->S <= 65535 && b->max_len > 0 &&
                  b->max_len <= b->M,
              T5D_EINVAL, "t5d_window_attention_run: M=%d S=%d max_len=%d", b->M,
              b->S, b->max_len);
  T5D_REQUIRE(a->ring > 0 && a->ring % 64 == 0 &&
                  (a->window == 0 || a->ring >= a->window - 1 + b->max_len),
              T5D_EINVAL,
              "t5d_window_attention_run: a ring of %d rows for a window of %d and "
              "portions of %d (multiple of 64, at least window - 1 + portion)",
              a->ring, a->window, b->max_len);
  T5D_REQUIRE(variant >= 0 && variant <= 3, T5D_EINVAL,
              "t5d_window_attention_run: variant %d", variant);
  WinArgs g = win_args(*a, *b, t5d_window_head_pad(a->D, a->Dv));
  T5D_REQUIRE(g.HP > 0, T5D_ELIMIT, "t5d_window_attention_run: head size %d / %d",
              a->D, a->Dv);
  hipStream_t s = as_stream(stream);
  const bool bf16 = a->dtype == T5D_BF16;
  const int GS = step_group(g.gs, g.HP);
  const bool can_step = bf16 && b->max_len == 1 && b->M == b->S && GS > 0;
  const bool can_rows = bf16 && g.HP <= 256 && a->ld_out % 4 == 0;
  T5D_REQUIRE((variant != 1 || can_step) && (variant != 2 || can_rows), T5D_EINVAL,
              "t5d_window_attention_run: variant %d does not cover this call",
              variant);
  if (variant == 1 || (variant == 0 && can_step)) {
    if (g.parts != nullptr) g.splits = step_splits(*a, b->S);
    const dim3 grid(b->S * a->G, g.splits), block(256);
#define T5D_WS(DT_, GS_)                                                     \
  if (g.HP == 32 * DT_ && GS == GS_)                                         \
    hipLaunchKernelGGL((window_step_kernel<DT_, GS_>), grid, block, 0, s, g)
    T5D_WS(1, 1); T5D_WS(1, 2); T5D_WS(1, 4); T5D_WS(1, 8); T5D_WS(1, 16);
    T5D_WS(2, 1); T5D_WS(2, 2); T5D_WS(2, 4); T5D_WS(2, 8); T5D_WS(2, 16);
    T5D_WS(4, 1); T5D_WS(4, 2); T5D_WS(4, 4); T5D_WS(4, 8); T5D_WS(4, 16);
    T5D_WS(8, 1); T5D_WS(8, 2); T5D_WS(8, 4); T5D_WS(8, 8);
#undef T5D_WS
    T5D_CHECK_LAUNCH("window attention (step)");
    if (g.splits > 1) {
      hipLaunchKernelGGL(window_merge_kernel, dim3(b->S * a->H), dim3(64), 0, s, g);
      T5D_CHECK_LAUNCH("window attention (merge)");
    }
    return T5D_OK;
  }
  const int64_t units = (int64_t)b->M * (a->H + 2 * a->G);
  const dim3 agrid((unsigned)((units + 3) / 4)), ablock(256);
  const bool pieces =
      bf16 && g.HP <= 256 &&
      ((a->D | a->Dv | a->off_q | a->off_k | a->off_v | a->ld_proj) & 7) == 0 &&
      (((uintptr_t)a->proj | (uintptr_t)a->q_rows | (uintptr_t)a->key_ring |
        (uintptr_t)a->value_ring | (uintptr_t)a->q_norm | (uintptr_t)a->k_norm) &
       15) == 0;
  if (pieces)
    hipLaunchKernelGGL(window_append_vec_kernel,
                       dim3((unsigned)((units * (g.HP / 8) + 255) / 256)), ablock, 0,
                       s, g);
  else if (bf16)
    hipLaunchKernelGGL(window_append_kernel<bf16_t>, agrid, ablock, 0, s, g);
  else
    hipLaunchKernelGGL(window_append_kernel<float>, agrid, ablock, 0, s, g);
  T5D_CHECK_LAUNCH("window attention (append)");
  if (variant == 2 || (variant == 0 && can_rows)) {
    const int64_t tiles = ((int64_t)b->max_len * g.gs + 127) / 128;
    const dim3 grid((unsigned)tiles, b->S, a->G), block(256);
    if (g.HP == 32) hipLaunchKernelGGL(window_rows_kernel<1>, grid, block, 0, s, g);
    else if (g.HP == 64) hipLaunchKernelGGL(window_rows_kernel<2>, grid, block, 0, s, g);
    else if (g.HP == 128) hipLaunchKernelGGL(window_rows_kernel<4>, grid, block, 0, s, g);
    else hipLaunchKernelGGL(window_rows_kernel<8>, grid, block, 0, s, g);
    T5D_CHECK_LAUNCH("window attention (rows)");
    return T5D_OK;
  }
  if (bf16) launch_wave<bf16_t>(s, g);
  else launch_wave<float>(s, g);
  T5D_CHECK_LAUNCH("window attention (wave)");
  return T5D_OK;
}
