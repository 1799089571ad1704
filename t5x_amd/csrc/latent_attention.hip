// Causal sliding-window attention whose keys and values are linear maps of one
// low-rank latent per position, with a sink in the denominator.  Only the latents
// are cached: position p of a slot's sequence is row p % ring of the slot's ring,
// shared by all heads (and by the layers that read another layer's latents).
//
// Two ways to attend, which differ by rounding only:
//   * spans: the latents that the call's queries can see are gathered and expanded
//     into keys and values by one dense layer, and window_rows_kernel attends over
//     those rows.  Least arithmetic per (query, key) pair; pays for the expansion,
//     so it is for portions that are long beside the window.
//   * absorbed: a head's key map moves to the query (q . W_uk c = W_uk^T q . c) and
//     its value map behind the weighted sum, so all heads attend to the latents
//     themselves, read once for up to 32 (token, head) rows.  For decoding and
//     short portions.
#include "common.h"
#include "gemm_tiles.h"

namespace t5d {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNoMax = -1e30f;  // running maximum before the first key
constexpr int kMaxSplits = 16;
constexpr int kMaxParts = 512;    // workgroups of a launch with split keys

struct LatentArgs {
  t5d_latent_attention a;
  t5d_ragged b;
  int HP, RP, QP, splits;
  float* parts;  // [M, H, splits, RP + 4]: sums, maximum, sum of weights
  const int32_t* gate;
};

// ---- norms of the new latents, ring update --------------------------------------
// One wavefront per (token, query latent or cached latent).  The projection's
// columns and the norm's weights are zero from the latent's size to the next
// multiple of 16 and RP / QP, so the padding of what is written is zero.
template <typename T>
__global__ void __launch_bounds__(256)
latent_append_kernel(LatentArgs g) {
  T5D_GATED(g.gate);
  const t5d_latent_attention& a = g.a;
  constexpr int E = Act<T>::kElemsPer16B;
  const int lane = threadIdx.x & 63;
  const int nvec = a.off_kv >= 0 ? 2 : 1;
  const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (int64_t)g.b.M * nvec) return;
  const int m = unit / nvec;
  const bool query = unit % nvec == 0;
  const int n = query ? a.q_rank : a.rank, pad = query ? g.QP : g.RP;
  const int have = (n + 15) & ~15;  // columns the projection has
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)m * a.ld_proj +
               (query ? a.off_q : a.off_kv);
  const float* w = query ? a.q_norm : a.kv_norm;
  T* dst = reinterpret_cast<T*>(a.cq) + (size_t)m * g.QP;
  if (!query)
    dst = reinterpret_cast<T*>(a.latent_ring) +
          ((size_t)g.b.seq_slot[g.b.tok_seq[m]] * a.ring + g.b.tok_pos[m] % a.ring) *
              g.RP;
  float ss = 0.f;
  for (int c = E * lane; c < have; c += E * 64) {
    float f[E];
    unpack16(*reinterpret_cast<const uint4*>(p + c), f);
#pragma unroll
    for (int e = 0; e < E; ++e) ss = fmaf(f[e], f[e], ss);
  }
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps);
  for (int c = E * lane; c < pad; c += E * 64) {
    float f[E];
    unpack16(c < have ? *reinterpret_cast<const uint4*>(p + c)
                      : make_uint4(0, 0, 0, 0), f);
#pragma unroll
    for (int e = 0; e < E; ++e) f[e] = f[e] * inv * w[c + e];
    uint4 v;
    if constexpr (sizeof(T) == 4)
      v = make_uint4(__float_as_uint(f[0]), __float_as_uint(f[1]),
                     __float_as_uint(f[2]), __float_as_uint(f[3]));
    else
      v = make_uint4(pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]),
                     pack_bf16x2(f[4], f[5]), pack_bf16x2(f[6], f[7]));
    *reinterpret_cast<uint4*>(dst + c) = v;
  }
}

// ---- spans ------------------------------------------------------------------------
// Row off[s] + i of a span is position first[s] + i of portion s; rows past the
// portion's end are zero.  One thread per 16 bytes.
__global__ void __launch_bounds__(256)
latent_gather_kernel(LatentArgs g, t5d_span span) {
  T5D_GATED(g.gate);
  const int per = g.RP / 8;
  const int64_t unit = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (unit >= (int64_t)span.rows * per) return;
  const int r = unit / per, c = 8 * (int)(unit % per);
  int lo = 0, hi = g.b.S;  // the portion: off[lo] <= r < off[lo + 1]
  while (hi - lo > 1) {
    const int mid = (lo + hi) / 2;
    if (span.off[mid] <= r) lo = mid;
    else hi = mid;
  }
  const int pos = span.first[lo] + r - span.off[lo];
  const int end = g.b.seq_start[lo] + g.b.seq_off[lo + 1] - g.b.seq_off[lo];
  uint4 v = make_uint4(0, 0, 0, 0);
  if (pos < end)
    v = *reinterpret_cast<const uint4*>(
        reinterpret_cast<const bf16_t*>(g.a.latent_ring) +
        ((size_t)g.b.seq_slot[lo] * g.a.ring + pos % g.a.ring) * g.RP + c);
  *reinterpret_cast<uint4*>(reinterpret_cast<bf16_t*>(g.a.lat) + (size_t)r * g.RP +
                            c) = v;
}

// ---- absorbed, bfloat16 --------------------------------------------------------------
__device__ __forceinline__ f32x4_v mfma(const Frag& x, const Frag& y, f32x4_v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.v, y.v, c, 0, 0, 0);
}

// A workgroup attends for 16 HG consecutive (token, head) rows of one portion over
// every splits-th tile of 64 positions.  The tile's latents go to LDS twice: as
// rows (scores S^T = C Q^T: wavefront w takes positions 16 w ..) and transposed
// (O^T = C^T P^T: wavefront w takes a quarter of the latent's columns).  Between
// the two the wavefronts exchange row maxima and weights through LDS; the weights
// are kept to 16 bits of mantissa as value + remainder.  RP = 32 DT.
template <int DT, int HG>
__global__ void __launch_bounds__(256, DT >= 16 ? 1 : 2)
latent_tile_kernel(LatentArgs g) {
  constexpr int RP = DT * 32, KB = 64, R = 16 * HG;
  constexpr int KS = RP + 8, VS = KB + 8, PS = KB + 8;  // LDS row strides
  constexpr int CT = RP / 16 / 4;                       // column tiles per wavefront
  constexpr int LPR = RP / 8;                           // lanes on one position
  constexpr int PPI = 64 / LPR;                         // positions per load
  constexpr int QUADS = 4 / PPI;                        // 4 positions, per thread
  static_assert(PPI >= 1 && PPI <= 4, "latents of 128, 256 or 512");
  __shared__ __align__(16) bf16_t s_k[KB * KS];         // [position][column]
  __shared__ __align__(16) bf16_t s_v[RP * VS];         // [column][position]
  __shared__ __align__(16) bf16_t s_p[2][R * PS];       // weights, remainders
  __shared__ float s_max[4][R];
  T5D_GATED(g.gate);
  const t5d_latent_attention& a = g.a;
  const int seq = blockIdx.y, part = blockIdx.z, H = a.H;
  const int off = g.b.seq_off[seq];
  const int rows = (g.b.seq_off[seq + 1] - off) * H;
  const int r0 = blockIdx.x * R;
  if (r0 >= rows) return;
  const int start = g.b.seq_start[seq];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n16 = lane & 15, gq = lane >> 4;
  const int W = a.window > 0 ? a.window : (1 << 30);
  const bf16_t* ring = reinterpret_cast<const bf16_t*>(a.latent_ring) +
                       (size_t)g.b.seq_slot[seq] * a.ring * RP;
  const float scale2 = a.scale * kLog2e;

  int pos[HG], vec[HG];  // of this lane's rows: position, (token, head) index
  float mx[HG], l[HG];
  Frag qf[HG][DT];
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    const int r = min(r0 + 16 * hg + n16, rows - 1);  // past the end: not stored
    const int t = r / H;
    pos[hg] = start + t;
    vec[hg] = (off + t) * H + (r - t * H);
    mx[hg] = kNoMax;
    l[hg] = 0.f;
    const bf16_t* q =
        reinterpret_cast<const bf16_t*>(a.ql) + (size_t)vec[hg] * RP + 8 * gq;
#pragma unroll
    for (int kk = 0; kk < DT; ++kk)
      qf[hg][kk].u = *reinterpret_cast<const uint4*>(q + 32 * kk);
  }
  f32x4_v o[CT][HG];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct)
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) o[ct][hg] = (f32x4_v){0.f, 0.f, 0.f, 0.f};

  const int i_lo = start + r0 / H;
  const int i_hi = start + min(r0 + R - 1, rows - 1) / H;
  const int j_begin = (max(0, i_lo - W + 1) & ~(KB - 1)) + KB * part;
  const int j_step = KB * g.splits;

  // A thread loads 8 columns of 4 consecutive positions (whole positions per
  // wavefront and load: consecutive memory), so the transposed copy takes 8 bytes
  // per column.  Its 16-byte pieces (8 positions) are XOR-swizzled by the column.
  uint4 lat[QUADS][4];
  const int piece = lane % LPR;
  const int quad0 = 4 * wave + lane / LPR;  // positions 4 quad ..
  auto fetch = [&](int jt) {
    const bf16_t* c = ring + ((size_t)(jt % a.ring) + 4 * quad0) * RP + 8 * piece;
#pragma unroll
    for (int i = 0; i < QUADS; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k)
        lat[i][k] = *reinterpret_cast<const uint4*>(c + (4 * PPI * i + k) * RP);
  };
  if (j_begin <= i_hi) fetch(j_begin);
  for (int jt = j_begin; jt <= i_hi; jt += j_step) {
    __syncthreads();  // the previous tile has been read
#pragma unroll
    for (int i = 0; i < QUADS; ++i) {
      const int quad = quad0 + PPI * i;
#pragma unroll
      for (int k = 0; k < 4; ++k)
        *reinterpret_cast<uint4*>(s_k + (4 * quad + k) * KS + 8 * piece) = lat[i][k];
      bf16_t* dst = s_v + (size_t)(8 * piece) * VS +
                    8 * ((quad >> 1) ^ ((piece >> 1) & 7)) + 4 * (quad & 1);
      auto put = [&](int e, uint32_t p, uint32_t q, uint32_t r, uint32_t s) {
        *reinterpret_cast<uint2*>(dst + (2 * e) * VS) =
            make_uint2((p & 0xFFFFu) | (q << 16), (r & 0xFFFFu) | (s << 16));
        *reinterpret_cast<uint2*>(dst + (2 * e + 1) * VS) = make_uint2(
            (p >> 16) | (q & 0xFFFF0000u), (r >> 16) | (s & 0xFFFF0000u));
      };
      put(0, lat[i][0].x, lat[i][1].x, lat[i][2].x, lat[i][3].x);
      put(1, lat[i][0].y, lat[i][1].y, lat[i][2].y, lat[i][3].y);
      put(2, lat[i][0].z, lat[i][1].z, lat[i][2].z, lat[i][3].z);
      put(3, lat[i][0].w, lat[i][1].w, lat[i][2].w, lat[i][3].w);
    }
    __syncthreads();
    if (jt + j_step <= i_hi) fetch(jt + j_step);

    f32x4_v s[HG];
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) s[hg] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < DT; ++kk) {
      Frag kf;
      kf.u = *reinterpret_cast<const uint4*>(s_k + (16 * wave + n16) * KS + 32 * kk +
                                             8 * gq);
#pragma unroll
      for (int hg = 0; hg < HG; ++hg) s[hg] = mfma(kf, qf[hg][kk], s[hg]);
    }
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) {
      float top = kNoMax;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dist = pos[hg] - jt - 16 * wave - 4 * gq - i;
        const float v = dist >= 0 && dist < W ? s[hg][i] * scale2 : -INFINITY;
        s[hg][i] = v;
        top = fmaxf(top, v);
      }
      top = rows_max(top);
      if (gq == 0) s_max[wave][16 * hg + n16] = top;
    }
    __syncthreads();
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) {
      const int r = 16 * hg + n16;
      const float top = fmaxf(mx[hg], fmaxf(fmaxf(s_max[0][r], s_max[1][r]),
                                            fmaxf(s_max[2][r], s_max[3][r])));
      const float alpha = __builtin_amdgcn_exp2f(mx[hg] - top);
      mx[hg] = top;
      float p[4], sum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        p[i] = __builtin_amdgcn_exp2f(s[hg][i] - top);
        sum += p[i];
      }
      l[hg] = l[hg] * alpha + sum;
      const uint32_t h0 = pack_bf16x2(p[0], p[1]), h1 = pack_bf16x2(p[2], p[3]);
      const int at = r * PS + 16 * wave + 4 * gq;
      *reinterpret_cast<uint2*>(s_p[0] + at) = make_uint2(h0, h1);
      *reinterpret_cast<uint2*>(s_p[1] + at) = make_uint2(
          pack_bf16x2(p[0] - bf16lo_to_f32(h0), p[1] - bf16hi_to_f32(h0)),
          pack_bf16x2(p[2] - bf16lo_to_f32(h1), p[3] - bf16hi_to_f32(h1)));
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int i = 0; i < 4; ++i) o[ct][hg][i] *= alpha;
    }
    __syncthreads();
#pragma unroll
    for (int kb = 0; kb < KB / 32; ++kb) {
      Frag hi[HG], lo[HG];
#pragma unroll
      for (int hg = 0; hg < HG; ++hg) {
        const int at = (16 * hg + n16) * PS + 32 * kb + 8 * gq;
        hi[hg].u = *reinterpret_cast<const uint4*>(s_p[0] + at);
        lo[hg].u = *reinterpret_cast<const uint4*>(s_p[1] + at);
      }
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        const int tile = CT * wave + ct;  // (two pieces of 8 columns)
        Frag vf;
        vf.u = *reinterpret_cast<const uint4*>(
            s_v + (16 * tile + n16) * VS + 8 * ((4 * kb + gq) ^ (tile & 7)));
#pragma unroll
        for (int hg = 0; hg < HG; ++hg) {
          o[ct][hg] = mfma(vf, hi[hg], o[ct][hg]);
          o[ct][hg] = mfma(vf, lo[hg], o[ct][hg]);
        }
      }
    }
  }
  // The sums of the wavefronts' weights meet in s_max (its last readers passed a
  // barrier; a workgroup without a tile has none).
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    const float sum = rows_sum(l[hg]);
    if (gq == 0) s_max[wave][16 * hg + n16] = sum;
  }
  __syncthreads();
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    const int r = 16 * hg + n16;
    if (r0 + r >= rows) continue;
    float den = (s_max[0][r] + s_max[1][r]) + (s_max[2][r] + s_max[3][r]);
    if (g.splits > 1) {
      float* out = g.parts + ((size_t)vec[hg] * g.splits + part) * (RP + 4);
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
        *reinterpret_cast<float4*>(out + 16 * (CT * wave + ct) + 4 * gq) =
            make_float4(o[ct][hg][0], o[ct][hg][1], o[ct][hg][2], o[ct][hg][3]);
      if (wave == 0 && gq == 0) {
        out[RP] = mx[hg];
        out[RP + 1] = den;
      }
      continue;
    }
    float c = 1.f;  // what the accumulated sums are scaled by
    if (a.sink != nullptr) {
      const float sink2 = a.sink[vec[hg] % H] * kLog2e;
      const float top = fmaxf(mx[hg], sink2);
      c = exp2f(mx[hg] - top);
      den = den * c + exp2f(sink2 - top);
    }
    const float inv = c / den;
    bf16_t* out = reinterpret_cast<bf16_t*>(a.ol) + (size_t)vec[hg] * RP;
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
      *reinterpret_cast<uint2*>(out + 16 * (CT * wave + ct) + 4 * gq) = make_uint2(
          pack_bf16x2(o[ct][hg][0] * inv, o[ct][hg][1] * inv),
          pack_bf16x2(o[ct][hg][2] * inv, o[ct][hg][3] * inv));
  }
}

// The parts of latent_tile_kernel: one workgroup of RP / 4 threads per (token,
// head), every part's loads in flight together.
template <int SPLITS>
__global__ void __launch_bounds__(128)
latent_merge_kernel(LatentArgs g) {
  T5D_GATED(g.gate);
  const t5d_latent_attention& a = g.a;
  const int vec = blockIdx.x, RP = g.RP, stride = RP + 4;
  const float* p = g.parts + (size_t)vec * SPLITS * stride;
  const int d = 4 * threadIdx.x;
  float4 o[SPLITS];
  float2 ml[SPLITS];
#pragma unroll
  for (int s = 0; s < SPLITS; ++s) {
    o[s] = *reinterpret_cast<const float4*>(p + s * stride + d);
    ml[s] = *reinterpret_cast<const float2*>(p + s * stride + RP);
  }
  const float sink2 = a.sink != nullptr ? a.sink[vec % a.H] * kLog2e : kNoMax;
  float top = sink2;
#pragma unroll
  for (int s = 0; s < SPLITS; ++s) top = fmaxf(top, ml[s].x);
  float den = a.sink != nullptr ? exp2f(sink2 - top) : 0.f;
  float4 num = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int s = 0; s < SPLITS; ++s) {
    const float f = exp2f(ml[s].x - top);
    den = fmaf(f, ml[s].y, den);
    num.x = fmaf(f, o[s].x, num.x);
    num.y = fmaf(f, o[s].y, num.y);
    num.z = fmaf(f, o[s].z, num.z);
    num.w = fmaf(f, o[s].w, num.w);
  }
  const float inv = 1.0f / den;
  *reinterpret_cast<uint2*>(reinterpret_cast<bf16_t*>(a.ol) + (size_t)vec * RP + d) =
      make_uint2(pack_bf16x2(num.x * inv, num.y * inv),
                 pack_bf16x2(num.z * inv, num.w * inv));
}

static int tile_groups(int H) { return H > 16 ? 2 : 1; }

static int tile_splits(const t5d_latent_attention& a, const t5d_ragged& b) {
  const int R = 16 * tile_groups(a.H);
  const int64_t wgs = (int64_t)b.S * (((int64_t)b.max_len * a.H + R - 1) / R);
  const int span = a.window > 0 ? min(a.window + b.max_len, a.ring) : a.ring;
  int n = 1;
  while (n < kMaxSplits && wgs * n < kMaxParts / 2 && span >= 128 * n) n *= 2;
  return n;
}

}  // namespace t5d

using namespace t5d;

extern "C" int t5d_latent_pad(int rank) {
  if (rank <= 0 || rank > 1024) return -1;
  for (int p = 128; p <= 512; p *= 2)
    if (rank <= p) return p;
  return (rank + 63) / 64 * 64;
}

extern "C" int64_t t5d_latent_workspace_bytes(int rank) {
  const int rp = t5d_latent_pad(rank);
  return rp < 0 ? -1 : (int64_t)kMaxParts * 32 * (rp + 4) * 4;
}

#define T5D_TRY(call)        \
  do {                       \
    int rc_ = (call);        \
    if (rc_ != T5D_OK) return rc_; \
  } while (0)

extern "C" int t5d_latent_attention_run(void* stream, const t5d_latent_attention* a,
                                        const t5d_ragged* b, int variant) {
  T5D_REQUIRE(a && b, T5D_EINVAL, "t5d_latent_attention_run: null arguments");
  T5D_REQUIRE(a->dtype == T5D_F32 || a->dtype == T5D_BF16, T5D_EINVAL,
              "t5d_latent_attention_run: dtype %d", a->dtype);
  T5D_REQUIRE(a->H > 0 && a->H <= 65535 && a->D > 0 && a->Dv > 0 && a->rank > 0 &&
                  a->q_rank > 0 && a->window >= 0,
              T5D_EINVAL, "t5d_latent_attention_run: H=%d D=%d Dv=%d rank=%d / %d "
              "window=%d", a->H, a->D, a->Dv, a->rank, a->q_rank, a->window);
  T5D_REQUIRE(a->proj && a->latent_ring && a->uq && a->absorb && a->expand && a->cq &&
                  a->q && a->ql && a->ol && a->out && a->q_norm &&
                  (a->off_kv < 0 || a->kv_norm) && b->tok_pos && b->tok_seq &&
                  b->seq_off && b->seq_start && b->seq_slot,
              T5D_EINVAL, "t5d_latent_attention_run: null buffer");
  T5D_REQUIRE(b->M > 0 && b->S > 0 && b->S <= 65535 && b->max_len > 0 &&
                  b->max_len <= b->M,
              T5D_EINVAL, "t5d_latent_attention_run: M=%d S=%d max_len=%d", b->M,
              b->S, b->max_len);
  T5D_REQUIRE(a->ring > 0 && a->ring % 64 == 0 &&
                  (a->window == 0 || a->ring >= a->window - 1 + b->max_len),
              T5D_EINVAL,
              "t5d_latent_attention_run: a ring of %d rows for a window of %d and "
              "portions of %d (multiple of 64, at least window - 1 + portion)",
              a->ring, a->window, b->max_len);
  T5D_REQUIRE(variant >= 0 && variant <= 3, T5D_EINVAL,
              "t5d_latent_attention_run: variant %d", variant);
  LatentArgs g;
  g.a = *a; g.b = *b;
  g.HP = t5d_window_head_pad(a->D, a->Dv);
  g.RP = t5d_latent_pad(a->rank);
  g.QP = (a->q_rank + 63) / 64 * 64;
  T5D_REQUIRE(g.HP > 0 && g.RP > 0, T5D_ELIMIT,
              "t5d_latent_attention_run: head size %d / %d, rank %d", a->D, a->Dv,
              a->rank);
  const bool bf16 = a->dtype == T5D_BF16;
  T5D_REQUIRE((((uintptr_t)a->proj | (uintptr_t)a->cq | (uintptr_t)a->latent_ring |
                (uintptr_t)a->lat | (uintptr_t)a->kv | (uintptr_t)a->ql |
                (uintptr_t)a->ol) % 16) == 0 &&
                  ((a->ld_proj | a->off_q | (a->off_kv < 0 ? 0 : a->off_kv)) & 7) == 0,
              T5D_EINVAL, "t5d_latent_attention_run: operand alignment");
  g.splits = 1; g.parts = (float*)a->workspace;
  g.gate = tls_gate;
  hipStream_t s = as_stream(stream);
  const t5d_span* span = nullptr;
  for (int i = 0; i < b->n_spans; ++i)
    if (b->spans[i].window == a->window) span = b->spans + i;
  const bool can_span = bf16 && span != nullptr && g.HP <= 256 && a->ukv && a->lat &&
                        a->kv && span->rows > 0 && span->rows <= a->span_rows &&
                        a->ld_out % 4 == 0;
  const bool can_tile = bf16 && g.RP <= 512;
  T5D_REQUIRE((variant != 1 || can_tile) && (variant != 2 || can_span), T5D_EINVAL,
              "t5d_latent_attention_run: variant %d does not cover this call",
              variant);

  const int64_t units = (int64_t)b->M * (a->off_kv >= 0 ? 2 : 1);
  const dim3 agrid((unsigned)((units + 3) / 4)), block(256);
  if (bf16)
    hipLaunchKernelGGL(latent_append_kernel<bf16_t>, agrid, block, 0, s, g);
  else
    hipLaunchKernelGGL(latent_append_kernel<float>, agrid, block, 0, s, g);
  T5D_CHECK_LAUNCH("latent attention (append)");
  const int QN = a->H * g.HP;
  T5D_TRY(t5d_dense(stream, a->dtype, a->dtype, a->cq, g.QP, a->uq, a->q, QN, QN, b->M,
                    g.QP, QN, T5D_EPI_NONE, 0.f, 0.f, 0.f));

  if (variant == 2 || (variant == 0 && can_span)) {
    const int64_t n = (int64_t)span->rows * (g.RP / 8);
    hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((n + 255) / 256)), block,
                       0, s, g, *span);
    T5D_CHECK_LAUNCH("latent attention (gather)");
    T5D_TRY(t5d_dense(stream, a->dtype, a->dtype, a->lat, g.RP, a->ukv, a->kv, 2 * QN,
                      2 * QN, span->rows, g.RP, 2 * QN, T5D_EPI_NONE, 0.f, 0.f, 0.f));
    t5d_window_attention w = {};
    w.dtype = a->dtype; w.H = w.G = a->H; w.D = a->D; w.Dv = a->Dv;
    w.ring = a->ring; w.window = a->window; w.scale = a->scale; w.sink = a->sink;
    w.q_rows = a->q; w.out = a->out; w.ld_out = a->ld_out;
    w.key_ring = a->kv;
    w.value_ring = (char*)a->kv + (size_t)QN * 2;
    return launch_window_span(s, w, *b, *span, 2 * QN);
  }
  // q [M, H, HP] -> ql [M, H, RP], a kernel per head
  t5d_grouped_dense d = {};
  d.dtype = a->dtype; d.epilogue = T5D_EPI_NONE;
  d.M = b->M; d.groups = a->H;
  d.A = a->q; d.lda = QN; d.a_step = g.HP; d.K = g.HP;
  d.W = a->absorb; d.N = d.n_store = g.RP;
  d.w_stride = (int64_t)g.HP * g.RP * (bf16 ? 2 : 4);
  d.C = a->ql; d.ldc = a->H * g.RP; d.c_step = g.RP;
  T5D_TRY(t5d_grouped_dense_run(stream, &d));
  if (variant == 1 || (variant == 0 && can_tile)) {
    const int HG = tile_groups(a->H), R = 16 * HG;
    if (g.parts != nullptr) g.splits = tile_splits(*a, *b);
    const dim3 grid((unsigned)(((int64_t)b->max_len * a->H + R - 1) / R), b->S,
                    g.splits);
#define T5D_LT(DT_, HG_)                                                       \
  if (g.RP == 32 * DT_ && HG == HG_)                                           \
    hipLaunchKernelGGL((latent_tile_kernel<DT_, HG_>), grid, block, 0, s, g)
    T5D_LT(4, 1); T5D_LT(8, 1); T5D_LT(16, 1);
    T5D_LT(4, 2); T5D_LT(8, 2); T5D_LT(16, 2);
#undef T5D_LT
    T5D_CHECK_LAUNCH("latent attention (tile)");
    if (g.splits > 1) {
      const dim3 mgrid(b->M * a->H), mblock(g.RP / 4);
      if (g.splits == 2)
        hipLaunchKernelGGL(latent_merge_kernel<2>, mgrid, mblock, 0, s, g);
      else if (g.splits == 4)
        hipLaunchKernelGGL(latent_merge_kernel<4>, mgrid, mblock, 0, s, g);
      else if (g.splits == 8)
        hipLaunchKernelGGL(latent_merge_kernel<8>, mgrid, mblock, 0, s, g);
      else
        hipLaunchKernelGGL(latent_merge_kernel<16>, mgrid, mblock, 0, s, g);
      T5D_CHECK_LAUNCH("latent attention (merge)");
    }
  } else {
    t5d_window_attention w = {};
    w.dtype = a->dtype; w.H = a->H; w.G = 1; w.D = w.Dv = g.RP;
    w.ring = a->ring; w.window = a->window; w.scale = a->scale; w.sink = a->sink;
    w.q_rows = a->ql; w.out = a->ol; w.ld_out = a->H * g.RP;
    w.key_ring = w.value_ring = a->latent_ring;
    T5D_TRY(launch_window_wave(s, w, *b, g.RP));
  }
  // ol [M, H, RP] -> out [M, H, Dv]
  d.A = a->ol; d.lda = a->H * g.RP; d.a_step = g.RP; d.K = g.RP;
  d.W = a->expand; d.N = (a->Dv + 15) / 16 * 16; d.n_store = a->Dv;
  d.w_stride = (int64_t)g.RP * d.N * (bf16 ? 2 : 4);
  d.C = a->out; d.ldc = a->ld_out; d.c_step = a->Dv;
  return t5d_grouped_dense_run(stream, &d);
}
