// The residual stream of models that keep it in float32: the embedding with its
// sinusoidal position vector, and the row kernel that sits between two dense
// layers — norm of a branch's output, the residual sum, an added vector, and the
// norm in front of the next branch — as one pass over the row.  Models with
// hyper-connections carry several such streams per token: hyper_norm_kernel mixes
// them, adds the branch's output (also one that is still in parts: the chosen
// experts' rows and a gated shared one) and norms their weighted sum for the next
// branch, again in one pass.
#include "common.h"

namespace t5d {

// ---- embedding + sinusoidal position ------------------------------------------
// One workgroup per token.  The angle p * 10000^(-2i/d) is formed and reduced to
// one turn in float64 (a float32 product of a position in the thousands is off by
// 1e-4 radians), its sine and cosine in float32.
template <typename T>
__global__ void __launch_bounds__(256)
embed_sinusoid_kernel(const T* __restrict__ table, const int32_t* __restrict__ ids,
                      const int32_t* __restrict__ pos, float* __restrict__ out,
                      float* __restrict__ out2, int d, int ld, int V,
                      const int32_t* gate) {
  T5D_GATED(gate);
  const int m = blockIdx.x;
  int id = ids[m];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);
  const double p = (double)pos[m];
  const T* row = table + (size_t)id * ld;
  const double step = -2.0 * 9.210340371976182736 / (double)d;  // ln 10000
  for (int i = threadIdx.x; 2 * i < ld; i += 256) {
    float s = 0.f, c = 0.f;
    const bool in = 2 * i < d;
    if (in) {
      const double turns = p * exp(step * (double)i) * 0.15915494309189533577;
      sincosf((float)((turns - floor(turns)) * 6.283185307179586477), &s, &c);
    }
    const float a = in ? to_f32<T>(row[2 * i]) + s : 0.f;
    const float b = in ? to_f32<T>(row[2 * i + 1]) + c : 0.f;
    const float2 v = make_float2(a, 2 * i + 1 < d ? b : 0.f);
    *reinterpret_cast<float2*>(out + (size_t)m * ld + 2 * i) = v;
    if (out2 != nullptr)
      *reinterpret_cast<float2*>(out2 + (size_t)m * ld + 2 * i) = v;
  }
}

// ---- the row kernel between two dense layers -------------------------------------
struct StreamNormArgs {
  const void* y;        // branch output [M, ld] (y_f32: float32, else activations)
  const float* y_norm;  // [d] norm of y (null: y is added as it is)
  const float* add;     // [d] added to the stream
  float* x;             // [M, ld] the stream, read and (if changed) written
  const float* norm;    // [d] norm of the stream -> out [M, ld]
  void* out;
  const float* x0;      // with it out is [M, 2 ld] = the stream | x0, not normed
  const int32_t* rows;  // out row m is stream row rows[m]
  int y_f32, d, ld;
  float eps;
  const int32_t* gate;
};

__device__ __forceinline__ float block_sum(float v, float* s4) {
  v = wave_sum(v);
  __syncthreads();  // the previous sum's readers are done
  if ((threadIdx.x & 63) == 0) s4[threadIdx.x >> 6] = v;
  __syncthreads();
  return (s4[0] + s4[1]) + (s4[2] + s4[3]);
}

// 256 threads per row, VPT groups of 4 columns per thread.  Columns d .. ld - 1
// of every row are zero and stay zero.
template <typename T, int VPT>
__global__ void __launch_bounds__(256)
stream_norm_kernel(StreamNormArgs g) {
  T5D_GATE_READ(g.gate);
  __shared__ float s4[4];
  const int m = blockIdx.x;
  const int src = g.rows != nullptr ? g.rows[m] : m;
  float* xrow = g.x + (size_t)src * g.ld;
  float4 x[VPT];
  bool on[VPT];
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int c = 4 * (threadIdx.x + 256 * v);
    on[v] = c < g.ld;
    x[v] = on[v] ? *reinterpret_cast<const float4*>(xrow + c)
                 : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  T5D_GATE_TEST();
  auto column = [&](const float* p, int c) {  // 4 entries of a [d] vector
    float4 r = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c + 4 <= g.d) return *reinterpret_cast<const float4*>(p + c);
    if (c < g.d) r.x = p[c];
    if (c + 1 < g.d) r.y = p[c + 1];
    if (c + 2 < g.d) r.z = p[c + 2];
    return r;
  };
  if (g.y != nullptr) {
    float4 y[VPT];
    float ss = 0.f;
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int c = 4 * (threadIdx.x + 256 * v);
      y[v] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (on[v]) {
        const size_t o = (size_t)src * g.ld + c;
        if (g.y_f32) {
          y[v] = *reinterpret_cast<const float4*>(
              reinterpret_cast<const float*>(g.y) + o);
        } else {
          const uint2 q = *reinterpret_cast<const uint2*>(
              reinterpret_cast<const bf16_t*>(g.y) + o);
          y[v] = make_float4(bf16lo_to_f32(q.x), bf16hi_to_f32(q.x),
                             bf16lo_to_f32(q.y), bf16hi_to_f32(q.y));
        }
      }
      ss = fmaf(y[v].x, y[v].x, ss);
      ss = fmaf(y[v].y, y[v].y, ss);
      ss = fmaf(y[v].z, y[v].z, ss);
      ss = fmaf(y[v].w, y[v].w, ss);
    }
    const bool normed = g.y_norm != nullptr;
    const float inv =
        normed ? 1.0f / sqrtf(block_sum(ss, s4) / (float)g.d + g.eps) : 1.f;
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int c = 4 * (threadIdx.x + 256 * v);
      if (!on[v]) continue;
      const float4 w =
          normed ? column(g.y_norm, c) : make_float4(1.f, 1.f, 1.f, 1.f);
      x[v].x += y[v].x * inv * w.x;
      x[v].y += y[v].y * inv * w.y;
      x[v].z += y[v].z * inv * w.z;
      x[v].w += y[v].w * inv * w.w;
    }
  }
  if (g.add != nullptr) {
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int c = 4 * (threadIdx.x + 256 * v);
      if (!on[v]) continue;
      const float4 w = column(g.add, c);
      x[v].x += w.x; x[v].y += w.y; x[v].z += w.z; x[v].w += w.w;
    }
  }
  if (g.y != nullptr || g.add != nullptr) {
#pragma unroll
    for (int v = 0; v < VPT; ++v)
      if (on[v])
        *reinterpret_cast<float4*>(xrow + 4 * (threadIdx.x + 256 * v)) = x[v];
  }
  if (g.out == nullptr) return;
  auto put = [&](size_t o, const float4& v) {
    if constexpr (sizeof(T) == 4)
      *reinterpret_cast<float4*>(reinterpret_cast<float*>(g.out) + o) = v;
    else
      *reinterpret_cast<uint2*>(reinterpret_cast<bf16_t*>(g.out) + o) =
          make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
  };
  if (g.x0 != nullptr) {
    const float* x0 = g.x0 + (size_t)src * g.ld;
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int c = 4 * (threadIdx.x + 256 * v);
      if (!on[v]) continue;
      put((size_t)m * 2 * g.ld + c, x[v]);
      put((size_t)m * 2 * g.ld + g.ld + c, *reinterpret_cast<const float4*>(x0 + c));
    }
    return;
  }
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    ss = fmaf(x[v].x, x[v].x, ss);
    ss = fmaf(x[v].y, x[v].y, ss);
    ss = fmaf(x[v].z, x[v].z, ss);
    ss = fmaf(x[v].w, x[v].w, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, s4) / (float)g.d + g.eps);
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int c = 4 * (threadIdx.x + 256 * v);
    if (!on[v]) continue;
    const float4 w = column(g.norm, c);
    put((size_t)m * g.ld + c,
        make_float4(x[v].x * inv * w.x, x[v].y * inv * w.y, x[v].z * inv * w.z,
                    x[v].w * inv * w.w));
  }
}

// ---- several streams ----------------------------------------------------------------
template <typename T>
__device__ __forceinline__ float4 load4(const T* p) {
  if constexpr (sizeof(T) == 4) {
    return *reinterpret_cast<const float4*>(p);
  } else {
    const uint2 q = *reinterpret_cast<const uint2*>(p);
    return make_float4(bf16lo_to_f32(q.x), bf16hi_to_f32(q.x), bf16lo_to_f32(q.y),
                       bf16hi_to_f32(q.y));
  }
}
__device__ __forceinline__ void fma4(float4& acc, float w, const float4& v) {
  acc.x = fmaf(w, v.x, acc.x);
  acc.y = fmaf(w, v.y, acc.y);
  acc.z = fmaf(w, v.z, acc.z);
  acc.w = fmaf(w, v.w, acc.w);
}
__device__ __forceinline__ float dot4(const float4& a, const float4& b) {
  return fmaf(a.x, b.x, fmaf(a.y, b.y, fmaf(a.z, b.z, a.w * b.w)));
}

// Every stream of a token starts as its scaled embedding.  (Columns d .. ld - 1 of
// the table are zero.)
template <typename T>
__global__ void __launch_bounds__(256)
embed_streams_kernel(const T* __restrict__ table, const int32_t* __restrict__ ids,
                     float scale, float* __restrict__ out, int ld, int streams,
                     int V, const int32_t* gate) {
  T5D_GATED(gate);
  const int m = blockIdx.x;
  int id = ids[m];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);
  const T* row = table + (size_t)id * ld;
  float* dst = out + (size_t)m * streams * ld;
  for (int c = 4 * threadIdx.x; c < ld; c += 1024) {
    const float4 e = load4<T>(row + c);
    const float4 v = make_float4(e.x * scale, e.y * scale, e.z * scale, e.w * scale);
    for (int s = 0; s < streams; ++s)
      *reinterpret_cast<float4*>(dst + (size_t)s * ld + c) = v;
  }
}

struct HyperArgs {
  t5d_hyper_norm a;
  const int32_t* gate;
};

// One workgroup per row; S streams (template: an upper bound, the real number is
// a.streams) of VPT groups of 4 columns per thread.  A thread holds one group of
// columns of every stream at a time and keeps only their weighted sum for the
// norm.  Columns d .. ld - 1 are zero and stay zero.
template <typename T, int S, int VPT>
__global__ void __launch_bounds__(256)
hyper_norm_kernel(HyperArgs h) {
  T5D_GATED(h.gate);
  const t5d_hyper_norm& g = h.a;
  __shared__ float s4[4];
  __shared__ float s_mix[S * S], s_spread[S], s_collect[S];
  const int n = g.streams;
  const bool add = g.y != nullptr || g.parts != nullptr;
  for (int i = threadIdx.x; i < S * S; i += 256) {
    const int from = i / S, to = i % S;
    float v = from == to ? 1.f : 0.f;
    if (g.mix != nullptr && from < n && to < n) v = g.mix[from * n + to];
    s_mix[i] = v;
  }
  if (threadIdx.x < S) {
    const int s = threadIdx.x;
    s_spread[s] = s < n ? (g.spread != nullptr ? g.spread[s] : 1.f) : 0.f;
    s_collect[s] = s < n ? (g.collect != nullptr ? g.collect[s] : 1.f) : 0.f;
  }
  __syncthreads();
  const int m = blockIdx.x;
  const int src = g.rows != nullptr ? g.rows[m] : m;
  float* xrow = g.x + (size_t)src * n * g.ld;
  const T* y = reinterpret_cast<const T*>(g.y);
  const T* parts = reinterpret_cast<const T*>(g.parts);
  const float y_gate = add && g.y_gate != nullptr ? g.y_gate[src] : 1.f;
  float4 u[VPT];
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int c = 4 * (threadIdx.x + 256 * v);
    u[v] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c >= g.ld) continue;
    float4 x[S];
#pragma unroll
    for (int s = 0; s < S; ++s)
      x[s] = s < n ? *reinterpret_cast<const float4*>(xrow + (size_t)s * g.ld + c)
                   : make_float4(0.f, 0.f, 0.f, 0.f);
    if (add) {
      float4 b = make_float4(0.f, 0.f, 0.f, 0.f);
      if (parts != nullptr)
        for (int t = 0; t < g.top; ++t) {
          const int r = g.part_row[(size_t)src * g.top + t];
          fma4(b, g.part_weight, load4<T>(parts + (size_t)r * g.ld + c));
        }
      if (y != nullptr) fma4(b, y_gate, load4<T>(y + (size_t)src * g.ld + c));
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (t >= n) continue;
        float4 z = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < S; ++s) fma4(z, s_mix[s * S + t], x[s]);
        fma4(z, s_spread[t], b);
        *reinterpret_cast<float4*>(xrow + (size_t)t * g.ld + c) = z;
        fma4(u[v], s_collect[t], z);
      }
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) fma4(u[v], s_collect[s], x[s]);
    }
    if (g.sum != nullptr)
      *reinterpret_cast<float4*>(g.sum + (size_t)m * g.ld + c) = u[v];
  }
  if (g.out == nullptr) return;
  auto column = [&](const float* p, int c) {  // 4 entries of a [d] vector
    float4 r = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c + 4 <= g.d) return *reinterpret_cast<const float4*>(p + c);
    if (c < g.d) r.x = p[c];
    if (c + 1 < g.d) r.y = p[c + 1];
    if (c + 2 < g.d) r.z = p[c + 2];
    return r;
  };
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) ss += dot4(u[v], u[v]);
  const float inv = 1.0f / sqrtf(block_sum(ss, s4) / (float)g.d + g.eps);
  float dot = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int c = 4 * (threadIdx.x + 256 * v);
    if (c >= g.ld) continue;
    const float4 w = column(g.norm, c);
    const float4 r = make_float4(u[v].x * inv * w.x, u[v].y * inv * w.y,
                                 u[v].z * inv * w.z, u[v].w * inv * w.w);
    const size_t o = (size_t)m * g.ld + c;
    if constexpr (sizeof(T) == 4)
      *reinterpret_cast<float4*>(reinterpret_cast<float*>(g.out) + o) = r;
    else
      *reinterpret_cast<uint2*>(reinterpret_cast<bf16_t*>(g.out) + o) =
          make_uint2(pack_bf16x2(r.x, r.y), pack_bf16x2(r.z, r.w));
    if (g.gate_w != nullptr) dot += dot4(r, column(g.gate_w, c));
  }
  if (g.gate_w != nullptr) {
    dot = block_sum(dot, s4);
    if (threadIdx.x == 0) g.gate_out[m] = 1.0f / (1.0f + expf(-dot));
  }
}

template <typename T, int S>
static void launch_hyper(hipStream_t s, const HyperArgs& h, int M) {
  const int vpt = (h.a.ld + 1023) / 1024;
#define T5D_HN(V_) \
  hipLaunchKernelGGL((hyper_norm_kernel<T, S, V_>), dim3(M), dim3(256), 0, s, h)
  if (vpt <= 1) T5D_HN(1);
  else if (vpt <= 2) T5D_HN(2);
  else if (vpt <= 4) T5D_HN(4);
  else T5D_HN(16);
#undef T5D_HN
}

template <typename T>
static void launch_stream_norm(hipStream_t s, const StreamNormArgs& g, int M) {
  const int vpt = (g.ld + 1023) / 1024;
#define T5D_SN(V_) \
  hipLaunchKernelGGL((stream_norm_kernel<T, V_>), dim3(M), dim3(256), 0, s, g)
  if (vpt <= 1) T5D_SN(1);
  else if (vpt <= 2) T5D_SN(2);
  else if (vpt <= 4) T5D_SN(4);
  else if (vpt <= 8) T5D_SN(8);
  else T5D_SN(16);
#undef T5D_SN
}

}  // namespace t5d

using namespace t5d;

extern "C" int t5d_embed_sinusoid(void* stream, int dtype, const void* table,
                                  const int32_t* ids, const int32_t* positions,
                                  float* out, float* out2, int M, int d, int ld,
                                  int V) {
  T5D_REQUIRE(dtype == T5D_F32 || dtype == T5D_BF16, T5D_EINVAL,
              "t5d_embed_sinusoid: dtype %d", dtype);
  T5D_REQUIRE(table && ids && positions && out, T5D_EINVAL,
              "t5d_embed_sinusoid: null pointer");
  T5D_REQUIRE(M > 0 && d > 0 && ld >= d && ld % 4 == 0 && V > 0 &&
                  (((uintptr_t)out | (uintptr_t)out2) % 16) == 0,
              T5D_EINVAL, "t5d_embed_sinusoid: M=%d d=%d ld=%d V=%d", M, d, ld, V);
  if (dtype == T5D_F32)
    hipLaunchKernelGGL(embed_sinusoid_kernel<float>, dim3(M), dim3(256), 0,
                       as_stream(stream), (const float*)table, ids, positions, out,
                       out2, d, ld, V, tls_gate);
  else
    hipLaunchKernelGGL(embed_sinusoid_kernel<bf16_t>, dim3(M), dim3(256), 0,
                       as_stream(stream), (const bf16_t*)table, ids, positions,
                       out, out2, d, ld, V, tls_gate);
  T5D_CHECK_LAUNCH("t5d_embed_sinusoid");
  return T5D_OK;
}

extern "C" int t5d_stream_norm(void* stream, int dtype, int y_dtype, const void* y,
                               const float* y_norm, const float* add, float* x,
                               const float* norm, const float* x0,
                               const int32_t* rows, void* out, int M, int d,
                               int ld, float eps) {
  T5D_REQUIRE((dtype == T5D_F32 || dtype == T5D_BF16) &&
                  (y_dtype == T5D_F32 || y_dtype == T5D_BF16),
              T5D_EINVAL, "t5d_stream_norm: dtypes %d %d", dtype, y_dtype);
  T5D_REQUIRE(x && (y || !y_norm) && (!out || norm || x0) && !(norm && x0),
              T5D_EINVAL, "t5d_stream_norm: null pointer");
  T5D_REQUIRE(M > 0 && d > 0 && ld >= d && ld % 8 == 0 && ld <= 16384, T5D_EINVAL,
              "t5d_stream_norm: M=%d d=%d ld=%d", M, d, ld);
  T5D_REQUIRE(!rows || (!y && !add), T5D_EINVAL,
              "t5d_stream_norm: picked rows are only read");
  T5D_REQUIRE((((uintptr_t)x | (uintptr_t)y | (uintptr_t)y_norm | (uintptr_t)add |
                (uintptr_t)norm | (uintptr_t)x0 | (uintptr_t)out) % 16) == 0,
              T5D_EINVAL, "t5d_stream_norm: operands must be 16-byte aligned");
  StreamNormArgs g;
  g.y = y; g.y_norm = y_norm; g.add = add; g.x = x; g.norm = norm; g.out = out;
  g.x0 = x0; g.rows = rows; g.y_f32 = y_dtype == T5D_F32; g.d = d; g.ld = ld;
  g.eps = eps; g.gate = tls_gate;
  if (dtype == T5D_F32) launch_stream_norm<float>(as_stream(stream), g, M);
  else launch_stream_norm<bf16_t>(as_stream(stream), g, M);
  T5D_CHECK_LAUNCH("t5d_stream_norm");
  return T5D_OK;
}

extern "C" int t5d_embed_streams(void* stream, int dtype, const void* table,
                                 const int32_t* ids, float scale, float* out, int M,
                                 int d, int ld, int streams, int V) {
  T5D_REQUIRE(dtype == T5D_F32 || dtype == T5D_BF16, T5D_EINVAL,
              "t5d_embed_streams: dtype %d", dtype);
  T5D_REQUIRE(table && ids && out && M > 0 && d > 0 && ld >= d && ld % 4 == 0 &&
                  V > 0 && streams > 0 &&
                  (((uintptr_t)table | (uintptr_t)out) % 16) == 0,
              T5D_EINVAL, "t5d_embed_streams: M=%d d=%d ld=%d streams=%d V=%d", M, d,
              ld, streams, V);
  if (dtype == T5D_F32)
    hipLaunchKernelGGL(embed_streams_kernel<float>, dim3(M), dim3(256), 0,
                       as_stream(stream), (const float*)table, ids, scale, out, ld,
                       streams, V, tls_gate);
  else
    hipLaunchKernelGGL(embed_streams_kernel<bf16_t>, dim3(M), dim3(256), 0,
                       as_stream(stream), (const bf16_t*)table, ids, scale, out, ld,
                       streams, V, tls_gate);
  T5D_CHECK_LAUNCH("t5d_embed_streams");
  return T5D_OK;
}

extern "C" int t5d_hyper_norm_run(void* stream, const t5d_hyper_norm* a, int M) {
  T5D_REQUIRE(a && a->x && M > 0, T5D_EINVAL, "t5d_hyper_norm_run: null pointer");
  T5D_REQUIRE(a->dtype == T5D_F32 || a->dtype == T5D_BF16, T5D_EINVAL,
              "t5d_hyper_norm_run: dtype %d", a->dtype);
  T5D_REQUIRE(a->streams > 0 && a->streams <= 16 && a->d > 0 && a->ld >= a->d &&
                  a->ld % 8 == 0 && a->ld <= 16384,
              a->streams > 16 || a->ld > 16384 ? T5D_ELIMIT : T5D_EINVAL,
              "t5d_hyper_norm_run: %d streams of %d / %d columns (at most 16 of "
              "16384)", a->streams, a->d, a->ld);
  T5D_REQUIRE((!a->out || a->norm) && (!a->parts || (a->part_row && a->top > 0)) &&
                  (!a->gate_w || (a->gate_out && a->out)),
              T5D_EINVAL, "t5d_hyper_norm_run: missing operand");
  T5D_REQUIRE(!a->rows || (!a->y && !a->parts), T5D_EINVAL,
              "t5d_hyper_norm_run: picked rows are only read");
  T5D_REQUIRE((((uintptr_t)a->x | (uintptr_t)a->y | (uintptr_t)a->parts |
                (uintptr_t)a->norm | (uintptr_t)a->out | (uintptr_t)a->sum |
                (uintptr_t)a->gate_w) % 16) == 0,
              T5D_EINVAL, "t5d_hyper_norm_run: operands must be 16-byte aligned");
  HyperArgs h;
  h.a = *a;
  h.gate = tls_gate;
  hipStream_t s = as_stream(stream);
  const bool f32 = a->dtype == T5D_F32;
  if (a->streams == 1) {
    if (f32) launch_hyper<float, 1>(s, h, M);
    else launch_hyper<bf16_t, 1>(s, h, M);
  } else if (a->streams <= 4) {
    if (f32) launch_hyper<float, 4>(s, h, M);
    else launch_hyper<bf16_t, 4>(s, h, M);
  } else {
    if (f32) launch_hyper<float, 16>(s, h, M);
    else launch_hyper<bf16_t, 16>(s, h, M);
  }
  T5D_CHECK_LAUNCH("t5d_hyper_norm_run");
  return T5D_OK;
}
