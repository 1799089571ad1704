// Which expert every token goes to, for mixtures whose experts are listed per
// token id in a table: the tokens of a call sorted by expert, as the tiles of rows
// that t5d_grouped_dense_run works on.  The choice depends on the token ids alone,
// so one launch at the start of a forward serves all layers, a workgroup per layer.
#include "common.h"

namespace t5d {

constexpr int kRouteThreads = 1024;
constexpr int kMaxExperts = 1024;
constexpr int kRouteLayers = 16;  // per launch

struct RouteArgs {
  const int32_t* tokens;
  int M, V;
  const int32_t* gate;
  t5d_route layer[kRouteLayers];
};

__global__ void __launch_bounds__(kRouteThreads)
route_kernel(RouteArgs g) {
  T5D_GATED(g.gate);
  const t5d_route& r = g.layer[blockIdx.x];
  __shared__ int s_first[kMaxExperts];   // count, then the expert's next free entry
  __shared__ int s_scan[2][kRouteThreads];
  const int t = threadIdx.x, E = r.experts, total = g.M * r.top;
  s_first[t] = 0;
  __syncthreads();
  auto expert_of = [&](int i) {
    const int m = i / r.top;
    int id = g.tokens[m];
    id = id < 0 ? 0 : (id >= g.V ? g.V - 1 : id);
    const int e = r.table[(size_t)id * r.top + (i - m * r.top)];
    return e < 0 ? 0 : (e >= E ? E - 1 : e);
  };
  for (int i = t; i < total; i += kRouteThreads) atomicAdd(&s_first[expert_of(i)], 1);
  __syncthreads();
  // Sums over the experts before this one: of entries, and of tiles.
  const int count = s_first[t];
  const int n_tiles = (count + r.tile_rows - 1) / r.tile_rows;
  int before[2];
#pragma unroll
  for (int pass = 0; pass < 2; ++pass) {
    const int mine = pass == 0 ? count : n_tiles;
    int cur = 0;
    s_scan[0][t] = mine;
    __syncthreads();
    for (int step = 1; step < kRouteThreads; step *= 2) {
      const int v = s_scan[cur][t] + (t >= step ? s_scan[cur][t - step] : 0);
      s_scan[cur ^ 1][t] = v;
      cur ^= 1;
      __syncthreads();
    }
    before[pass] = s_scan[cur][t] - mine;
    if (pass == 1) {
      // tiles that no expert needs
      const int used = s_scan[cur][kRouteThreads - 1];
      for (int i = used + t; i < r.max_tiles; i += kRouteThreads)
        reinterpret_cast<int4*>(r.tiles)[i] = make_int4(-1, 0, 0, 0);
    }
    __syncthreads();
  }
  for (int i = 0; i < n_tiles; ++i)
    if (before[1] + i < r.max_tiles)
      reinterpret_cast<int4*>(r.tiles)[before[1] + i] =
          make_int4(t, before[0] + i * r.tile_rows,
                    min(r.tile_rows, count - i * r.tile_rows), 0);
  s_first[t] = before[0];
  __syncthreads();
  for (int i = t; i < total; i += kRouteThreads) {
    const int p = atomicAdd(&s_first[expert_of(i)], 1);
    r.token_of[p] = i / r.top;
    r.entry_of[i] = p;
  }
}

}  // namespace t5d

using namespace t5d;

extern "C" int t5d_route_max_tiles(int entries, int experts, int tile_rows) {
  if (entries <= 0 || experts <= 0 || tile_rows <= 0) return -1;
  return entries / tile_rows + (experts < entries ? experts : entries);
}

extern "C" int t5d_route_tokens(void* stream, const int32_t* tokens, int M, int V,
                                const t5d_route* layers, int n_layers) {
  T5D_REQUIRE(tokens && layers && M > 0 && V > 0 && n_layers > 0, T5D_EINVAL,
              "t5d_route_tokens: M=%d V=%d layers=%d", M, V, n_layers);
  for (int i = 0; i < n_layers; ++i) {
    const t5d_route& r = layers[i];
    T5D_REQUIRE(r.experts > 0 && r.experts <= kMaxExperts,
                r.experts > kMaxExperts ? T5D_ELIMIT : T5D_EINVAL,
                "t5d_route_tokens: %d experts (at most %d)", r.experts, kMaxExperts);
    T5D_REQUIRE(r.table && r.tiles && r.token_of && r.entry_of && r.top > 0 &&
                    (int64_t)M * r.top < (1 << 30) &&
                    r.max_tiles >= t5d_route_max_tiles(M * r.top, r.experts,
                                                       r.tile_rows) &&
                    r.tile_rows > 0 && ((uintptr_t)r.tiles % 16) == 0,
                T5D_EINVAL, "t5d_route_tokens: top=%d tiles=%d of %d rows", r.top,
                r.max_tiles, r.tile_rows);
  }
  for (int i = 0; i < n_layers; i += kRouteLayers) {
    RouteArgs g;
    g.tokens = tokens; g.M = M; g.V = V; g.gate = tls_gate;
    const int n = n_layers - i < kRouteLayers ? n_layers - i : kRouteLayers;
    for (int k = 0; k < n; ++k) g.layer[k] = layers[i + k];
    hipLaunchKernelGGL(route_kernel, dim3(n), dim3(kRouteThreads), 0,
                       as_stream(stream), g);
    T5D_CHECK_LAUNCH("t5d_route_tokens");
  }
  return T5D_OK;
}
