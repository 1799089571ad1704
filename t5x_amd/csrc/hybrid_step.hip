// One host call enqueues a whole forward of a decoder-only model with windowed
// attention, latent attention and recurrent layers, for portions of any lengths.
// Between two dense layers there is one row kernel (t5d_stream_norm, or
// t5d_hyper_norm for models with several streams) that adds the previous branch to
// the float32 residual and norms it for the next one.
#include "common.h"

using namespace t5d;

namespace {

struct GateScope {
  explicit GateScope(const int32_t* g) { tls_gate = g; }
  ~GateScope() { tls_gate = nullptr; }
};

#define T5D_TRY(call)        \
  do {                       \
    int rc_ = (call);        \
    if (rc_ != T5D_OK) return rc_; \
  } while (0)

int check_hybrid(const t5d_hybrid_model* m, const t5d_ragged* b) {
  T5D_REQUIRE(m && b && m->layers && m->runs, T5D_EINVAL,
              "t5d_hybrid_step: null model description");
  T5D_REQUIRE(m->dtype == T5D_F32 || m->dtype == T5D_BF16, T5D_EINVAL,
              "t5d_hybrid_step: dtype %d", m->dtype);
  T5D_REQUIRE(m->d > 0 && m->ld >= m->d && m->ld % 64 == 0 && m->V > 0 &&
                  m->head_n >= m->V && m->n_layers > 0 && m->n_runs > 0,
              T5D_EINVAL, "t5d_hybrid_step: d=%d ld=%d V=%d head_n=%d layers=%d "
              "runs=%d", m->d, m->ld, m->V, m->head_n, m->n_layers, m->n_runs);
  T5D_REQUIRE(m->embedding && m->head && m->final_norm && m->x && m->h && m->proj &&
                  m->y && b->tokens && b->tok_pos && b->M > 0,
              T5D_EINVAL, "t5d_hybrid_step: null buffer");
  for (int r = 0; r < m->n_runs; ++r) {
    const t5d_hybrid_run& run = m->runs[r];
    T5D_REQUIRE(run.layer >= 0 && run.layer < m->n_layers, T5D_EINVAL,
                "t5d_hybrid_step: run %d names layer %d", r, run.layer);
    T5D_REQUIRE(!run.enter || (m->loop_in && m->x0 && m->cat), T5D_EINVAL,
                "t5d_hybrid_step: run %d enters a loop without its input layer", r);
    const t5d_hybrid_layer& l = m->layers[run.layer];
    T5D_REQUIRE(l.proj && l.out && l.norm1 && l.mix_rows &&
                    (!l.low || m->low) &&
                    (!l.glu || (l.down && l.norm2 && l.ff_rows)),
                T5D_EINVAL, "t5d_hybrid_step: layer %d: null weights or buffers",
                run.layer);
    const t5d_experts& e = l.experts;
    T5D_REQUIRE(e.n == 0 ||
                    (m->streams > 0 && !l.glu && l.norm2 && e.top > 0 && e.F > 0 &&
                     e.glu && e.down && e.table && e.tiles && e.token_of &&
                     e.entry_of && e.rows && e.out &&
                     (e.shared_F == 0 || (e.shared_glu && e.shared_down &&
                                          e.shared_gate && e.shared_rows && e.gate))),
                T5D_EINVAL, "t5d_hybrid_step: layer %d: experts", run.layer);
    T5D_REQUIRE(m->streams >= 0 && (m->streams == 0 || !run.enter), T5D_EINVAL,
                "t5d_hybrid_step: %d streams, run %d", m->streams, r);
  }
  return T5D_OK;
}

int mixer(void* stream, const t5d_hybrid_model* m, const t5d_hybrid_layer& l,
          const t5d_hybrid_run& run, const t5d_ragged* b) {
  if (l.mix == T5D_MIX_WINDOW_ATTENTION) {
    t5d_window_attention a = l.attention;
    a.dtype = m->dtype; a.proj = m->proj; a.ld_proj = l.proj_n;
    a.key_ring = run.cache0; a.value_ring = run.cache1;
    a.q_rows = m->q_rows; a.out = l.mix_rows; a.ld_out = l.out_k;
    a.workspace =
        m->workspace_bytes >= t5d_window_workspace_bytes(b->S, a.H, a.D, a.Dv)
            ? m->workspace : nullptr;
    return t5d_window_attention_run(stream, &a, b, 0);
  }
  if (l.mix == T5D_MIX_LATENT_ATTENTION) {
    t5d_latent_attention a = l.latent;
    a.dtype = m->dtype; a.proj = m->proj; a.ld_proj = l.proj_n;
    a.latent_ring = run.cache0;
    a.out = l.mix_rows; a.ld_out = l.out_k;
    a.workspace = m->workspace_bytes >= t5d_latent_workspace_bytes(a.rank)
                      ? m->workspace : nullptr;
    return t5d_latent_attention_run(stream, &a, b, 0);
  }
  T5D_REQUIRE(l.mix == T5D_MIX_RECURRENCE, T5D_EINVAL, "t5d_hybrid_step: mixer %d",
              l.mix);
  t5d_recurrence a = l.recurrence;
  a.dtype = m->dtype; a.proj = m->proj; a.ld_proj = l.proj_n;
  a.low = m->low; a.ld_low = l.low_n;
  a.state = (float*)run.cache0; a.conv_ring = run.cache1;
  a.out = l.mix_rows; a.ld_out = l.out_k;
  a.workspace = m->workspace;
  a.workspace_bytes = m->workspace_bytes;
  return t5d_recurrence_run(stream, &a, b, 0);
}

// Tokens of the call by expert, for all layers that have experts.
int route(void* stream, const t5d_hybrid_model* m, const t5d_ragged* b) {
  t5d_route layers[16];
  int n = 0;
  for (int i = 0; i < m->n_layers; ++i) {
    const t5d_experts& e = m->layers[i].experts;
    if (e.n > 0) {
      t5d_route& r = layers[n++];
      r.experts = e.n; r.top = e.top;
      r.tile_rows = t5d_grouped_tile_rows(m->dtype, b->M * e.top, e.n);
      r.max_tiles = t5d_route_max_tiles(b->M * e.top, e.n, r.tile_rows);
      T5D_REQUIRE(r.max_tiles <= e.max_tiles, T5D_EINVAL,
                  "t5d_hybrid_step: layer %d has room for %d tiles of %d", i,
                  e.max_tiles, r.max_tiles);
      r.table = e.table; r.tiles = e.tiles;
      r.token_of = e.token_of; r.entry_of = e.entry_of;
    }
    if (n == 16 || (n > 0 && i + 1 == m->n_layers)) {
      T5D_TRY(t5d_route_tokens(stream, b->tokens, b->M, m->V, layers, n));
      n = 0;
    }
  }
  return T5D_OK;
}

// The chosen experts' outputs (rows of e.out) and the shared one's (m->y).
int experts(void* stream, const t5d_hybrid_model* m, const t5d_experts& e, int M) {
  const int dt = m->dtype, ld = m->ld;
  t5d_grouped_dense d = {};
  d.dtype = dt;
  d.tile_rows = t5d_grouped_tile_rows(dt, M * e.top, e.n);
  d.n_tiles = t5d_route_max_tiles(M * e.top, e.n, d.tile_rows);
  d.tiles = e.tiles;
  d.A = m->h; d.lda = ld; d.rows = e.token_of; d.K = ld;
  d.W = e.glu; d.w_stride = e.glu_stride; d.N = d.n_store = 2 * e.F;
  d.C = e.rows; d.ldc = e.F;
  d.epilogue = T5D_EPI_CLAMPED_GLU;
  d.glu_limit = e.limit; d.glu_alpha = e.alpha; d.glu_add = e.add;
  T5D_TRY(t5d_grouped_dense_run(stream, &d));
  d.A = e.rows; d.lda = e.F; d.rows = nullptr; d.K = e.F;
  d.W = e.down; d.w_stride = e.down_stride; d.N = d.n_store = ld;
  d.C = e.out; d.ldc = ld;
  d.epilogue = T5D_EPI_NONE;
  T5D_TRY(t5d_grouped_dense_run(stream, &d));
  if (e.shared_F == 0) return T5D_OK;
  const int F = e.shared_F;
  T5D_TRY(t5d_dense(stream, dt, dt, m->h, ld, e.shared_glu, e.shared_rows, F, 2 * F, M,
                    ld, 2 * F, T5D_EPI_CLAMPED_GLU, e.shared_limit, e.alpha, e.add));
  return t5d_dense(stream, dt, dt, e.shared_rows, F, e.shared_down, m->y, ld, ld, M, F,
                   ld, T5D_EPI_NONE, 0.f, 0.f, 0.f);
}

}  // namespace

extern "C" int t5d_hybrid_step(void* stream, const t5d_hybrid_model* m,
                               const t5d_ragged* b, const int32_t* want_rows,
                               int n_want, float* logits) {
  T5D_TRY(check_hybrid(m, b));
  T5D_REQUIRE(n_want >= 0 && (n_want == 0 || logits) &&
                  (want_rows || n_want == 0 || n_want == b->M),
              T5D_EINVAL, "t5d_hybrid_step: n_want=%d", n_want);
  GateScope gate(m->gate);
  const int dt = m->dtype, M = b->M, d = m->d, ld = m->ld;
  bool looped = false;
  for (int r = 0; r < m->n_runs; ++r) looped = looped || m->runs[r].enter;
  const bool hyper = m->streams > 0;
  if (hyper) {
    T5D_TRY(t5d_embed_streams(stream, dt, m->embedding, b->tokens, m->embed_scale,
                              m->x, M, d, ld, m->streams, m->V));
    T5D_TRY(route(stream, m, b));
  } else {
    T5D_TRY(t5d_embed_sinusoid(stream, dt, m->embedding, b->tokens, b->tok_pos, m->x,
                               looped ? m->x0 : nullptr, M, d, ld, m->V));
  }
  // A branch output waiting in m->y for the next row kernel, and its norm.
  const void* y = nullptr;
  const float* y_norm = nullptr;
  // With several streams: everything of the waiting branch (y, parts, how it
  // spreads), the rest filled in per call.
  t5d_hyper_norm wait = {};
  wait.dtype = dt; wait.d = d; wait.ld = ld; wait.streams = m->streams;
  wait.eps = m->eps; wait.x = m->x;
  const t5d_hyper_norm none = wait;
  struct Collect {  // what is formed of the streams
    const float *weights, *norm;
    void* out;
    float* sum;
    const int32_t* rows;
    const float* gate_w;
    float* gate;
  };
  auto collect = [&](const Collect& c, int n) {
    t5d_hyper_norm a = wait;
    wait = none;
    a.collect = c.weights; a.norm = c.norm; a.out = c.out; a.sum = c.sum;
    a.rows = c.rows; a.gate_w = c.gate_w; a.gate_out = c.gate;
    return t5d_hyper_norm_run(stream, &a, n);
  };
  auto row = [&](const float* add, const float* norm, const float* x0, void* out) {
    const int rc = t5d_stream_norm(stream, dt, dt, y, y_norm, add, m->x, norm, x0,
                                   nullptr, out, M, d, ld, m->eps);
    y = nullptr;
    y_norm = nullptr;
    return rc;
  };
  auto branch = [&](const void* in, int k, const void* w, const float* norm) {
    y = m->y;
    y_norm = norm;
    return t5d_dense(stream, dt, dt, in, k, w, m->y, ld, ld, M, k, ld, T5D_EPI_NONE,
                     0.f, 0.f, 0.f);
  };
  for (int r = 0; r < m->n_runs; ++r) {
    const t5d_hybrid_run& run = m->runs[r];
    const t5d_hybrid_layer& l = m->layers[run.layer];
    if (run.enter) {
      T5D_TRY(row(nullptr, nullptr, m->x0, m->cat));
      T5D_TRY(t5d_dense(stream, dt, T5D_F32, m->cat, 2 * ld, m->loop_in, m->x, ld,
                        ld, M, 2 * ld, ld, T5D_EPI_NONE, 0.f, 0.f, 0.f));
    }
    if (hyper)
      T5D_TRY(collect({l.in1, l.norm1, m->h}, M));
    else
      T5D_TRY(row(run.enter ? run.enter_add : nullptr, l.norm1, nullptr, m->h));
    T5D_TRY(t5d_dense(stream, dt, dt, m->h, ld, l.proj, m->proj, l.proj_n, l.proj_n,
                      M, ld, l.proj_n, T5D_EPI_NONE, 0.f, 0.f, 0.f));
    if (l.low) {
      const char* a = (const char*)m->proj + (size_t)l.off_low * (dt == T5D_F32 ? 4 : 2);
      T5D_TRY(t5d_dense(stream, dt, T5D_F32, a, l.proj_n, l.low, m->low, l.low_n,
                        l.low_n, M, l.low_k, l.low_n, T5D_EPI_NONE, 0.f, 0.f, 0.f));
    }
    T5D_TRY(mixer(stream, m, l, run, b));
    T5D_TRY(branch(l.mix_rows, l.out_k, l.out, l.norm1b));
    if (hyper) {
      wait.y = m->y; wait.mix = l.mix1; wait.spread = l.out1;
    }
    if (l.experts.n > 0) {
      const t5d_experts& e = l.experts;
      T5D_TRY(collect({l.in2, l.norm2, m->h, nullptr, nullptr,
                       e.shared_F ? e.shared_gate : nullptr, e.gate}, M));
      T5D_TRY(experts(stream, m, e, M));
      wait.parts = e.out; wait.part_row = e.entry_of; wait.top = e.top;
      wait.part_weight = 1.0f / (float)e.top;
      if (e.shared_F) {
        wait.y = m->y;
        wait.y_gate = e.gate;
      }
      wait.mix = l.mix2; wait.spread = l.out2;
    }
    if (l.glu) {
      if (hyper)
        T5D_TRY(collect({l.in2, l.norm2, m->h}, M));
      else
        T5D_TRY(row(nullptr, l.norm2, nullptr, m->h));
      T5D_TRY(t5d_dense(stream, dt, dt, m->h, ld, l.glu, l.ff_rows, l.F, 2 * l.F, M,
                        ld, 2 * l.F, T5D_EPI_CLAMPED_GLU, l.glu_limit, l.glu_alpha, l.glu_add));
      T5D_TRY(branch(l.ff_rows, l.F, l.down, l.norm2b));
      if (hyper) {
        wait.y = m->y; wait.mix = l.mix2; wait.spread = l.out2;
      }
    }
    if (m->trace && hyper) {
      T5D_TRY(collect({nullptr, nullptr, nullptr, m->trace + (size_t)r * M * ld}, M));
    } else if (m->trace) {
      T5D_TRY(row(nullptr, nullptr, nullptr, nullptr));
      const size_t n = (size_t)M * ld;
      const hipError_t e =
          hipMemcpyAsync(m->trace + (size_t)r * n, m->x, n * sizeof(float),
                         hipMemcpyDeviceToDevice, as_stream(stream));
      T5D_REQUIRE(e == hipSuccess, T5D_EHIP, "t5d_hybrid_step: trace copy: %s",
                  hipGetErrorString(e));
    }
  }
  if (n_want == 0) return T5D_OK;  // the last branch feeds nothing but the logits
  if (hyper) {
    if (want_rows && (wait.y || wait.parts))
      T5D_TRY(collect({nullptr, nullptr, nullptr, nullptr}, M));
    T5D_TRY(collect({nullptr, m->final_norm, m->h, nullptr, want_rows}, n_want));
  } else if (want_rows) {
    if (y) T5D_TRY(row(nullptr, nullptr, nullptr, nullptr));
    T5D_TRY(t5d_stream_norm(stream, dt, dt, nullptr, nullptr, nullptr, m->x,
                            m->final_norm, nullptr, want_rows, m->h, n_want, d, ld,
                            m->eps));
  } else {
    T5D_TRY(row(nullptr, m->final_norm, nullptr, m->h));
  }
  return t5d_dense(stream, dt, T5D_F32, m->h, ld, m->head, logits, m->V, m->V, n_want,
                   ld, m->head_n, T5D_EPI_NONE, 0.f, 0.f, 0.f);
}
