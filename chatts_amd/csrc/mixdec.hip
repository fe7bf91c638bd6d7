// mixdec.hip - host-side composition of decoders with mixed layers (latent attention / gated delta rule, norms before and after each
// sublayer, looped layer ranges).  Like decoder.hip: nothing here allocates or synchronises, a decode step is capturable.
//
// A layer:   norm1 (in the previous residual_norm launch) -> stacked input projection -> mixer kernels -> out projection
//            -> residual_norm (x += norm1b(y); norm2(x)) -> up (squared relu in the epilogue) -> down -> residual_norm (..., next norm1)
// Operands between the launches travel in the format the next projection's kernel takes for this row count: bf16 hi / lo planes
// (2 .. 16 rows: weight-streaming kernel; >= 96 rows: the prefill kernel) or float32.
#include <new>
#include <vector>

#include "common.h"

namespace chatts {

__global__ __launch_bounds__(256) void rows_from_pos_kernel(ChattsRow* __restrict__ rows, const int32_t* __restrict__ pos, int n) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) rows[i] = ChattsRow{i, pos[i], i, 0};
}

__global__ __launch_bounds__(256) void gather_rows_kernel(const float* __restrict__ x, const int32_t* __restrict__ index, float* __restrict__ out, int ld) {
  const float* src = x + (size_t)index[blockIdx.x] * ld;
  float* dst = out + (size_t)blockIdx.x * ld;
  for (int c = threadIdx.x * 4; c < ld; c += 1024) *reinterpret_cast<f32x4*>(dst + c) = *reinterpret_cast<const f32x4*>(src + c);
}

}  // namespace chatts

using namespace chatts;

struct ChattsMixDecoder {
  ChattsMixConfig c;
  ChattsMixBuffers b;
  std::vector<ChattsMixLayer> layers;
  std::vector<ChattsMixRun> runs;
};

static bool mix_planes(const ChattsMixConfig& c, int m, int k) { return !c.exact && k % 64 == 0 && ((m >= 2 && m <= 16) || m >= 96); }

extern "C" size_t chatts_mixdec_workspace(const ChattsMixConfig* c, const ChattsMixLayer* layers) {
  if (!c || !layers) return 0;
  std::vector<std::pair<int, int>> shapes;
  auto add = [&](int n, int k) {
    for (auto& s : shapes) if (s.first == n && s.second == k) return;
    if (n > 0 && k > 0) shapes.emplace_back(n, k);
  };
  for (int i = 0; i < c->n_layers; ++i) {
    const ChattsMixLayer& l = layers[i];
    add(l.in_n, c->width_p);
    add(c->width_p, l.out_k);
    if (l.up) { add(l.ff, c->width_p); add(c->width_p, l.ff); }
    if (l.kind == CHATTS_MIX_DELTA) { add(l.dt_n, l.delta.ld_a2); add(l.gate_n, l.delta.ld_g2); }
  }
  add((int)c->vocab_p, c->width_p);
  size_t ws = argmax_scratch_bytes(c->max_slots > 1 ? c->max_slots : 1);
  for (int t = 2; t <= c->t_max; ++t)
    for (auto& s : shapes) {
      const size_t w = chatts_linear_workspace(t, s.first, s.second);
      if (w > ws) ws = w;
    }
  return ws + 256;
}

extern "C" ChattsMixDecoder* chatts_mixdec_create(const ChattsMixConfig* c, const ChattsMixLayer* layers, const ChattsMixRun* runs, const ChattsMixBuffers* b) {
  if (!c || !layers || !runs || !b) { set_error("mixdec_create: null argument"); return nullptr; }
  if (c->n_layers < 1 || c->n_runs < 1 || c->width < 1 || c->width_p < c->width || c->width_p % 64) { set_error("mixdec_create: bad sizes"); return nullptr; }
  if (kv_log_block(c->block_size) < 0) { set_error("mixdec_create: pages of %d tokens (power of two, 64 .. 32768)", c->block_size); return nullptr; }
  for (int i = 0; i < c->n_runs; ++i)
    if (runs[i].layer < 0 || runs[i].layer >= c->n_layers) { set_error("mixdec_create: run %d names layer %d", i, runs[i].layer); return nullptr; }
  for (int i = 0; i < c->n_layers; ++i) {
    const ChattsMixLayer& l = layers[i];
    if ((l.kind != CHATTS_MIX_LATENT && l.kind != CHATTS_MIX_DELTA) || !l.in || !l.out || !l.norm1 || (l.up && !(l.down && l.norm2))) {
      set_error("mixdec_create: layer %d is incomplete", i);
      return nullptr;
    }
  }
  ChattsMixDecoder* d = new (std::nothrow) ChattsMixDecoder();
  if (!d) { set_error("mixdec_create: out of host memory"); return nullptr; }
  d->c = *c;
  d->b = *b;
  d->layers.assign(layers, layers + c->n_layers);
  d->runs.assign(runs, runs + c->n_runs);
  return d;
}

extern "C" void chatts_mixdec_destroy(ChattsMixDecoder* d) { delete d; }

// operand buffer A (normed stream) or B (mixer output, activation) in the form a projection over k takes for m rows
static ChattsOperand operand(const ChattsMixDecoder* d, bool second, int m, int k) {
  ChattsOperand o{};
  o.ld = k;
  if (mix_planes(d->c, m, k)) {
    o.hi = second ? d->b.b_hi : d->b.a_hi;
    o.lo = second ? d->b.b_lo : d->b.a_lo;
  } else {
    o.f32 = second ? d->b.b_f32 : d->b.a_f32;
  }
  return o;
}

static int mix_linear(const ChattsMixDecoder* d, const ChattsOperand& in, const chatts_bf16* w, const chatts_bf16* w_t, int m, int n, int k, int epilogue,
                      const ChattsOperand& out, chatts_stream_t s) {
  ChattsLinearArgs a{};
  a.a = in.f32;
  a.lda = in.ld;
  if (!in.f32) { a.a_hi = in.hi; a.a_lo = in.lo; a.ld_planes = in.ld; }
  a.w = w; a.ldw = k; a.w_tiled = w_t;
  a.m = m; a.n = n; a.k = k; a.epilogue = epilogue;
  a.c = out.f32; a.ldc = out.ld;
  if (!out.f32) { a.c_hi = out.hi; a.c_lo = out.lo; a.ld_cplanes = out.ld; }
  a.exact_f32 = d->c.exact;
  a.workspace = d->b.workspace; a.workspace_bytes = d->b.workspace_bytes;
  return chatts_linear(&a, s);
}
static ChattsOperand f32_out(float* p, int ld) {
  ChattsOperand o{};
  o.f32 = p;
  o.ld = ld;
  return o;
}

static int mix_latent(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, const ChattsOperand& out, chatts_stream_t s) {
  StageRange stage("chatts.mix.latent");
  ChattsLatentArgs a = l.latent;
  const int cw = a.rank_p + a.rot_p;
  a.proj = d->b.proj; a.ld_proj = l.in_n;
  a.cache = run.cache; a.cache_f32 = d->c.exact;
  a.table = d->b.table; a.table_stride = d->c.table_stride; a.log_block = kv_log_block(d->c.block_size);
  a.rows = d->b.rows; a.n_rows = t; a.eps = d->c.eps;
  a.q = ChattsOperand{};
  a.q.ld = a.heads * cw;
  if (d->c.exact) a.q.f32 = d->b.q_f32;
  else { a.q.hi = d->b.q_hi; a.q.lo = d->b.q_lo; }
  a.o = d->b.o_lat;
  int rc;
  if ((rc = chatts_latent_prep(&a, s)) != 0) return rc;
  ChattsHeadLinearArgs h{};
  h.a = d->b.proj + a.off_q; h.lda = l.in_n; h.a_head = l.dim_p;
  h.w = l.uk; h.m = t; h.heads = a.heads; h.n = a.rank_p; h.k = l.dim_p; h.out = a.q; h.out_head = cw; h.exact = d->c.exact;
  if ((rc = chatts_head_linear(&h, s)) != 0) return rc;
  // few rows: the keys of a row are spread over workgroups until the chip has ~2 per CU
  const int tiles = (a.heads + 15) / 16 * t;
  int splits = tiles >= 512 ? 1 : 512 / tiles;
  if (splits > 64) splits = 64;
  const int most = (d->c.max_ctx + 63) / 64;
  if (splits > most) splits = most;
  while (splits > 1 && (size_t)t * a.heads * splits * (a.rank_p + 2) > d->b.partial_elems) --splits;
  a.n_splits = splits; a.partial = d->b.partial;
  if ((rc = chatts_latent_attend(&a, s)) != 0) return rc;
  h.a = d->b.o_lat; h.lda = a.heads * a.rank_p; h.a_head = a.rank_p;
  h.w = l.uv; h.n = l.vdim_p; h.k = a.rank_p; h.out = out; h.out_head = l.out_head;
  return chatts_head_linear(&h, s);
}

static int mix_delta(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, int n_spans, bool single, const ChattsOperand& out,
                     chatts_stream_t s) {
  StageRange stage("chatts.mix.delta");
  ChattsDeltaArgs a = l.delta;
  a.proj = d->b.proj; a.ld_proj = l.in_n; a.eps = d->c.eps;
  a.state = run.state; a.ring = run.ring;
  a.rows = d->b.rows; a.n_rows = t; a.spans = d->b.spans; a.n_spans = n_spans;
  a.out = out;
  if (single) return chatts_delta_decode(&a, s);
  a.q = d->b.dq; a.k = d->b.dk; a.v = d->b.dv; a.g = d->b.dg; a.gate = d->b.dgate; a.beta = d->b.dbeta; a.o = d->b.dout;
  a.dt = d->b.ddt; a.ld_dt = l.dt_n; a.ld_gate = l.gate_n;
  int rc;
  if ((rc = mix_linear(d, f32_out(d->b.proj + a.off_a, l.in_n), a.a2, nullptr, t, l.dt_n, a.ld_a2, CHATTS_EPI_NONE, f32_out(d->b.ddt, l.dt_n), s)) != 0) return rc;
  if ((rc = mix_linear(d, f32_out(d->b.proj + a.off_g, l.in_n), a.g2, nullptr, t, l.gate_n, a.ld_g2, CHATTS_EPI_NONE, f32_out(d->b.dgate, l.gate_n), s)) != 0) return rc;
  if ((rc = chatts_delta_prep(&a, s)) != 0) return rc;
  if ((rc = chatts_delta_scan(&a, s)) != 0) return rc;
  return chatts_delta_out(&a, s);
}

static int mix_norm(const ChattsMixDecoder* d, int t, const float* y, const float* post, const float* add, const float* pre, const ChattsOperand& out,
                    chatts_stream_t s) {
  ChattsResidualNormArgs a{};
  a.x = d->b.x; a.y = y; a.post_w = post; a.add = add; a.pre_w = pre; a.out = out;
  a.t = t; a.width = d->c.width; a.ldx = a.ldy = d->c.width_p; a.eps = d->c.eps;
  return chatts_residual_norm(&a, s);
}

extern "C" int chatts_mixdec_forward(ChattsMixDecoder* d, const int64_t* tokens, int t, int n_spans, int single, chatts_stream_t s) {
  CHATTS_REQUIRE(d && tokens, CHATTS_E_BADARG, "mixdec_forward: null argument");
  const ChattsMixConfig& c = d->c;
  CHATTS_REQUIRE(t >= 1 && t <= c.t_max && (single || (n_spans >= 1 && n_spans <= c.max_slots)), CHATTS_E_SHAPE, "mixdec_forward: %d rows in %d segments", t, n_spans);
  StageRange stage(single ? "chatts.mix.decode" : "chatts.mix.prefill");
  int rc;
  if ((rc = chatts_embed_token_batched(tokens, t, d->b.embed, 0, c.vocab, c.width_p, d->b.x, s)) != 0) return rc;
  const ChattsOperand A = operand(d, false, t, c.width_p), Y = f32_out(d->b.y, c.width_p);
  if ((rc = mix_norm(d, t, nullptr, nullptr, d->runs[0].add, d->layers[d->runs[0].layer].norm1, A, s)) != 0) return rc;
  for (int r = 0; r < c.n_runs; ++r) {
    const ChattsMixRun& run = d->runs[r];
    const ChattsMixLayer& l = d->layers[run.layer];
    const ChattsMixRun* next = r + 1 < c.n_runs ? &d->runs[r + 1] : nullptr;
    const float* next_add = next ? next->add : nullptr;
    const float* next_norm = next ? d->layers[next->layer].norm1 : nullptr;
    if ((rc = mix_linear(d, A, l.in, l.in_t, t, l.in_n, c.width_p, CHATTS_EPI_NONE, f32_out(d->b.proj, l.in_n), s)) != 0) return rc;
    const ChattsOperand B = operand(d, true, t, l.out_k);
    rc = l.kind == CHATTS_MIX_LATENT ? mix_latent(d, l, run, t, B, s) : mix_delta(d, l, run, t, n_spans, single != 0, B, s);
    if (rc) return rc;
    if ((rc = mix_linear(d, B, l.out, l.out_t, t, c.width_p, l.out_k, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    if (!l.up) {
      if ((rc = mix_norm(d, t, d->b.y, l.norm1b, next_add, next_norm, A, s)) != 0) return rc;
      continue;
    }
    if ((rc = mix_norm(d, t, d->b.y, l.norm1b, nullptr, l.norm2, A, s)) != 0) return rc;
    const ChattsOperand F = operand(d, true, t, l.ff);
    if ((rc = mix_linear(d, A, l.up, l.up_t, t, l.ff, c.width_p, CHATTS_EPI_RELU2, F, s)) != 0) return rc;
    if ((rc = mix_linear(d, F, l.down, l.down_t, t, c.width_p, l.ff, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    if ((rc = mix_norm(d, t, d->b.y, l.norm2b, next_add, next_norm, A, s)) != 0) return rc;
  }
  return CHATTS_OK;
}

extern "C" int chatts_mixdec_logits(ChattsMixDecoder* d, const int32_t* index, int n, float* logits, chatts_stream_t s) {
  CHATTS_REQUIRE(d && logits, CHATTS_E_BADARG, "mixdec_logits: null argument");
  const ChattsMixConfig& c = d->c;
  CHATTS_REQUIRE(n >= 0 && n <= c.t_max, CHATTS_E_SHAPE, "mixdec_logits: %d rows", n);
  if (n == 0) return CHATTS_OK;
  StageRange stage("chatts.mix.logits");
  ChattsResidualNormArgs a{};
  a.x = d->b.x;
  if (index) {
    hipLaunchKernelGGL(gather_rows_kernel, dim3(n), dim3(256), 0, as_stream(s), d->b.x, index, d->b.y, c.width_p);
    CHATTS_CHECK_LAUNCH("gather_rows");
    a.x = d->b.y;
  }
  a.pre_w = d->b.final_norm;
  a.out = operand(d, false, n, c.width_p);
  a.t = n; a.width = c.width; a.ldx = a.ldy = c.width_p; a.eps = c.eps;
  if (const int rc = chatts_residual_norm(&a, s)) return rc;
  return mix_linear(d, a.out, d->b.head, d->b.head_t, n, (int)c.vocab_p, c.width_p, CHATTS_EPI_NONE, f32_out(logits, (int)c.vocab_p), s);
}

extern "C" int chatts_mixdec_decode(ChattsMixDecoder* d, int batch, const int64_t* token, const int32_t* pos, float* logits, chatts_stream_t s) {
  CHATTS_REQUIRE(d && token && pos && batch >= 1 && batch <= d->c.max_slots, CHATTS_E_BADARG, "mixdec_decode: batch %d", batch);
  hipLaunchKernelGGL(rows_from_pos_kernel, dim3((batch + 255) / 256), dim3(256), 0, as_stream(s), d->b.rows, pos, batch);
  CHATTS_CHECK_LAUNCH("rows_from_pos");
  if (const int rc = chatts_mixdec_forward(d, token, batch, 0, 1, s)) return rc;
  return chatts_mixdec_logits(d, nullptr, batch, logits, s);
}
