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
  }
  add((int)c->vocab_p, c->width_p);
  // keys and values written out from the latents: rows in whole tiles of 64
  size_t ws = 0;
  for (int i = 0; i < c->n_layers; ++i) {
    const ChattsMixLayer& l = layers[i];
    bool seen = l.kind != CHATTS_MIX_LATENT || !l.ukx;
    for (int j = 0; j < i && !seen; ++j)
      seen = layers[j].kind == CHATTS_MIX_LATENT && layers[j].ukx && layers[j].latent.heads == l.latent.heads && layers[j].dim_p == l.dim_p &&
             layers[j].vdim_p == l.vdim_p && layers[j].latent.rank_p == l.latent.rank_p;
    for (int n = 64; !seen && n <= c->expand_rows; n += 64) {
      const size_t a = chatts_linear_workspace(n, l.latent.heads * l.dim_p, l.latent.rank_p), b = chatts_linear_workspace(l.latent.heads * l.vdim_p, n, l.latent.rank_p);
      if (a > ws) ws = a;
      if (b > ws) ws = b;
    }
  }
  const size_t am = argmax_scratch_bytes(c->max_slots > 1 ? c->max_slots : 1);
  if (am > ws) ws = am;
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

static ChattsOperand rows_from(ChattsOperand o, int row) {
  const size_t at = (size_t)row * o.ld;
  if (o.f32) o.f32 += at;
  if (o.hi) o.hi += at;
  if (o.lo) o.lo += at;
  return o;
}

// absorbed attention for rows r0 .. r0 + n (a: prepared for the whole batch)
static int mix_latent_absorbed(const ChattsMixDecoder* d, const ChattsMixLayer& l, ChattsLatentArgs a, int r0, int n, const ChattsOperand& out, chatts_stream_t s) {
  const int cw = a.rank_p + a.rot_p;
  a.rows += r0; a.n_rows = n;
  a.q = rows_from(a.q, r0);
  a.o = d->b.o_lat + (size_t)r0 * a.heads * a.rank_p;
  int rc;
  ChattsHeadLinearArgs h{};
  h.a = a.proj + (size_t)r0 * a.ld_proj + a.off_q; h.lda = a.ld_proj; h.a_head = l.dim_p;
  h.w = l.uk; h.m = n; h.heads = a.heads; h.n = a.rank_p; h.k = l.dim_p; h.out = a.q; h.out_head = cw; h.exact = d->c.exact;
  if ((rc = chatts_head_linear(&h, s)) != 0) return rc;
  // few rows: the keys of a row are spread over workgroups (32 at a time) until there is about one per CU
  const int groups = (a.heads + 31) / 32 * n;
  int splits = groups >= 256 ? 1 : 256 / groups;
  const int most = (d->c.max_ctx + 63) / 64;
  if (splits > most) splits = most;
  if (splits > 64) splits = 64;
  while (splits > 1 && (size_t)n * a.heads * splits * (a.rank_p + 4) > d->b.partial_elems) --splits;
  a.n_splits = splits; a.partial = d->b.partial;
  if ((rc = chatts_latent_attend(&a, s)) != 0) return rc;
  h.a = a.o; h.lda = a.heads * a.rank_p; h.a_head = a.rank_p;
  h.w = l.uv; h.n = l.vdim_p; h.k = a.rank_p; h.out = rows_from(out, r0); h.out_head = l.out_head;
  return chatts_head_linear(&h, s);
}

static int mix_latent(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, const ChattsSpan* spans, int n_spans, bool single,
                      const ChattsOperand& out, chatts_stream_t s) {
  StageRange stage("chatts.mix.latent");
  ChattsLatentArgs a = l.latent;
  a.proj = d->b.proj; a.ld_proj = l.in_n; a.dim_p = l.dim_p;
  a.cache = run.cache; a.cache_f32 = d->c.exact;
  a.table = d->b.table; a.table_stride = d->c.table_stride; a.log_block = kv_log_block(d->c.block_size);
  a.rows = d->b.rows; a.n_rows = t; a.eps = d->c.eps; a.n_splits = 1;
  a.q = ChattsOperand{};
  a.q.ld = a.heads * (a.rank_p + a.rot_p);
  int expanded = 0;
  if (!single && l.ukx)
    for (int i = 0; i < n_spans; ++i) expanded += spans[i].base >= 0;
  if (single || expanded < n_spans) {      // some rows run absorbed
    if (d->c.exact) a.q.f32 = d->b.q_f32;
    else { a.q.hi = d->b.q_hi; a.q.lo = d->b.q_lo; }
  }
  if (expanded) a.qx = d->b.qx;
  int rc;
  if ((rc = chatts_latent_prep(&a, s)) != 0) return rc;
  if (expanded) {
    ChattsLatentExpandArgs x{};
    x.latent = &a; x.spans = spans; x.spans_dev = d->b.spans; x.n_spans = n_spans; x.vdim_p = l.vdim_p; x.out_head = l.out_head; x.max_rows = d->c.expand_rows;
    x.uk = l.ukx; x.uv = l.uvx; x.cbuf = d->b.cbuf; x.krbuf = d->b.krbuf; x.zero = d->b.zero;
    x.k_hi = d->b.kx_hi; x.k_lo = d->b.kx_lo; x.v_hi = d->b.vx_hi; x.v_lo = d->b.vx_lo;
    x.out = out; x.workspace = d->b.workspace; x.workspace_bytes = d->b.workspace_bytes;
    if ((rc = chatts_latent_expanded(&x, s)) != 0) return rc;
    if (expanded == n_spans) return CHATTS_OK;
  }
  if (!expanded) return mix_latent_absorbed(d, l, a, 0, t, out, s);
  for (int i = 0; i < n_spans;) {          // runs of neighbouring spans that are not expanded
    if (spans[i].base >= 0) { ++i; continue; }
    const int r0 = spans[i].row0;
    int n = 0;
    for (; i < n_spans && spans[i].base < 0; ++i) n += spans[i].t;
    if ((rc = mix_latent_absorbed(d, l, a, r0, n, out, s)) != 0) return rc;
  }
  return CHATTS_OK;
}

// The absorbed form costs ~(2 rank + rot) products per query, key and head, the expanded one (dim + rot + vdim) plus rank (dim + vdim) per key and
// head for writing keys and values out (two passes).  The absorbed kernel serves 16 heads of ONE query per workgroup and fetches the keys again
// for every query: measured, a product costs about four times as much there.
extern "C" int chatts_mixdec_plan(ChattsMixDecoder* d, ChattsSpan* spans, int n_spans) {
  CHATTS_REQUIRE(d && spans && n_spans >= 0, CHATTS_E_BADARG, "mixdec_plan: null argument");
  const ChattsMixLayer* l = nullptr;
  for (const ChattsMixLayer& x : d->layers)
    if (x.kind == CHATTS_MIX_LATENT && x.ukx) { l = &x; break; }
  int rows = 0;
  for (int i = 0; i < n_spans; ++i) {
    ChattsSpan& sp = spans[i];
    sp.base = -1;
    if (!l || d->c.expand_rows <= 0 || sp.t < 8) continue;
    const double own = 4.0 * sp.t * (2.0 * l->latent.rank_p + l->latent.rot_p);
    const double exp = sp.t * (double)(l->dim_p + l->latent.rot_p + l->vdim_p) + 2.0 * l->latent.rank_p * (l->dim_p + l->vdim_p);
    const int need = (sp.pos0 + sp.t + 63) & ~63;
    if (own <= exp || rows + need > d->c.expand_rows) continue;
    sp.base = rows;
    rows += need;
  }
  return CHATTS_OK;
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
  a.q = d->b.dq; a.k = d->b.dk; a.v = d->b.dv; a.g = d->b.dg; a.gate = d->b.dgate; a.beta = d->b.dbeta; a.chunks = d->b.dchunks; a.o = d->b.dout;
  a.exact = d->c.exact;
  int rc;
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

extern "C" int chatts_mixdec_forward(ChattsMixDecoder* d, const int64_t* tokens, int t, const ChattsSpan* spans, int n_spans, int single, chatts_stream_t s) {
  CHATTS_REQUIRE(d && tokens && (single || spans), CHATTS_E_BADARG, "mixdec_forward: null argument");
  const ChattsMixConfig& c = d->c;
  CHATTS_REQUIRE(t >= 1 && t <= c.t_max && (single || (n_spans >= 1 && n_spans <= c.max_slots)), CHATTS_E_SHAPE, "mixdec_forward: %d rows in %d segments", t, n_spans);
  if (!single) {
    int rows = 0;
    for (int i = 0; i < n_spans; ++i) {
      CHATTS_REQUIRE(spans[i].row0 == rows && spans[i].t >= 1, CHATTS_E_SHAPE, "mixdec_forward: segment %d starts at row %d, not %d", i, spans[i].row0, rows);
      rows += spans[i].t;
    }
    CHATTS_REQUIRE(rows == t, CHATTS_E_SHAPE, "mixdec_forward: segments hold %d of %d rows", rows, t);
  }
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
    rc = l.kind == CHATTS_MIX_LATENT ? mix_latent(d, l, run, t, spans, n_spans, single != 0, B, s) : mix_delta(d, l, run, t, n_spans, single != 0, B, s);
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
  if (const int rc = chatts_mixdec_forward(d, token, batch, nullptr, 0, 1, s)) return rc;
  return chatts_mixdec_logits(d, nullptr, batch, logits, s);
}
