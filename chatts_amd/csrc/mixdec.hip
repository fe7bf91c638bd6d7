// mixdec.hip - host-side composition of decoders with mixed layers (latent attention, gated delta rule, gated linear recurrences, windowed attention, minimal
// gated recurrence, selective scan; feed-forwards or experts; looped layer ranges).  Like decoder.hip: nothing here allocates or synchronises, a decode step is capturable.
//
// Sequential layer (norms before and after each sublayer):
//   norm1 (in the previous residual_norm launch) -> stacked input projection -> mixer kernels -> out projection
//   -> residual_norm (x += norm1b(y); norm2(x)) -> up (squared relu in the epilogue) -> down -> residual_norm (..., next norm1)
// Parallel layer (two norms of the same x):
//   pair_norm (norm1(x), norm2(x), with the experts' sum of the layer before, the token shift of a decoded token) -> input projections -> mixer kernels
//   -> out projection, added to x -> gate_up (gated unit in the epilogue) -> down, added to x;  or router -> experts, added by the next pair_norm
// Layer with its norms after the sums (sublayers read x itself):
//   input projections -> mixer kernels -> out projection -> post_norm (x = norm1(alpha x + y), as the next operand too)
//   -> gate_up (gated unit in the epilogue) -> down;  or router -> experts, beside a shared one: up -> down -> post_norm (x = norm2(alpha x + y + experts))
// Layer with norms before its sublayers only (a factor of what is added; the streams of all layers averaged after each):
//   input projections -> mixer kernels, two mixers side by side writing neighbouring columns of one operand -> out projection
//   -> depth_norm (x += mult y; norm2(x)) -> router -> experts, beside a shared one: gate_up -> down
//   -> depth_norm (x += mult (y + experts); average over depth; the next layer's norm1)
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

static int mix_equal_blocks(const ChattsMixLayer& l, int i) {      // how many operand blocks from i on have the size of block i
  const int rows = l.mix_row[i + 1] - l.mix_row[i];
  int n = 1;
  while (i + n < l.n_mix && l.mix_row[i + n + 1] - l.mix_row[i + n] == rows) ++n;
  return n;
}

static bool mix_pairs(const ChattsMixLayer& l) {      // `up` holds gate and up rows
  return l.ff_kind == CHATTS_FF_CLAMPGLU || l.ff_kind == CHATTS_FF_GEGLU || (l.ff_kind == CHATTS_FF_MOE && l.pre);
}
static bool mix_has(const ChattsMixLayer& l, int kind) { return l.kind == kind || l.beside == kind; }

extern "C" size_t chatts_mixdec_workspace(const ChattsMixConfig* c, const ChattsMixLayer* layers) {
  if (!c || !layers) return 0;
  std::vector<std::pair<int, int>> shapes;
  auto add = [&](int n, int k) {
    for (auto& s : shapes) if (s.first == n && s.second == k) return;
    if (n > 0 && k > 0) shapes.emplace_back(n, k);
  };
  for (int i = 0; i < c->n_layers; ++i) {
    const ChattsMixLayer& l = layers[i];
    for (int j = 0; j < l.n_mix; ++j) add(l.mix_row[j + 1] - l.mix_row[j], c->width_p);
    if (!l.n_mix) add(l.in_n, c->width_p);
    add(c->width_p, l.out_k);
    if (l.w2) add(l.w2_n, l.recur.rank);
    if (l.up) { add(mix_pairs(l) ? 2 * l.ff : l.ff, c->width_p); add(c->width_p, l.ff); }
    if (l.router) add(l.router_n, c->width_p);
    if (l.sel_low) { add(l.select.ld_low, l.sel_k); add(l.sel_dt_n, l.select.rank); }
  }
  add(c->width_p, 2 * c->width_p);
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
  for (int i = 0; i < c->n_layers; ++i)
    for (int j = 0, n; j < layers[i].n_mix; j += n) {
      n = mix_equal_blocks(layers[i], j);
      for (int t = 2; t <= 16 && t <= c->t_max; ++t) {
        const size_t w = chatts_linear_workspace_batch(t, layers[i].mix_row[j + 1] - layers[i].mix_row[j], c->width_p, n);
        if (w > ws) ws = w;
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
  for (int i = 0; i < c->n_runs; ++i)
    if (layers[runs[i].layer].depth && b->stream_stride < (int64_t)c->t_max * c->width_p) { set_error("mixdec_create: streams of %lld values", (long long)b->stream_stride); return nullptr; }
  for (int i = 0; i < c->n_layers; ++i) {
    const ChattsMixLayer& l = layers[i];
    const bool pair = l.kind == CHATTS_MIX_RECUR || l.kind == CHATTS_MIX_WINDOW;
    if (l.kind < CHATTS_MIX_LATENT || l.kind > CHATTS_MIX_SELECT || !l.in || !l.out || !l.norm1 || (l.up && !(l.down && l.norm2)) ||
        (l.ff_kind == CHATTS_FF_MOE && !(l.router && l.norm2 && l.moe.gate_up && l.moe.down)) || l.n_mix < 0 || l.n_mix > 7 || (l.n_mix && !l.mu)) {
      set_error("mixdec_create: layer %d is incomplete", i);
      return nullptr;
    }
    if (l.pre || layers[0].pre) {
      auto fits = [&](int kind) { return kind == CHATTS_MIX_WINDOW || kind == CHATTS_MIX_GRU || kind == CHATTS_MIX_SELECT; };
      if (!l.pre || !layers[0].pre || l.parallel || l.post || !fits(l.kind) || (l.beside && (!fits(l.beside) || l.beside == l.kind || l.beside_col < 0 || l.beside_col >= l.out_k)) ||
          (l.ff_kind != CHATTS_FF_NONE && l.ff_kind != CHATTS_FF_CLAMPGLU && l.ff_kind != CHATTS_FF_MOE) || (l.ff_kind != CHATTS_FF_NONE && !l.norm2) ||
          (l.ff_kind == CHATTS_FF_CLAMPGLU && !l.up) || (l.depth && !b->streams) || (mix_has(l, CHATTS_MIX_WINDOW) && l.window.ld_vfirst && !b->vfirst) ||
          (mix_has(l, CHATTS_MIX_SELECT) && !(l.sel_low && l.sel_dt && b->sel_u && b->sel_low && b->sel_delta && (c->exact || (b->sel_u_hi && b->sel_dt_hi))))) {
        set_error("mixdec_create: layer %d: a layer with norms before its sublayers has attention, minimal recurrence or selective scan (one or two of them) and a clamped "
                  "gated unit, experts or nothing", i);
        return nullptr;
      }
      continue;
    }
    if (l.kind > CHATTS_MIX_WINDOW || l.beside) { set_error("mixdec_create: layer %d: this mixer needs norms before its sublayers only", i); return nullptr; }
    if (l.post || layers[0].post) {
      if (!l.post || !layers[0].post || l.parallel || l.kind != CHATTS_MIX_WINDOW || (l.ff_kind != CHATTS_FF_NONE && !l.norm2) ||
          (l.ff_kind == CHATTS_FF_GEGLU ? !l.up : (l.ff_kind != CHATTS_FF_NONE && l.ff_kind != CHATTS_FF_MOE)) || (l.window.vfirst_write && !b->vfirst)) {
        set_error("mixdec_create: layer %d: a layer with norms after the sums has windowed attention and a gated unit, experts or nothing", i);
        return nullptr;
      }
      continue;
    }
    if (l.parallel != layers[0].parallel || (pair && !l.parallel) || (l.ff_kind > CHATTS_FF_RELU2 && !l.parallel) || (l.ff_kind == CHATTS_FF_RELU2 && l.parallel)) {
      set_error("mixdec_create: layer %d: sequential and parallel layers do not mix", i);
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
                      const ChattsOperand& out, chatts_stream_t s, float limit = 0.f, float alpha = 0.f, const float* bias = nullptr) {
  ChattsLinearArgs a{};
  a.bias = bias;
  a.glu_limit = limit; a.glu_alpha = alpha;
  a.resid = epilogue == CHATTS_EPI_RESID ? out.f32 : nullptr;
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


static ChattsOperand second_norm(const ChattsMixDecoder* d, const ChattsMixLayer& l, int m) {
  ChattsOperand o{};
  o.ld = d->c.width_p;
  const bool planes = mix_planes(d->c, m, o.ld);
  if (planes || (l.ff_kind == CHATTS_FF_MOE && !d->c.exact)) { o.hi = d->b.n_hi; o.lo = d->b.n_lo; }      // (experts take planes, the router what its kernel wants)
  if (!planes) o.f32 = d->b.n_f32;
  return o;
}
static ChattsOperand linear_form(const ChattsOperand& o) {      // one of the two forms
  ChattsOperand r = o;
  if (r.f32) r.hi = r.lo = nullptr;
  return r;
}
static ChattsOperand shift_operand(const ChattsMixDecoder* d, int m, int block) {
  ChattsOperand o{};
  o.ld = d->c.width_p;
  const int64_t at = block * d->b.mix_stride;
  if (mix_planes(d->c, m, o.ld)) { o.hi = d->b.m_hi + at; o.lo = d->b.m_lo + at; }
  else o.f32 = d->b.m_f32 + at;
  return o;
}

static int mix_recur(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, int n_spans, bool single, const ChattsOperand& out,
                     chatts_stream_t s) {
  StageRange stage("chatts.mix.recur");
  ChattsRecurArgs a = l.recur;
  a.proj = d->b.proj; a.ld_proj = l.in_n; a.eps = d->c.eps;
  a.state = run.state; a.n_state = run.n_state; a.m_state = run.m_state;
  a.rows = d->b.rows; a.n_rows = t; a.spans = d->b.spans; a.n_spans = n_spans;
  a.out = out;
  if (single) return chatts_recur_decode(&a, s);
  a.gates = d->b.gates; a.chunks = d->b.dchunks; a.o = d->b.dout; a.den = d->b.den;
  int rc;
  if (a.kind == CHATTS_RECUR_WKV) {
    const ChattsOperand low = operand(d, true, t, a.rank);
    if ((rc = chatts_recur_tanh(&a, &low, s)) != 0) return rc;
    if ((rc = mix_linear(d, low, l.w2, nullptr, t, l.w2_n, a.rank, CHATTS_EPI_NONE, f32_out(d->b.dg, l.w2_n), s)) != 0) return rc;
    a.decay = d->b.dg; a.ld_decay = l.w2_n;
    a.h = d->b.h; a.prev = run.ring; a.ld_h = d->c.width_p;
  }
  if ((rc = chatts_recur_scan(&a, s)) != 0) return rc;
  return chatts_recur_out(&a, s);
}

static int mix_window(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, const ChattsSpan* spans, int n_spans, bool single,
                      const ChattsOperand& out, chatts_stream_t s) {
  StageRange stage("chatts.mix.window");
  ChattsWindowArgs a = l.window;
  a.proj = d->b.proj; a.ld_proj = l.in_n; a.eps = d->c.eps;
  a.kcache = run.cache; a.vcache = run.vcache; a.cache_f32 = d->c.exact;
  a.ring = run.ring;
  if (a.ld_vfirst) { a.vfirst = d->b.vfirst; a.ld_vfirst = d->b.ld_vfirst; }
  a.table = d->b.table; a.table_stride = d->c.table_stride; a.log_block = kv_log_block(d->c.block_size);
  a.rows = d->b.rows; a.n_rows = t; a.spans = d->b.spans; a.n_spans = single ? 0 : n_spans;
  a.q.ld = a.heads * a.dim_p;
  if (d->c.exact) a.q.f32 = d->b.q_f32;
  else a.q.hi = d->b.q_hi;
  a.out = out; a.n_splits = 1; a.longest = 0;
  for (int i = 0; !single && i < n_spans; ++i)
    if (spans[i].t > a.longest) a.longest = spans[i].t;
  if (const int rc = chatts_window_prep(&a, s)) return rc;
  if (a.longest >= 8 && !d->c.exact && chatts_window_can_prefill(a.dim_p, a.vdim_p)) return chatts_window_prefill(&a, s);
  if (!d->c.exact) {      // few rows: a row's tiles (32 keys a wave, 4 waves) are spread over workgroups, about three per CU, the same number to every wave
    const int group = a.heads / a.kv_heads, wgs = a.kv_heads * ((group + 15) / 16) * t;
    const int most = a.window > 0 ? a.window + a.keep_first + 64 : (a.chunk > 0 ? a.chunk + a.keep_first + 64 : d->c.max_ctx);
    const int tiles = (most < d->c.max_ctx ? most : d->c.max_ctx) / 32;
    int splits = 3 * device_cus() / wgs;
    if (splits < 1) splits = 1;
    const int each = (tiles + 4 * splits - 1) / (4 * splits);
    splits = (tiles + 4 * each - 1) / (4 * each);
    if (splits > 64) splits = 64;
    while (splits > 1 && (size_t)t * a.heads * splits * (a.vdim_p + 4) > d->b.partial_elems) --splits;
    a.n_splits = splits < 1 ? 1 : splits;
    a.partial = d->b.partial;
  }
  return chatts_window_attend(&a, s);
}

static ChattsMoeArgs mix_moe_args(const ChattsMixDecoder* d, const ChattsMixLayer& l, int t, const ChattsOperand& h) {
  const ChattsMixBuffers& b = d->b;
  ChattsMoeArgs a = l.moe;
  a.logits = b.moe_logits; a.ld_logits = l.router_n;
  a.h = h;
  if (!d->c.exact) a.h.f32 = nullptr;
  a.rows = b.rows; a.n_rows = t; a.exact = d->c.exact;
  a.ids = b.moe_ids; a.place = b.moe_place; a.order = b.moe_order; a.offsets = b.moe_offsets; a.tiles = b.moe_tiles;
  a.weight = b.moe_weight; a.kept = b.moe_kept; a.y = b.moe_y;
  a.act = ChattsOperand{};
  a.act.ld = a.ff_p;
  if (d->c.exact) a.act.f32 = b.act_f32;
  else { a.act.hi = b.act_hi; a.act.lo = b.act_lo; }
  return a;
}

// x += what the experts of `moe` owe it; then the norms of `next` (or its joined input)
static int mix_pair_norm(const ChattsMixDecoder* d, int t, const ChattsMixLayer* moe, const float* w1, const float* w2, const ChattsOperand& out1, const ChattsOperand& out2,
                         bool join, const ChattsMixLayer* shift, float* prev, chatts_stream_t s) {
  ChattsPairNormArgs a{};
  a.x = d->b.x; a.t = t; a.width = d->c.width; a.ldx = d->c.width_p; a.groups = d->c.norm_groups; a.eps = d->c.eps;
  if (moe) {
    a.y = d->b.moe_y; a.place = d->b.moe_place; a.weight = d->b.moe_weight; a.kept = d->b.moe_kept; a.top = moe->moe.top;
    a.h = linear_form(second_norm(d, *moe, t));
  }
  if (join) a.x0 = d->b.x0;
  a.w1 = w1; a.w2 = w2; a.out1 = out1; a.out2 = out2;
  if (shift) {
    a.n_mix = shift->n_mix; a.mu = shift->mu; a.mix = shift_operand(d, t, 0); a.mix_stride = d->b.mix_stride; a.prev = prev; a.rows = d->b.rows;
  }
  return chatts_pair_norm(&a, s);
}

static int mix_parallel_forward(ChattsMixDecoder* d, const int64_t* tokens, int t, const ChattsSpan* spans, int n_spans, bool single, chatts_stream_t s) {
  const ChattsMixConfig& c = d->c;
  const int wp = c.width_p;
  const ChattsOperand none{}, X = f32_out(d->b.x, wp);
  int rc;
  {
    ChattsEmbedPairArgs e{};
    e.tokens = tokens; e.rows = d->b.rows; e.t = t; e.single = single; e.width_p = wp; e.vocab = (int)c.vocab;
    e.embed = d->b.embed; e.scale = c.embed_scale; e.bigram = d->b.bigram; e.buckets = c.bigram_buckets; e.mul_prev = c.bigram_prev; e.mul_cur = c.bigram_cur;
    e.prev = d->b.prev_token; e.x = d->b.x; e.x0 = d->b.x0;
    if ((rc = chatts_embed_pair(&e, s)) != 0) return rc;
  }
  const ChattsMixLayer* owed = nullptr;      // the layer whose experts' outputs x still misses
  for (int r = 0; r < c.n_runs; ++r) {
    const ChattsMixRun& run = d->runs[r];
    const ChattsMixLayer& l = d->layers[run.layer];
    if (run.join) {
      const ChattsOperand J = operand(d, true, t, 2 * wp);
      if ((rc = mix_pair_norm(d, t, owed, nullptr, nullptr, J, none, true, nullptr, nullptr, s)) != 0) return rc;
      owed = nullptr;
      if ((rc = mix_linear(d, J, run.join, run.join_t, t, wp, 2 * wp, CHATTS_EPI_NONE, X, s)) != 0) return rc;
    }
    const bool shift = l.n_mix > 0, ff = l.ff_kind != CHATTS_FF_NONE;
    const ChattsOperand A = shift && !single ? f32_out(d->b.h, wp) : operand(d, false, t, wp), N = second_norm(d, l, t);
    if ((rc = mix_pair_norm(d, t, owed, l.norm1, ff ? l.norm2 : nullptr, A, N, false, shift && single ? &l : nullptr, run.ring, s)) != 0) return rc;
    owed = nullptr;
    if (shift) {
      if (!single) {
        ChattsTokenShiftArgs a{};
        a.h = d->b.h; a.t = t; a.ldx = wp; a.n_mix = l.n_mix; a.mu = l.mu; a.mix = shift_operand(d, t, 0); a.mix_stride = d->b.mix_stride; a.prev = run.ring;
        a.rows = d->b.rows;
        if ((rc = chatts_token_shift(&a, s)) != 0) return rc;
      }
      for (int i = 0, n; i < l.n_mix; i += n) {      // blocks of equal size are one batch
        n = mix_equal_blocks(l, i);
        const ChattsOperand in = shift_operand(d, t, i);
        const int rows = l.mix_row[i + 1] - l.mix_row[i];
        ChattsLinearArgs a{};
        a.a = in.f32; a.lda = wp;
        if (!in.f32) { a.a_hi = in.hi; a.a_lo = in.lo; a.ld_planes = wp; }
        a.w = l.in + (size_t)l.mix_row[i] * wp; a.ldw = wp; a.w_tiled = l.mix_t[i]; a.w_tiled_batch = l.mix_t + i;
        a.m = t; a.n = rows; a.k = wp; a.epilogue = CHATTS_EPI_NONE; a.c = d->b.proj + l.mix_row[i]; a.ldc = l.in_n;
        a.batch = n; a.a_stride = d->b.mix_stride; a.w_stride = (int64_t)rows * wp; a.c_stride = rows;
        a.exact_f32 = c.exact; a.workspace = d->b.workspace; a.workspace_bytes = d->b.workspace_bytes;
        if ((rc = chatts_linear(&a, s)) != 0) return rc;
      }
    } else if ((rc = mix_linear(d, A, l.in, l.in_t, t, l.in_n, wp, CHATTS_EPI_NONE, f32_out(d->b.proj, l.in_n), s)) != 0) {
      return rc;
    }
    const ChattsOperand B = operand(d, true, t, l.out_k);
    rc = l.kind == CHATTS_MIX_WINDOW ? mix_window(d, l, run, t, spans, n_spans, single, B, s) : mix_recur(d, l, run, t, n_spans, single, B, s);
    if (rc) return rc;
    if ((rc = mix_linear(d, B, l.out, l.out_t, t, wp, l.out_k, CHATTS_EPI_RESID, X, s)) != 0) return rc;
    if (l.ff_kind == CHATTS_FF_CLAMPGLU) {
      const ChattsOperand F = operand(d, true, t, l.ff);
      if ((rc = mix_linear(d, linear_form(N), l.up, l.up_t, t, 2 * l.ff, wp, CHATTS_EPI_CLAMPGLU, F, s, l.glu_limit, l.glu_alpha)) != 0) return rc;
      if ((rc = mix_linear(d, F, l.down, l.down_t, t, wp, l.ff, CHATTS_EPI_RESID, X, s)) != 0) return rc;
    } else if (l.ff_kind == CHATTS_FF_MOE) {
      StageRange stage("chatts.mix.experts");
      if ((rc = mix_linear(d, linear_form(N), l.router, l.router_t, t, l.router_n, wp, CHATTS_EPI_NONE, f32_out(d->b.moe_logits, l.router_n), s)) != 0) return rc;
      const ChattsMoeArgs m = mix_moe_args(d, l, t, N);
      if ((rc = chatts_moe_route(&m, s)) != 0) return rc;
      if ((rc = chatts_moe_experts(&m, s)) != 0) return rc;
      owed = &l;
    }
  }
  if (owed) return mix_pair_norm(d, t, owed, nullptr, nullptr, none, none, false, nullptr, nullptr, s);
  return CHATTS_OK;
}

// ---- norms after the sums ----
// x as the operand of what reads it next: x itself where float32 is taken, planes beside it for wide steps and for experts
static ChattsOperand stream_operand(const ChattsMixDecoder* d, int m, bool experts) {
  ChattsOperand o{};
  o.ld = d->c.width_p;
  const bool planes = mix_planes(d->c, m, o.ld);
  if (planes || (experts && !d->c.exact)) { o.hi = d->b.a_hi; o.lo = d->b.a_lo; }
  if (!planes) o.f32 = d->b.x;
  return o;
}
static int mix_post_norm(const ChattsMixDecoder* d, int t, const float* y, const ChattsMixLayer* moe, const float* w, ChattsOperand out, chatts_stream_t s) {
  ChattsPostNormArgs a{};
  a.x = d->b.x; a.t = t; a.width = d->c.width; a.ldx = d->c.width_p; a.alpha = d->c.alpha; a.eps = d->c.eps; a.y = y; a.w = w;
  if (moe) { a.ey = d->b.moe_y; a.place = d->b.moe_place; a.weight = d->b.moe_weight; a.top = moe->moe.top; }
  out.f32 = nullptr;      // (x itself)
  a.out = out;
  return chatts_post_norm(&a, s);
}

static int mix_post_forward(ChattsMixDecoder* d, const int64_t* tokens, int t, const ChattsSpan* spans, int n_spans, bool single, chatts_stream_t s) {
  const ChattsMixConfig& c = d->c;
  const int wp = c.width_p;
  const ChattsOperand Y = f32_out(d->b.y, wp);
  int rc;
  if ((rc = chatts_embed_token_batched(tokens, t, d->b.embed, 0, c.vocab, wp, d->b.x, s)) != 0) return rc;
  ChattsOperand X = stream_operand(d, t, false);
  if (X.hi && (rc = chatts_split_bf16x2(d->b.x, t, wp, wp, X.hi, X.lo, wp, s)) != 0) return rc;
  for (int r = 0; r < c.n_runs; ++r) {
    const ChattsMixRun& run = d->runs[r];
    const ChattsMixLayer& l = d->layers[run.layer];
    if ((rc = mix_linear(d, linear_form(X), l.in, l.in_t, t, l.in_n, wp, CHATTS_EPI_NONE, f32_out(d->b.proj, l.in_n), s, 0.f, 0.f, l.in_bias)) != 0) return rc;
    const ChattsOperand B = operand(d, true, t, l.out_k);
    if ((rc = mix_window(d, l, run, t, spans, n_spans, single, B, s)) != 0) return rc;
    if ((rc = mix_linear(d, B, l.out, l.out_t, t, wp, l.out_k, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    const bool moe = l.ff_kind == CHATTS_FF_MOE;
    X = stream_operand(d, t, moe);
    if ((rc = mix_post_norm(d, t, d->b.y, nullptr, l.norm1, X, s)) != 0) return rc;
    if (l.ff_kind == CHATTS_FF_NONE) continue;
    if (l.up) {
      const ChattsOperand F = operand(d, true, t, l.ff);
      if ((rc = mix_linear(d, linear_form(X), l.up, l.up_t, t, moe ? l.ff : 2 * l.ff, wp, moe ? CHATTS_EPI_RELU2 : CHATTS_EPI_GEGLU, F, s)) != 0) return rc;
      if ((rc = mix_linear(d, F, l.down, l.down_t, t, wp, l.ff, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    }
    if (moe) {
      StageRange stage("chatts.mix.experts");
      if ((rc = mix_linear(d, linear_form(X), l.router, l.router_t, t, l.router_n, wp, CHATTS_EPI_NONE, f32_out(d->b.moe_logits, l.router_n), s)) != 0) return rc;
      const ChattsMoeArgs m = mix_moe_args(d, l, t, X);
      if ((rc = chatts_moe_route(&m, s)) != 0) return rc;
      if ((rc = chatts_moe_experts(&m, s)) != 0) return rc;
    }
    X = stream_operand(d, t, false);
    if ((rc = mix_post_norm(d, t, l.up ? d->b.y : nullptr, moe ? &l : nullptr, l.norm2, X, s)) != 0) return rc;
  }
  return CHATTS_OK;
}

// ---- norms before the sublayers only ----
static int mix_gru(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, int n_spans, bool single, const ChattsOperand& out, chatts_stream_t s) {
  StageRange stage("chatts.mix.gru");
  ChattsGruArgs a = l.gru;
  a.proj = d->b.proj; a.ld_proj = l.in_n;
  a.state = run.gru_state;
  a.rows = d->b.rows; a.n_rows = t; a.spans = d->b.spans; a.n_spans = n_spans;
  a.out = out;
  return single ? chatts_gru_decode(&a, s) : chatts_gru_scan(&a, s);
}

static int mix_select(const ChattsMixDecoder* d, const ChattsMixLayer& l, const ChattsMixRun& run, int t, int n_spans, bool single, const ChattsOperand& out, chatts_stream_t s) {
  StageRange stage("chatts.mix.select");
  const ChattsMixBuffers& b = d->b;
  ChattsSelectArgs a = l.select;
  a.proj = b.proj; a.ld_proj = l.in_n;
  a.s = run.sel_state; a.ring = run.sel_ring;
  a.rows = b.rows; a.n_rows = t; a.spans = b.spans; a.n_spans = single ? 0 : n_spans;
  a.u.f32 = b.sel_u; a.u.ld = l.sel_k;
  ChattsOperand in = f32_out(b.sel_u, l.sel_k);
  if (mix_planes(d->c, t, l.sel_k)) {
    a.u.hi = b.sel_u_hi; a.u.lo = b.sel_u_lo;
    in.f32 = nullptr; in.hi = b.sel_u_hi; in.lo = b.sel_u_lo;
  }
  a.low = b.sel_low; a.out = out;
  int rc;
  if ((rc = chatts_select_conv(&a, s)) != 0) return rc;
  if ((rc = mix_linear(d, in, l.sel_low, l.sel_low_t, t, a.ld_low, l.sel_k, CHATTS_EPI_NONE, f32_out(b.sel_low, a.ld_low), s)) != 0) return rc;
  if (single) return chatts_select_decode(&a, s);
  ChattsOperand dt = f32_out(b.sel_low + a.off_dt, a.ld_low);
  a.delta = b.sel_delta; a.ld_delta = l.sel_dt_n;
  if (t >= 96 && a.w_dt_f) {
    a.delta_steps = 1; a.dt_hi = b.sel_dt_hi; a.dt_lo = b.sel_dt_lo;
    if ((rc = chatts_select_steps(&a, s)) != 0) return rc;
    return chatts_select_scan(&a, s);
  }
  if (mix_planes(d->c, t, a.rank)) {
    if ((rc = chatts_split_bf16x2(dt.f32, t, a.rank, a.ld_low, b.sel_dt_hi, b.sel_dt_lo, a.rank, s)) != 0) return rc;
    dt.f32 = nullptr; dt.hi = b.sel_dt_hi; dt.lo = b.sel_dt_lo; dt.ld = a.rank;
  }
  if ((rc = mix_linear(d, dt, l.sel_dt, nullptr, t, l.sel_dt_n, a.rank, CHATTS_EPI_NONE, f32_out(b.sel_delta, l.sel_dt_n), s)) != 0) return rc;
  return chatts_select_scan(&a, s);
}

static int mix_one(const ChattsMixDecoder* d, const ChattsMixLayer& l, int kind, const ChattsMixRun& run, int t, const ChattsSpan* spans, int n_spans, bool single,
                   const ChattsOperand& out, chatts_stream_t s) {
  if (kind == CHATTS_MIX_WINDOW) return mix_window(d, l, run, t, spans, n_spans, single, out, s);
  return kind == CHATTS_MIX_GRU ? mix_gru(d, l, run, t, n_spans, single, out, s) : mix_select(d, l, run, t, n_spans, single, out, s);
}

// x += mult (y + what the experts of `moe` owe it), averaged over depth after the run number `stream` of a layer with such weights; then the next norm
static int mix_depth_norm(const ChattsMixDecoder* d, int t, const float* y, const ChattsMixLayer* moe, const float* depth, int stream, const float* w, const ChattsOperand& out,
                          chatts_stream_t s) {
  ChattsDepthNormArgs a{};
  a.x = d->b.x; a.t = t; a.width = d->c.width; a.ldx = d->c.width_p; a.mult = d->c.mult; a.eps = d->c.eps; a.y = y;
  if (moe) { a.ey = d->b.moe_y; a.place = d->b.moe_place; a.weight = d->b.moe_weight; a.top = moe->moe.top; }
  a.depth = depth; a.streams = d->b.streams; a.stream_stride = d->b.stream_stride; a.n_streams = stream + 1; a.keep = depth && stream + 1 < d->c.n_runs;
  a.w = w; a.out = out;
  return chatts_depth_norm(&a, s);
}

static int mix_pre_forward(ChattsMixDecoder* d, const int64_t* tokens, int t, const ChattsSpan* spans, int n_spans, bool single, chatts_stream_t s) {
  const ChattsMixConfig& c = d->c;
  const int wp = c.width_p;
  const ChattsOperand none{}, A = operand(d, false, t, wp), Y = f32_out(d->b.y, wp);
  int rc;
  {
    ChattsEmbedPairArgs e{};
    e.tokens = tokens; e.rows = d->b.rows; e.t = t; e.single = single; e.width_p = wp; e.vocab = (int)c.vocab; e.embed = d->b.embed; e.scale = c.embed_scale;
    e.x = d->b.x; e.x0 = d->b.streams; e.width = c.width; e.pos_fine = d->b.pos_fine; e.pos_coarse = d->b.pos_coarse;
    if ((rc = chatts_embed_pair(&e, s)) != 0) return rc;
  }
  if ((rc = mix_depth_norm(d, t, nullptr, nullptr, nullptr, 0, d->layers[d->runs[0].layer].norm1, A, s)) != 0) return rc;
  for (int r = 0; r < c.n_runs; ++r) {
    const ChattsMixRun& run = d->runs[r];
    const ChattsMixLayer& l = d->layers[run.layer];
    const float* next = r + 1 < c.n_runs ? d->layers[d->runs[r + 1].layer].norm1 : nullptr;
    if ((rc = mix_linear(d, A, l.in, l.in_t, t, l.in_n, wp, CHATTS_EPI_NONE, f32_out(d->b.proj, l.in_n), s, 0.f, 0.f, l.in_bias)) != 0) return rc;
    const ChattsOperand B = operand(d, true, t, l.out_k);
    if ((rc = mix_one(d, l, l.kind, run, t, spans, n_spans, single, B, s)) != 0) return rc;
    if (l.beside) {
      ChattsOperand C = B;
      if (C.f32) C.f32 += l.beside_col;
      else { C.hi += l.beside_col; C.lo += l.beside_col; }
      if ((rc = mix_one(d, l, l.beside, run, t, spans, n_spans, single, C, s)) != 0) return rc;
    }
    if ((rc = mix_linear(d, B, l.out, l.out_t, t, wp, l.out_k, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    const bool moe = l.ff_kind == CHATTS_FF_MOE;
    if (l.ff_kind == CHATTS_FF_NONE) {
      if ((rc = mix_depth_norm(d, t, d->b.y, nullptr, l.depth, r, next, next ? A : none, s)) != 0) return rc;
      continue;
    }
    const ChattsOperand N = second_norm(d, l, t);
    if ((rc = mix_depth_norm(d, t, d->b.y, nullptr, nullptr, 0, l.norm2, N, s)) != 0) return rc;
    if (moe) {
      StageRange stage("chatts.mix.experts");
      if ((rc = mix_linear(d, linear_form(N), l.router, l.router_t, t, l.router_n, wp, CHATTS_EPI_NONE, f32_out(d->b.moe_logits, l.router_n), s)) != 0) return rc;
      const ChattsMoeArgs m = mix_moe_args(d, l, t, N);
      if ((rc = chatts_moe_route(&m, s)) != 0) return rc;
      if ((rc = chatts_moe_experts(&m, s)) != 0) return rc;
    }
    if (l.up) {
      const ChattsOperand F = operand(d, true, t, l.ff);
      if ((rc = mix_linear(d, linear_form(N), l.up, l.up_t, t, 2 * l.ff, wp, CHATTS_EPI_CLAMPGLU, F, s, l.glu_limit, l.glu_alpha)) != 0) return rc;
      if ((rc = mix_linear(d, F, l.down, l.down_t, t, wp, l.ff, CHATTS_EPI_NONE, Y, s)) != 0) return rc;
    }
    if ((rc = mix_depth_norm(d, t, l.up ? d->b.y : nullptr, moe ? &l : nullptr, l.depth, r, next, next ? A : none, s)) != 0) return rc;
  }
  return CHATTS_OK;
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
  if (d->layers[0].pre) return mix_pre_forward(d, tokens, t, spans, n_spans, single != 0, s);
  if (d->layers[0].post) return mix_post_forward(d, tokens, t, spans, n_spans, single != 0, s);
  if (d->layers[0].parallel) return mix_parallel_forward(d, tokens, t, spans, n_spans, single != 0, s);
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
  const float* x = d->b.x;
  if (index) {
    hipLaunchKernelGGL(gather_rows_kernel, dim3(n), dim3(256), 0, as_stream(s), d->b.x, index, d->b.y, c.width_p);
    CHATTS_CHECK_LAUNCH("gather_rows");
    x = d->b.y;
  }
  const ChattsOperand A = operand(d, false, n, c.width_p);
  int rc;
  if (d->layers[0].parallel) {
    ChattsPairNormArgs a{};
    a.x = const_cast<float*>(x); a.t = n; a.width = c.width; a.ldx = c.width_p; a.groups = c.norm_groups; a.eps = c.eps;
    a.w1 = d->b.final_norm; a.out1 = A;
    rc = chatts_pair_norm(&a, s);
  } else {
    ChattsResidualNormArgs a{};
    a.x = const_cast<float*>(x); a.pre_w = d->b.final_norm; a.out = A;
    a.t = n; a.width = c.width; a.ldx = a.ldy = c.width_p; a.eps = c.eps;
    rc = chatts_residual_norm(&a, s);
  }
  if (rc) return rc;
  if ((rc = mix_linear(d, A, d->b.head, d->b.head_t, n, (int)c.vocab_p, c.width_p, CHATTS_EPI_NONE, f32_out(logits, (int)c.vocab_p), s)) != 0) return rc;
  return c.logit_cap > 0.f ? chatts_soft_cap(logits, n * c.vocab_p, c.logit_cap, s) : CHATTS_OK;
}

extern "C" int chatts_mixdec_decode(ChattsMixDecoder* d, int batch, const int64_t* token, const int32_t* pos, float* logits, chatts_stream_t s) {
  CHATTS_REQUIRE(d && token && pos && batch >= 1 && batch <= d->c.max_slots, CHATTS_E_BADARG, "mixdec_decode: batch %d", batch);
  hipLaunchKernelGGL(rows_from_pos_kernel, dim3((batch + 255) / 256), dim3(256), 0, as_stream(s), d->b.rows, pos, batch);
  CHATTS_CHECK_LAUNCH("rows_from_pos");
  if (const int rc = chatts_mixdec_forward(d, token, batch, nullptr, 0, 1, s)) return rc;
  return chatts_mixdec_logits(d, nullptr, batch, logits, s);
}
