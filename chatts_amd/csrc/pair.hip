// pair.hip - the residual stream of layers whose mixer and feed-forward read two norms of the same x: embedding (optionally with a row per token pair, or
// with sinusoidal positions), the two norms (in groups) in one launch together with what else touches the row - the experts' weighted sum, the input of
// a joining projection, the operands of a token shift.
#include "common.h"

namespace chatts {

// a workgroup per row
__global__ __launch_bounds__(256) void embed_pair_kernel(ChattsEmbedPairArgs p) {
  const int row = blockIdx.x, tid = threadIdx.x;
  const ChattsRow R = p.rows[row];
  int64_t tok = p.tokens[row];
  if (tok < 0 || tok >= p.vocab) tok = 0;      // (the host has refused such tokens; parked rows hold anything)
  const uint16_t* e = p.embed + (size_t)tok * p.width_p;
  const uint16_t* g = nullptr;
  if (p.bigram) {
    int64_t r = p.buckets;
    if (R.pos > 0) {
      const int64_t before = row > R.first ? p.tokens[row - 1] : p.prev[R.slot];
      r = (before * p.mul_prev + tok * p.mul_cur) % p.buckets;
      if (r < 0) r += p.buckets;
    }
    g = p.bigram + (size_t)r * p.width_p;
  }
  for (int c = tid * 4; c < p.width_p; c += 1024) {
    const u32x2 ev = *reinterpret_cast<const u32x2*>(e + c);
    f32x4 x = {bf16_lo(ev[0]) * p.scale, bf16_hi(ev[0]) * p.scale, bf16_lo(ev[1]) * p.scale, bf16_hi(ev[1]) * p.scale};
    if (g) {
      const u32x2 gv = *reinterpret_cast<const u32x2*>(g + c);
      x[0] += bf16_lo(gv[0]);
      x[1] += bf16_hi(gv[0]);
      x[2] += bf16_lo(gv[1]);
      x[3] += bf16_hi(gv[1]);
    }
    if (p.pos_fine) {
      const int pos = R.pos > 0 ? R.pos : 0;
      const f32x4 a = *reinterpret_cast<const f32x4*>(p.pos_fine + (size_t)(pos & 63) * p.width_p + c);
      const f32x4 b = *reinterpret_cast<const f32x4*>(p.pos_coarse + (size_t)(pos >> 6) * p.width_p + c);
#pragma unroll
      for (int k = 0; k < 4; k += 2) {
        x[k] += c + k < p.width ? a[k] * b[k + 1] + a[k + 1] * b[k] : 0.f;
        x[k + 1] += c + k + 1 < p.width ? a[k + 1] * b[k + 1] - a[k] * b[k] : 0.f;
      }
    }
    *reinterpret_cast<f32x4*>(p.x + (size_t)row * p.width_p + c) = x;
    if (p.x0) *reinterpret_cast<f32x4*>(p.x0 + (size_t)row * p.width_p + c) = x;
  }
  if (p.single && p.bigram && R.pos >= 0) {
    __syncthreads();      // (everyone has read the old one)
    if (tid == 0) p.prev[R.slot] = tok;
  }
}
__global__ __launch_bounds__(256) void last_token_kernel(ChattsEmbedPairArgs p) {
  const int row = blockIdx.x * 256 + threadIdx.x;
  if (row >= p.t) return;
  const ChattsRow R = p.rows[row];
  if (R.pos >= 0 && R.rest == 0) p.prev[R.slot] = p.tokens[row];
}

__device__ __forceinline__ f32x4 load_operand4(const ChattsOperand& o, size_t row, int c) {
  const size_t at = row * o.ld + c;
  if (o.f32) return *reinterpret_cast<const f32x4*>(o.f32 + at);
  const u32x2 h = *reinterpret_cast<const u32x2*>(o.hi + at), l = *reinterpret_cast<const u32x2*>(o.lo + at);
  return (f32x4){bf16_lo(h[0]) + bf16_lo(l[0]), bf16_hi(h[0]) + bf16_hi(l[0]), bf16_lo(h[1]) + bf16_lo(l[1]), bf16_hi(h[1]) + bf16_hi(l[1])};
}
__device__ __forceinline__ ChattsOperand operand_block(ChattsOperand o, int64_t at) {
  if (o.f32) o.f32 += at;
  if (o.hi) o.hi += at;
  if (o.lo) o.lo += at;
  return o;
}
__device__ __forceinline__ void store_row4(const ChattsOperand& o, size_t row, int c, const f32x4& x) {
  const float v[4] = {x[0], x[1], x[2], x[3]};
  store_operand4(o, row, c, v);
}

// a workgroup per row; a thread keeps its columns in registers.  QUADS: the groups are made of whole quads of columns.  NT: threads (more of them
// for a few rows: then every load of a row is in flight at once)
template <int NT, int NV, bool QUADS>
__global__ __launch_bounds__(NT) void pair_norm_kernel(ChattsPairNormArgs p, int padded) {
  extern __shared__ float sm[];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, part = p.width / p.groups;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  ChattsRow R{0, -1, 0, 0};
  if (p.n_mix) R = p.rows[row];
  f32x4 x[NV], wa[NV], wb[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    x[i] = c < padded ? *reinterpret_cast<const f32x4*>(p.x + row * p.ldx + c) : zero;
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {      // (the weights travel while the row is reduced)
    const int c = (i * NT + tid) * 4;
    wa[i] = p.w1 && c < padded ? *reinterpret_cast<const f32x4*>(p.w1 + c) : zero;
    wb[i] = p.w2 && c < padded ? *reinterpret_cast<const f32x4*>(p.w2 + c) : zero;
  }
  if (p.y) {
    constexpr int U = 4;      // experts' rows requested at once
    for (int j0 = 0; j0 < p.top; j0 += U) {
      int at[U];
      float w[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int j = j0 + u < p.top ? j0 + u : j0;
        at[u] = j0 + u < p.top ? p.place[row * p.top + j] : -1;      // (uniform)
        w[u] = p.weight[row * p.top + j];
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * NT + tid) * 4;
        if (c >= padded) continue;
        f32x4 y[U];
#pragma unroll
        for (int u = 0; u < U; ++u) y[u] = at[u] >= 0 ? *reinterpret_cast<const f32x4*>(p.y + (size_t)at[u] * p.ldx + c) : zero;
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < 4; ++k) x[i][k] += at[u] >= 0 ? w[u] * y[u][k] : 0.f;
      }
    }
    const float kept = p.kept[row];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * NT + tid) * 4;
      if (c < padded) {
        if (kept != 0.f) {
          const f32x4 h = load_operand4(p.h, row, c);
#pragma unroll
          for (int k = 0; k < 4; ++k) x[i][k] += kept * h[k];
        }
        *reinterpret_cast<f32x4*>(p.x + row * p.ldx + c) = x[i];
      }
    }
  }
  if (p.x0) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * NT + tid) * 4;
      if (c >= padded) continue;
      store_row4(p.out1, row, c, x[i]);
      store_row4(p.out1, row, p.ldx + c, *reinterpret_cast<const f32x4*>(p.x0 + row * p.ldx + c));
    }
    return;
  }
  if (!p.w1) return;
  // sums of squares per quad (or column) meet in LDS, a wave adds up a group
  const int units = QUADS ? p.width / 4 : p.width, per = QUADS ? part / 4 : part;
  float* inv = sm + units;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    if (QUADS) {
      if (c < p.width) sm[c >> 2] = (x[i][0] * x[i][0] + x[i][1] * x[i][1]) + (x[i][2] * x[i][2] + x[i][3] * x[i][3]);
    } else {
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (c + k < p.width) sm[c + k] = x[i][k] * x[i][k];
    }
  }
  f32x4 before[NV];      // the token shift: h of the slot's previous token
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    before[i] = R.pos > 0 && c < padded ? *reinterpret_cast<const f32x4*>(p.prev + (size_t)R.slot * p.ldx + c) : zero;
  }
  __syncthreads();
  for (int g = wave; g < p.groups; g += NT / 64) {
    float ss = 0.f;
    for (int u = lane; u < per; u += 64) ss += sm[g * per + u];
    ss = wave_sum(ss);
    if (lane == 0) inv[g] = 1.0f / sqrtf(ss / (float)part + p.eps);
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    if (c >= padded) continue;
    f32x4 n, h, d;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      n[k] = c + k < p.width ? x[i][k] * inv[(c + (QUADS ? 0 : k)) / part] : 0.f;
      h[k] = n[k] * wa[i][k];
      d[k] = before[i][k] - h[k];
    }
    if (p.n_mix) {
      constexpr int U = 5;
      for (int s0 = 0; s0 < p.n_mix; s0 += U) {
        f32x4 mu[U];
#pragma unroll
        for (int u = 0; u < U; ++u) mu[u] = *reinterpret_cast<const f32x4*>(p.mu + (size_t)(s0 + u < p.n_mix ? s0 + u : s0) * p.ldx + c);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          if (s0 + u >= p.n_mix) break;
          f32x4 m;
#pragma unroll
          for (int k = 0; k < 4; ++k) m[k] = h[k] + d[k] * mu[u][k];
          store_row4(operand_block(p.mix, (s0 + u) * p.mix_stride), row, c, m);
        }
      }
      if (R.pos >= 0) *reinterpret_cast<f32x4*>(p.prev + (size_t)R.slot * p.ldx + c) = h;
    } else {
      store_row4(p.out1, row, c, h);
    }
    if (p.w2) {
#pragma unroll
      for (int k = 0; k < 4; ++k) h[k] = n[k] * wb[i][k];
      store_row4(p.out2, row, c, h);
    }
  }
}

// grid (rows, columns / 1024)
__global__ __launch_bounds__(256) void token_shift_kernel(ChattsTokenShiftArgs p) {
  const int row = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (c >= p.ldx) return;
  const ChattsRow R = p.rows[row];
  const f32x4 h = *reinterpret_cast<const f32x4*>(p.h + (size_t)row * p.ldx + c);
  f32x4 d = {0.f, 0.f, 0.f, 0.f};
  if (row > R.first) d = *reinterpret_cast<const f32x4*>(p.h + (size_t)(row - 1) * p.ldx + c);
  else if (R.pos > 0) d = *reinterpret_cast<const f32x4*>(p.prev + (size_t)R.slot * p.ldx + c);
#pragma unroll
  for (int k = 0; k < 4; ++k) d[k] -= h[k];
  for (int s = 0; s < p.n_mix; ++s) {
    const f32x4 mu = *reinterpret_cast<const f32x4*>(p.mu + (size_t)s * p.ldx + c);
    f32x4 m;
#pragma unroll
    for (int k = 0; k < 4; ++k) m[k] = h[k] + d[k] * mu[k];
    store_row4(operand_block(p.mix, s * p.mix_stride), row, c, m);
  }
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_embed_pair(const ChattsEmbedPairArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->tokens && a->rows && a->embed && a->x && a->t >= 0 && a->width_p > 0 && a->width_p % 4 == 0 && a->vocab > 0, CHATTS_E_BADARG,
                 "embed_pair: bad arguments");
  CHATTS_REQUIRE(!a->bigram || (a->buckets > 0 && a->prev), CHATTS_E_BADARG, "embed_pair: %lld buckets", (long long)a->buckets);
  CHATTS_REQUIRE(!a->pos_fine || (a->pos_coarse && a->width > 0 && a->width <= a->width_p && (((uintptr_t)a->pos_fine | (uintptr_t)a->pos_coarse) % 16) == 0),
                 CHATTS_E_BADARG, "embed_pair: positions");
  if (a->t == 0) return CHATTS_OK;
  hipLaunchKernelGGL(embed_pair_kernel, dim3(a->t), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("embed_pair");
  if (a->bigram && !a->single) {
    hipLaunchKernelGGL(last_token_kernel, dim3((a->t + 255) / 256), dim3(256), 0, as_stream(stream), *a);
    CHATTS_CHECK_LAUNCH("last_token");
  }
  return CHATTS_OK;
}

template <int NT, int NV>
static void launch_pair_norm(const ChattsPairNormArgs* a, hipStream_t s) {
  const bool quads = a->width % (4 * a->groups) == 0;
  const size_t lds = (size_t)((quads ? a->width / 4 : a->width) + a->groups) * sizeof(float);
  if (quads) hipLaunchKernelGGL((pair_norm_kernel<NT, NV, true>), dim3(a->t), dim3(NT), lds, s, *a, a->ldx);
  else hipLaunchKernelGGL((pair_norm_kernel<NT, NV, false>), dim3(a->t), dim3(NT), lds, s, *a, a->ldx);
}

extern "C" int chatts_pair_norm(const ChattsPairNormArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->x && a->t >= 0 && a->width > 0 && a->groups > 0 && a->width % a->groups == 0, CHATTS_E_BADARG, "pair_norm: a width of %d in %d groups",
                 a ? a->width : 0, a ? a->groups : 0);
  CHATTS_REQUIRE(a->ldx >= a->width && a->ldx % 4 == 0 && a->ldx <= 16384 && a->width + a->groups <= 16000, CHATTS_E_SHAPE, "pair_norm: row stride %d", a->ldx);
  CHATTS_REQUIRE(!a->y || (a->place && a->weight && a->kept && a->top > 0 && (a->h.f32 || (a->h.hi && a->h.lo))), CHATTS_E_BADARG, "pair_norm: experts");
  auto ok = [](const ChattsOperand& o, int ld) { return (o.f32 || o.hi) && o.ld >= ld && o.ld % 4 == 0; };
  CHATTS_REQUIRE(!a->x0 || ok(a->out1, 2 * a->ldx), CHATTS_E_BADARG, "pair_norm: no output for a joined row");
  CHATTS_REQUIRE(a->x0 || !a->w1 || a->n_mix || ok(a->out1, a->ldx), CHATTS_E_BADARG, "pair_norm: no output");
  CHATTS_REQUIRE(!a->w2 || ok(a->out2, a->ldx), CHATTS_E_BADARG, "pair_norm: no second output");
  CHATTS_REQUIRE(!a->n_mix || (a->mu && a->prev && a->rows && ok(a->mix, a->ldx) && a->mix_stride % 4 == 0), CHATTS_E_BADARG, "pair_norm: token shift");
  if (a->t == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  if (a->ldx <= 1024) launch_pair_norm<256, 1>(a, s);
  else if (a->t <= 64 && a->ldx <= 4096) launch_pair_norm<1024, 1>(a, s);
  else if (a->t <= 64 && a->ldx <= 8192) launch_pair_norm<1024, 2>(a, s);
  else if (a->ldx <= 2048) launch_pair_norm<256, 2>(a, s);
  else if (a->ldx <= 4096) launch_pair_norm<256, 4>(a, s);
  else if (a->ldx <= 8192) launch_pair_norm<256, 8>(a, s);
  else launch_pair_norm<1024, 4>(a, s);
  CHATTS_CHECK_LAUNCH("pair_norm");
  return CHATTS_OK;
}

extern "C" int chatts_token_shift(const ChattsTokenShiftArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->h && a->mu && a->prev && a->rows && a->t >= 0 && a->n_mix > 0 && a->ldx > 0 && a->ldx % 4 == 0 && (a->mix.f32 || a->mix.hi) &&
                     a->mix.ld >= a->ldx && a->mix.ld % 4 == 0 && a->mix_stride % 4 == 0, CHATTS_E_BADARG, "token_shift: bad arguments");
  if (a->t == 0) return CHATTS_OK;
  hipLaunchKernelGGL(token_shift_kernel, dim3(a->t, (a->ldx + 1023) / 1024), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("token_shift");
  return CHATTS_OK;
}
