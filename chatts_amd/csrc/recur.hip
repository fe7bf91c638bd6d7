// recur.hip - gated linear recurrences:  S <- diag(g_t) S + k_t v_t^T per head, S [dim, vdim] in float32, with a read-out per token.
//   wkv    decays per key channel from a low-rank product; the token reads S before its own write, its own value through a bonus u
//   mlstm  one decay per head from exponential gates under a running maximum; the token reads S after its write, divided by a normaliser
// Kernels:
//  * recur_decode_kernel: one token per sequence, everything of a (sequence, head) in one workgroup: decay, state update (the state passes
//    through registers once), read-out, norm, gate.
//  * recur_gates_kernel (mlstm), recur_chunk_kernel, recur_scan_kernel, recur_out_kernel: several tokens per sequence.  Chunks of 16 tokens: what
//    depends on the inputs only is formed for all chunks in parallel, scan passes the state along on the float32 matrix pipe.
#include "common.h"

namespace chatts {

// ---- one token per sequence: thread (tx, ty) = 4 consecutive value columns tx * 4, key rows ty + TY * r ----
template <int KIND, int NT, int NR>
__global__ __launch_bounds__(NT) void recur_decode_kernel(ChattsRecurArgs p, int TX) {
  constexpr bool WKV = KIND == CHATTS_RECUR_WKV;
  extern __shared__ float sm[];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
  const int pos = p.rows[row].pos, slot = p.rows[row].slot;
  if (pos < 0) return;
  const int dim = p.dim, vdim = p.vdim, v4 = (vdim + 3) & ~3;
  float* red = sm;                      // NT * 4 (read as float4)
  float* sv = red + NT * 4;             // v4
  float* sq = sv + v4;                  // dim
  float* sk = sq + dim;
  float* sg = sk + dim;
  float* sa = sg + dim;                 // rank
  float* scratch = sa + (WKV ? p.rank : 0);
  const int tx = tid & (TX - 1), ty = tid / TX, TY = NT / TX;
  const bool live = tx * 4 < v4;
  const float* pr = p.proj + (size_t)row * p.ld_proj;
  // small inputs first, the state last: the gates are formed while it is on its way
  const int dq = tid < dim ? tid : dim - 1, dv = tid < vdim ? tid : vdim - 1;
  const float q_in = pr[p.off_q + h * dim + dq], k_in = pr[p.off_k + h * dim + dq], v_in = pr[p.off_v + h * vdim + dv];
  const float gate_in = pr[p.off_gate + h * vdim + dv], nw = p.norm_w[h * vdim + dv];
  constexpr int kW = 8;
  u32x4 wv[kW];
  float w0 = 0.f, u_in = 0.f, n_in = 0.f, m_in = 0.f, i_in = 0.f, f_in = 0.f;
  const int rows = p.heads * dim, lrow = h * dim + dq, rank8 = p.rank >> 3;
  if constexpr (WKV) {
#pragma unroll
    for (int c = 0; c < kW; ++c) wv[c] = *reinterpret_cast<const u32x4*>(p.w2d + ((size_t)(c < rank8 ? c : 0) * rows + lrow) * 8);
    w0 = p.w0[lrow];
    u_in = p.u[lrow];
  } else {
    i_in = pr[p.off_i + h] + p.bias_i[h];
    f_in = pr[p.off_f + h] + p.bias_f[h];
    if (pos > 0) {
      m_in = p.m_state[(size_t)slot * p.heads + h];
      n_in = p.n_state[((size_t)slot * p.heads + h) * dim + dq];
    }
  }
  float* S = p.state + ((size_t)slot * p.heads + h) * dim * v4;
  f32x4 s[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int i = ty + TY * r < dim ? ty + TY * r : dim - 1;
    s[r] = *reinterpret_cast<const f32x4*>(S + (size_t)i * v4 + (live ? tx * 4 : 0));
  }
  if constexpr (WKV)
    for (int i = tid; i < p.rank; i += NT) sa[i] = tanhf(pr[p.off_a + i]);
  if (tid < v4) sv[tid] = tid < vdim ? v_in : 0.f;
  float a = 1.f, b = 1.f, floor_m = 0.f, m1 = 0.f, mine = 0.f;      // mine: this thread's channel of the scalar product that every column shares
  if constexpr (!WKV) {
    const float i = p.cap * tanhf(i_in / p.cap), f = -softplus_f(-p.cap * tanhf(f_in / p.cap));
    m1 = fmaxf(f + m_in, i);
    a = exp_hw(f + m_in - m1);
    b = exp_hw(i - m1);
    floor_m = exp_hw(-m1);
    if (tid < dim) {
      const float k = b * k_in, n = a * n_in + k, q = q_in * rsqrtf((float)dim);
      sq[tid] = q;
      sk[tid] = k;
      mine = n * q;
      p.n_state[((size_t)slot * p.heads + h) * dim + tid] = n;
    }
  }
  __syncthreads();      // (mlstm: every thread has read m)
  if constexpr (WKV) {
    if (tid < dim) {
      float z = w0;
      auto dot8 = [&](const u32x4& w, const float* x) {
#pragma unroll
        for (int j = 0; j < 4; ++j) { z += bf16_lo(w[j]) * x[2 * j]; z += bf16_hi(w[j]) * x[2 * j + 1]; }
      };
#pragma unroll
      for (int c = 0; c < kW; ++c)
        if (c < rank8) dot8(wv[c], sa + c * 8);
      for (int c = kW; c < rank8; ++c) dot8(*reinterpret_cast<const u32x4*>(p.w2d + ((size_t)c * rows + lrow) * 8), sa + c * 8);
      sg[tid] = exp_hw(-exp_hw(z));
      sq[tid] = q_in;
      sk[tid] = k_in;
      mine = q_in * u_in * k_in;
    }
  } else if (tid == 0) {
    p.m_state[(size_t)slot * p.heads + h] = m1;
  }
  const float shared = block_sum<NT / 64>(mine, scratch);      // wkv: q . (u k);  mlstm: n . q   (its barriers also publish sg, sq, sk)
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  if (live) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(sv + tx * 4);
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const int i = ty + TY * r;
      if (i < dim) {
        const float q = sq[i], k = sk[i], g = WKV ? sg[i] : a;
        if (pos == 0) s[r] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if constexpr (WKV) acc[j] += s[r][j] * q;
          s[r][j] = g * s[r][j] + k * v[j];
          if constexpr (!WKV) acc[j] += s[r][j] * q;
        }
        *reinterpret_cast<f32x4*>(S + (size_t)i * v4 + tx * 4) = s[r];
      }
    }
  }
  *reinterpret_cast<f32x4*>(red + tid * 4) = acc;
  __syncthreads();
  float o = 0.f;
  if (tid < vdim) {
    for (int y = 0; y < TY; ++y) o += red[(y * TX + (tid >> 2)) * 4 + (tid & 3)];
    if constexpr (WKV) o += shared * v_in;
    else o = o / (fmaxf(fabsf(shared), floor_m) + 1e-6f);
  }
  const float ss = block_sum<NT / 64>(tid < vdim ? o * o : 0.f, scratch);
  if (tid < vdim) {
    const float gs = sigmoid_f(gate_in);
    store_operand(p.out, row, h * vdim + tid, o * (1.0f / sqrtf(ss / (float)vdim + p.eps)) * nw * (WKV ? gate_in * gs : gs));
  }
}

// ---- several tokens ----
__global__ __launch_bounds__(256) void recur_tanh_kernel(ChattsRecurArgs p, ChattsOperand out) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  const int quads = p.rank >> 2;
  const size_t row = i / quads;
  const int c = (int)(i - row * quads) * 4;
  if (row >= (size_t)p.n_rows) return;
  const f32x4 x = *reinterpret_cast<const f32x4*>(p.proj + row * p.ld_proj + p.off_a + c);
  const float v[4] = {tanhf(x[0]), tanhf(x[1]), tanhf(x[2]), tanhf(x[3])};
  store_operand4(out, row, c, v);
}

// mlstm: a workgroup = one head of one span, 1024 tokens at a time.  (sum of f, running maximum) pairs combine associatively:
// m_t = max(m_0 + F_t, M_t) with (F, M) o (F', M') = (F + F', max(M + F', M')).
__global__ __launch_bounds__(1024) void recur_gates_kernel(ChattsRecurArgs p) {
  __shared__ float wf[16], wm[16];
  const ChattsSpan sp = p.spans[blockIdx.y];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  if (sp.t < 1) return;
  float m0 = sp.pos0 > 0 ? p.m_state[(size_t)sp.slot * p.heads + h] : 0.f;
  const float bi = p.bias_i[h], bf = p.bias_f[h];
  for (int t0 = 0; t0 < sp.t; t0 += 1024) {
    const int t = t0 + tid;
    const bool ok = t < sp.t;
    const float* pr = p.proj + (size_t)(sp.row0 + (ok ? t : sp.t - 1)) * p.ld_proj;
    const float i = ok ? p.cap * tanhf((pr[p.off_i + h] + bi) / p.cap) : -INFINITY, f = ok ? -softplus_f(-p.cap * tanhf((pr[p.off_f + h] + bf) / p.cap)) : 0.f;
    float F = f, M = i;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const float F1 = __shfl_up(F, d, 64), M1 = __shfl_up(M, d, 64);
      if (lane >= d) { M = fmaxf(M1 + F, M); F += F1; }
    }
    __syncthreads();
    if (lane == 63) { wf[wave] = F; wm[wave] = M; }
    __syncthreads();
    float mw = m0, end = m0;      // the running maximum before this wave's tokens, after all of them
    for (int w = 0; w < 16; ++w) {
      if (w == wave) mw = end;
      end = fmaxf(end + wf[w], wm[w]);
    }
    const float m = fmaxf(mw + F, M);
    float before = __shfl_up(m, 1, 64);
    if (lane == 0) before = mw;
    if (ok) {
      const f32x4 g = {exp_hw(f + before - m), exp_hw(i - m), exp_hw(-m), 0.f};
      *reinterpret_cast<f32x4*>(p.gates + ((size_t)(sp.row0 + t) * p.heads + h) * 4) = g;
    }
    m0 = end;
  }
  if (tid == 0) p.m_state[(size_t)sp.slot * p.heads + h] = m0;
}

// With G_t = g_0 .. g_t from the chunk's start and D(s, t) = g_{s+1} .. g_t (every product runs forward: factors <= 1, nothing is divided), a chunk
// that starts from S is
//   o_t = S^T (R_t q_t) + sum_s P_ts v_s,   S <- G_15 S + sum_s (D(s, 15) k_s) v_s^T
//   read after the write:  R_t = G_t,      P_ts = q_t . (D(s, t) k_s)      (s <= t)
//   read before it:        R_t = G_{t-1},  P_ts = q_t . (D(s, t-1) k_s)    (s < t),  P_tt = q_t . (u k_t)
// A (chunk, head) holds, in floats, D = 64 NC channels:  R q [D / 16][64][4] | D(., 15) k [D / 16][64][4] | P [64][4] | G_15 [D], in the order in which
// the 64 lanes of a wave read matrix fragments.  Chunk c of span i is number row0 / 16 + i + c.  Rows past the end of a span: k = q = 0, g = 1.
constexpr int kRcChunk = 16;
__host__ __device__ constexpr int rc_chunk_floats(int nc) { return 64 * nc * (2 * kRcChunk + 1) + 256; }

template <int KIND, int NC>
__global__ __launch_bounds__(256) void recur_chunk_kernel(ChattsRecurArgs p) {
  constexpr bool WKV = KIND == CHATTS_RECUR_WKV;
  constexpr int D = NC * 64, D4 = D / 4;
  __shared__ __attribute__((aligned(16))) float sk[kRcChunk][D], sq[kRcChunk][D], sg[WKV ? kRcChunk : 1][D];
  __shared__ float sa[kRcChunk];
  const int h = blockIdx.x, chunk = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int row = -1, n = 0;      // first row and rows of this chunk
  for (int i = 0; i < p.n_spans; ++i) {
    const int r0 = p.spans[i].row0, t = p.spans[i].t, c = chunk - (r0 / kRcChunk + i);
    if (c >= 0 && c * kRcChunk < t) { row = r0 + c * kRcChunk; n = t - c * kRcChunk; }
  }
  if (row < 0) return;
  if (n > kRcChunk) n = kRcChunk;
  const int dim = p.dim;
  const float qscale = WKV ? 1.f : rsqrtf((float)dim);
  float* out = p.chunks + ((size_t)chunk * p.heads + h) * rc_chunk_floats(NC);
#pragma unroll
  for (int e = 0; e < kRcChunk * D / 256; ++e) {
    const int j = e * 256 + tid, t = j / D, c = j % D;
    const bool ok = t < n && c < dim;
    const size_t r = row + (t < n ? t : 0);
    const int cc = h * dim + (c < dim ? c : 0);
    const float* pr = p.proj + r * p.ld_proj;
    const float q = pr[p.off_q + cc], k = pr[p.off_k + cc];
    float b = 1.f;
    if constexpr (WKV) {
      const float z = p.decay[r * p.ld_decay + cc] + p.w0[cc];
      sg[t][c] = ok ? exp_hw(-exp_hw(z)) : 1.f;
    } else {
      b = p.gates[(r * p.heads + h) * 4 + 1];
    }
    sk[t][c] = ok ? k * b : 0.f;
    sq[t][c] = ok ? q * qscale : 0.f;
  }
  if constexpr (!WKV)
    if (tid < kRcChunk) sa[tid] = tid < n ? p.gates[((size_t)(row + tid) * p.heads + h) * 4] : 1.f;
  __syncthreads();
  {
    // P: thread = (token s, 1 / 16 of the channels), w = D(s, t) k_s walks forward in t
    const int s = tid >> 4, l16 = tid & 15;
    f32x4 w[NC], own[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      w[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
      own[c] = *reinterpret_cast<const f32x4*>(&sk[s][c * 64 + l16 * 4]);
    }
    float kp = 0.f;      // of token t = l16
#pragma unroll 4
    for (int t = 0; t < kRcChunk; ++t) {
      float b = 0.f;
      const float a = WKV ? 1.f : sa[t];
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        const int ch = c * 64 + l16 * 4;
        const f32x4 q = *reinterpret_cast<const f32x4*>(&sq[t][ch]);
        f32x4 g = {a, a, a, a};
        if constexpr (WKV) g = *reinterpret_cast<const f32x4*>(&sg[t][ch]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if constexpr (WKV) {
            b += q[j] * w[c][j];
            w[c][j] = t == s ? own[c][j] : w[c][j] * g[j];
          } else {
            w[c][j] = t == s ? own[c][j] : w[c][j] * g[j];
            b += q[j] * w[c][j];
          }
        }
      }
      b = row16_sum(b);
      kp = l16 == t ? b : kp;
    }
    if constexpr (WKV) {
      float b = 0.f;
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int ch = c * 64 + l16 * 4 + j;
          if (ch < dim) b += sq[s][ch] * sk[s][ch] * p.u[h * dim + ch];
        }
      b = row16_sum(b);
      if (l16 == s) kp = b;
    }
    out[2 * kRcChunk * D + ((s >> 2) * 16 + l16) * 4 + (s & 3)] = l16 >= s ? kp : 0.f;      // P[t = l16][s]
  }
  // R q and D(., 15) k of (token, 4 channels)
  constexpr int PER = D4 * kRcChunk / 256;
  f32x4 kt[PER];
#pragma unroll
  for (int e = 0; e < PER; ++e) {
    const int ct = e * 4 + wave, t = lane & 15, c = ct * 16 + (lane >> 4) * 4;
    f32x4 f = {1.f, 1.f, 1.f, 1.f}, b = {1.f, 1.f, 1.f, 1.f}, last = {1.f, 1.f, 1.f, 1.f};
#pragma unroll
    for (int r = 0; r < kRcChunk; ++r) {
      const float a = WKV ? 1.f : sa[r];
      f32x4 g = {a, a, a, a};
      if constexpr (WKV) g = *reinterpret_cast<const f32x4*>(&sg[r][c]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f[j] *= r < t || (!WKV && r == t) ? g[j] : 1.f;
        b[j] *= r > t ? g[j] : 1.f;
        if (WKV && r == kRcChunk - 1) last[j] = g[j];
      }
    }
    const f32x4 k = *reinterpret_cast<const f32x4*>(&sk[t][c]), q = *reinterpret_cast<const f32x4*>(&sq[t][c]);
    f32x4 gq;
#pragma unroll
    for (int j = 0; j < 4; ++j) { gq[j] = f[j] * q[j]; kt[e][j] = b[j] * k[j]; }
    *reinterpret_cast<f32x4*>(out + ct * 256 + lane * 4) = gq;
    if (t == kRcChunk - 1) {
#pragma unroll
      for (int j = 0; j < 4; ++j) f[j] *= last[j];
      *reinterpret_cast<f32x4*>(out + 2 * kRcChunk * D + 256 + c) = f;
    }
  }
  __syncthreads();      // (sq is free)
#pragma unroll
  for (int e = 0; e < PER; ++e)
    *reinterpret_cast<f32x4*>(&sq[lane & 15][(e * 4 + wave) * 16 + (lane >> 4) * 4]) = kt[e];
  __syncthreads();
#pragma unroll
  for (int e = 0; e < PER; ++e) {      // transposed: lane = (4 tokens lane >> 4, channel lane & 15)
    const int ct = e * 4 + wave;
    f32x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = sq[(lane >> 4) * 4 + j][ct * 16 + (lane & 15)];
    *reinterpret_cast<f32x4*>(out + kRcChunk * D + ct * 256 + lane * 4) = v;
  }
}

// grid (heads * column blocks of 16, spans), 4 waves: a wave holds NC tiles (16 channels x 16 columns) of the state as accumulators of the matrix
// pipe, which are also the right-hand operands of S^T (R q) - K slot g of product r means channel 4 g + r of a tile, token 4 g + r in the others, on
// both sides, so nothing is shuffled.  The waves' sums of the read-outs meet in LDS once per chunk and leave a chunk later: no wave waits for
// another's products.  mlstm: one column block more, whose first column is the normaliser n (v = 1).
template <int KIND, int NC>
__global__ __launch_bounds__(256, NC <= 2 ? 2 : 1) void recur_scan_kernel(ChattsRecurArgs p) {
  constexpr int D = NC * 64;
  __shared__ float so[2][4][4][64];
  const ChattsSpan sp = p.spans[blockIdx.y];
  if (sp.t < 1) return;
  const int cb = blockIdx.x / p.heads, h = blockIdx.x - cb * p.heads, tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dim = p.dim, vdim = p.vdim, v4 = (vdim + 3) & ~3, fr = lane & 15, fg = lane >> 4;
  const bool ones = KIND == CHATTS_RECUR_MLSTM && cb == (vdim + 15) / 16;      // (uniform)
  const int col = ones ? fr : cb * 16 + fr, cols = ones ? 1 : vdim;
  const bool live = col < cols;
  float* S = ones ? p.n_state + ((size_t)sp.slot * p.heads + h) * dim : p.state + ((size_t)sp.slot * p.heads + h) * dim * v4;
  const int lds = ones ? 1 : v4;
  f32x4 s[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = (wave * NC + c) * 16 + fg * 4 + r;
      s[c][r] = sp.pos0 > 0 && live && i < dim ? S[(size_t)i * lds + col] : 0.f;
    }
  const int t_all = __builtin_amdgcn_readfirstlane(sp.t), row0 = __builtin_amdgcn_readfirstlane(sp.row0), nch = (t_all + kRcChunk - 1) / kRcChunk;
  const float* ops = p.chunks + ((size_t)(row0 / kRcChunk + blockIdx.y) * p.heads + h) * rc_chunk_floats(NC);
  const size_t step = (size_t)p.heads * rc_chunk_floats(NC);
  const float* gv = p.proj + (size_t)row0 * p.ld_proj + p.off_v + h * vdim;
  const int orow = ones ? p.heads : p.heads * vdim;
  float* go = ones ? p.den + (size_t)row0 * p.heads + h : p.o + (size_t)row0 * orow + h * vdim;
  const uint32_t lane16 = lane * 16, tile0 = wave * NC * 1024, gain0 = (wave * NC * 16 + fg * 4) * 4, p0 = lane16 + wave * 4;
  const uint32_t vrow = p.ld_proj, vcol = live && !ones ? col : 0, v_last = ((uint32_t)(t_all - 1) * vrow + vcol) * 4;
  uint32_t v_at[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) v_at[r] = ((uint32_t)(fg * 4 + r) * vrow + vcol) * 4;
  const float mine[4] = {wave == 0 ? 1.f : 0.f, wave == 1 ? 1.f : 0.f, wave == 2 ? 1.f : 0.f, wave == 3 ? 1.f : 0.f};
  struct Ops { f32x4 q[NC], kt[NC], g[NC], v; float pw; };
  auto at4 = [](const float* base, uint32_t off) __attribute__((always_inline)) { return *reinterpret_cast<const f32x4*>(reinterpret_cast<const char*>(base) + off); };
  auto at1 = [](const float* base, uint32_t off) __attribute__((always_inline)) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + off); };
  auto fetch = [&](int c, Ops& o) __attribute__((always_inline)) {
    if (c > nch - 1) c = nch - 1;
    const float* b = ops + (size_t)c * step;
#pragma unroll
    for (int i = 0; i < NC; ++i) o.q[i] = at4(b + i * 256, tile0 + lane16);
    const uint32_t skip = (uint32_t)c * kRcChunk * vrow * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t off = v_at[r] + skip;
      o.v[r] = at1(gv, off < v_last ? off : v_last);
    }
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      o.g[i] = at4(b + 2 * kRcChunk * D + 256 + i * 16, gain0);
      o.kt[i] = at4(b + kRcChunk * D + i * 256, tile0 + lane16);
    }
    o.pw = at1(b + 2 * kRcChunk * D, p0);
  };
  auto emit = [&](int c, const float (&x)[4]) __attribute__((always_inline)) {      // this wave writes the tokens 4 g + wave of a chunk
    const int t = c * kRcChunk + fg * 4 + wave;
    if (c >= 0 && live && t < t_all) go[(size_t)t * orow + col] = (x[0] + x[1]) + (x[2] + x[3]);
  };
  auto meet = [&]() __attribute__((always_inline)) {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  auto chunk = [&](int c, Ops& o, Ops& later) __attribute__((always_inline)) {
    const int b = c & 1;
    float past[4];
#pragma unroll
    for (int w = 0; w < 4; ++w) past[w] = c > 0 ? so[b ^ 1][w][wave][lane] : 0.f;
    fetch(c + 2, later);
    __builtin_amdgcn_sched_barrier(0);
    if (ones) o.v = (f32x4){1.f, 1.f, 1.f, 1.f};
    const float vw = o.v[0] * mine[0] + o.v[1] * mine[1] + o.v[2] * mine[2] + o.v[3] * mine[3];      // = v[wave], without branches
    f32x4 e = {0.f, 0.f, 0.f, 0.f};
    e = __builtin_amdgcn_mfma_f32_16x16x4f32(o.pw, vw, e, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4 * NC; ++i) e = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i >> 2][i & 3], s[i >> 2][i & 3], e, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NC; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[i][r] *= o.g[i][r];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < NC; ++i) s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kt[i][r], o.v[r], s[i], 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) so[b][wave][r][lane] = e[r];
    emit(c - 1, past);
    meet();
  };
  Ops ops3[3];
  fetch(0, ops3[0]);
  fetch(1, ops3[1]);
  int c = 0;
  for (; c + 3 <= nch; c += 3) {
    chunk(c, ops3[0], ops3[2]);
    chunk(c + 1, ops3[1], ops3[0]);
    chunk(c + 2, ops3[2], ops3[1]);
  }
  if (c < nch) chunk(c, ops3[0], ops3[2]);
  if (c + 1 < nch) chunk(c + 1, ops3[1], ops3[0]);
  float past[4];
#pragma unroll
  for (int w = 0; w < 4; ++w) past[w] = so[(nch - 1) & 1][w][wave][lane];
  emit(nch - 1, past);
  if (live)
#pragma unroll
    for (int c2 = 0; c2 < NC; ++c2)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = (wave * NC + c2) * 16 + fg * 4 + r;
        if (i < dim) S[(size_t)i * lds + col] = s[c2][r];
      }
}

// norm + gate of the read-outs; the last row of a segment leaves its mixer input behind.  A head belongs to G lanes (a power of two, 4 G >= vdim),
// 4 consecutive columns each.
template <int KIND, bool QUADS>      // vdim % 4 == 0
__global__ __launch_bounds__(256) void recur_out_kernel(ChattsRecurArgs p, int G) {
  constexpr bool WKV = KIND == CHATTS_RECUR_WKV;
  const int row = blockIdx.x, tid = threadIdx.x, per = 256 / G, i = (tid & (G - 1)) * 4;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const int vdim = p.vdim, vrow = p.heads * vdim;
  const float* o = p.o + (size_t)row * vrow;
  const float* gate = p.proj + (size_t)row * p.ld_proj + p.off_gate;
  for (int h = blockIdx.y * per + tid / G; h < p.heads; h += gridDim.y * per) {      // (h is the same in all lanes of a group)
    float v[4] = {0.f, 0.f, 0.f, 0.f}, g[4] = {0.f, 0.f, 0.f, 0.f}, w[4] = {0.f, 0.f, 0.f, 0.f};
    const int at = h * vdim + i;
    if (QUADS) {
      if (i < vdim) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(o + at), y = *reinterpret_cast<const f32x4*>(gate + at), z = *reinterpret_cast<const f32x4*>(p.norm_w + at);
#pragma unroll
        for (int j = 0; j < 4; ++j) { v[j] = x[j]; g[j] = y[j]; w[j] = z[j]; }
      }
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < vdim) { v[j] = o[at + j]; g[j] = gate[at + j]; w[j] = p.norm_w[at + j]; }
    }
    if constexpr (!WKV) {
      const float d = fmaxf(fabsf(p.den[(size_t)row * p.heads + h]), p.gates[((size_t)row * p.heads + h) * 4 + 2]) + 1e-6f;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] /= d;
    }
    float ss = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    for (int x = 1; x < G; x <<= 1) ss += __shfl_xor(ss, x, 64);
    const float f = 1.0f / sqrtf(ss / (float)vdim + p.eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float sg = sigmoid_f(g[j]);
      v[j] = v[j] * f * w[j] * (WKV ? g[j] * sg : sg);
    }
    if (QUADS) {
      if (i < vdim) store_operand4(p.out, row, at, v);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < vdim) store_operand(p.out, row, at + j, v[j]);
    }
  }
  if (p.prev && R.rest == 0)
    for (int c = blockIdx.y * 256 + tid; c < p.ld_h; c += gridDim.y * 256) p.prev[(size_t)R.slot * p.ld_h + c] = p.h[(size_t)row * p.ld_h + c];
}

static int check_recur(const ChattsRecurArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->proj && a->rows && a->state && a->norm_w, CHATTS_E_BADARG, "%s: null pointer", who);
  CHATTS_REQUIRE(a->kind == CHATTS_RECUR_WKV || a->kind == CHATTS_RECUR_MLSTM, CHATTS_E_BADARG, "%s: kind %d", who, a->kind);
  CHATTS_REQUIRE(a->heads > 0 && a->dim >= 1 && a->dim <= 256 && a->vdim >= 1 && a->vdim <= 256, CHATTS_E_SHAPE, "%s: %d heads of %d x %d (at most 256 x 256)", who,
                 a->heads, a->dim, a->vdim);
  CHATTS_REQUIRE(a->n_rows >= 0 && a->ld_proj % 4 == 0 && a->off_q >= 0 && a->off_k >= 0 && a->off_v >= 0 && a->off_gate >= 0 &&
                     a->off_q + a->heads * a->dim <= a->ld_proj && a->off_k + a->heads * a->dim <= a->ld_proj && a->off_v + a->heads * a->vdim <= a->ld_proj &&
                     a->off_gate + a->heads * a->vdim <= a->ld_proj, CHATTS_E_SHAPE, "%s: column blocks", who);
  if (a->kind == CHATTS_RECUR_WKV)
    CHATTS_REQUIRE(a->w0 && a->u && a->rank > 0 && a->rank % 8 == 0 && a->rank <= 4096 && a->off_a % 4 == 0 && a->off_a + a->rank <= a->ld_proj, CHATTS_E_SHAPE,
                   "%s: low-rank input of %d columns", who, a->rank);
  else
    CHATTS_REQUIRE(a->bias_i && a->bias_f && a->n_state && a->m_state && a->cap > 0.f && a->off_i + a->heads <= a->ld_proj && a->off_f + a->heads <= a->ld_proj,
                   CHATTS_E_BADARG, "%s: gates", who);
  return CHATTS_OK;
}

template <int KIND>
static void launch_recur_decode(const ChattsRecurArgs* a, int TX, int nt, int nr, size_t lds, hipStream_t s) {
  const dim3 g(a->heads, a->n_rows);
  if (nt == 512) hipLaunchKernelGGL((recur_decode_kernel<KIND, 512, 32>), g, dim3(512), lds, s, *a, TX);
  else if (nr <= 4) hipLaunchKernelGGL((recur_decode_kernel<KIND, 256, 4>), g, dim3(256), lds, s, *a, TX);
  else if (nr <= 8) hipLaunchKernelGGL((recur_decode_kernel<KIND, 256, 8>), g, dim3(256), lds, s, *a, TX);
  else if (nr <= 16) hipLaunchKernelGGL((recur_decode_kernel<KIND, 256, 16>), g, dim3(256), lds, s, *a, TX);
  else hipLaunchKernelGGL((recur_decode_kernel<KIND, 256, 32>), g, dim3(256), lds, s, *a, TX);
}

template <int KIND>
static void launch_recur_scan(const ChattsRecurArgs* a, hipStream_t s) {
  const dim3 gc(a->heads, a->n_rows / kRcChunk + a->n_spans), gs(a->heads * ((a->vdim + 15) / 16 + (KIND == CHATTS_RECUR_MLSTM)), a->n_spans), b(256);
#define CHATTS_RECUR_SCAN(NC)                                                   \
  do {                                                                          \
    hipLaunchKernelGGL((recur_chunk_kernel<KIND, NC>), gc, b, 0, s, *a);        \
    hipLaunchKernelGGL((recur_scan_kernel<KIND, NC>), gs, b, 0, s, *a);         \
  } while (0)
  switch ((a->dim + 63) / 64) {
    case 1: CHATTS_RECUR_SCAN(1); break;
    case 2: CHATTS_RECUR_SCAN(2); break;
    case 3: CHATTS_RECUR_SCAN(3); break;
    default: CHATTS_RECUR_SCAN(4); break;
  }
#undef CHATTS_RECUR_SCAN
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_recur_decode(const ChattsRecurArgs* a, chatts_stream_t stream) {
  if (const int rc = check_recur(a, "recur_decode")) return rc;
  const bool wkv = a->kind == CHATTS_RECUR_WKV;
  CHATTS_REQUIRE((!wkv || a->w2d) && (a->out.f32 || a->out.hi) && a->out.ld >= a->heads * a->vdim, CHATTS_E_BADARG, "recur_decode: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  const int v4 = (a->vdim + 3) & ~3;
  int TX = 1;
  while (TX * 4 < v4) TX *= 2;
  auto rows_for = [&](int nt) { return (a->dim + nt / TX - 1) / (nt / TX); };
  const int nt = rows_for(256) > 32 ? 512 : 256, nr = rows_for(nt);
  const size_t lds = (size_t)(nt * 4 + v4 + 3 * a->dim + (wkv ? a->rank : 0) + 16) * sizeof(float);
  if (wkv) launch_recur_decode<CHATTS_RECUR_WKV>(a, TX, nt, nr, lds, as_stream(stream));
  else launch_recur_decode<CHATTS_RECUR_MLSTM>(a, TX, nt, nr, lds, as_stream(stream));
  CHATTS_CHECK_LAUNCH("recur_decode");
  return CHATTS_OK;
}

extern "C" int chatts_recur_tanh(const ChattsRecurArgs* a, const ChattsOperand* out, chatts_stream_t stream) {
  if (const int rc = check_recur(a, "recur_tanh")) return rc;
  CHATTS_REQUIRE(a->kind == CHATTS_RECUR_WKV && out && (out->f32 || out->hi) && out->ld >= a->rank && out->ld % 4 == 0, CHATTS_E_BADARG, "recur_tanh: bad arguments");
  if (a->n_rows == 0) return CHATTS_OK;
  const size_t total = (size_t)a->n_rows * (a->rank / 4);
  hipLaunchKernelGGL(recur_tanh_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, as_stream(stream), *a, *out);
  CHATTS_CHECK_LAUNCH("recur_tanh");
  return CHATTS_OK;
}

extern "C" int64_t chatts_recur_chunk_floats(int heads, int dim, int n_rows, int n_spans) {
  return (int64_t)(n_rows / kRcChunk + n_spans) * heads * rc_chunk_floats((dim + 63) / 64);
}

extern "C" int chatts_recur_scan(const ChattsRecurArgs* a, chatts_stream_t stream) {
  if (const int rc = check_recur(a, "recur_scan")) return rc;
  const bool wkv = a->kind == CHATTS_RECUR_WKV;
  CHATTS_REQUIRE(a->chunks && ((uintptr_t)a->chunks % 16) == 0 && a->o && a->spans && (wkv ? a->decay && a->ld_decay >= a->heads * a->dim : a->gates && a->den),
                 CHATTS_E_BADARG, "recur_scan: null scratch");
  if (a->n_spans == 0 || a->n_rows == 0) return CHATTS_OK;
  if (wkv) {
    launch_recur_scan<CHATTS_RECUR_WKV>(a, as_stream(stream));
  } else {
    hipLaunchKernelGGL(recur_gates_kernel, dim3(a->heads, a->n_spans), dim3(1024), 0, as_stream(stream), *a);
    CHATTS_CHECK_LAUNCH("recur_gates");
    launch_recur_scan<CHATTS_RECUR_MLSTM>(a, as_stream(stream));
  }
  CHATTS_CHECK_LAUNCH("recur_scan");
  return CHATTS_OK;
}

extern "C" int chatts_recur_out(const ChattsRecurArgs* a, chatts_stream_t stream) {
  if (const int rc = check_recur(a, "recur_out")) return rc;
  const bool wkv = a->kind == CHATTS_RECUR_WKV;
  CHATTS_REQUIRE(a->o && (wkv || (a->den && a->gates)) && (a->out.f32 || a->out.hi) && a->out.ld >= a->heads * a->vdim && (!a->prev || a->h), CHATTS_E_BADARG,
                 "recur_out: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  int lanes = 1;
  while (lanes * 4 < a->vdim) lanes *= 2;
  const int per = 256 / lanes;
  const dim3 g(a->n_rows, (a->heads + 2 * per - 1) / (2 * per)), b(256);
  hipStream_t s = as_stream(stream);
  const bool quads = a->vdim % 4 == 0 && a->out.ld % 4 == 0 && a->off_gate % 4 == 0;
  if (wkv && quads) hipLaunchKernelGGL((recur_out_kernel<CHATTS_RECUR_WKV, true>), g, b, 0, s, *a, lanes);
  else if (wkv) hipLaunchKernelGGL((recur_out_kernel<CHATTS_RECUR_WKV, false>), g, b, 0, s, *a, lanes);
  else if (quads) hipLaunchKernelGGL((recur_out_kernel<CHATTS_RECUR_MLSTM, true>), g, b, 0, s, *a, lanes);
  else hipLaunchKernelGGL((recur_out_kernel<CHATTS_RECUR_MLSTM, false>), g, b, 0, s, *a, lanes);
  CHATTS_CHECK_LAUNCH("recur_out");
  return CHATTS_OK;
}
