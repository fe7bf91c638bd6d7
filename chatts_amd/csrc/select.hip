// select.hip - selective scan: per channel c and state n  S <- exp(d_c A[c, n]) S + d_c u_c B_n,  y_c = sum_n S C_n + D_c u_c  with step sizes d, inputs u and
// the vectors B, C of every token; the read-out y silu(z) leaves as the next projection's operand.  Float32.
//   select_conv_kernel    u = silu(short convolution), with the inputs before a segment from a ring per slot
//   select_ring_kernel    the last convolution inputs of every segment
//   select_decode_kernel  one token per sequence: the step sizes' projection, the state's update and the read-out in one launch
//   select_split_kernel   dt of many rows as bf16 hi + lo matrix fragments (a fragment is 1 KB of consecutive memory: sixteen cache lines a load would cost four
//                         times as much)
//   select_steps_kernel   their step sizes: W_dt in registers, the fragments streamed past it, softplus in the epilogue
//   select_scan_kernel    segments of several tokens, in tiles through LDS
// A channel's states lie in LPC neighbouring lanes, SPL in each.
#include "gemm_common.h"

namespace chatts {

// a thread owns four channels of ROWS consecutive rows; TAPS 0: any number, one input after the other
template <int TAPS, int ROWS>
__global__ __launch_bounds__(256) void select_conv_kernel(ChattsSelectArgs p) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4, row0 = blockIdx.y * ROWS;
  if (c >= p.conv_ch || c >= ((p.inner + 3) & ~3)) return;
  const int taps = TAPS ? TAPS : p.taps;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f}, bias = *reinterpret_cast<const f32x4*>(p.conv_b + c);
  ChattsRow R[ROWS];
  f32x4 now[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    R[r] = row0 + r < p.n_rows ? p.rows[row0 + r] : ChattsRow{0, -1, 0, 0};
    now[r] = R[r].pos >= 0 ? *reinterpret_cast<const f32x4*>(p.proj + (size_t)(row0 + r) * p.ld_proj + p.off_x + c) : zero;
  }
  auto before = [&](const ChattsRow& r, int row, int back) __attribute__((always_inline)) {      // the input `back` tokens before a row's
    if (row - back >= r.first) return *reinterpret_cast<const f32x4*>(p.proj + (size_t)(row - back) * p.ld_proj + p.off_x + c);
    const int q = r.pos - back;
    return q >= 0 ? *reinterpret_cast<const f32x4*>(p.ring + ((size_t)r.slot * taps + q % taps) * p.conv_ch + c) : zero;
  };
  constexpr int H = TAPS > 1 ? TAPS - 1 : 1;
  f32x4 w[TAPS ? TAPS : 1], hist[H];      // [tokens back], [tokens back - 1]
  if (TAPS)
#pragma unroll
    for (int g = 0; g < TAPS; ++g) w[g] = *reinterpret_cast<const f32x4*>(p.conv_w + (size_t)(TAPS - 1 - g) * p.conv_ch + c);
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int row = row0 + r;
    if (R[r].pos < 0) continue;
    f32x4 y = bias;
    if (TAPS) {
      if (r == 0 || R[r].first == row) {
#pragma unroll
        for (int g = 1; g < TAPS; ++g) hist[g - 1] = before(R[r], row, g);
      }
#pragma unroll
      for (int g = TAPS - 1; g > 0; --g) y += w[g] * hist[g - 1];
      y += w[0] * now[r];
#pragma unroll
      for (int g = H - 1; g > 0; --g) hist[g] = hist[g - 1];
      hist[0] = now[r];
    } else {
      for (int g = taps - 1; g > 0; --g) y += *reinterpret_cast<const f32x4*>(p.conv_w + (size_t)(taps - 1 - g) * p.conv_ch + c) * before(R[r], row, g);
      y += *reinterpret_cast<const f32x4*>(p.conv_w + (size_t)(taps - 1) * p.conv_ch + c) * now[r];
    }
    float v[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = y[k] * sigmoid_f(y[k]);
    store_operand4(p.u, row, c, v);
    if (p.n_spans == 0)      // segments of one token: nobody else reads this entry of the ring
      *reinterpret_cast<f32x4*>(p.ring + ((size_t)R[r].slot * taps + R[r].pos % taps) * p.conv_ch + c) = now[r];
  }
}

// grid (taps - 1, spans, columns / 1024): the inputs that the next step's convolutions read
__global__ __launch_bounds__(256) void select_ring_kernel(ChattsSelectArgs p) {
  const ChattsSpan sp = p.spans[blockIdx.y];
  const int i = blockIdx.x, c = (blockIdx.z * 256 + threadIdx.x) * 4;
  if (i >= sp.t || c >= p.conv_ch || c >= ((p.inner + 3) & ~3)) return;
  const int last = sp.t - 1 - i;
  *reinterpret_cast<f32x4*>(p.ring + ((size_t)sp.slot * p.taps + (sp.pos0 + last) % p.taps) * p.conv_ch + c) =
      *reinterpret_cast<const f32x4*>(p.proj + (size_t)(sp.row0 + last) * p.ld_proj + p.off_x + c);
}

// sum over LPC neighbouring lanes (aligned), in every one of them
template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) {
  v += lane_xor1(v);
  v += lane_xor2(v);
  if (LPC >= 8) v += half_mirror(v);
  if (LPC >= 16) v += row_ror8(v);
  if (LPC >= 32) v += __shfl_xor(v, 16, 64);
  return v;
}

// the SPL states of a lane, from n4 values (a multiple of 4) of its channel
template <int SPL>
__device__ __forceinline__ void states_load(const float* src, int l, int n4, float (&s)[SPL]) {
  constexpr int V = SPL < 4 ? SPL : 4;
#pragma unroll
  for (int i = 0; i < SPL; i += V) {
    const bool ok = l * SPL + i < n4;
#pragma unroll
    for (int k = 0; k < V; ++k) s[i + k] = 0.f;
    if (!ok) continue;
    if constexpr (V == 4) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(src + l * SPL + i);
#pragma unroll
      for (int k = 0; k < 4; ++k) s[i + k] = x[k];
    } else if constexpr (V == 1) {
      s[i] = src[l + i];
    } else {
      const float2 x = *reinterpret_cast<const float2*>(src + l * SPL + i);
      s[i] = x.x;
      s[i + 1] = x.y;
    }
  }
}
template <int SPL>
__device__ __forceinline__ void states_store(float* dst, int l, int n4, const float (&s)[SPL]) {
  constexpr int V = SPL < 4 ? SPL : 4;
#pragma unroll
  for (int i = 0; i < SPL; i += V) {
    if (l * SPL + i >= n4) continue;
    if constexpr (V == 4) *reinterpret_cast<f32x4*>(dst + l * SPL + i) = (f32x4){s[i], s[i + 1], s[i + 2], s[i + 3]};
    else if constexpr (V == 1) dst[l + i] = s[i];
    else *reinterpret_cast<float2*>(dst + l * SPL + i) = make_float2(s[i], s[i + 1]);
  }
}

// grid (channels / (256 / LPC), rows / NR): NR sequences share what a workgroup reads of W_dt
template <int SPL, int LPC, int NR>
__global__ __launch_bounds__(256) void select_decode_kernel(ChattsSelectArgs p) {
  constexpr int CH = 256 / LPC;
  const int row0 = blockIdx.y * NR, l = threadIdx.x & (LPC - 1), c = blockIdx.x * CH + threadIdx.x / LPC, n4 = (p.state + 3) & ~3;
  const bool live = c < p.inner;
  const int cc = live ? c : 0;
  int pos[NR], row[NR];
  float* S[NR];
  float s[NR][SPL], u[NR], z[NR], acc[NR], a[SPL];
  bool any = false;
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    row[r] = row0 + r < p.n_rows ? row0 + r : p.n_rows - 1;
    const ChattsRow R = p.rows[row[r]];
    pos[r] = row0 + r < p.n_rows ? R.pos : -1;
    any = any || pos[r] >= 0;
    S[r] = p.s + ((size_t)(pos[r] >= 0 ? R.slot : 0) * p.inner + cc) * n4;
    acc[r] = 0.f;
  }
  if (!any) return;
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    states_load<SPL>(S[r], l, n4, s[r]);
    u[r] = p.u.f32[(size_t)row[r] * p.u.ld + cc];
    z[r] = p.proj[(size_t)row[r] * p.ld_proj + p.off_z + cc];
  }
  states_load<SPL>(p.a + (size_t)cc * n4, l, n4, a);
  const float bias = p.dt_bias[cc], d = p.d[cc];
  // the step sizes: a channel's lanes share its row of W_dt
  const uint16_t* w = p.w_dt + (size_t)cc * p.rank;
  for (int i = l * 8; i < p.rank; i += LPC * 8) {
    const u32x4 wv = *reinterpret_cast<const u32x4*>(w + i);
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const float* x = p.low + (size_t)row[r] * p.ld_low + p.off_dt + i;
      const f32x4 x0 = *reinterpret_cast<const f32x4*>(x), x1 = *reinterpret_cast<const f32x4*>(x + 4);
      acc[r] += (bf16_lo(wv[0]) * x0[0] + bf16_hi(wv[0]) * x0[1]) + (bf16_lo(wv[1]) * x0[2] + bf16_hi(wv[1]) * x0[3]);
      acc[r] += (bf16_lo(wv[2]) * x1[0] + bf16_hi(wv[2]) * x1[1]) + (bf16_lo(wv[3]) * x1[2] + bf16_hi(wv[3]) * x1[3]);
    }
  }
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const float* low = p.low + (size_t)row[r] * p.ld_low;
    float B[SPL], Cn[SPL], y = 0.f;
    states_load<SPL>(low + p.off_b, l, n4, B);
    states_load<SPL>(low + p.off_c, l, n4, Cn);
    const float dt = softplus_f(lanes_sum<LPC>(acc[r]) + bias), du = dt * u[r];
#pragma unroll
    for (int i = 0; i < SPL; ++i) {
      s[r][i] = __builtin_amdgcn_exp2f(dt * a[i]) * (pos[r] > 0 ? s[r][i] : 0.f) + du * B[i];
      y += s[r][i] * Cn[i];
    }
    y = lanes_sum<LPC>(y);
    if (!live || pos[r] < 0) continue;
    states_store<SPL>(S[r], l, n4, s[r]);
    if (l == 0) store_operand(p.out, row[r], c, (y + d * u[r]) * z[r] * sigmoid_f(z[r]) * p.out_scale);
  }
}

// grid (channels / 128, rows / kStepRows), 4 waves of 32 channels each.  rank = 32 KS; a wave keeps its rows of W_dt, the fragments of 16 rows of dt pass through LDS
// (LDS-DMA, the next ones while these are multiplied); D = W . A^T: a lane holds four neighbouring channels of one row
constexpr int kStepRows = 128;
// grid (rows / 16, rank / 128): a thread = 8 K-values of a row
__global__ __launch_bounds__(256) void select_split_kernel(ChattsSelectArgs p) {
  const int l = threadIdx.x & 63, kt = blockIdx.y * 4 + (threadIdx.x >> 6), row = blockIdx.x * 16 + (l & 15), nk = p.rank >> 5;
  if (kt >= nk) return;
  const float* src = p.low + (size_t)(row < p.n_rows ? row : p.n_rows - 1) * p.ld_low + p.off_dt + kt * 32 + (l >> 4) * 8;
  const f32x4 a = *reinterpret_cast<const f32x4*>(src), b = *reinterpret_cast<const f32x4*>(src + 4);
  const float v0[4] = {a[0], a[1], a[2], a[3]}, v1[4] = {b[0], b[1], b[2], b[3]};
  ChattsOperand o{};
  o.hi = p.dt_hi; o.lo = p.dt_lo;
  const int at = l * 8;
  const size_t block = ((size_t)blockIdx.x * nk + kt) * 512;
  o.hi += block; o.lo += block;
  store_operand4(o, 0, at, v0);
  store_operand4(o, 0, at + 4, v1);
}
template <int KS>
__global__ __launch_bounds__(256, 2) void select_steps_kernel(ChattsSelectArgs p) {
  constexpr int CT = 2;
  __shared__ __attribute__((aligned(16))) uint16_t sa[2][2 * KS * 512];      // hi fragments, lo fragments
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), fr = lane & 15, fg = lane >> 4;
  const int c0 = (blockIdx.x * 4 + wave) * 16 * CT, r0 = blockIdx.y * kStepRows, c4 = (p.inner + 3) & ~3, last = ((p.inner + 63) >> 4 & ~3) - 1;      // (W_dt's last fragment)
  bf16x8_t w[CT][KS];
  f32x4 bias[CT], d[CT];
#pragma unroll
  for (int t = 0; t < CT; ++t) {
    const int c = c0 + t * 16 + fg * 4, f = (c0 >> 4) + t < last ? (c0 >> 4) + t : last;
#pragma unroll
    for (int k = 0; k < KS; ++k) w[t][k] = *reinterpret_cast<const bf16x8_t*>(p.w_dt_f + ((size_t)f * KS + k) * 512 + lane * 8);
    d[t] = bias[t] = *reinterpret_cast<const f32x4*>(p.dt_bias + (c < c4 ? c : 0));
  }
  const int end = r0 + kStepRows < p.n_rows ? r0 + kStepRows : p.n_rows;
  auto request = [&](int r, int buf) __attribute__((always_inline)) {      // a wave takes every fourth fragment
    const size_t at = (size_t)(r >> 4) * KS * 512 + lane * 8;
#pragma unroll
    for (int i = 0; i < KS / 2; ++i) {
      const int f = i * 4 + wave;      // (uniform)
      const uint16_t* src = (f < KS ? p.dt_hi + f * 512 : p.dt_lo + (f - KS) * 512) + at;
      __builtin_amdgcn_global_load_lds((gptr_t)src, (lptr_t)(&sa[buf][f * 512]), 16, 0, 0);
    }
  };
  auto store = [&](int r) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < CT; ++t) {
      const int c = c0 + t * 16 + fg * 4;
      if (r + fr < end && c < c4) *reinterpret_cast<f32x4*>(p.delta + (size_t)(r + fr) * p.ld_delta + c) = d[t];
    }
  };
  auto meet = []() __attribute__((always_inline)) {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  request(r0, 0);
  meet();
  int buf = 0;
  for (int r = r0; r < end; r += 16, buf ^= 1) {
    if (r > r0) store(r - 16);      // (behind the barrier that follows they have had a tile's time)
    if (r + 16 < end) request(r + 16, buf ^ 1);
#pragma unroll
    for (int t = 0; t < CT; ++t) d[t] = bias[t];
    const uint16_t* a = &sa[buf][lane * 8];
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const bf16x8_t h = *reinterpret_cast<const bf16x8_t*>(a + k * 512), l = *reinterpret_cast<const bf16x8_t*>(a + (KS + k) * 512);
#pragma unroll
      for (int t = 0; t < CT; ++t) d[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t][k], l, d[t], 0, 0, 0);
#pragma unroll
      for (int t = 0; t < CT; ++t) d[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t][k], h, d[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < CT; ++t)
#pragma unroll
      for (int j = 0; j < 4; ++j) d[t][j] = softplus_f(d[t][j]);
    meet();
  }
  store(r0 + (end - r0 - 1) / 16 * 16);
}

// grid (channels / (256 / LPC), spans), 8 waves.  Waves 0 .. 3 run the recurrence of 64 / LPC channels each and do nothing else; wave 4 + w prepares the next
// tile for wave w (step sizes as quads of tokens, B and C for everyone) and finishes the previous one (adds the lanes' shares of the read-outs, gates and
// stores them).  Everything between them lies in LDS twice; one barrier per tile.
template <int SPL, int LPC, int TT>
constexpr int select_lds() {      // floats, each twice: step sizes, step sizes times u [channels][TT + 4], shares [4][TT / 4][64][4], B, C [states][TT + 4]
  return 2 * (2 * (256 / LPC) * (TT + 4) + 256 * TT + 2 * SPL * LPC * (TT + 4));
}
template <int SPL, int LPC, int TT>
__global__ __launch_bounds__(512, TT == 16 ? 4 : 2) void select_scan_kernel(ChattsSelectArgs p) {
  constexpr int LD = TT + 4, T4 = TT / 4, CW = 64 / LPC, NP = SPL * LPC, NQ = NP / 4, KB = (TT * NQ + 255) / 256, NT = TT * CW > 64 ? TT * CW / 64 : 1;
  constexpr bool kRows = NQ <= 4;      // B and C: neighbouring lanes take a row's quads (whole lines), or - many states - neighbouring rows (no bank met twice)
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ChattsSpan sp = p.spans[blockIdx.y];
  if (sp.t < 1) return;
  const int tid = threadIdx.x & 255, lane = tid & 63, role = __builtin_amdgcn_readfirstlane(threadIdx.x >> 8), wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n4 = (p.state + 3) & ~3, c0 = (blockIdx.x * 4 + wave) * CW, t_all = __builtin_amdgcn_readfirstlane(sp.t), tiles = (t_all + 2 * TT - 1) / (2 * TT) * 2;      // (an empty one at the end of some)
  constexpr int kStep = 4 * CW * LD, kShare = 256 * TT;      // floats of a buffer
  float* sdt = sm + wave * CW * LD;                          // + buffer * kStep; step sizes times u: 2 kStep further
  float* sy = sm + 4 * kStep + wave * 64 * TT;               // + buffer * kShare
  float* sbc = sm + 4 * kStep + 2 * kShare;                  // [buffer][B, C][NP][LD]
  auto meet = [&]() __attribute__((always_inline)) {         // (LDS alone: what goes to and from memory stays on its way)
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  if (role == 0) {
    const int l = lane & (LPC - 1), c = c0 + lane / LPC, cc = c < p.inner ? c : 0;
    float a[SPL], s[SPL];
    float* S = p.s + ((size_t)sp.slot * p.inner + cc) * n4;
    states_load<SPL>(p.a + (size_t)cc * n4, l, n4, a);
#pragma unroll
    for (int i = 0; i < SPL; ++i) s[i] = 0.f;
    if (sp.pos0 > 0 && c < p.inner) states_load<SPL>(S, l, n4, s);
    meet();
    for (int k = 0; k < tiles; ++k) {
      const int buf = k & 1;
      const float* rdt = sdt + buf * kStep + (lane / LPC) * LD;
      const float* rdu = rdt + 2 * kStep;
      const float* b = sbc + (buf * 2 * NP + l * SPL) * LD;
      float* y0 = sy + buf * kShare + lane * 4;
      struct Quad { f32x4 dt, du, B[SPL], C[SPL]; };      // four tokens
      auto request = [&](int g, Quad& q) __attribute__((always_inline)) {
        q.dt = *reinterpret_cast<const f32x4*>(rdt + g * 4);
        q.du = *reinterpret_cast<const f32x4*>(rdu + g * 4);
#pragma unroll
        for (int i = 0; i < SPL; ++i) {
          q.B[i] = *reinterpret_cast<const f32x4*>(b + i * LD + g * 4);
          q.C[i] = *reinterpret_cast<const f32x4*>(b + (NP + i) * LD + g * 4);
        }
      };
      auto run = [&](int g, const Quad& q) __attribute__((always_inline)) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
        float e[SPL][4];
#pragma unroll
        for (int i = 0; i < SPL; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) e[i][j] = __builtin_amdgcn_exp2f(q.dt[j] * a[i]);
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int i = 0; i < SPL; ++i) {
            s[i] = e[i][j] * s[i] + q.du[j] * q.B[i][j];
            y[j] += s[i] * q.C[i][j];
          }
        *reinterpret_cast<f32x4*>(y0 + g * 256) = y;
      };
      if constexpr (SPL <= 4) {      // the next quad travels while one is worked on
        Quad quad[2];
        request(0, quad[0]);
#pragma unroll
        for (int g = 0; g < T4; ++g) {
          if (g + 1 < T4) request(g + 1, quad[(g + 1) & 1]);
          __builtin_amdgcn_sched_barrier(0);
          run(g, quad[g & 1]);
          __builtin_amdgcn_sched_barrier(0);
        }
      } else {
#pragma unroll 1
        for (int g = 0; g < T4; ++g) {
          Quad quad;
          request(g, quad);
          run(g, quad);
        }
      }
      meet();
    }
    if (c < p.inner) states_store<SPL>(S, l, n4, s);
    return;
  }
  // lane = (channel oc, tokens NT og ..)
  const bool mine = TT * CW >= 64 || lane / CW < TT;      // (few channels: not every lane has a token)
  const int oc = lane & (CW - 1), og = mine ? lane / CW : 0, och = c0 + oc;
  const bool stage = mine && och < p.inner;
  const int at = stage ? och : 0;
  const float bias = p.dt_bias[at], dw = p.d[at];
  struct Inputs { float d[NT], u[NT], z[NT]; f32x4 b[KB], c[KB]; };      // of a tile; two tiles are on their way
  Inputs in[2];
  float out[NT], u[3][NT], z[3][NT];      // u, z: of the tile prepared last, the one before, ...
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    out[j] = 0.f;
    u[0][j] = u[1][j] = u[2][j] = z[0][j] = z[1][j] = z[2][j] = 0.f;
  }
  auto at1 = [](const float* base, uint32_t off) __attribute__((always_inline)) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + off); };
  // (no branches: requests stay in flight across them only if no two paths meet.  Beyond the end: the last row)
  auto fetch = [&](int k, Inputs& x) __attribute__((always_inline)) {
    const int t0 = k * TT < t_all ? k * TT : t_all - 1, last = t_all - 1 - t0;
    const size_t row = sp.row0 + t0;
    const float* d0 = p.delta + row * p.ld_delta;
    const float* u0 = p.u.f32 + row * p.u.ld;
    const float* z0 = p.proj + row * p.ld_proj + p.off_z;
    const float* low = p.low + row * p.ld_low;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int own = og * NT + j, t = own < last ? own : last;
      x.d[j] = at1(d0, (uint32_t)(__mul24(t, p.ld_delta) + at) * 4u);
      x.u[j] = at1(u0, (uint32_t)(__mul24(t, p.u.ld) + at) * 4u);
      x.z[j] = at1(z0, (uint32_t)(__mul24(t, p.ld_proj) + at) * 4u);
    }
#pragma unroll
    for (int e = 0; e < KB; ++e) {
      const int i = e * 256 + tid, own = kRows ? i / NQ : i % TT, t = own < last ? own : last, n = (kRows ? i % NQ : i / TT) * 4;
      const float* src = low + (uint32_t)(__mul24(t, p.ld_low) + (n < n4 ? n : 0));
      x.b[e] = *reinterpret_cast<const f32x4*>(src + p.off_b);
      x.c[e] = *reinterpret_cast<const f32x4*>(src + p.off_c);
    }
  };
  auto prepare = [&](int k, Inputs& x) __attribute__((always_inline)) {      // tile k from registers to LDS
    const int buf = k & 1;
    float dt[NT], du[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      u[2][j] = u[1][j];
      z[2][j] = z[1][j];
      u[1][j] = u[0][j];
      z[1][j] = z[0][j];
      u[0][j] = x.u[j];
      z[0][j] = x.z[j];
      const uint32_t keep = stage && k * TT + og * NT + j < t_all ? 0xffffffffu : 0u;      // (beyond the end: the state stays)
      dt[j] = __uint_as_float(__float_as_uint(p.delta_steps ? x.d[j] : softplus_f(x.d[j] + bias)) & keep);
      du[j] = dt[j] * x.u[j];
    }
    float* d = sdt + buf * kStep + oc * LD + og * NT;
    if (mine) {
      if constexpr (NT == 4) {
        *reinterpret_cast<f32x4*>(d) = (f32x4){dt[0], dt[1], dt[2], dt[3]};
        *reinterpret_cast<f32x4*>(d + 2 * kStep) = (f32x4){du[0], du[1], du[2], du[3]};
      } else {
#pragma unroll
        for (int j = 0; j < NT; ++j) {
          d[j] = dt[j];
          d[2 * kStep + j] = du[j];
        }
      }
    }
#pragma unroll
    for (int e = 0; e < KB; ++e) {
      const int i = e * 256 + tid, t = kRows ? i / NQ : i % TT, n = (kRows ? i % NQ : i / TT) * 4;
      if (i < TT * NQ) {
        float* dst = sbc + (buf * 2 * NP + n) * LD + t;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          dst[q * LD] = n < n4 ? x.b[e][q] : 0.f;
          dst[(NP + q) * LD] = n < n4 ? x.c[e][q] : 0.f;
        }
      }
    }
  };
  auto finish = [&](int k, const float (&uk)[NT], const float (&zk)[NT]) __attribute__((always_inline)) {      // shares -> read-outs
    const float* part = sy + (k & 1) * kShare + ((og * NT >> 2) * 64 + oc * LPC) * 4 + (og * NT & 3);
    float y[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) y[j] = 0.f;
    constexpr int G = LPC < 8 ? LPC : 8;      // shares requested at once
#pragma unroll
    for (int i0 = 0; i0 < LPC; i0 += G) {
      float v[G][NT];
#pragma unroll
      for (int i = 0; i < G; ++i) {      // (in turn, so that neighbouring channels meet different banks)
        const float* q = part + ((i0 + i + oc) & (LPC - 1)) * 4;
        if constexpr (NT == 4) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(q);
#pragma unroll
          for (int j = 0; j < 4; ++j) v[i][j] = x[j];
        } else {
#pragma unroll
          for (int j = 0; j < NT; ++j) v[i][j] = q[j];
        }
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        float t[G];
#pragma unroll
        for (int i = 0; i < G; ++i) t[i] = v[i][j];
#pragma unroll
        for (int d = G / 2; d > 0; d >>= 1)
#pragma unroll
          for (int i = 0; i < d; ++i) t[i] += t[i + d];
        y[j] += t[0];
      }
    }
#pragma unroll
    for (int j = 0; j < NT; ++j) out[j] = (y[j] + dw * uk[j]) * zk[j] * sigmoid_f(zk[j]) * p.out_scale;
  };
  auto emit = [&](int k) __attribute__((always_inline)) {
    const int left = t_all - k * TT;
    const size_t row = (size_t)(sp.row0 + k * TT) * p.out.ld;
    ChattsOperand o = p.out;
    if (o.f32) o.f32 += row;
    if (o.hi) o.hi += row;
    if (o.lo) o.lo += row;
    if (stage)
#pragma unroll
      for (int j = 0; j < NT; ++j)
        if (left >= TT || og * NT + j < left) store_operand(o, 0, __mul24(og * NT + j, o.ld) + och, out[j]);
  };
  fetch(0, in[0]);
  prepare(0, in[0]);
  fetch(1, in[1]);
  fetch(2, in[0]);
  meet();
  auto tile = [&](int k, Inputs& x) __attribute__((always_inline)) {      // (read-outs are stored a tile late, ahead of the requests that are waited for next)
    prepare(k + 1, x);
    if (k > 1) emit(k - 2);
    fetch(k + 3, x);
    if (k > 0) finish(k - 1, u[2], z[2]);
    meet();
  };
  for (int k = 0; k < tiles; k += 2) {
    tile(k, in[1]);
    tile(k + 1, in[0]);
  }
  emit(tiles - 2);
  finish(tiles - 1, u[1], z[1]);
  emit(tiles - 1);
}

static int check_select(const ChattsSelectArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->proj && a->rows && a->n_rows >= 0 && a->u.f32, CHATTS_E_BADARG, "%s: null pointer", who);
  const int c4 = (a->inner + 3) & ~3;
  CHATTS_REQUIRE(a->inner > 0 && a->state >= 1 && a->state <= 256 && a->taps >= 1, CHATTS_E_SHAPE, "%s: %d channels of %d states (at most 256), %d taps", who, a->inner, a->state,
                 a->taps);
  CHATTS_REQUIRE((a->ld_proj | a->off_x | a->off_z | a->conv_ch | a->u.ld) % 4 == 0 && a->off_x >= 0 && a->off_z >= 0 && a->off_x + c4 <= a->ld_proj &&
                     a->off_z + c4 <= a->ld_proj && a->conv_ch >= c4 && a->u.ld >= c4, CHATTS_E_SHAPE, "%s: column blocks", who);
  CHATTS_REQUIRE((((uintptr_t)a->proj | (uintptr_t)a->u.f32) % 16) == 0, CHATTS_E_SHAPE, "%s: alignment", who);
  return CHATTS_OK;
}
static int check_select_state(const ChattsSelectArgs* a, const char* who) {
  const int n4 = (a->state + 3) & ~3;
  CHATTS_REQUIRE(a->low && a->dt_bias && a->a && a->d && a->s && (a->out.f32 || a->out.hi), CHATTS_E_BADARG, "%s: null pointer", who);
  CHATTS_REQUIRE((a->ld_low | a->off_b | a->off_c | a->off_dt) % 4 == 0 && a->off_b >= 0 && a->off_c >= 0 && a->off_dt >= 0 && a->off_b + n4 <= a->ld_low &&
                     a->off_c + n4 <= a->ld_low && a->rank > 0 && a->rank % 8 == 0 && a->off_dt + a->rank <= a->ld_low && a->out.ld >= ((a->inner + 3) & ~3) &&
                     a->out.ld % 4 == 0, CHATTS_E_SHAPE, "%s: step sizes of rank %d, rows of %d", who, a->rank, a->ld_low);
  CHATTS_REQUIRE((((uintptr_t)a->low | (uintptr_t)a->dt_bias | (uintptr_t)a->a | (uintptr_t)a->d | (uintptr_t)a->s | (uintptr_t)a->w_dt | (uintptr_t)a->delta |
                   (uintptr_t)a->out.f32) % 16) == 0 && (((uintptr_t)a->out.hi | (uintptr_t)a->out.lo) % 8) == 0, CHATTS_E_SHAPE, "%s: alignment", who);
  return CHATTS_OK;
}

template <int SPL, int LPC>
static int launch_select_decode(const ChattsSelectArgs* a, hipStream_t s) {
  const int blocks = (a->inner + 256 / LPC - 1) / (256 / LPC);
  if (a->n_rows < 4) hipLaunchKernelGGL((select_decode_kernel<SPL, LPC, 1>), dim3(blocks, a->n_rows), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL((select_decode_kernel<SPL, LPC, 4>), dim3(blocks, (a->n_rows + 3) / 4), dim3(256), 0, s, *a);
  CHATTS_CHECK_LAUNCH("select_decode");
  return CHATTS_OK;
}
template <int SPL, int LPC, int TT>
static int launch_select_scan(const ChattsSelectArgs* a, hipStream_t s) {
  constexpr size_t lds = select_lds<SPL, LPC, TT>() * sizeof(float);
  static_assert(lds <= 160 * 1024, "LDS");
  static bool done = false;
  if (!done) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&select_scan_kernel<SPL, LPC, TT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "select_scan: cannot reserve LDS: %s", hipGetErrorString(e));
    done = true;
  }
  hipLaunchKernelGGL((select_scan_kernel<SPL, LPC, TT>), dim3((a->inner + 256 / LPC - 1) / (256 / LPC), a->n_spans), dim3(512), lds, s, *a);
  CHATTS_CHECK_LAUNCH("select_scan");
  return CHATTS_OK;
}
static int launch_select_decode_for(const ChattsSelectArgs* a, hipStream_t s) {
  if (a->state <= 8) return launch_select_decode<2, 4>(a, s);
  if (a->state <= 16) return launch_select_decode<2, 8>(a, s);
  if (a->state <= 32) return launch_select_decode<4, 8>(a, s);
  if (a->state <= 64) return launch_select_decode<8, 8>(a, s);
  return a->state <= 128 ? launch_select_decode<8, 16>(a, s) : launch_select_decode<8, 32>(a, s);
}
// tiles of 32 tokens: one workgroup per CU; of 16: two.  More states a lane where the lanes do not run out
static int launch_select_scan_for(const ChattsSelectArgs* a, hipStream_t s) {
  const int64_t wide = (int64_t)((a->inner + 63) / 64) * a->n_spans, groups = (int64_t)((a->inner + 31) / 32) * a->n_spans;
  const bool many = wide >= device_cus(), alone = groups <= device_cus();
  if (a->state <= 8) return many ? launch_select_scan<2, 4, 16>(a, s) : (alone ? launch_select_scan<1, 8, 32>(a, s) : launch_select_scan<1, 8, 16>(a, s));
  if (a->state <= 16) return many ? launch_select_scan<4, 4, 16>(a, s) : (alone ? launch_select_scan<2, 8, 32>(a, s) : launch_select_scan<2, 8, 16>(a, s));
  if (a->state <= 32) return alone ? launch_select_scan<4, 8, 32>(a, s) : launch_select_scan<4, 8, 16>(a, s);
  if (a->state <= 64) return launch_select_scan<8, 8, 16>(a, s);
  return a->state <= 128 ? launch_select_scan<8, 16, 16>(a, s) : launch_select_scan<8, 32, 16>(a, s);
}

template <int TAPS>
static void launch_select_conv(const ChattsSelectArgs* a, hipStream_t s) {
  constexpr int ROWS = 8;
  const int cols = ((a->inner + 3) / 4 + 255) / 256;
  if (a->n_rows <= 64) hipLaunchKernelGGL((select_conv_kernel<TAPS, 1>), dim3(cols, a->n_rows), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL((select_conv_kernel<TAPS, ROWS>), dim3(cols, (a->n_rows + ROWS - 1) / ROWS), dim3(256), 0, s, *a);
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_select_conv(const ChattsSelectArgs* a, chatts_stream_t stream) {
  if (const int rc = check_select(a, "select_conv")) return rc;
  CHATTS_REQUIRE(a->conv_w && a->conv_b && a->ring && (a->n_spans == 0 || a->spans) && (((uintptr_t)a->conv_w | (uintptr_t)a->conv_b | (uintptr_t)a->ring) % 16) == 0 &&
                     (((uintptr_t)a->u.hi | (uintptr_t)a->u.lo) % 8) == 0, CHATTS_E_BADARG, "select_conv: bad arguments");
  if (a->n_rows == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  switch (a->taps) {
    case 1: launch_select_conv<1>(a, s); break;
    case 2: launch_select_conv<2>(a, s); break;
    case 3: launch_select_conv<3>(a, s); break;
    case 4: launch_select_conv<4>(a, s); break;
    default: launch_select_conv<0>(a, s); break;
  }
  if (a->n_spans > 0 && a->taps > 1)
    hipLaunchKernelGGL(select_ring_kernel, dim3(a->taps - 1, a->n_spans, ((a->inner + 3) / 4 + 255) / 256), dim3(256), 0, s, *a);
  CHATTS_CHECK_LAUNCH("select_conv");
  return CHATTS_OK;
}

extern "C" int chatts_select_decode(const ChattsSelectArgs* a, chatts_stream_t stream) {
  if (const int rc = check_select(a, "select_decode")) return rc;
  if (const int rc = check_select_state(a, "select_decode")) return rc;
  CHATTS_REQUIRE(a->w_dt, CHATTS_E_BADARG, "select_decode: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  return launch_select_decode_for(a, as_stream(stream));
}

extern "C" int chatts_select_can_steps(int rank) { return rank > 0 && rank % 64 == 0 && rank <= 384; }

extern "C" int chatts_select_steps(const ChattsSelectArgs* a, chatts_stream_t stream) {
  if (const int rc = check_select(a, "select_steps")) return rc;
  CHATTS_REQUIRE(a->low && a->w_dt_f && a->dt_hi && a->dt_lo && a->dt_bias && a->delta && (a->ld_low | a->off_dt) % 4 == 0 && a->off_dt >= 0 && a->off_dt + a->rank <= a->ld_low && chatts_select_can_steps(a->rank) && a->ld_delta >= ((a->inner + 3) & ~3) && a->ld_delta % 4 == 0,
                 CHATTS_E_SHAPE, "select_steps: step sizes of rank %d (multiples of 64, at most 384)", a->rank);
  CHATTS_REQUIRE((((uintptr_t)a->low | (uintptr_t)a->w_dt_f | (uintptr_t)a->dt_hi | (uintptr_t)a->dt_lo | (uintptr_t)a->dt_bias | (uintptr_t)a->delta) % 16) == 0, CHATTS_E_SHAPE,
                 "select_steps: alignment");
  if (a->n_rows == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  const unsigned rows = (a->n_rows + kStepRows - 1) / kStepRows;
  const dim3 g((a->inner + 127) / 128, rows), b(256);
  hipLaunchKernelGGL(select_split_kernel, dim3((a->n_rows + 15) / 16, (a->rank + 127) / 128), b, 0, s, *a);
  switch (a->rank / 64) {
    case 1: hipLaunchKernelGGL(select_steps_kernel<2>, g, b, 0, s, *a); break;
    case 2: hipLaunchKernelGGL(select_steps_kernel<4>, g, b, 0, s, *a); break;
    case 3: hipLaunchKernelGGL(select_steps_kernel<6>, g, b, 0, s, *a); break;
    case 4: hipLaunchKernelGGL(select_steps_kernel<8>, g, b, 0, s, *a); break;
    case 5: hipLaunchKernelGGL(select_steps_kernel<10>, g, b, 0, s, *a); break;
    default: hipLaunchKernelGGL(select_steps_kernel<12>, g, b, 0, s, *a); break;
  }
  CHATTS_CHECK_LAUNCH("select_steps");
  return CHATTS_OK;
}

extern "C" int chatts_select_scan(const ChattsSelectArgs* a, chatts_stream_t stream) {
  if (const int rc = check_select(a, "select_scan")) return rc;
  if (const int rc = check_select_state(a, "select_scan")) return rc;
  CHATTS_REQUIRE(a->delta && a->ld_delta >= ((a->inner + 3) & ~3) && a->ld_delta % 4 == 0 && a->spans && a->n_spans >= 0, CHATTS_E_BADARG, "select_scan: step sizes");
  if (a->n_rows == 0 || a->n_spans == 0) return CHATTS_OK;
  return launch_select_scan_for(a, as_stream(stream));
}
