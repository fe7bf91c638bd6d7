// select.hip - selective scan: per channel c and state n  S <- exp(d_c A[c, n]) S + d_c u_c B_n,  y_c = sum_n S C_n + D_c u_c  with step sizes d, inputs u and
// the vectors B, C of every token; the read-out y silu(z) leaves as the next projection's operand.  Float32.
//   select_conv_kernel    u = silu(short convolution), with the inputs before a segment from a ring per slot
//   select_ring_kernel    the last convolution inputs of every segment
//   select_decode_kernel  one token per sequence: the step sizes' projection, the state's update and the read-out in one launch
//   select_scan_kernel    segments of several tokens: a channel's states lie in LPC neighbouring lanes, SPL in each; tokens in tiles through LDS
#include "common.h"

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
    else *reinterpret_cast<float2*>(dst + l * SPL + i) = make_float2(s[i], s[i + 1]);
  }
}

// grid (channels / (256 / LPC), rows)
template <int SPL, int LPC>
__global__ __launch_bounds__(256) void select_decode_kernel(ChattsSelectArgs p) {
  constexpr int CH = 256 / LPC;
  const int row = blockIdx.y, l = threadIdx.x & (LPC - 1), c = blockIdx.x * CH + threadIdx.x / LPC, n4 = (p.state + 3) & ~3;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const bool live = c < p.inner;
  const int cc = live ? c : 0;
  const float* low = p.low + (size_t)row * p.ld_low;
  const float u = p.u.f32[(size_t)row * p.u.ld + cc], z = p.proj[(size_t)row * p.ld_proj + p.off_z + cc], bias = p.dt_bias[cc], d = p.d[cc];
  float a[SPL], B[SPL], Cn[SPL], s[SPL];
  states_load<SPL>(p.a + (size_t)cc * n4, l, n4, a);
  states_load<SPL>(low + p.off_b, l, n4, B);
  states_load<SPL>(low + p.off_c, l, n4, Cn);
  float* S = p.s + ((size_t)R.slot * p.inner + cc) * n4;
  states_load<SPL>(S, l, n4, s);
  // the step size: the channel's lanes share its row of W_dt
  float acc = 0.f;
  const uint16_t* w = p.w_dt + (size_t)cc * p.rank;
  for (int i = l * 8; i < p.rank; i += LPC * 8) {
    const u32x4 wv = *reinterpret_cast<const u32x4*>(w + i);
    const f32x4 x0 = *reinterpret_cast<const f32x4*>(low + p.off_dt + i), x1 = *reinterpret_cast<const f32x4*>(low + p.off_dt + i + 4);
    acc += (bf16_lo(wv[0]) * x0[0] + bf16_hi(wv[0]) * x0[1]) + (bf16_lo(wv[1]) * x0[2] + bf16_hi(wv[1]) * x0[3]);
    acc += (bf16_lo(wv[2]) * x1[0] + bf16_hi(wv[2]) * x1[1]) + (bf16_lo(wv[3]) * x1[2] + bf16_hi(wv[3]) * x1[3]);
  }
  const float dt = softplus_f(lanes_sum<LPC>(acc) + bias), du = dt * u;
  float y = 0.f;
#pragma unroll
  for (int i = 0; i < SPL; ++i) {
    s[i] = __builtin_amdgcn_exp2f(dt * a[i]) * (R.pos > 0 ? s[i] : 0.f) + du * B[i];
    y += s[i] * Cn[i];
  }
  y = lanes_sum<LPC>(y);
  if (!live) return;
  states_store<SPL>(S, l, n4, s);
  if (l == 0) store_operand(p.out, row, c, (y + d * u) * z * sigmoid_f(z) * p.out_scale);
}

// grid (channels / (256 / LPC), spans)
template <int SPL, int LPC>
__global__ __launch_bounds__(256) void select_scan_kernel(ChattsSelectArgs p) {
  constexpr int CH = 256 / LPC, TT = 4 * LPC < 32 ? 4 * LPC : 32, NP = SPL * LPC, CQ = CH / 4, KB = TT * NP / 4 > 256 ? TT * NP / 1024 : 1;
  __shared__ __attribute__((aligned(16))) float sdt[TT][CH], sdu[TT][CH], sy[TT][CH], sb[TT][NP], sc[TT][NP];
  const ChattsSpan sp = p.spans[blockIdx.y];
  if (sp.t < 1) return;
  const int tid = threadIdx.x, l = tid & (LPC - 1), ch = tid / LPC, c0 = blockIdx.x * CH, c = c0 + ch, n4 = (p.state + 3) & ~3;
  const bool live = c < p.inner;
  const int cc = live ? c : 0;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  float a[SPL], s[SPL];
  float* S = p.s + ((size_t)sp.slot * p.inner + cc) * n4;
  states_load<SPL>(p.a + (size_t)cc * n4, l, n4, a);
#pragma unroll
  for (int i = 0; i < SPL; ++i) s[i] = 0.f;
  if (sp.pos0 > 0 && live) states_load<SPL>(S, l, n4, s);
  // staging: thread = (token, four channels)
  const int lt = tid / CQ, lc = c0 + (tid - lt * CQ) * 4;
  const bool stage = tid < TT * CQ && lc < ((p.inner + 3) & ~3);
  f32x4 bias = zero, dw = zero;
  if (stage) {
    bias = *reinterpret_cast<const f32x4*>(p.dt_bias + lc);
    dw = *reinterpret_cast<const f32x4*>(p.d + lc);
  }
  f32x4 dl = zero, un = zero, zn = zero, rb[KB], rc[KB];
  auto fetch = [&](int t0) __attribute__((always_inline)) {
    if (stage) {
      const size_t row = sp.row0 + (t0 + lt < sp.t ? t0 + lt : sp.t - 1);
      dl = *reinterpret_cast<const f32x4*>(p.delta + row * p.ld_delta + lc);
      un = *reinterpret_cast<const f32x4*>(p.u.f32 + row * p.u.ld + lc);
      zn = *reinterpret_cast<const f32x4*>(p.proj + row * p.ld_proj + p.off_z + lc);
    }
#pragma unroll
    for (int e = 0; e < KB; ++e) {
      const int i = e * 256 + tid, t = i / (NP / 4), n = (i - t * (NP / 4)) * 4;
      rb[e] = rc[e] = zero;
      if (i < TT * NP / 4 && n < n4) {
        const float* low = p.low + (size_t)(sp.row0 + (t0 + t < sp.t ? t0 + t : sp.t - 1)) * p.ld_low;
        rb[e] = *reinterpret_cast<const f32x4*>(low + p.off_b + n);
        rc[e] = *reinterpret_cast<const f32x4*>(low + p.off_c + n);
      }
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < sp.t; t0 += TT) {
    const f32x4 u = un, z = zn;
    if (tid < TT * CQ) {
      f32x4 dt, du;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        dt[k] = stage && t0 + lt < sp.t ? softplus_f(dl[k] + bias[k]) : 0.f;      // (beyond the end: the state stays)
        du[k] = dt[k] * u[k];
      }
      *reinterpret_cast<f32x4*>(&sdt[lt][lc - c0]) = dt;
      *reinterpret_cast<f32x4*>(&sdu[lt][lc - c0]) = du;
    }
#pragma unroll
    for (int e = 0; e < KB; ++e) {
      const int i = e * 256 + tid, t = i / (NP / 4), n = (i - t * (NP / 4)) * 4;
      if (i < TT * NP / 4) {
        *reinterpret_cast<f32x4*>(&sb[t][n]) = rb[e];
        *reinterpret_cast<f32x4*>(&sc[t][n]) = rc[e];
      }
    }
    __syncthreads();
    if (t0 + TT < sp.t) fetch(t0 + TT);
    for (int tb = 0; tb < TT; tb += LPC) {
      float mine = 0.f;
#pragma unroll LPC < 16 ? LPC : 16
      for (int j = 0; j < LPC; ++j) {
        const float dt = sdt[tb + j][ch], du = sdu[tb + j][ch];
        float B[SPL], Cn[SPL], y = 0.f;
        states_load<SPL>(sb[tb + j], l, NP, B);
        states_load<SPL>(sc[tb + j], l, NP, Cn);
#pragma unroll
        for (int i = 0; i < SPL; ++i) {
          s[i] = __builtin_amdgcn_exp2f(dt * a[i]) * s[i] + du * B[i];
          y += s[i] * Cn[i];
        }
        y = lanes_sum<LPC>(y);
        mine = l == j ? y : mine;
      }
      sy[tb + l][ch] = mine;
    }
    __syncthreads();
    if (stage && t0 + lt < sp.t) {
      const f32x4 y = *reinterpret_cast<const f32x4*>(&sy[lt][lc - c0]);
      float v[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) v[k] = (y[k] + dw[k] * u[k]) * z[k] * sigmoid_f(z[k]) * p.out_scale;
      store_operand4(p.out, sp.row0 + t0 + lt, lc, v);
    }
  }
  if (live) states_store<SPL>(S, l, n4, s);
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
static void launch_select(const ChattsSelectArgs* a, bool decode, hipStream_t s) {
  const int blocks = (a->inner + 256 / LPC - 1) / (256 / LPC);
  if (decode) hipLaunchKernelGGL((select_decode_kernel<SPL, LPC>), dim3(blocks, a->n_rows), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL((select_scan_kernel<SPL, LPC>), dim3(blocks, a->n_spans), dim3(256), 0, s, *a);
}
static void launch_select_for(const ChattsSelectArgs* a, bool decode, hipStream_t s) {
  if (a->state <= 8) launch_select<2, 4>(a, decode, s);
  else if (a->state <= 16) launch_select<2, 8>(a, decode, s);
  else if (a->state <= 32) launch_select<2, 16>(a, decode, s);
  else if (a->state <= 64) launch_select<4, 16>(a, decode, s);
  else if (a->state <= 128) launch_select<4, 32>(a, decode, s);
  else launch_select<8, 32>(a, decode, s);
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
  launch_select_for(a, true, as_stream(stream));
  CHATTS_CHECK_LAUNCH("select_decode");
  return CHATTS_OK;
}

extern "C" int chatts_select_scan(const ChattsSelectArgs* a, chatts_stream_t stream) {
  if (const int rc = check_select(a, "select_scan")) return rc;
  if (const int rc = check_select_state(a, "select_scan")) return rc;
  CHATTS_REQUIRE(a->delta && a->ld_delta >= ((a->inner + 3) & ~3) && a->ld_delta % 4 == 0 && a->spans && a->n_spans >= 0, CHATTS_E_BADARG, "select_scan: step sizes");
  if (a->n_rows == 0 || a->n_spans == 0) return CHATTS_OK;
  launch_select_for(a, false, as_stream(stream));
  CHATTS_CHECK_LAUNCH("select_scan");
  return CHATTS_OK;
}
