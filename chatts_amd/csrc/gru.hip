// gru.hip - a gated recurrence whose gates read the current token alone (minGRU): S <- (1 - s) S + s c per channel, s = sigmoid(z), c = x + 1/2 for x >= 0
// and sigmoid(x) below; the read-out S silu(g) leaves as the next projection's operand.  Float32.
//   gru_decode_kernel  one token per sequence, elementwise
//   gru_scan_kernel    segments of several tokens: every step is an affine map S -> a S + b and maps compose, so a workgroup owns 16 channels and walks the
//                      tokens in tiles: a thread composes its four tokens, a wave and then the workgroup put the threads' maps together, and every thread
//                      runs its tokens again from the state it then knows.  Every input is read once.
#include "common.h"

namespace chatts {

__device__ __forceinline__ float gru_candidate(float x) { return x >= 0.f ? x + 0.5f : sigmoid_f(x); }
__device__ __forceinline__ float silu4(float g) { return g * sigmoid_f(g); }

// grid (width / 1024, rows): a thread owns four channels
__global__ __launch_bounds__(256) void gru_decode_kernel(ChattsGruArgs p) {
  const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
  const ChattsRow R = p.rows[row];
  const int w4 = (p.width + 3) & ~3;
  if (R.pos < 0 || c >= w4) return;
  const float* pr = p.proj + (size_t)row * p.ld_proj + c;
  const f32x4 z = *reinterpret_cast<const f32x4*>(pr + p.off_z), x = *reinterpret_cast<const f32x4*>(pr + p.off_x), g = *reinterpret_cast<const f32x4*>(pr + p.off_g);
  float* st = p.state + (size_t)R.slot * w4 + c;
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  if (R.pos > 0) S = *reinterpret_cast<const f32x4*>(st);
  float v[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    S[k] = sigmoid_f(-z[k]) * S[k] + sigmoid_f(z[k]) * gru_candidate(x[k]);
    v[k] = S[k] * silu4(g[k]) * p.out_scale;
  }
  *reinterpret_cast<f32x4*>(st) = S;
  store_operand4(p.out, row, c, v);
}

// grid (blocks of 16 channels, spans): lane = (4 channels lane & 3, tokens 4 (16 wave + lane >> 2) ..) of a tile of NT tokens
template <int NT>
__global__ __launch_bounds__(NT) void gru_scan_kernel(ChattsGruArgs p) {
  constexpr int NW = NT / 64;
  __shared__ f32x4 wa[2][NW][4], wb[2][NW][4];
  const ChattsSpan sp = p.spans[blockIdx.y];
  if (sp.t < 1) return;
  // neighbouring blocks share cache lines of a row: XCD x (= blockIdx % 8; speed only) takes a contiguous eighth of them
  const int share = gridDim.x >> 3, rem = gridDim.x & 7, xcd = blockIdx.x & 7, block = xcd * share + (xcd < rem ? xcd : rem) + (blockIdx.x >> 3);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, q = lane & 3, seg = lane >> 2, w4 = (p.width + 3) & ~3, c = block * 16 + q * 4;
  const bool live = c < w4;
  const int cc = live ? c : 0;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f}, one = {1.f, 1.f, 1.f, 1.f};
  float* st = p.state + (size_t)sp.slot * w4 + cc;
  f32x4 S = zero;      // the state before the tile
  if (sp.pos0 > 0) S = *reinterpret_cast<const f32x4*>(st);
  __syncthreads();      // (every wave has read it before the last one writes it)
  int buf = 0;
  for (int t0 = 0; t0 < sp.t; t0 += NT, buf ^= 1) {
    const int t = t0 + (wave * 16 + seg) * 4;
    f32x4 z[4], x[4], g[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = t + j < sp.t ? t + j : sp.t - 1;
      const float* pr = p.proj + (size_t)(sp.row0 + r) * p.ld_proj + cc;
      z[j] = *reinterpret_cast<const f32x4*>(pr + p.off_z);
      x[j] = *reinterpret_cast<const f32x4*>(pr + p.off_x);
      g[j] = *reinterpret_cast<const f32x4*>(pr + p.off_g);
    }
    f32x4 A = one, B = zero;      // this thread's tokens as one map
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const bool ok = t + j < sp.t;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float a = ok ? sigmoid_f(-z[j][k]) : 1.f, b = ok ? sigmoid_f(z[j][k]) * gru_candidate(x[j][k]) : 0.f;
        z[j][k] = a;
        x[j][k] = b;
        A[k] *= a;
        B[k] = a * B[k] + b;
      }
    }
#pragma unroll
    for (int d = 1; d < 16; d <<= 1)      // earlier lanes' maps first
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float a = __shfl_up(A[k], 4 * d, 64), b = __shfl_up(B[k], 4 * d, 64);
        if (seg >= d) {
          B[k] = A[k] * b + B[k];
          A[k] *= a;
        }
      }
    if (seg == 15) { wa[buf][wave][q] = A; wb[buf][wave][q] = B; }
    __syncthreads();
    f32x4 end = S;      // the state after each wave in turn
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      if (w == wave) S = end;
      const f32x4 a = wa[buf][w][q], b = wb[buf][w][q];
#pragma unroll
      for (int k = 0; k < 4; ++k) end[k] = a[k] * end[k] + b[k];
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float a = __shfl_up(A[k], 4, 64), b = __shfl_up(B[k], 4, 64);
      if (seg > 0) S[k] = a * S[k] + b;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float v[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        S[k] = z[j][k] * S[k] + x[j][k];
        v[k] = S[k] * silu4(g[j][k]) * p.out_scale;
      }
      if (live && t + j < sp.t) store_operand4(p.out, sp.row0 + t + j, c, v);
    }
    S = end;
  }
  if (tid < 4 && live) *reinterpret_cast<f32x4*>(st) = S;
}

static int check_gru(const ChattsGruArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->proj && a->state && a->rows && a->width > 0 && a->n_rows >= 0, CHATTS_E_BADARG, "%s: null pointer", who);
  const int w4 = (a->width + 3) & ~3;
  CHATTS_REQUIRE((a->ld_proj | a->off_z | a->off_x | a->off_g) % 4 == 0 && a->off_z >= 0 && a->off_x >= 0 && a->off_g >= 0 && a->off_z + w4 <= a->ld_proj &&
                     a->off_x + w4 <= a->ld_proj && a->off_g + w4 <= a->ld_proj, CHATTS_E_SHAPE, "%s: column blocks", who);
  CHATTS_REQUIRE((a->out.f32 || a->out.hi) && a->out.ld >= w4 && a->out.ld % 4 == 0, CHATTS_E_SHAPE, "%s: operand rows of %d", who, a->out.ld);
  CHATTS_REQUIRE((((uintptr_t)a->proj | (uintptr_t)a->state | (uintptr_t)a->out.f32) % 16) == 0 && (((uintptr_t)a->out.hi | (uintptr_t)a->out.lo) % 8) == 0,
                 CHATTS_E_SHAPE, "%s: pointers must be aligned", who);
  return CHATTS_OK;
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_gru_decode(const ChattsGruArgs* a, chatts_stream_t stream) {
  if (const int rc = check_gru(a, "gru_decode")) return rc;
  if (a->n_rows == 0) return CHATTS_OK;
  hipLaunchKernelGGL(gru_decode_kernel, dim3((a->width + 1023) / 1024, a->n_rows), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("gru_decode");
  return CHATTS_OK;
}

extern "C" int chatts_gru_scan(const ChattsGruArgs* a, chatts_stream_t stream) {
  if (const int rc = check_gru(a, "gru_scan")) return rc;
  CHATTS_REQUIRE(a->spans && a->n_spans >= 0, CHATTS_E_BADARG, "gru_scan: no spans");
  if (a->n_rows == 0 || a->n_spans == 0) return CHATTS_OK;
  const dim3 g((a->width + 15) / 16, a->n_spans);
  if (a->n_rows <= 256) hipLaunchKernelGGL(gru_scan_kernel<256>, g, dim3(256), 0, as_stream(stream), *a);
  else hipLaunchKernelGGL(gru_scan_kernel<1024>, g, dim3(1024), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("gru_scan");
  return CHATTS_OK;
}
