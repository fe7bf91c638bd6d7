// postnorm.hip - the residual stream of layers whose norm stands after the sum: x <- norm(alpha x + sublayer), a workgroup per row; the experts' weighted
// sum and the next projection's operand in the same launch.
#include "common.h"

namespace chatts {

// a thread keeps its columns in registers.  NT: threads (more of them for a few rows: then every load of a row is in flight at once)
template <int NT, int NV>
__global__ __launch_bounds__(NT) void post_norm_kernel(ChattsPostNormArgs p) {
  __shared__ float red[NT / 64];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 x[NV], w[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    x[i] = w[i] = zero;
    if (c >= p.ldx) continue;
    x[i] = *reinterpret_cast<const f32x4*>(p.x + row * p.ldx + c);
    w[i] = *reinterpret_cast<const f32x4*>(p.w + c);      // (the weights travel while the row is reduced)
    const f32x4 y = p.y ? *reinterpret_cast<const f32x4*>(p.y + row * p.ldx + c) : zero;
#pragma unroll
    for (int k = 0; k < 4; ++k) x[i][k] = p.alpha * x[i][k] + y[k];
  }
  if (p.ey) {
    constexpr int U = 4;      // experts' rows requested at once
    for (int j0 = 0; j0 < p.top; j0 += U) {
      int at[U];
      float f[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int j = j0 + u < p.top ? j0 + u : j0;
        at[u] = j0 + u < p.top ? p.place[row * p.top + j] : -1;      // (uniform)
        f[u] = p.weight[row * p.top + j];
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * NT + tid) * 4;
        if (c >= p.ldx) continue;
        f32x4 y[U];
#pragma unroll
        for (int u = 0; u < U; ++u) y[u] = at[u] >= 0 ? *reinterpret_cast<const f32x4*>(p.ey + (size_t)at[u] * p.ldx + c) : zero;
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < 4; ++k) x[i][k] += at[u] >= 0 ? f[u] * y[u][k] : 0.f;
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (c + k < p.width) ss += x[i][k] * x[i][k];
  }
  ss = block_sum<NT / 64>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)p.width + p.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    if (c >= p.ldx) continue;
    float v[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = c + k < p.width ? x[i][k] * inv * w[i][k] : 0.f;
    *reinterpret_cast<f32x4*>(p.x + row * p.ldx + c) = (f32x4){v[0], v[1], v[2], v[3]};
    store_operand4(p.out, row, c, v);
  }
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_post_norm(const ChattsPostNormArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->x && a->w && a->t >= 0 && a->width > 0, CHATTS_E_BADARG, "post_norm: bad arguments");
  CHATTS_REQUIRE(a->ldx >= a->width && a->ldx % 4 == 0 && a->ldx <= 16384, CHATTS_E_SHAPE, "post_norm: a width of %d in rows of %d (at most 16384)", a->width, a->ldx);
  CHATTS_REQUIRE(!a->ey || (a->place && a->weight && a->top > 0), CHATTS_E_BADARG, "post_norm: experts");
  CHATTS_REQUIRE((!a->out.f32 && !a->out.hi) || (a->out.ld >= a->ldx && a->out.ld % 4 == 0), CHATTS_E_SHAPE, "post_norm: operand rows of %d", a->out.ld);
  CHATTS_REQUIRE((((uintptr_t)a->x | (uintptr_t)a->y | (uintptr_t)a->ey | (uintptr_t)a->w | (uintptr_t)a->out.f32) % 16) == 0 &&
                     (((uintptr_t)a->out.hi | (uintptr_t)a->out.lo) % 8) == 0, CHATTS_E_SHAPE, "post_norm: pointers must be aligned (16 bytes, planes 8)");
  if (a->t == 0) return CHATTS_OK;
  const dim3 g(a->t);
  hipStream_t s = as_stream(stream);
  if (a->ldx <= 1024) hipLaunchKernelGGL((post_norm_kernel<256, 1>), g, dim3(256), 0, s, *a);
  else if (a->t <= 64 && a->ldx <= 4096) hipLaunchKernelGGL((post_norm_kernel<1024, 1>), g, dim3(1024), 0, s, *a);
  else if (a->t <= 64 && a->ldx <= 8192) hipLaunchKernelGGL((post_norm_kernel<1024, 2>), g, dim3(1024), 0, s, *a);
  else if (a->ldx <= 2048) hipLaunchKernelGGL((post_norm_kernel<256, 2>), g, dim3(256), 0, s, *a);
  else if (a->ldx <= 4096) hipLaunchKernelGGL((post_norm_kernel<256, 4>), g, dim3(256), 0, s, *a);
  else if (a->ldx <= 8192) hipLaunchKernelGGL((post_norm_kernel<256, 8>), g, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL((post_norm_kernel<1024, 4>), g, dim3(1024), 0, s, *a);
  CHATTS_CHECK_LAUNCH("post_norm");
  return CHATTS_OK;
}
