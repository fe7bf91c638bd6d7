// depth.hip - the residual stream of layers with norms before their sublayers only: a sublayer's share (its output, the experts' weighted sum) enters x
// with a factor, the streams of all earlier layers are averaged, and the next norm's operand leaves in the same launch, a workgroup per row.
// Also the cap of the logits.
#include "common.h"

namespace chatts {

// a thread keeps its columns in registers.  NT: threads (more of them for a few rows: then every load of a row is in flight at once)
template <int NT, int NV>
__global__ __launch_bounds__(NT) void depth_norm_kernel(ChattsDepthNormArgs p) {
  __shared__ float red[NT / 64];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  constexpr int U = NV <= 2 ? 4 : 2;      // rows requested at once
  f32x4 x[NV], add[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    x[i] = c < p.ldx ? *reinterpret_cast<const f32x4*>(p.x + row * p.ldx + c) : zero;
    add[i] = p.y && c < p.ldx ? *reinterpret_cast<const f32x4*>(p.y + row * p.ldx + c) : zero;
  }
  if (p.ey) {
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
          for (int k = 0; k < 4; ++k) add[i][k] += at[u] >= 0 ? f[u] * y[u][k] : 0.f;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int k = 0; k < 4; ++k) x[i][k] += p.mult * add[i][k];
  if (p.depth) {
    const float own = p.depth[p.n_streams];
    float* st = p.streams + row * p.ldx;
    if (p.keep) {
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * NT + tid) * 4;
        if (c < p.ldx) *reinterpret_cast<f32x4*>(st + p.n_streams * p.stream_stride + c) = x[i];
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k) x[i][k] *= own;
    for (int j0 = 0; j0 < p.n_streams; j0 += U) {
      float f[U];
#pragma unroll
      for (int u = 0; u < U; ++u) f[u] = j0 + u < p.n_streams ? p.depth[j0 + u] : 0.f;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * NT + tid) * 4;
        if (c >= p.ldx) continue;
        f32x4 s[U];
#pragma unroll
        for (int u = 0; u < U; ++u) s[u] = j0 + u < p.n_streams ? *reinterpret_cast<const f32x4*>(st + (j0 + u) * p.stream_stride + c) : zero;
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < 4; ++k) x[i][k] += f[u] * s[u][k];
      }
    }
  }
  if (p.y || p.ey || p.depth) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * NT + tid) * 4;
      if (c < p.ldx) *reinterpret_cast<f32x4*>(p.x + row * p.ldx + c) = x[i];
    }
  }
  if (!p.w) return;
  f32x4 w[NV];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * NT + tid) * 4;
    w[i] = c < p.ldx ? *reinterpret_cast<const f32x4*>(p.w + c) : zero;      // (the weights travel while the row is reduced)
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
    store_operand4(p.out, row, c, v);
  }
}

__global__ __launch_bounds__(256) void soft_cap_kernel(float* __restrict__ x, int64_t quads, int64_t n, float cap, float k) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  auto f = [&](float v) { return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(v * k)); };
  if (i < quads) {
    f32x4 v = *reinterpret_cast<const f32x4*>(x + i * 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = f(v[j]);
    *reinterpret_cast<f32x4*>(x + i * 4) = v;
  } else if (i == quads) {
    for (int64_t j = quads * 4; j < n; ++j) x[j] = f(x[j]);
  }
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_depth_norm(const ChattsDepthNormArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->x && a->t >= 0 && a->width > 0, CHATTS_E_BADARG, "depth_norm: bad arguments");
  CHATTS_REQUIRE(a->ldx >= a->width && a->ldx % 4 == 0 && a->ldx <= 16384, CHATTS_E_SHAPE, "depth_norm: a width of %d in rows of %d (at most 16384)", a->width, a->ldx);
  CHATTS_REQUIRE(!a->ey || (a->place && a->weight && a->top > 0), CHATTS_E_BADARG, "depth_norm: experts");
  CHATTS_REQUIRE(!a->depth || (a->n_streams >= 0 && (a->streams || (a->n_streams == 0 && !a->keep)) && a->stream_stride % 4 == 0), CHATTS_E_BADARG,
                 "depth_norm: an average over %d streams", a->n_streams);
  CHATTS_REQUIRE(!a->w || ((a->out.f32 || a->out.hi) && a->out.ld >= a->ldx && a->out.ld % 4 == 0), CHATTS_E_SHAPE, "depth_norm: operand rows of %d", a->out.ld);
  CHATTS_REQUIRE((((uintptr_t)a->x | (uintptr_t)a->y | (uintptr_t)a->ey | (uintptr_t)a->w | (uintptr_t)a->streams | (uintptr_t)a->out.f32) % 16) == 0 &&
                     (((uintptr_t)a->out.hi | (uintptr_t)a->out.lo) % 8) == 0, CHATTS_E_SHAPE, "depth_norm: pointers must be aligned (16 bytes, planes 8)");
  if (a->t == 0) return CHATTS_OK;
  const dim3 g(a->t);
  hipStream_t s = as_stream(stream);
  if (a->ldx <= 1024) hipLaunchKernelGGL((depth_norm_kernel<256, 1>), g, dim3(256), 0, s, *a);
  else if (a->t <= 64 && a->ldx <= 4096) hipLaunchKernelGGL((depth_norm_kernel<1024, 1>), g, dim3(1024), 0, s, *a);
  else if (a->t <= 64 && a->ldx <= 8192) hipLaunchKernelGGL((depth_norm_kernel<1024, 2>), g, dim3(1024), 0, s, *a);
  else if (a->ldx <= 2048) hipLaunchKernelGGL((depth_norm_kernel<256, 2>), g, dim3(256), 0, s, *a);
  else if (a->ldx <= 4096) hipLaunchKernelGGL((depth_norm_kernel<256, 4>), g, dim3(256), 0, s, *a);
  else if (a->ldx <= 8192) hipLaunchKernelGGL((depth_norm_kernel<256, 8>), g, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL((depth_norm_kernel<1024, 4>), g, dim3(1024), 0, s, *a);
  CHATTS_CHECK_LAUNCH("depth_norm");
  return CHATTS_OK;
}

extern "C" int chatts_soft_cap(float* x, int64_t n, float cap, chatts_stream_t stream) {
  CHATTS_REQUIRE(x && n >= 0 && cap > 0.f && ((uintptr_t)x % 16) == 0, CHATTS_E_BADARG, "soft_cap: %lld values, cap %g", (long long)n, (double)cap);
  if (n == 0) return CHATTS_OK;
  const int64_t quads = n / 4;
  hipLaunchKernelGGL(soft_cap_kernel, dim3((unsigned)((quads + 1 + 255) / 256)), dim3(256), 0, as_stream(stream), x, quads, n, cap, 2.0f * 1.44269504088896341f / cap);
  CHATTS_CHECK_LAUNCH("soft_cap");
  return CHATTS_OK;
}
