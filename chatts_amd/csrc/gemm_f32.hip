// gemm_f32.hip - projections in true 32-bit: C[M,N] = epilogue(A[M,K] . W[N,K]^T) with float32 A, the bf16 weights widened (exactly) and
// v_mfma_f32_16x16x4_f32, i.e. float32 products and float32 sums.  ChattsLinearArgs.exact_f32 and the 32-bit form of chatts_head_linear:
// the runs that check a model in 32-bit, not a serving path.  grid (N / 64, M / 64, batch), 4 waves of 32 x 32 outputs.
#include "gemm_common.h"

namespace chatts {

struct GemmF32Params {
  const float* a;
  const uint16_t* w;
  const float* bias;
  const float* resid;
  float* c;
  int m, n, k, lda, ldw, ldc, epilogue;
  float glu_limit, glu_alpha;
  int64_t a_batch, w_batch, c_batch;
};

constexpr int kF32Ld = 36;      // LDS row of 32 K-values, padded: 16-byte aligned, rows 4 banks apart

__global__ __launch_bounds__(256) void gemm_f32_kernel(GemmF32Params p) {
  __shared__ __attribute__((aligned(16))) float sa[64 * kF32Ld], sw[64 * kF32Ld];
  const int n0 = blockIdx.x * 64, m0 = blockIdx.y * 64, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const float* a = p.a + (int64_t)blockIdx.z * p.a_batch;
  const uint16_t* w = p.w + (int64_t)blockIdx.z * p.w_batch;
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
  f32x4 acc[2][2] = {};
  const int r = tid >> 2, kc = (tid & 3) * 8;      // staging: 8 consecutive K-values of one row per thread
  const int ar = m0 + r < p.m ? m0 + r : p.m - 1, wr = n0 + r < p.n ? n0 + r : p.n - 1;
  for (int k0 = 0; k0 < p.k; k0 += 32) {
    const f32x4 a0 = *reinterpret_cast<const f32x4*>(a + (size_t)ar * p.lda + k0 + kc);
    const f32x4 a1 = *reinterpret_cast<const f32x4*>(a + (size_t)ar * p.lda + k0 + kc + 4);
    const u32x4 wv = *reinterpret_cast<const u32x4*>(w + (size_t)wr * p.ldw + k0 + kc);
    __syncthreads();
    *reinterpret_cast<f32x4*>(sa + r * kF32Ld + kc) = a0;
    *reinterpret_cast<f32x4*>(sa + r * kF32Ld + kc + 4) = a1;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sw[r * kF32Ld + kc + 2 * j] = bf16_lo(wv[j]);
      sw[r * kF32Ld + kc + 2 * j + 1] = bf16_hi(wv[j]);
    }
    __syncthreads();
    const int fr = lane & 15, fk = lane >> 4;
#pragma unroll
    for (int kk = 0; kk < 32; kk += 4) {
      float av[2], bv[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        av[i] = sa[(wm + i * 16 + fr) * kF32Ld + kk + fk];
        bv[i] = sw[(wn + i * 16 + fr) * kF32Ld + kk + fk];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i], bv[j], acc[i][j], 0, 0, 0);
    }
  }
  float* c = p.c + (int64_t)blockIdx.z * p.c_batch;
  if (epi_is_glu(p.epilogue)) {      // the two 16-column halves of a wave: gate and up of the same outputs
    const int col = n0 + wn + (lane & 15);
    if (col + 16 >= p.n) return;
    const float bg = p.bias ? p.bias[col] : 0.f, bu = p.bias ? p.bias[col + 16] : 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int row = m0 + wm + i * 16 + (lane >> 4) * 4 + q;
        if (row < p.m) c[(size_t)row * p.ldc + ((n0 + wn) >> 1) + (lane & 15)] = glu_value(p.epilogue, acc[i][0][q] + bg, acc[i][1][q] + bu, p.glu_limit, p.glu_alpha);
      }
    return;
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int col = n0 + wn + j * 16 + (lane & 15);
      if (col >= p.n) continue;
      const float b = p.bias ? p.bias[col] : 0.f;
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int row = m0 + wm + i * 16 + (lane >> 4) * 4 + q;
        if (row >= p.m) continue;
        float v = acc[i][j][q] + b;
        if (p.epilogue == CHATTS_EPI_GELU) v = gelu_erf_f(v);
        if (p.epilogue == CHATTS_EPI_RELU2) v = relu2_f(v);
        if (p.epilogue == CHATTS_EPI_RESID) v = p.resid[(size_t)row * p.ldc + col] + v;
        c[(size_t)row * p.ldc + col] = v;
      }
    }
}

int launch_gemm_f32_batched(const float* a, int64_t a_batch, int lda, const uint16_t* w, int64_t w_batch, int ldw, float* c, int64_t c_batch, int ldc,
                            int m, int n, int k, int batch, hipStream_t s) {
  GemmF32Params p{a, w, nullptr, nullptr, c, m, n, k, lda, ldw, ldc, CHATTS_EPI_NONE, 0.f, 0.f, a_batch, w_batch, c_batch};
  hipLaunchKernelGGL(gemm_f32_kernel, dim3((n + 63) / 64, (m + 63) / 64, batch), dim3(256), 0, s, p);
  CHATTS_CHECK_LAUNCH("gemm_f32");
  return CHATTS_OK;
}

int launch_gemm_f32(const ChattsLinearArgs* a, hipStream_t s) {
  GemmF32Params p{a->a, a->w, a->bias, a->resid, a->c, a->m, a->n, a->k, a->lda, a->ldw, a->ldc, a->epilogue, a->glu_limit, a->glu_alpha, 0, 0, 0};
  hipLaunchKernelGGL(gemm_f32_kernel, dim3((a->n + 63) / 64, (a->m + 63) / 64, 1), dim3(256), 0, s, p);
  CHATTS_CHECK_LAUNCH("gemm_f32");
  return CHATTS_OK;
}

}  // namespace chatts
