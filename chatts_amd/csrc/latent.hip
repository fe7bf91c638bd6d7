// latent.hip - latent attention: keys and values of all heads are linear maps of one cached latent per token, beside one rotated key part
// that the heads share.  The cache holds only [latent | rotated part] per token, in pages.
//   score_h(i, j) = (q_un_h(i) . W_uk_h c_j + q_rot_h(i) . k_rot_j) * scale = ([W_uk_h^T q_un_h | q_rot_h](i) . [c | k_rot](j)) * scale
//   out_h(i) = W_uv_h sum_j softmax(score)_ij c_j
// The absorbed form (second half of each line) is multi-query attention over the cached rows: one row feeds every head, so decoding reads
// the cache once per head tile.
//   * latent_prep_kernel: rotation of the query parts, norm of the latent, rotation of the key part, cache write
//   * head_linear_kernel: W_uk^T on the queries, W_uv on the weighted latents (a product per head)
//   * latent_attend_kernel: one (row, head) per workgroup on the vector units, float32 or bf16 cache: the 32-bit runs and odd sizes
//   * latent_decode_kernel: 16 heads of a row per workgroup on the matrix pipe over every n_splits-th key tile, bf16 cache, partials merged by
//     latent_merge_kernel
#include "gemm_common.h"

namespace chatts {

int launch_gemm_f32_batched(const float* a, int64_t a_batch, int lda, const uint16_t* w, int64_t w_batch, int ldw, float* c, int64_t c_batch, int ldc,
                            int m, int n, int k, int batch, hipStream_t s);

template <typename T> __device__ __forceinline__ T to_cache(float v);
template <> __device__ __forceinline__ float to_cache<float>(float v) { return v; }
template <> __device__ __forceinline__ uint16_t to_cache<uint16_t>(float v) { return __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ f32x4 load_cache4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load_cache4(const uint16_t* p) {
  const u32x2 v = *reinterpret_cast<const u32x2*>(p);
  return (f32x4){bf16_lo(v.x), bf16_hi(v.x), bf16_lo(v.y), bf16_hi(v.y)};
}

// element offset of the cache row of position `pos` of slot `slot`
__device__ __forceinline__ size_t latent_row(const ChattsLatentArgs& p, int slot, int pos, int cw) {
  const int blk = p.table[(size_t)slot * p.table_stride + (pos >> p.log_block)];
  return (((size_t)blk << p.log_block) + (pos & ((1 << p.log_block) - 1))) * cw;
}

// ---- rotation, norm, cache write: one workgroup per row ----
template <typename CT>
__global__ __launch_bounds__(256) void latent_prep_kernel(ChattsLatentArgs p) {
  __shared__ float red[4];
  const int row = blockIdx.x, tid = threadIdx.x, cw = p.rank_p + p.rot_p;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  float* pr = p.proj + (size_t)row * p.ld_proj;
  const int half = p.rot >> 1;
  const float* ct = p.cos_tab + (size_t)R.pos * half;
  const float* st = p.sin_tab + (size_t)R.pos * half;
  for (int e = tid; e < p.heads * p.rot_p; e += 256) {      // the rotated part of every head's absorbed query, padding included
    const int h = e / p.rot_p, i = e - h * p.rot_p;
    float v = 0.f;
    if (i < p.rot) {
      const float* q = pr + p.off_qr + h * p.rot;
      const int f = i < half ? i : i - half;
      const float u = q[f], w = q[f + half];
      v = i < half ? u * ct[f] - w * st[f] : w * ct[f] + u * st[f];
    }
    store_operand(p.q, row, h * cw + p.rank_p + i, v);
  }
  float ss = 0.f;
  for (int i = tid; i < p.rank; i += 256) { const float v = pr[p.off_c + i]; ss += v * v; }
  ss = block_sum<4>(ss, red);
  const float f = 1.0f / sqrtf(ss / (float)p.rank + p.eps);
  CT* dst = reinterpret_cast<CT*>(p.cache) + latent_row(p, R.slot, R.pos, cw);
  for (int i = tid; i < cw; i += 256) {
    float v = 0.f;
    if (i < p.rank) v = pr[p.off_c + i] * f * p.c_norm[i];
    else if (i >= p.rank_p && i - p.rank_p < p.rot) {
      const float* k = pr + p.off_kr;
      const int j = i - p.rank_p, g = j < half ? j : j - half;
      const float u = k[g], w = k[g + half];
      v = j < half ? u * ct[g] - w * st[g] : w * ct[g] + u * st[g];
    }
    dst[i] = to_cache<CT>(v);
  }
}

// ---- absorbed attention on the vector units: grid (heads, rows) ----
template <typename CT>
__global__ __launch_bounds__(256) void latent_attend_kernel(ChattsLatentArgs p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, cw = p.rank_p + p.rot_p;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  float* sq = sm;              // [cw]
  float* sc = sq + cw;         // [64] scores, then weights
  for (int i = tid; i < cw; i += 256) {
    const size_t at = (size_t)row * p.q.ld + h * cw + i;
    sq[i] = p.q.f32 ? p.q.f32[at] : bf16_to_f32(p.q.hi[at]) + (p.q.lo ? bf16_to_f32(p.q.lo[at]) : 0.f);
  }
  const CT* cache = reinterpret_cast<const CT*>(p.cache);
  float m = -INFINITY, l = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};      // columns tid + 256 j
  const int n = R.pos + 1;
  for (int k0 = 0; k0 < n; k0 += 64) {      // (a page holds a multiple of 64 rows: a tile is contiguous)
    __syncthreads();
    const CT* tile = cache + latent_row(p, R.slot, k0, cw);
    const int key = tid >> 2, part = tid & 3;
    float d = 0.f;
    if (k0 + key < n)
      for (int c = part * 4; c < cw; c += 16) {
        const f32x4 kv = load_cache4(tile + (size_t)key * cw + c), qv = *reinterpret_cast<const f32x4*>(sq + c);
        d += kv.x * qv.x + kv.y * qv.y + kv.z * qv.z + kv.w * qv.w;
      }
    d += lane_xor1(d);
    d += lane_xor2(d);
    if (part == 0) sc[key] = k0 + key < n ? d * p.scale : -INFINITY;
    __syncthreads();
    const float s = sc[tid & 63];
    const float mn = fmaxf(m, wave_max(s));
    const float e = expf(s - mn), alpha = expf(m - mn);
    l = l * alpha + wave_sum(e);
    m = mn;
    __syncthreads();
    if (tid < 64) sc[tid] = e;
    __syncthreads();
    const int lim = n - k0 < 64 ? n - k0 : 64;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = tid + 256 * j;
      if (c >= p.rank_p) break;
      float a = o[j] * alpha;
      for (int k = 0; k < lim; ++k) {
        float v;
        if constexpr (sizeof(CT) == 4) v = tile[(size_t)k * cw + c];
        else v = bf16_to_f32(tile[(size_t)k * cw + c]);
        a += sc[k] * v;
      }
      o[j] = a;
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int c = tid + 256 * j;
    if (c < p.rank_p) p.o[((size_t)row * p.heads + h) * p.rank_p + c] = o[j] / l;
  }
}

// ---- absorbed attention on the matrix pipe: grid (head tiles, rows, splits), 16 heads x 64 keys per step ----
// S = Q K^T: wave w takes keys 16 w .. + 15 of the tile; the scores meet in LDS, 16 lanes per head do the online softmax; O += P C: wave w
// takes latent columns [w, w + 1) * rank_p / 4, its B fragments gathered from the same LDS rows (8 keys of one column per lane).  Q enters
// as bf16 hi + lo, P too: only the cache's own rounding to bf16 is left.
constexpr int kLdP = 72;
template <int NT>      // 16-column fragments of the latent per wave (rank_p <= 64 NT)
__global__ __launch_bounds__(256) void latent_decode_kernel(ChattsLatentArgs p) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int ht = blockIdx.x, row = blockIdx.y, split = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int cw = p.rank_p + p.rot_p, ldk = cw + 8, cv = cw >> 3;
  const ChattsRow R = p.rows[row];
  uint16_t* kt = reinterpret_cast<uint16_t*>(smem);          // [64][ldk]
  uint16_t* qh = kt + 64 * ldk;                              // [16][ldk]
  uint16_t* ql = qh + 16 * ldk;
  uint16_t* ph = ql + 16 * ldk;                              // [16][kLdP]
  uint16_t* pl = ph + 16 * kLdP;
  float* ss = reinterpret_cast<float*>(pl + 16 * kLdP);      // [16][68]
  float* sal = ss + 16 * 68;                                 // [16] rescale factors
  const int n = R.pos + 1, ntiles = (n + 63) >> 6;
  if (R.pos < 0) return;
  for (int e = tid; e < 16 * cv; e += 256) {
    const int r = e / cv, c = (e - r * cv) * 8;
    int h = ht * 16 + r;
    if (h >= p.heads) h = p.heads - 1;
    const size_t at = (size_t)row * p.q.ld + (size_t)h * cw + c;
    *reinterpret_cast<u32x4*>(qh + r * ldk + c) = *reinterpret_cast<const u32x4*>(p.q.hi + at);
    *reinterpret_cast<u32x4*>(ql + r * ldk + c) = *reinterpret_cast<const u32x4*>(p.q.lo + at);
  }
  const uint16_t* cache = reinterpret_cast<const uint16_t*>(p.cache);
  float m = -INFINITY, l = 0.f;      // of head tid >> 4
  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const int nf = p.rank_p >> 4, fr = lane & 15, fg = lane >> 4;
  for (int t = split; t < ntiles; t += p.n_splits) {
    const uint16_t* tile = cache + latent_row(p, R.slot, t * 64, cw);
    const int lim = n - t * 64 < 64 ? n - t * 64 : 64;
    for (int e = tid; e < 64 * cv; e += 256) {
      const int r = e / cv, c = (e - r * cv) * 8;
      // rows past the last key: zeros, so that 0 * row stays 0 whatever an unused cache row holds
      u32x4 v = {0u, 0u, 0u, 0u};
      if (r < lim) v = *reinterpret_cast<const u32x4*>(tile + (size_t)r * cw + c);
      *reinterpret_cast<u32x4*>(kt + r * ldk + c) = v;
    }
    __syncthreads();
    f32x4 sacc = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < cw; k += 32) {
      const bf16x8_t b = *reinterpret_cast<const bf16x8_t*>(kt + (wave * 16 + fr) * ldk + k + fg * 8);
      const bf16x8_t a0 = *reinterpret_cast<const bf16x8_t*>(qh + fr * ldk + k + fg * 8);
      const bf16x8_t a1 = *reinterpret_cast<const bf16x8_t*>(ql + fr * ldk + k + fg * 8);
      sacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0, b, sacc, 0, 0, 0);
      sacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1, b, sacc, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) ss[(fg * 4 + r) * 68 + wave * 16 + fr] = sacc[r];
    __syncthreads();
    {
      const int h = tid >> 4, c = tid & 15;
      float v[4], mx = -INFINITY;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = j * 16 + c;
        v[j] = key < lim ? ss[h * 68 + key] * p.scale : -INFINITY;
        mx = fmaxf(mx, v[j]);
      }
      const float mn = fmaxf(m, row16_max(mx)), alpha = expf(m - mn);
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float e = expf(v[j] - mn);
        sum += e;
        uint16_t hi, lo;
        split_bf16x2(e, hi, lo);
        ph[h * kLdP + j * 16 + c] = hi;
        pl[h * kLdP + j * 16 + c] = lo;
      }
      l = l * alpha + row16_sum(sum);
      m = mn;
      if (c == 0) sal[h] = alpha;
    }
    __syncthreads();
    float al[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) al[r] = sal[fg * 4 + r];
    bf16x8_t a[2][2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      a[k][0] = *reinterpret_cast<const bf16x8_t*>(ph + fr * kLdP + k * 32 + fg * 8);
      a[k][1] = *reinterpret_cast<const bf16x8_t*>(pl + fr * kLdP + k * 32 + fg * 8);
    }
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int f = wave + 4 * i;
      if (f < nf) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[i][r] *= al[r];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          union { uint16_t u[8]; bf16x8_t v; } b;
#pragma unroll
          for (int j = 0; j < 8; ++j) b.u[j] = kt[(k * 32 + fg * 8 + j) * ldk + f * 16 + fr];
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[k][0], b.v, acc[i], 0, 0, 0);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[k][1], b.v, acc[i], 0, 0, 0);
        }
      }
    }
    __syncthreads();
  }
  // write out: C layout col = lane & 15 (latent column), row = 4 * (lane >> 4) + r (head)
  if ((tid & 15) == 0) { ss[tid >> 4] = m; ss[16 + (tid >> 4)] = l; }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int hh = fg * 4 + r, h = ht * 16 + hh;
    if (h >= p.heads) continue;
    const float ll = ss[16 + hh];
    if (p.n_splits == 1) {
      float* o = p.o + ((size_t)row * p.heads + h) * p.rank_p;
#pragma unroll
      for (int i = 0; i < NT; ++i)
        if (wave + 4 * i < nf) o[(wave + 4 * i) * 16 + fr] = acc[i][r] / ll;
    } else {
      float* o = p.partial + (((size_t)row * p.heads + h) * p.n_splits + split) * (p.rank_p + 2);
#pragma unroll
      for (int i = 0; i < NT; ++i)
        if (wave + 4 * i < nf) o[(wave + 4 * i) * 16 + fr] = acc[i][r];
      if (wave == 0 && fr == 0) { o[p.rank_p] = ss[hh]; o[p.rank_p + 1] = ll; }
    }
  }
}

// merge of the splits: one workgroup per (head, row)
__global__ __launch_bounds__(256) void latent_merge_kernel(ChattsLatentArgs p) {
  const int h = blockIdx.x, row = blockIdx.y;
  if (p.rows[row].pos < 0) return;
  const float* part = p.partial + ((size_t)row * p.heads + h) * p.n_splits * (p.rank_p + 2);
  const int ld = p.rank_p + 2;
  float M = -INFINITY;
  for (int s = 0; s < p.n_splits; ++s) M = fmaxf(M, part[(size_t)s * ld + p.rank_p]);
  float L = 0.f;
  for (int s = 0; s < p.n_splits; ++s) L += expf(part[(size_t)s * ld + p.rank_p] - M) * part[(size_t)s * ld + p.rank_p + 1];
  for (int c = threadIdx.x; c < p.rank_p; c += 256) {
    float o = 0.f;
    for (int s = 0; s < p.n_splits; ++s) o += expf(part[(size_t)s * ld + p.rank_p] - M) * part[(size_t)s * ld + c];
    p.o[((size_t)row * p.heads + h) * p.rank_p + c] = o / L;
  }
}

// ---- a product per head: wave = 16 rows x 16 columns, A split hi / lo in registers ----
__global__ __launch_bounds__(256) void head_linear_kernel(ChattsHeadLinearArgs p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, h = blockIdx.z;
  const int n0 = (blockIdx.x * 4 + wave) * 16, m0 = blockIdx.y * 16;
  if (n0 >= p.n) return;
  const int fr = lane & 15, fg = lane >> 4;
  const int r = m0 + fr < p.m ? m0 + fr : p.m - 1;
  const float* a = p.a + (size_t)r * p.lda + (size_t)h * p.a_head + fg * 8;
  const uint16_t* w = p.w + ((size_t)h * p.n + n0 + fr) * p.k + fg * 8;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < p.k; k += 32) {
    const f32x4 x0 = *reinterpret_cast<const f32x4*>(a + k), x1 = *reinterpret_cast<const f32x4*>(a + k + 4);
    const bf16x8_t b = *reinterpret_cast<const bf16x8_t*>(w + k);
    bf16x8_t hi, lo;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float x = j < 4 ? x0[j] : x1[j - 4];
      hi[j] = (__bf16)x;
      lo[j] = (__bf16)(x - (float)hi[j]);
    }
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, b, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, b, acc, 0, 0, 0);
  }
#pragma unroll
  for (int q = 0; q < 4; ++q)
    if (m0 + fg * 4 + q < p.m) store_operand(p.out, m0 + fg * 4 + q, h * p.out_head + n0 + fr, acc[q]);
}

static int check_latent(const ChattsLatentArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->cache && a->table && a->rows && a->q.ld > 0, CHATTS_E_BADARG, "%s: null pointer", who);
  CHATTS_REQUIRE(a->heads > 0 && a->dim > 0 && a->rot >= 0 && a->rot % 2 == 0 && a->rank > 0 && a->rank_p % 32 == 0 && a->rot_p % 32 == 0 &&
                     a->rank_p >= a->rank && a->rot_p >= a->rot, CHATTS_E_SHAPE, "%s: heads %d, dim %d + %d, latent %d (padded %d + %d)", who, a->heads, a->dim,
                 a->rot, a->rank, a->rank_p, a->rot_p);
  CHATTS_REQUIRE(a->rank_p <= 1024 && a->rot_p <= 256, CHATTS_E_SHAPE, "%s: latent %d (at most 1024) / rotated part %d (at most 256)", who, a->rank, a->rot);
  CHATTS_REQUIRE(a->log_block >= 6 && a->log_block <= 15, CHATTS_E_SHAPE, "%s: pages of 2^%d tokens (64 .. 32768)", who, a->log_block);
  CHATTS_REQUIRE(((uintptr_t)a->cache % 16) == 0 && a->q.ld >= a->heads * (a->rank_p + a->rot_p) && a->q.ld % 8 == 0, CHATTS_E_SHAPE, "%s: alignment / strides", who);
  return CHATTS_OK;
}

template <int NT>
static int launch_latent_decode(const ChattsLatentArgs* a, hipStream_t s) {
  const int cw = a->rank_p + a->rot_p;
  const size_t lds = (size_t)(64 + 32) * (cw + 8) * 2 + 2 * 16 * kLdP * 2 + (16 * 68 + 16) * 4;
  CHATTS_REQUIRE(lds <= 160 * 1024, CHATTS_E_SHAPE, "latent_attend: a cache row of %d elements does not fit", cw);
  static bool configured = false;
  if (!configured) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<NT>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "latent_attend: cannot reserve LDS: %s", hipGetErrorString(e));
    configured = true;
  }
  hipLaunchKernelGGL(latent_decode_kernel<NT>, dim3((a->heads + 15) / 16, a->n_rows, a->n_splits), dim3(256), lds, s, *a);
  CHATTS_CHECK_LAUNCH("latent_decode");
  return CHATTS_OK;
}

static int latent_attend_impl(const ChattsLatentArgs* a, hipStream_t s) {
  if (const int rc = check_latent(a, "latent_attend")) return rc;
  CHATTS_REQUIRE(a->o && (a->q.f32 || a->q.hi), CHATTS_E_BADARG, "latent_attend: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  const int cw = a->rank_p + a->rot_p;
  const bool matrix = !a->cache_f32 && a->q.hi && a->q.lo && (size_t)(64 + 32) * (cw + 8) * 2 + 2 * 16 * kLdP * 2 + (16 * 68 + 16) * 4 <= 160 * 1024;
  if (!matrix) {
    const size_t lds = (size_t)(cw + 64) * sizeof(float);
    const dim3 g(a->heads, a->n_rows);
    if (a->cache_f32) hipLaunchKernelGGL(latent_attend_kernel<float>, g, dim3(256), lds, s, *a);
    else hipLaunchKernelGGL(latent_attend_kernel<uint16_t>, g, dim3(256), lds, s, *a);
    CHATTS_CHECK_LAUNCH("latent_attend");
    return CHATTS_OK;
  }
  CHATTS_REQUIRE(a->n_splits >= 1 && (a->n_splits == 1 || a->partial), CHATTS_E_BADARG, "latent_attend: %d splits without a buffer", a->n_splits);
  int rc;
  if (a->rank_p <= 128) rc = launch_latent_decode<2>(a, s);
  else if (a->rank_p <= 256) rc = launch_latent_decode<4>(a, s);
  else if (a->rank_p <= 512) rc = launch_latent_decode<8>(a, s);
  else rc = launch_latent_decode<16>(a, s);
  if (rc) return rc;
  if (a->n_splits > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(a->heads, a->n_rows), dim3(256), 0, s, *a);
    CHATTS_CHECK_LAUNCH("latent_merge");
  }
  return CHATTS_OK;
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_latent_prep(const ChattsLatentArgs* a, chatts_stream_t stream) {
  if (const int rc = check_latent(a, "latent_prep")) return rc;
  CHATTS_REQUIRE(a->proj && a->c_norm && (a->rot == 0 || (a->cos_tab && a->sin_tab)) && (a->q.f32 || a->q.hi), CHATTS_E_BADARG, "latent_prep: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  if (a->cache_f32) hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(a->n_rows), dim3(256), 0, as_stream(stream), *a);
  else hipLaunchKernelGGL(latent_prep_kernel<uint16_t>, dim3(a->n_rows), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("latent_prep");
  return CHATTS_OK;
}

extern "C" int chatts_latent_attend(const ChattsLatentArgs* a, chatts_stream_t stream) { return latent_attend_impl(a, as_stream(stream)); }

extern "C" int chatts_head_linear(const ChattsHeadLinearArgs* a, chatts_stream_t stream) {
  CHATTS_REQUIRE(a && a->a && a->w && (a->out.f32 || a->out.hi), CHATTS_E_BADARG, "head_linear: null pointer");
  CHATTS_REQUIRE(a->m >= 0 && a->heads > 0 && a->n > 0 && a->n % 16 == 0 && a->k > 0 && a->k % 32 == 0, CHATTS_E_SHAPE, "head_linear: m=%d n=%d k=%d", a->m, a->n, a->k);
  CHATTS_REQUIRE(a->lda % 4 == 0 && a->a_head % 4 == 0 && ((uintptr_t)a->a % 16) == 0 && ((uintptr_t)a->w % 16) == 0, CHATTS_E_SHAPE,
                 "head_linear: A rows and heads must be 16-byte aligned (lda=%d, head stride %d)", a->lda, a->a_head);
  if (a->m == 0) return CHATTS_OK;
  if (a->exact) {
    CHATTS_REQUIRE(a->out.f32 && !a->out.hi, CHATTS_E_BADARG, "head_linear: the exact form writes float32");
    return launch_gemm_f32_batched(a->a, a->a_head, a->lda, a->w, (int64_t)a->n * a->k, a->k, a->out.f32, a->out_head, a->out.ld, a->m, a->n, a->k,
                                   a->heads, as_stream(stream));
  }
  hipLaunchKernelGGL(head_linear_kernel, dim3((a->n / 16 + 3) / 4, (a->m + 15) / 16, a->heads), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("head_linear");
  return CHATTS_OK;
}
