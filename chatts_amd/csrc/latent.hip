// latent.hip - latent attention: keys and values of all heads are linear maps of one cached latent per token, beside one rotated key part
// that the heads share.  The cache holds only [latent | rotated part] per token, in pages.
//   score_h(i, j) = (q_un_h(i) . W_uk_h c_j + q_rot_h(i) . k_rot_j) * scale = ([W_uk_h^T q_un_h | q_rot_h](i) . [c | k_rot](j)) * scale
//   out_h(i) = W_uv_h sum_j softmax(score)_ij c_j
// The absorbed form (second half of each line) is multi-query attention over the cached rows: one row feeds every head, so decoding reads
// the cache once per head tile.
//   * latent_prep_kernel: rotation of the query parts, norm of the latent, rotation of the key part, cache write
//   * head_linear_kernel: W_uk^T on the queries, W_uv on the weighted latents (a product per head)
//   * latent_attend_kernel: one (row, head) per workgroup on the vector units, float32 or bf16 cache: the 32-bit runs and odd sizes
//   * latent_decode_kernel: up to 32 heads of a row per workgroup on the matrix pipe, bf16 cache, the keys spread over workgroups, partials
//     merged by latent_merge_kernel
// The expanded form (first half of each line) does fewer products per key once many queries share it: prompts take it
//   * latent_gather_kernel, two projections (keys; values, transposed by exchanging the operands) and latent_prefill_kernel, a flash loop
#include "ring_store.h"

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
  if (p.qx)                                                  // expanded form: the unrotated part as it is
    for (int e = tid; e < p.heads * (p.dim_p >> 2); e += 256) {
      const int h = e / (p.dim_p >> 2), c = (e - h * (p.dim_p >> 2)) * 4;
      const f32x4 v = *reinterpret_cast<const f32x4*>(pr + p.off_q + h * p.dim_p + c);
      typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
      *reinterpret_cast<bf16x4_t*>(p.qx + (size_t)row * p.heads * (p.dim_p + p.rot_p) + h * (p.dim_p + p.rot_p) + c) =
          (bf16x4_t){(__bf16)v.x, (__bf16)v.y, (__bf16)v.z, (__bf16)v.w};
    }
  for (int e = tid; e < p.heads * p.rot_p; e += 256) {      // the rotated part of every head's query, padding included
    const int h = e / p.rot_p, i = e - h * p.rot_p;
    float v = 0.f;
    if (i < p.rot) {
      const float* q = pr + p.off_qr + h * p.rot;
      const int f = i < half ? i : i - half;
      const float u = q[f], w = q[f + half];
      v = i < half ? u * ct[f] - w * st[f] : w * ct[f] + u * st[f];
    }
    if (p.q.f32 || p.q.hi) store_operand(p.q, row, h * cw + p.rank_p + i, v);
    if (p.qx) p.qx[(size_t)row * p.heads * (p.dim_p + p.rot_p) + h * (p.dim_p + p.rot_p) + p.dim_p + i] = to_cache<uint16_t>(v);
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

// ---- absorbed attention on the matrix pipe: grid (splits, rows, head tiles / HT), HT x 16 heads per workgroup ----------------------------
// Tiles of 32 keys pass through a ring of four in LDS, filled by two loader waves (LDS-DMA) and read by four compute waves; compute wave = (head
// tile, slice of the latent columns).  S^T = K Q^T reads rows of the tile as A fragments, so a lane ends up with 8 scores of one head (column =
// lane & 15); O^T = C^T P^T reads the tile transposed, and its B fragment IS the 8 probabilities of the lane.  K slot 8 g + j of that product means
// key 4 g + j (j < 4) or 16 + 4 g + j - 4, on both sides.  The waves of a head tile compute the same scores (that is cheaper than handing them
// round) and own different latent columns: nothing is merged inside a workgroup.
// 16-byte chunk c of row r lies at position c ^ (r & swizzle): neither way of reading meets the same banks in every row.
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4* lds_s16x4;
constexpr int kLatStages = 4, kLatLoaders = 2, kLatThreads = 64 * (4 + kLatLoaders);

// at most n (wave-uniform) of this wave's requests outstanding
__device__ __forceinline__ void latent_wait(int n) {
#define CHATTS_VM(N) case N: asm volatile("s_waitcnt vmcnt(" #N ")" ::: "memory"); break;
#define CHATTS_VM4(A, B, C, D) CHATTS_VM(A) CHATTS_VM(B) CHATTS_VM(C) CHATTS_VM(D)
  switch (n) {
    CHATTS_VM4(1, 2, 3, 4) CHATTS_VM4(5, 6, 7, 8) CHATTS_VM4(9, 10, 11, 12) CHATTS_VM4(13, 14, 15, 16) CHATTS_VM4(17, 18, 20, 22) CHATTS_VM4(24, 26, 28, 30)
    CHATTS_VM(32) CHATTS_VM(34) CHATTS_VM(36)
    default: asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); break;
  }
#undef CHATTS_VM4
#undef CHATTS_VM
}

template <int NF, int NK, int HT, bool FULL>      // rank_p <= 16 NF, cw <= 32 NK; FULL: equal
__global__ __launch_bounds__(kLatThreads, 2) void latent_decode_kernel(ChattsLatentArgs p) {
  extern __shared__ __attribute__((aligned(1024))) char smem[];
  constexpr int RS = 4 / HT, NFW = NF / RS;      // slices of the latent columns, fragments per wave
  const int split = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int cw = FULL ? 32 * NK : p.rank_p + p.rot_p, cv = cw >> 3, nf = FULL ? NF : p.rank_p >> 4, nk = FULL ? NK : cw >> 5, sw = (cv & 7) == 0 ? 7 : 3;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const int n = R.pos + 1, ntiles = (n + 31) >> 5, fr = lane & 15, fg = lane >> 4;
  const int count = split < ntiles ? (ntiles - split + p.n_splits - 1) / p.n_splits : 0;      // tiles split, split + n_splits, ...
  const int stage = cw * 64;
  if (wave >= 4) {
    // ---- loader: every kLatLoaders-th of the cw / 16 pieces (64 chunks of 16 bytes) of a tile
    const int L = wave - 4, pieces = cw >> 4, mine = (pieces - L + kLatLoaders - 1) / kLatLoaders;
    const int e0 = L * 64 + lane, r0 = e0 / cv, c0 = e0 - r0 * cv, dr = kLatLoaders * 64 / cv, dc = kLatLoaders * 64 - dr * cv;
    const char* cache = reinterpret_cast<const char*>(p.cache);
    auto issue = [&](int k) {
      const char* tile = cache + latent_row(p, R.slot, (split + k * p.n_splits) * 32, cw) * 2;
      char* base = smem + (k & (kLatStages - 1)) * stage + L * 1024;
      int r = r0, c = c0;
      for (int i = 0; i < mine; ++i) {
        __builtin_amdgcn_global_load_lds((gptr_t)(tile + (uint32_t)(r * cw + ((c ^ (r & sw)) << 3)) * 2), (lptr_t)(base + i * (kLatLoaders * 1024)), 16, 0, 0);
        r += dr;
        c += dc;
        if (c >= cv) { c -= cv; ++r; }
      }
    };
    for (int k = 0; k < kLatStages - 1 && k < count; ++k) issue(k);
    for (int k = 0; k < count; ++k) {
      const int later = count - 1 - k < kLatStages - 2 ? count - 1 - k : kLatStages - 2;
      latent_wait(later * mine);                              // tile k has landed
      __builtin_amdgcn_s_barrier();                           // ... and everyone has read tile k - 1
      if (n - (split + k * p.n_splits) * 32 < 32) __builtin_amdgcn_s_barrier();
      if (k + kLatStages - 1 < count) issue(k + kLatStages - 1);
    }
    return;
  }
  const int ht = blockIdx.z * HT + wave / RS, f0 = (wave % RS) * NFW;
  bf16x8_t q[NK];
  {
    int h = ht * 16 + fr;
    if (h >= p.heads) h = p.heads - 1;
    const uint16_t* src = p.q.hi + (size_t)row * p.q.ld + (size_t)h * cw + fg * 8;
#pragma unroll
    for (int k = 0; k < NK; ++k)
      if (k < nk) q[k] = *reinterpret_cast<const bf16x8_t*>(src + k * 32);
  }
  float m = -INFINITY, l = 0.f;      // of head fr; l: this lane's keys only
  f32x4 acc[NFW];
#pragma unroll
  for (int i = 0; i < NFW; ++i) acc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < count; ++k) {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");      // this wave has read tile k - 1
    __builtin_amdgcn_s_barrier();                           // tile k is complete
    char* kt = smem + (k & (kLatStages - 1)) * stage;
    const int lim = n - (split + k * p.n_splits) * 32;
    if (lim < 32) {      // keys past the last one become zeros, whatever an unused cache row holds
      for (int e = lim * cv + tid; e < 32 * cv; e += 256) *reinterpret_cast<u32x4*>(kt + e * 16) = (u32x4){0u, 0u, 0u, 0u};
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      __builtin_amdgcn_s_barrier();
    }
    f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    {
      const char* a0 = kt + fr * cw * 2;
      const char* a1 = kt + (16 + fr) * cw * 2;
      const int x = fr & sw;      // (16 is a multiple of the swizzle's period)
      // fragments of G K-steps are requested while those before are multiplied
      constexpr int G = 3, NG = (NK + G - 1) / G;
      bf16x8_t kf[2][G][2];
      auto request = [&](int g, bf16x8_t (&dst)[G][2]) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < G; ++u) {
          const int k2 = g * G + u;
          if (k2 < NK && k2 < nk) {
            const int c = ((k2 * 4 + fg) ^ x) << 4;
            dst[u][0] = *reinterpret_cast<const bf16x8_t*>(a0 + c);
            dst[u][1] = *reinterpret_cast<const bf16x8_t*>(a1 + c);
          }
        }
      };
      request(0, kf[0]);
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        if (g + 1 < NG) request(g + 1, kf[(g + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int u = 0; u < G; ++u) {
          const int k2 = g * G + u;
          if (k2 < NK && k2 < nk) {
            s[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[g & 1][u][0], q[k2], s[0], 0, 0, 0);
            s[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[g & 1][u][1], q[k2], s[1], 0, 0, 0);
          }
        }
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    float v[8], mx = -INFINITY;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int key = (j >> 2) * 16 + fg * 4 + (j & 3);
      v[j] = key < lim ? s[j >> 2][j & 3] * p.scale : -INFINITY;
      mx = fmaxf(mx, v[j]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx), alpha = exp_hw(m - mn);
    m = mn;
    bf16x8_t ph, pl;
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float e = exp_hw(v[j] - mn);
      sum += e;
      ph[j] = (__bf16)e;
      pl[j] = (__bf16)(e - (float)ph[j]);
    }
    l = l * alpha + sum;
    if (__any(alpha != 1.0f)) {
#pragma unroll
      for (int i = 0; i < NFW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[i][r] *= alpha;
    }
    {
      // transposing reads: lane -> row 4 g + (fr >> 2) (and + 16), 4 columns (fr & 3) * 4 of the fragment's 16: chunk 2 f + (fr >> 1 & 1), half fr & 1
      const int tr = fg * 4 + (fr >> 2), x = tr & sw, cb = (fr >> 1) & 1;
      const char* t0 = kt + tr * cw * 2 + (fr & 1) * 8;
      constexpr int G = NFW < 4 ? NFW : 4, NG = NFW / G;
      union Tr { s16x4 h[2]; bf16x8_t v; };
      Tr a[2][G];
      auto request = [&](int g, Tr (&dst)[G]) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < G; ++u) {
          const int f = f0 + g * G + u;
          if (FULL || f < nf) {
            const int c = ((2 * f + cb) ^ x) << 4;
            dst[u].h[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(t0 + c));
            dst[u].h[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(t0 + 32 * cw + c));
          }
        }
      };
      request(0, a[0]);
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        if (g + 1 < NG) request(g + 1, a[(g + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int u = 0; u < G; ++u)
          if (FULL || f0 + g * G + u < nf) acc[g * G + u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[g & 1][u].v, ph, acc[g * G + u], 0, 0, 0);
#pragma unroll
        for (int u = 0; u < G; ++u)
          if (FULL || f0 + g * G + u < nf) acc[g * G + u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[g & 1][u].v, pl, acc[g * G + u], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  const int h = ht * 16 + fr;
  if (h >= p.heads) return;
  // a lane: 4 consecutive latent columns of its head per fragment
  const bool whole = p.n_splits == 1;
  float* dst = whole ? p.o + ((size_t)row * p.heads + h) * p.rank_p : p.partial + (((size_t)row * p.heads + h) * p.n_splits + split) * (p.rank_p + 4);
  const float f = whole ? 1.0f / l : 1.0f;
#pragma unroll
  for (int i = 0; i < NFW; ++i)
    if (FULL || f0 + i < nf) *reinterpret_cast<f32x4*>(dst + (f0 + i) * 16 + fg * 4) = (f32x4){acc[i][0] * f, acc[i][1] * f, acc[i][2] * f, acc[i][3] * f};
  if (!whole && f0 == 0 && fg == 0) { dst[p.rank_p] = m; dst[p.rank_p + 1] = l; }
}

// merge of the splits: one workgroup per (head, row)
__global__ __launch_bounds__(128) void latent_merge_kernel(ChattsLatentArgs p) {
  __shared__ float w[64];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, ld = p.rank_p + 4;
  if (p.rows[row].pos < 0) return;
  const float* part = p.partial + ((size_t)row * p.heads + h) * p.n_splits * ld;
  if (tid < 64) {
    const float m = tid < p.n_splits ? part[(size_t)tid * ld + p.rank_p] : -INFINITY, l = tid < p.n_splits ? part[(size_t)tid * ld + p.rank_p + 1] : 0.f;
    const float M = wave_max(m), f = m == -INFINITY ? 0.f : exp_hw(m - M);
    const float L = wave_sum(f * l);
    w[tid] = f / L;
  }
  __syncthreads();
  for (int c = tid * 4; c < p.rank_p; c += 512) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < p.n_splits; ++s) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(part + (size_t)s * ld + c);
      const float f = w[s];
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] += f * x[r];
    }
    *reinterpret_cast<f32x4*>(p.o + ((size_t)row * p.heads + h) * p.rank_p + c) = o;
  }
}

// ---- expanded form, for prompts: keys and values of every head are written out for the sequence, then ordinary flash attention ----------
// gather: the latents and rotated key parts of each expanded span's sequence from its pages into consecutive rows (span.base ..), a whole
// number of 64-row tiles per span, zeros past the last key.  grid (row groups of 16, spans)
__global__ __launch_bounds__(256) void latent_gather_kernel(ChattsLatentArgs p, const ChattsSpan* __restrict__ spans, uint16_t* __restrict__ cbuf,
                                                            uint16_t* __restrict__ krbuf) {
  const ChattsSpan sp = spans[blockIdx.y];
  if (sp.base < 0) return;
  const int n = sp.pos0 + sp.t, rows = (n + 63) & ~63, cw = p.rank_p + p.rot_p, cv = cw >> 3;
  const int j0 = blockIdx.x * 16;
  if (j0 >= rows) return;
  const uint16_t* src = reinterpret_cast<const uint16_t*>(p.cache) + (j0 < n ? latent_row(p, sp.slot, j0, cw) : 0);
  for (int e = threadIdx.x; e < 16 * cv; e += 256) {
    const int r = e / cv, c = (e - r * cv) * 8;
    u32x4 v = {0u, 0u, 0u, 0u};
    if (j0 + r < n) v = *reinterpret_cast<const u32x4*>(src + (size_t)r * cw + c);
    const size_t at = (size_t)(sp.base + j0 + r);
    if (c < p.rank_p) *reinterpret_cast<u32x4*>(cbuf + at * p.rank_p + c) = v;
    else *reinterpret_cast<u32x4*>(krbuf + at * p.rot_p + c - p.rank_p) = v;
  }
}

// grid (heads, query tiles of 128, spans) - the heads of an XCD (workgroup id modulo 8) stay the same, so their keys and values stay in its L2, and every
// XCD gets long and short query tiles alike -, a wave owns 32 queries of one head, 64 keys per step: S^T = K Q^T, O^T = V^T P^T - the probabilities of
// a lane are the B fragment of the second product (K slot 8 g + j = key 8 g + j: the rows of K are staged in the order that makes it so).
// Rows of the expanded keys and values are 256 bytes longer than their contents: at a power-of-two stride every row of a tile would lie in the
// same L2 channel.
constexpr int kExpandPad = CHATTS_LATENT_EXPAND_PAD;

struct LatentPrefill {
  const uint16_t* kx;      // [rows, ldk]: unrotated keys, head by head (dim_p each)
  const uint16_t* kr;      // [rows, rot_p]
  const uint16_t* vt;      // [heads * vdim_p, ldv]: values, transposed
  const uint16_t* qx;      // [T, ldq]: [unrotated | rotated] per head (dim_p + rot_p)
  int ldk, ldv, ldq, dim_p, rot_p, vdim_p, out_head;
  float scale;
  ChattsOperand out;
};
template <int NK, int NV, int OCC, bool FULL>      // dim_p + rot_p <= 32 NK, vdim_p <= 16 NV; FULL: equal
__global__ __launch_bounds__(256, OCC) void latent_prefill_kernel(LatentPrefill p, const ChattsSpan* __restrict__ spans) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const ChattsSpan sp = spans[blockIdx.z];
  const int qt0 = (gridDim.y - 1 - blockIdx.y) * 128, h = blockIdx.x;      // the longest key ranges first
  if (sp.base < 0 || qt0 >= sp.t) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int dq = FULL ? 32 * NK : p.dim_p + p.rot_p, vdim_p = FULL ? 16 * NV : p.vdim_p, ldl = dq + 8, nk = dq >> 5, nv = vdim_p >> 4;
  constexpr int kLdV = 72;
  uint16_t* ks = reinterpret_cast<uint16_t*>(smem);      // [64][ldl]
  uint16_t* vs = ks + 64 * ldl;                          // [vdim_p][72]
  const int qlast = qt0 + 127 < sp.t ? qt0 + 127 : sp.t - 1;
  const int ntiles = (sp.pos0 + qlast + 64) >> 6;        // keys 0 .. pos0 + qlast
  const int q0 = qt0 + wave * 32;
  bf16x8_t q[2][NK];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    int r = q0 + u * 16 + fr;
    if (r > sp.t - 1) r = sp.t - 1;
    const uint16_t* src = p.qx + (size_t)(sp.row0 + r) * p.ldq + h * dq + fg * 8;
#pragma unroll
    for (int k = 0; k < NK; ++k)
      if (k < nk) q[u][k] = *reinterpret_cast<const bf16x8_t*>(src + k * 32);
  }
  f32x4 o[NV][2];
#pragma unroll
  for (int i = 0; i < NV; ++i) o[i][0] = o[i][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  const float scale2 = p.scale * 1.44269504088896341f;      // scores in base 2
  // staging: K rows in 16-byte pieces (64 rows x dq / 8), V^T rows (vdim_p x 8)
  constexpr int KP = NK, VP = (NV + 1) / 2;
  u32x4 rk[KP], rv[VP];
  const int kc = dq >> 3, dc = p.dim_p >> 3;
  auto fetch = [&](int t) {
    const size_t base = (size_t)sp.base + t * 64;
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int e = i * 256 + tid;
      if (FULL || e < 64 * kc) {
        const int r = e / kc, c = e - r * kc;
        rk[i] = c < dc ? *reinterpret_cast<const u32x4*>(p.kx + (base + r) * p.ldk + h * p.dim_p + c * 8)
                       : *reinterpret_cast<const u32x4*>(p.kr + (base + r) * p.rot_p + (c - dc) * 8);
      }
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int e = i * 256 + tid;
      if (FULL ? NV % 2 == 0 || e < vdim_p * 8 : e < vdim_p * 8) rv[i] = *reinterpret_cast<const u32x4*>(p.vt + (size_t)(h * vdim_p + (e >> 3)) * p.ldv + base + (e & 7) * 8);
    }
  };
  fetch(0);
  for (int t = 0; t < ntiles; ++t) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int e = i * 256 + tid;
      if (FULL || e < 64 * kc) {      // key 32 G + 8 g + 4 h + j -> row 32 G + 16 h + 4 g + j: the rows of a fragment lie next to each other
        const int key = e / kc, r = (key & 35) | ((key & 4) << 2) | ((key & 24) >> 1);
        *reinterpret_cast<u32x4*>(ks + r * ldl + (e - key * kc) * 8) = rk[i];
      }
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int e = i * 256 + tid;
      if (FULL ? NV % 2 == 0 || e < vdim_p * 8 : e < vdim_p * 8) *reinterpret_cast<u32x4*>(vs + (e >> 3) * kLdV + (e & 7) * 8) = rv[i];
    }
    __syncthreads();
    if (t + 1 < ntiles) fetch(t + 1);
    if (t * 64 > sp.pos0 + q0 + 31) continue;      // (uniform per wave) nothing visible to this wave's queries
    f32x4 s[4][2];      // [32-key group * 2 + half][query block]
#pragma unroll
    for (int a = 0; a < 4; ++a) s[a][0] = s[a][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const uint16_t* kb = ks + fr * ldl + fg * 8;
    {
      bf16x8_t kf[2][4];      // the next K-step's fragments are requested while this one's are multiplied
      auto request = [&](int k, bf16x8_t (&dst)[4]) __attribute__((always_inline)) {
#pragma unroll
        for (int a = 0; a < 4; ++a) dst[a] = *reinterpret_cast<const bf16x8_t*>(kb + a * 16 * ldl + k * 32);
      };
      request(0, kf[0]);
#pragma unroll
      for (int k = 0; k < NK; ++k)
        if (k < nk) {
          if (k + 1 < NK && k + 1 < nk) request(k + 1, kf[(k + 1) & 1]);
          __builtin_amdgcn_sched_barrier(0);
#pragma unroll
          for (int a = 0; a < 4; ++a) {
            s[a][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[k & 1][a], q[0][k], s[a][0], 0, 0, 0);
            s[a][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[k & 1][a], q[1][k], s[a][1], 0, 0, 0);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
    }
    bf16x8_t pf[2][2];      // [32-key group][query block]
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int qpos = sp.pos0 + q0 + u * 16 + fr;
      const bool edge = t * 64 + 63 > sp.pos0 + q0 + u * 16;      // (uniform) some key of the tile is in the future of some query
      float mx = -INFINITY;
#pragma unroll
      for (int a = 0; a < 4; ++a)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float v = s[a][u][r] * scale2;
          if (edge && t * 64 + (a >> 1) * 32 + fg * 8 + (a & 1) * 4 + r > qpos) v = -INFINITY;
          s[a][u][r] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[u], mx), safe = mn == -INFINITY ? 0.f : mn, alpha = __builtin_amdgcn_exp2f(m[u] - safe);
      m[u] = mn;
      float sum = 0.f;
#pragma unroll
      for (int a = 0; a < 4; ++a)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = __builtin_amdgcn_exp2f(s[a][u][r] - safe);
          sum += e;
          pf[a >> 1][u][(a & 1) * 4 + r] = (__bf16)e;
        }
      l[u] = l[u] * alpha + sum;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[i][u][r] *= alpha;
      }
    }
    {
      bf16x8_t vf[2][2];
      auto request = [&](int i, bf16x8_t (&dst)[2]) __attribute__((always_inline)) {
#pragma unroll
        for (int g = 0; g < 2; ++g) dst[g] = *reinterpret_cast<const bf16x8_t*>(vs + (i * 16 + fr) * kLdV + g * 32 + fg * 8);
      };
      request(0, vf[0]);
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (i < nv) {
          if (i + 1 < NV && i + 1 < nv) request(i + 1, vf[(i + 1) & 1]);
          __builtin_amdgcn_sched_barrier(0);
#pragma unroll
          for (int g = 0; g < 2; ++g) {
            o[i][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i & 1][g], pf[g][0], o[i][0], 0, 0, 0);
            o[i][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i & 1][g], pf[g][1], o[i][1], 0, 0, 0);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
    }
  }
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int r = q0 + u * 16 + fr;
    float L = l[u];
    L += __shfl_xor(L, 16, 64);
    L += __shfl_xor(L, 32, 64);
    if (r >= sp.t) continue;
    const float inv = 1.0f / L;
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (i < nv) {
        const float v[4] = {o[i][u][0] * inv, o[i][u][1] * inv, o[i][u][2] * inv, o[i][u][3] * inv};
        store_operand4(p.out, sp.row0 + r, h * p.out_head + i * 16 + fg * 4, v);
      }
  }
}

// ---- a product per head: wave = 16 rows x 16 columns, A split hi / lo in registers ----
__global__ __launch_bounds__(256) void head_linear_kernel(ChattsHeadLinearArgs p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, h = blockIdx.z;
  const int n0 = (blockIdx.x * (blockDim.x >> 6) + wave) * 16, m0 = blockIdx.y * 16;
  if (n0 >= p.n) return;
  const int fr = lane & 15, fg = lane >> 4;
  const int r = m0 + fr < p.m ? m0 + fr : p.m - 1;
  const float* a = p.a + (size_t)r * p.lda + (size_t)h * p.a_head + fg * 8;
  const uint16_t* w = p.w + ((size_t)h * p.n + n0 + fr) * p.k + fg * 8;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
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

template <int NF, int NK, int HT, bool FULL>
static int launch_latent_decode_t(const ChattsLatentArgs* a, hipStream_t s) {
  static bool configured = false;
  if (!configured) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<NF, NK, HT, FULL>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                             kLatStages * 32 * NK * 64);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "latent_attend: cannot reserve LDS: %s", hipGetErrorString(e));
    configured = true;
  }
  const int tiles = (a->heads + 15) / 16;
  hipLaunchKernelGGL((latent_decode_kernel<NF, NK, HT, FULL>), dim3(a->n_splits, a->n_rows, (tiles + HT - 1) / HT), dim3(kLatThreads),
                     kLatStages * (a->rank_p + a->rot_p) * 64, s, *a);
  CHATTS_CHECK_LAUNCH("latent_decode");
  return CHATTS_OK;
}
template <int NF, int NK>
static int launch_latent_decode(const ChattsLatentArgs* a, hipStream_t s) {
  const bool full = a->rank_p == 16 * NF && a->rank_p + a->rot_p == 32 * NK;
  if (a->heads <= 16) return full ? launch_latent_decode_t<NF, NK, 1, true>(a, s) : launch_latent_decode_t<NF, NK, 1, false>(a, s);
  return full ? launch_latent_decode_t<NF, NK, 2, true>(a, s) : launch_latent_decode_t<NF, NK, 2, false>(a, s);
}

static int latent_attend_impl(const ChattsLatentArgs* a, hipStream_t s) {
  if (const int rc = check_latent(a, "latent_attend")) return rc;
  CHATTS_REQUIRE(a->o && (a->q.f32 || a->q.hi), CHATTS_E_BADARG, "latent_attend: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  const int cw = a->rank_p + a->rot_p;
  CHATTS_REQUIRE(a->n_splits >= 1 && a->n_splits <= 64 && (a->n_splits == 1 || a->partial), CHATTS_E_BADARG, "latent_attend: %d splits", a->n_splits);
  int rc;
  if (!a->cache_f32 && a->q.hi && a->rank_p <= 64 && cw <= 128) rc = launch_latent_decode<4, 4>(a, s);
  else if (!a->cache_f32 && a->q.hi && a->rank_p <= 128 && cw <= 192) rc = launch_latent_decode<8, 6>(a, s);
  else if (!a->cache_f32 && a->q.hi && a->rank_p <= 256 && cw <= 384) rc = launch_latent_decode<16, 12>(a, s);
  else if (!a->cache_f32 && a->q.hi && a->rank_p <= 512 && cw <= 576) rc = launch_latent_decode<32, 18>(a, s);
  else {
    const size_t lds = (size_t)(cw + 64) * sizeof(float);
    const dim3 g(a->heads, a->n_rows);
    if (a->cache_f32) hipLaunchKernelGGL(latent_attend_kernel<float>, g, dim3(256), lds, s, *a);
    else hipLaunchKernelGGL(latent_attend_kernel<uint16_t>, g, dim3(256), lds, s, *a);
    CHATTS_CHECK_LAUNCH("latent_attend");
    return CHATTS_OK;
  }
  if (rc) return rc;
  if (a->n_splits > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(a->heads, a->n_rows), dim3(128), 0, s, *a);
    CHATTS_CHECK_LAUNCH("latent_merge");
  }
  return CHATTS_OK;
}

template <int NK, int NV, int OCC, bool FULL>
static int launch_latent_prefill_t(const LatentPrefill& p, const ChattsSpan* spans, int n_spans, int heads, int longest, hipStream_t s) {
  const size_t lds = (size_t)(64 * (p.dim_p + p.rot_p + 8) + p.vdim_p * 72) * 2;
  static bool configured = false;
  if (!configured) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_prefill_kernel<NK, NV, OCC, FULL>), hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "latent_expanded: cannot reserve LDS: %s", hipGetErrorString(e));
    configured = true;
  }
  hipLaunchKernelGGL((latent_prefill_kernel<NK, NV, OCC, FULL>), dim3(heads, (longest + 127) / 128, n_spans), dim3(256), lds, s, p, spans);
  CHATTS_CHECK_LAUNCH("latent_prefill");
  return CHATTS_OK;
}
template <int NK, int NV, int OCC>
static int launch_latent_prefill(const LatentPrefill& p, const ChattsSpan* spans, int n_spans, int heads, int longest, hipStream_t s) {
  return p.dim_p + p.rot_p == 32 * NK && p.vdim_p == 16 * NV ? launch_latent_prefill_t<NK, NV, OCC, true>(p, spans, n_spans, heads, longest, s)
                                                             : launch_latent_prefill_t<NK, NV, OCC, false>(p, spans, n_spans, heads, longest, s);
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_latent_prep(const ChattsLatentArgs* a, chatts_stream_t stream) {
  if (const int rc = check_latent(a, "latent_prep")) return rc;
  CHATTS_REQUIRE(a->proj && a->c_norm && (a->rot == 0 || (a->cos_tab && a->sin_tab)) && (a->q.f32 || a->q.hi || a->qx), CHATTS_E_BADARG, "latent_prep: null pointer");
  CHATTS_REQUIRE(!a->qx || (a->dim_p % 4 == 0 && a->off_q % 4 == 0 && a->ld_proj % 4 == 0), CHATTS_E_SHAPE, "latent_prep: query columns");
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
  const int waves = a->m <= 16 ? 1 : 4;      // one row tile: spread over as many CUs as there are column tiles
  hipLaunchKernelGGL(head_linear_kernel, dim3((a->n / 16 + waves - 1) / waves, (a->m + 15) / 16, a->heads), dim3(64 * waves), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("head_linear");
  return CHATTS_OK;
}

extern "C" int chatts_latent_can_expand(int dim_p, int rot_p, int vdim_p, int rank_p) {
  return rank_p % 64 == 0 && dim_p % 32 == 0 && rot_p % 32 == 0 && vdim_p % 16 == 0 && dim_p + rot_p <= 384 && vdim_p <= 256;
}

extern "C" int chatts_latent_expanded(const ChattsLatentExpandArgs* x, chatts_stream_t stream) {
  CHATTS_REQUIRE(x && x->latent && x->spans && x->spans_dev && x->cbuf && x->krbuf && x->zero && x->k_hi && x->k_lo && x->v_hi && x->v_lo && x->uk && x->uv &&
                     x->latent->qx, CHATTS_E_BADARG, "latent_expanded: null pointer");
  const ChattsLatentArgs* a = x->latent;
  if (const int rc = check_latent(a, "latent_expanded")) return rc;
  CHATTS_REQUIRE(!a->cache_f32 && chatts_latent_can_expand(a->dim_p, a->rot_p, x->vdim_p, a->rank_p), CHATTS_E_SHAPE, "latent_expanded: head sizes %d + %d / %d, latent %d",
                 a->dim_p, a->rot_p, x->vdim_p, a->rank_p);
  CHATTS_REQUIRE((x->out.f32 || x->out.hi) && x->out.ld >= (a->heads - 1) * x->out_head + x->vdim_p && x->out.ld % 4 == 0 && x->out_head % 4 == 0, CHATTS_E_SHAPE,
                 "latent_expanded: output stride");
  int rows = 0, longest = 0, longest_ctx = 0;
  for (int i = 0; i < x->n_spans; ++i) {
    const ChattsSpan& sp = x->spans[i];
    if (sp.base < 0) continue;
    CHATTS_REQUIRE(sp.base == rows && sp.t >= 1 && sp.pos0 >= 0, CHATTS_E_SHAPE, "latent_expanded: span %d starts at row %d, not %d", i, sp.base, rows);
    rows += (sp.pos0 + sp.t + 63) & ~63;
    if (sp.t > longest) longest = sp.t;
    if (sp.pos0 + sp.t > longest_ctx) longest_ctx = sp.pos0 + sp.t;
  }
  if (rows == 0) return CHATTS_OK;
  CHATTS_REQUIRE(rows <= x->max_rows, CHATTS_E_SHAPE, "latent_expanded: %d rows exceed the buffers (%d)", rows, x->max_rows);
  hipStream_t s = as_stream(stream);
  hipLaunchKernelGGL(latent_gather_kernel, dim3((((longest_ctx + 63) & ~63) + 15) / 16, x->n_spans), dim3(256), 0, s, *a, x->spans_dev, x->cbuf, x->krbuf);
  CHATTS_CHECK_LAUNCH("latent_gather");
  ChattsLinearArgs g{};      // keys: [rows, heads * dim_p] = latents . W_uk^T;  values, transposed: [heads * vdim_p, rows] = W_uv . latents^T
  g.workspace = x->workspace; g.workspace_bytes = x->workspace_bytes;
  g.a_hi = x->cbuf; g.a_lo = x->zero; g.ld_planes = a->rank_p; g.w = x->uk; g.ldw = a->rank_p;
  g.m = rows; g.n = a->heads * a->dim_p; g.k = a->rank_p; g.ldc = g.n; g.c_hi = x->k_hi; g.c_lo = x->k_lo; g.ld_cplanes = g.n + kExpandPad; g.epilogue = CHATTS_EPI_NONE;
  int rc;
  if ((rc = chatts_linear(&g, stream)) != 0) return rc;
  g.a_hi = x->uv; g.w = x->cbuf;
  g.m = a->heads * x->vdim_p; g.n = rows; g.ldc = rows; g.c_hi = x->v_hi; g.c_lo = x->v_lo; g.ld_cplanes = rows + kExpandPad;
  if ((rc = chatts_linear(&g, stream)) != 0) return rc;
  LatentPrefill p{};
  p.kx = x->k_hi; p.kr = x->krbuf; p.vt = x->v_hi; p.qx = a->qx;
  p.ldk = a->heads * a->dim_p + kExpandPad; p.ldv = rows + kExpandPad; p.ldq = a->heads * (a->dim_p + a->rot_p);
  p.dim_p = a->dim_p; p.rot_p = a->rot_p; p.vdim_p = x->vdim_p; p.out_head = x->out_head; p.scale = a->scale; p.out = x->out;
  const int dq = a->dim_p + a->rot_p;
  if (dq <= 96 && x->vdim_p <= 64) return launch_latent_prefill<3, 4, 2>(p, x->spans_dev, x->n_spans, a->heads, longest, s);
  if (dq <= 192 && x->vdim_p <= 128) return launch_latent_prefill<6, 8, 1>(p, x->spans_dev, x->n_spans, a->heads, longest, s);
  return launch_latent_prefill<12, 16, 1>(p, x->spans_dev, x->n_spans, a->heads, longest, s);
}
