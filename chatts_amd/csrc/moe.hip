// moe.hip - mixture of experts: choice by softmax values or logits, with a correction of the choice and choice groups; weights over the chosen ones, or the
// softmax values as they are times a factor; experts W_down (silu(W_gate h) * W_up h), the clamped gated unit or W_down max(W_up h, 0)^2, identity outputs.
//   moe_route_kernel      a wave per token: scores, the best groups, the best `top` outputs, their weights
//   moe_list_kernel       a workgroup per expert: its (token, choice) pairs as a list, in order; tiles of the lists for the tiled products
//   moe_route_small_kernel  both in one workgroup, for up to 16 rows; the tiles are then the experts in use
//   moe_stream_kernel     up to 16 rows: an expert's weights stream once for all of its tokens
//   moe_gemm_kernel       some more rows: tiles of 32 tokens x 128 weight rows, A gathered through the list
//   gemm_ring_kernel (gemm_ring.hip), grouped: many rows
//   moe_gemm_f32_kernel   32-bit runs
// Places: the pairs of expert e are places offsets[e] .. offsets[e + 1) of the packed buffers act and y; order[place] = token * top + choice.
// The weighted sum over a token's places is part of the norm that follows (chatts_pair_norm).
#include <type_traits>

#include "gemm_common.h"

namespace chatts {

constexpr int kMoeSmall = 16;       // rows of the streaming form
constexpr int kMoeMaxOut = 1024;    // router outputs
constexpr int kMoeListThreads = 1024;
static_assert(kMoeListThreads == 1024 && kMoeMaxOut <= 1024, "moe_list_kernel: 16 waves, one expert per thread");

__device__ __forceinline__ void wave_best(float& v, int& i) {      // largest value, lowest index
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(i, o, 64);
    if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
  }
}

// scratch: 2 N + groups floats of LDS owned by this wave
__device__ __forceinline__ void moe_route_row(const ChattsMoeArgs& p, int row, int lane, float* sc) {
  const int N = p.experts + p.identity, per = N / p.groups;
  float* ch = sc + N;
  float* gr = ch + N;
  const bool parked = p.rows[row].pos < 0;
  const bool logits = p.choose == CHATTS_CHOOSE_LOGITS;
  const float* z = p.logits + (size_t)row * p.ld_logits;
  if (logits) {
    for (int i = lane; i < N; i += 64) {
      sc[i] = z[i];
      ch[i] = z[i] + (p.correction ? p.correction[i] : 0.f);
    }
  } else {
    float mx = -INFINITY;
    for (int i = lane; i < N; i += 64) mx = fmaxf(mx, z[i]);
    mx = wave_max(mx);
    float sum = 0.f;
    for (int i = lane; i < N; i += 64) {
      const float e = expf(z[i] - mx);
      sc[i] = e;
      sum += e;
    }
    sum = wave_sum(sum);
    for (int i = lane; i < N; i += 64) {
      const float s = sc[i] / sum;
      sc[i] = s;
      ch[i] = s + (p.correction ? p.correction[i] : 0.f);
    }
  }
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");      // (the wave's own LDS: no barrier)
  if (p.keep < p.groups) {
    for (int g = lane; g < p.groups; g += 64) {
      float b = -INFINITY;
      for (int i = 0; i < per; ++i) b = fmaxf(b, ch[g * per + i]);
      gr[g] = b;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    // a group stays if fewer than `keep` groups come before it
    for (int g = lane; g < p.groups; g += 64) {
      int before = 0;
      for (int o = 0; o < p.groups; ++o) before += gr[o] > gr[g] || (gr[o] == gr[g] && o < g);
      if (before >= p.keep)
        for (int i = 0; i < per; ++i) ch[g * per + i] = -INFINITY;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  }
  float total = 0.f, kept = 0.f, mine = logits ? -INFINITY : 0.f;
  int id = -1, own = -1;      // lane j: choice j
  for (int j = 0; j < p.top; ++j) {
    float v = -INFINITY;
    int b = 1 << 30;
    for (int i = lane; i < N; i += 64)
      if (ch[i] > v) { v = ch[i]; b = i; }
    wave_best(v, b);
    const float s = b < N ? sc[b] : 0.f;
    if (b < N && lane == 0) ch[b] = -INFINITY;
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    total += s;
    if (b < N && b >= p.experts) kept += s;
    if (lane == j && b < N) { own = b; id = b < p.experts ? b : -1; mine = s; }
  }
  if (logits) {      // softmax over the chosen logits
    const float mx = wave_max(mine);
    mine = lane < p.top ? expf(mine - mx) : 0.f;
    total = wave_sum(mine);
    kept = wave_sum(own >= p.experts ? mine : 0.f);
  }
  const float inv = p.choose == CHATTS_CHOOSE_SCORES ? p.weight_scale : 1.0f / (total + 1e-20f);
  if (lane < p.top) {
    p.ids[(size_t)row * p.top + lane] = parked ? -1 : id;
    p.weight[(size_t)row * p.top + lane] = mine * inv;
    p.place[(size_t)row * p.top + lane] = -1;
  }
  if (lane == 0) p.kept[row] = parked ? 0.f : kept * inv;
}

__global__ __launch_bounds__(256) void moe_route_kernel(ChattsMoeArgs p) {
  extern __shared__ float sm[];
  const int wave = threadIdx.x >> 6, row = blockIdx.x * 4 + wave;
  if (row < p.n_rows) moe_route_row(p, row, threadIdx.x & 63, sm + wave * (2 * (p.experts + p.identity) + p.groups));
}

// grid (experts); tiles: {expert, first place, places, 0}, at most bm places each, an expert's 16-place fragments dealt evenly; the rest {-1, ..}
__global__ __launch_bounds__(kMoeListThreads) void moe_list_kernel(ChattsMoeArgs p, int bm, int n_tiles) {
  __shared__ int hist[kMoeMaxOut];
  __shared__ int wsum[2][16], sums[16][4];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = p.n_rows * p.top;
  for (int i = tid; i < p.experts; i += 1024) hist[i] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) {
    const int id = p.ids[i];
    if (id >= 0) atomicAdd(&hist[id], 1);
  }
  __syncthreads();
  {
    const int c = tid < p.experts ? hist[tid] : 0, t = (c + bm - 1) / bm;      // (experts <= 1024: one per thread)
    const int v[4] = {wave_sum_i(tid < e ? c : 0), wave_sum_i(tid < e ? t : 0), wave_sum_i(c), wave_sum_i(t)};
    if (lane == 0)
      for (int k = 0; k < 4; ++k) sums[wave][k] = v[k];
  }
  __syncthreads();
  int before = 0, tile0 = 0, all = 0, all_tiles = 0;
  for (int w = 0; w < 16; ++w) { before += sums[w][0]; tile0 += sums[w][1]; all += sums[w][2]; all_tiles += sums[w][3]; }
  const int mine = hist[e], tiles = (mine + bm - 1) / bm, frags = (mine + 15) >> 4;
  if (tid == 0) {
    p.offsets[e] = before;
    if (e == p.experts - 1) { p.offsets[p.experts] = all; p.offsets[p.experts + 1] = all_tiles; }
  }
  for (int t = tid; t < tiles; t += 1024) {
    const int base = frags / tiles, rem = frags % tiles, at = (t * base + (t < rem ? t : rem)) * 16, len = (base + (t < rem)) * 16;
    int32_t* o = p.tiles + (size_t)(tile0 + t) * 4;
    o[0] = e;
    o[1] = before + at;
    o[2] = mine - at < len ? mine - at : len;
    o[3] = 0;
  }
  if (e == 0)
    for (int t = all_tiles + tid; t < n_tiles; t += 1024) p.tiles[(size_t)t * 4] = -1;
  int at = before, b = 0;
  int next = tid < n ? p.ids[tid] : -1;
  for (int i0 = 0; i0 < n; i0 += 1024, b ^= 1) {
    const int i = i0 + tid;
    const bool hit = i < n && next == e;
    next = i + 1024 < n ? p.ids[i + 1024] : -1;
    const unsigned long long mask = __ballot(hit);
    if (lane == 0) wsum[b][wave] = __popcll(mask);
    __syncthreads();
    int w0 = 0, total = 0;
    for (int w = 0; w < 16; ++w) { if (w < wave) w0 += wsum[b][w]; total += wsum[b][w]; }
    if (hit) {
      const int pl = at + w0 + __popcll(mask & ((1ull << lane) - 1));
      p.order[pl] = i;
      p.place[i] = pl;
    }
    at += total;
  }
}

// one workgroup of 16 waves, up to 16 rows
__global__ __launch_bounds__(1024) void moe_route_small_kernel(ChattsMoeArgs p, int n_tiles) {
  extern __shared__ float sm[];
  __shared__ int hist[kMoeMaxOut], ids[kMoeSmall * 64], s_before[kMoeMaxOut];
  __shared__ int wc[16], wu[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = p.n_rows * p.top;
  if (wave < p.n_rows) moe_route_row(p, wave, lane, sm + wave * (2 * (p.experts + p.identity) + p.groups));
  if (tid < p.experts) hist[tid] = 0;
  __syncthreads();      // (global writes of this workgroup are visible to it)
  for (int i = tid; i < n; i += 1024) {
    const int id = p.ids[i];
    ids[i] = id;
    if (id >= 0) atomicAdd(&hist[id], 1);
  }
  __syncthreads();
  // exclusive sums of the counts and of the experts in use (experts <= 1024: one per thread)
  {
    const int c = tid < p.experts ? hist[tid] : 0;
    const unsigned long long used = __ballot(c > 0);
    int x = c;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const int y = __shfl_up(x, d, 64);
      if (lane >= d) x += y;
    }
    if (lane == 63) { wc[wave] = x; wu[wave] = __popcll(used); }
    __syncthreads();
    int bc = 0, bu = 0, all = 0, all_used = 0;
    for (int w = 0; w < 16; ++w) {
      if (w < wave) { bc += wc[w]; bu += wu[w]; }
      all += wc[w];
      all_used += wu[w];
    }
    const int before = bc + x - c, slot = bu + __popcll(used & ((1ull << lane) - 1));
    if (tid < p.experts) {
      s_before[tid] = before;
      p.offsets[tid] = before;
      if (c > 0) {
        int32_t* o = p.tiles + (size_t)slot * 4;
        o[0] = tid;
        o[1] = before;
        o[2] = c;
        o[3] = 0;
      }
    }
    if (tid == 0) { p.offsets[p.experts] = all; p.offsets[p.experts + 1] = all_used; }
    for (int t = all_used + tid; t < n_tiles; t += 1024) p.tiles[(size_t)t * 4] = -1;
  }
  __syncthreads();
  if (tid < n && ids[tid] >= 0) {
    int r = 0;
    for (int i = 0; i < tid; ++i) r += ids[i] == ids[tid];
    const int pl = s_before[ids[tid]] + r;
    p.order[pl] = tid;
    p.place[tid] = pl;
  }
}

__device__ __forceinline__ float moe_glu(float g, float u) { return g * sigmoid_f(g) * u; }

// the products of an expert: its input projection (kGated, kClamped: gate and up rows interleaved in blocks of 16, kRelu2: up rows alone), the output projection
enum { kDown = 0, kGated, kRelu2, kClamped };
__host__ __device__ constexpr bool moe_pairs(int step) { return step == kGated || step == kClamped; }
template <int STEP>
__device__ __forceinline__ float moe_unit(const ChattsMoeArgs& p, float g, float u) {
  return STEP == kClamped ? clamp_glu(g, u, p.glu_limit, p.glu_alpha) : moe_glu(g, u);
}
__device__ __host__ __forceinline__ int moe_in_rows(const ChattsMoeArgs& p) { return p.act_kind == CHATTS_EXPERT_RELU2 ? p.ff_p : 2 * p.ff_p; }
__device__ __forceinline__ void moe_relu2_4(const ChattsOperand& o, size_t row, int col, const f32x4& s) {
  float v[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) v[r] = relu2_f(s[r]);
  store_operand4(o, row, col, v);
}

// ---- up to 16 rows: grid (blocks of 16 RF weight rows, tiles), NW waves split K; D = W . A^T: a lane holds 4 consecutive outputs of one token.
// pairs (RF = 2): the two 16-row halves of a block are gate and up rows of the same outputs ----
// TILED: weights from the chatts_tile_bf16 copy: a fragment's 64 pieces are 1 KB of consecutive memory
template <int STEP, bool TILED, int NW, int RF>
__global__ __launch_bounds__(64 * NW) void moe_stream_kernel(ChattsMoeArgs p) {
  __shared__ f32x4 red[NW][RF][64];
  static_assert(!moe_pairs(STEP) || RF == 2, "a pair of fragments");
  constexpr bool IN = STEP != kDown;
  const int32_t* tile = p.tiles + (size_t)blockIdx.y * 4;
  const int e = tile[0];
  if (e < 0) return;
  const int place0 = tile[1], count = tile[2], lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), fr = lane & 15, fg = lane >> 4;
  const int K = IN ? p.width_p : p.ff_p, N = IN ? moe_in_rows(p) : p.width_p, n0 = blockIdx.x * 16 * RF;
  const uint16_t* w = TILED ? (IN ? p.gate_up_t : p.down_t) + ((size_t)e * N + n0) * K + (fr * 4 + (fg ^ ((fr >> 3) << 1))) * 8
                            : (IN ? p.gate_up : p.down) + ((size_t)e * N + n0 + fr) * K + fg * 8;
  constexpr int kStep = TILED ? 16 : 1;      // elements of w per K-value
  const int pl = place0 + (fr < count ? fr : 0);
  const size_t arow = IN ? (size_t)(p.order[pl] / p.top) * p.h.ld : (size_t)pl * p.act.ld;
  const uint16_t* ah = (IN ? p.h.hi : p.act.hi) + arow + fg * 8;
  const uint16_t* al = (IN ? p.h.lo : p.act.lo) + arow + fg * 8;
  f32x4 acc[RF];
#pragma unroll
  for (int f = 0; f < RF; ++f) acc[f] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // K-steps of 32: wave, wave + NW, ...; U of them requested at once
  auto run = [&](auto u_c, int k0) __attribute__((always_inline)) {
    constexpr int U = decltype(u_c)::value;
    bf16x8_t wv[U][RF], hv[U], lv[U];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int f = 0; f < RF; ++f)
        wv[u][f] = __builtin_bit_cast(bf16x8_t, __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(w + (size_t)16 * f * K + (k0 + NW * u) * 32 * kStep)));
#pragma unroll
    for (int u = 0; u < U; ++u) {
      hv[u] = *reinterpret_cast<const bf16x8_t*>(ah + (k0 + NW * u) * 32);
      lv[u] = *reinterpret_cast<const bf16x8_t*>(al + (k0 + NW * u) * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int f = 0; f < RF; ++f) {
        acc[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u][f], lv[u], acc[f], 0, 0, 0);
        acc[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u][f], hv[u], acc[f], 0, 0, 0);
      }
  };
  const int steps = K >> 5;
  int mine = wave < steps ? (steps - wave + NW - 1) / NW : 0, k0 = wave;
  for (; mine >= 4; mine -= 4, k0 += 4 * NW) run(std::integral_constant<int, 4>{}, k0);
  if (mine == 3) run(std::integral_constant<int, 3>{}, k0);
  else if (mine == 2) run(std::integral_constant<int, 2>{}, k0);
  else if (mine == 1) run(std::integral_constant<int, 1>{}, k0);
#pragma unroll
  for (int f = 0; f < RF; ++f) red[wave][f][lane] = acc[f];
  __syncthreads();
  if (wave >= (moe_pairs(STEP) ? 1 : RF)) return;
  f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};      // (a pair: gate and up; otherwise s[0] = this wave's fragment)
#pragma unroll
  for (int f = 0; f < (moe_pairs(STEP) ? 2 : 1); ++f)
#pragma unroll
    for (int x = 0; x < NW; x += 4) {
      const int g = moe_pairs(STEP) ? f : wave;
      s[f] += (red[x][g][lane] + red[x + 1][g][lane]) + (red[x + 2][g][lane] + red[x + 3][g][lane]);
    }
  if (fr >= count) return;
  if (STEP == kRelu2) {
    moe_relu2_4(p.act, place0 + fr, n0 + wave * 16 + fg * 4, s[0]);
  } else if (moe_pairs(STEP)) {
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = moe_unit<STEP>(p, s[0][r], s[1][r]);
    store_operand4(p.act, place0 + fr, (n0 >> 1) + fg * 4, v);
  } else {
    *reinterpret_cast<f32x4*>(p.y + (size_t)(place0 + fr) * p.width_p + n0 + wave * 16 + fg * 4) = s[0];
  }
}

// ---- more rows: grid (tiles, blocks of 128 weight rows), 4 waves; K in steps of 64 through LDS, the next step requested while this one is multiplied.
// D = W . A^T, wave = 128 / WN weight rows x BM / WM tokens ----
constexpr int kMoeLd = 72;      // LDS row of 64 K-values: 144 bytes, sixteen rows meet sixteen different groups of banks
template <int STEP, int BM, int WM, int WN>
__global__ __launch_bounds__(256, 2) void moe_gemm_kernel(ChattsMoeArgs p) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr bool IN = STEP != kDown;
  constexpr int FN = 8 / WN, FM = BM / 16 / WM;      // fragments of a wave: weight rows, tokens
  const int32_t* tile = p.tiles + (size_t)blockIdx.x * 4;
  const int e = tile[0];
  if (e < 0) return;
  const int place0 = tile[1], count = tile[2], tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int wm = wave / WN, wn = wave % WN, K = IN ? p.width_p : p.ff_p, N = IN ? moe_in_rows(p) : p.width_p, n0 = blockIdx.y * 128;
  uint16_t* sw = reinterpret_cast<uint16_t*>(smem);      // [128][kMoeLd]
  uint16_t* sh = sw + 128 * kMoeLd;                      // [BM][kMoeLd]
  uint16_t* sl = sh + BM * kMoeLd;
  // staging: 16-byte pieces, 8 per row
  constexpr int PW = 4, PA = BM / 32;
  const uint16_t* wsrc[PW];
  const uint16_t *hsrc[PA], *lsrc[PA];
  const int c = (tid & 7) * 8, r0 = tid >> 3;
#pragma unroll
  for (int i = 0; i < PW; ++i) {
    const int r = n0 + r0 + i * 32;
    wsrc[i] = (IN ? p.gate_up : p.down) + ((size_t)e * N + (r < N ? r : N - 1)) * K + c;
  }
#pragma unroll
  for (int i = 0; i < PA; ++i) {
    const int r = r0 + i * 32, pl = place0 + (r < count ? r : count - 1);
    const size_t at = (IN ? (size_t)(p.order[pl] / p.top) * p.h.ld : (size_t)pl * p.act.ld) + c;
    hsrc[i] = (IN ? p.h.hi : p.act.hi) + at;
    lsrc[i] = (IN ? p.h.lo : p.act.lo) + at;
  }
  u32x4 rw[PW], rh[PA], rl[PA];
  auto fetch = [&](int k) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < PW; ++i) rw[i] = *reinterpret_cast<const u32x4*>(wsrc[i] + k);
#pragma unroll
    for (int i = 0; i < PA; ++i) {
      rh[i] = *reinterpret_cast<const u32x4*>(hsrc[i] + k);
      rl[i] = *reinterpret_cast<const u32x4*>(lsrc[i] + k);
    }
  };
  f32x4 acc[FM][FN];
#pragma unroll
  for (int i = 0; i < FM; ++i)
#pragma unroll
    for (int j = 0; j < FN; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
  fetch(0);
  for (int k = 0; k < K; k += 64) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PW; ++i) *reinterpret_cast<u32x4*>(sw + (r0 + i * 32) * kMoeLd + c) = rw[i];
#pragma unroll
    for (int i = 0; i < PA; ++i) {
      *reinterpret_cast<u32x4*>(sh + (r0 + i * 32) * kMoeLd + c) = rh[i];
      *reinterpret_cast<u32x4*>(sl + (r0 + i * 32) * kMoeLd + c) = rl[i];
    }
    __syncthreads();
    if (k + 64 < K) fetch(k + 64);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8_t w[FN];
#pragma unroll
      for (int j = 0; j < FN; ++j) w[j] = *reinterpret_cast<const bf16x8_t*>(sw + ((wn * FN + j) * 16 + fr) * kMoeLd + kk * 32 + fg * 8);
#pragma unroll
      for (int i = 0; i < FM; ++i) {
        const int at = ((wm * FM + i) * 16 + fr) * kMoeLd + kk * 32 + fg * 8;
        const bf16x8_t h = *reinterpret_cast<const bf16x8_t*>(sh + at), l = *reinterpret_cast<const bf16x8_t*>(sl + at);
#pragma unroll
        for (int j = 0; j < FN; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[j], l, acc[i][j], 0, 0, 0);
#pragma unroll
        for (int j = 0; j < FN; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[j], h, acc[i][j], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < FM; ++i) {
    const int m = (wm * FM + i) * 16 + fr;
    if (m >= count) continue;
    if constexpr (STEP == kRelu2) {
#pragma unroll
      for (int j = 0; j < FN; ++j) {
        const int n = n0 + (wn * FN + j) * 16;
        if (n < N) moe_relu2_4(p.act, place0 + m, n + fg * 4, acc[i][j]);
      }
    } else if constexpr (moe_pairs(STEP)) {
#pragma unroll
      for (int j = 0; j < FN; j += 2) {
        const int n = n0 + (wn * FN + j) * 16;
        if (n >= N) continue;
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = moe_unit<STEP>(p, acc[i][j][r], acc[i][j + 1][r]);
        store_operand4(p.act, place0 + m, (n >> 1) + fg * 4, v);
      }
    } else {
#pragma unroll
      for (int j = 0; j < FN; ++j) {
        const int n = n0 + (wn * FN + j) * 16;
        if (n < N) *reinterpret_cast<f32x4*>(p.y + (size_t)(place0 + m) * p.width_p + n + fg * 4) = acc[i][j];
      }
    }
  }
}

// ---- 32-bit runs: grid (tiles of 64, N / 64), float32 products and sums; wave = 32 tokens x 32 weight rows ----
constexpr int kMoeF32Ld = 36;
template <int STEP>
__global__ __launch_bounds__(256) void moe_gemm_f32_kernel(ChattsMoeArgs p) {
  __shared__ __attribute__((aligned(16))) float sa[64 * kMoeF32Ld], sw[64 * kMoeF32Ld];
  constexpr bool IN = STEP != kDown;
  const int32_t* tile = p.tiles + (size_t)blockIdx.x * 4;
  const int e = tile[0];
  if (e < 0) return;
  const int place0 = tile[1], count = tile[2], tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int K = IN ? p.width_p : p.ff_p, N = IN ? moe_in_rows(p) : p.width_p, n0 = blockIdx.y * 64, wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
  const int r = tid >> 2, kc = (tid & 3) * 8, pl = place0 + (r < count ? r : count - 1);
  const float* a = IN ? p.h.f32 + (size_t)(p.order[pl] / p.top) * p.h.ld : p.act.f32 + (size_t)pl * p.act.ld;
  const uint16_t* w = (IN ? p.gate_up : p.down) + ((size_t)e * N + n0 + r) * K;
  f32x4 acc[2][2] = {};
  for (int k0 = 0; k0 < K; k0 += 32) {
    const f32x4 a0 = *reinterpret_cast<const f32x4*>(a + k0 + kc), a1 = *reinterpret_cast<const f32x4*>(a + k0 + kc + 4);
    const u32x4 wv = *reinterpret_cast<const u32x4*>(w + k0 + kc);
    __syncthreads();
    *reinterpret_cast<f32x4*>(sa + r * kMoeF32Ld + kc) = a0;
    *reinterpret_cast<f32x4*>(sa + r * kMoeF32Ld + kc + 4) = a1;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sw[r * kMoeF32Ld + kc + 2 * j] = bf16_lo(wv[j]);
      sw[r * kMoeF32Ld + kc + 2 * j + 1] = bf16_hi(wv[j]);
    }
    __syncthreads();
    const int fr = lane & 15, fk = lane >> 4;
#pragma unroll
    for (int kk = 0; kk < 32; kk += 4) {
      float av[2], bv[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        av[i] = sa[(wm + i * 16 + fr) * kMoeF32Ld + kk + fk];
        bv[i] = sw[(wn + i * 16 + fr) * kMoeF32Ld + kk + fk];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i], bv[j], acc[i][j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int m = wm + i * 16 + (lane >> 4) * 4 + q;
      if (m >= count) continue;
      if (STEP == kRelu2) {
#pragma unroll
        for (int j = 0; j < 2; ++j) p.act.f32[(size_t)(place0 + m) * p.act.ld + n0 + wn + j * 16 + (lane & 15)] = relu2_f(acc[i][j][q]);
      } else if (moe_pairs(STEP)) {
        p.act.f32[(size_t)(place0 + m) * p.act.ld + ((n0 + wn) >> 1) + (lane & 15)] = moe_unit<STEP>(p, acc[i][0][q], acc[i][1][q]);
      } else {
#pragma unroll
        for (int j = 0; j < 2; ++j) p.y[(size_t)(place0 + m) * p.width_p + n0 + wn + j * 16 + (lane & 15)] = acc[i][j][q];
      }
    }
}

static int check_moe(const ChattsMoeArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->rows && a->ids && a->place && a->order && a->offsets && a->tiles && a->weight && a->kept && a->n_rows >= 0, CHATTS_E_BADARG, "%s: null pointer", who);
  const int n = a->experts + a->identity;
  CHATTS_REQUIRE(a->experts >= 1 && a->identity >= 0 && n <= kMoeMaxOut && a->top >= 1 && a->top <= 64 && a->groups >= 1 && n % a->groups == 0 && a->keep >= 1 &&
                     a->keep <= a->groups && a->top <= n / a->groups * a->keep, CHATTS_E_SHAPE, "%s: %d experts + %d, top %d, %d of %d groups", who, a->experts,
                 a->identity, a->top, a->keep, a->groups);
  CHATTS_REQUIRE(a->choose >= CHATTS_CHOOSE_SOFTMAX && a->choose <= CHATTS_CHOOSE_SCORES && a->act_kind >= CHATTS_EXPERT_SWIGLU && a->act_kind <= CHATTS_EXPERT_CLAMPGLU,
                 CHATTS_E_BADARG, "%s: choice %d, experts of kind %d", who, a->choose, a->act_kind);
  CHATTS_REQUIRE(a->width_p > 0 && a->width_p % 64 == 0 && a->ff_p > 0 && a->ff_p % 64 == 0, CHATTS_E_SHAPE, "%s: widths %d, %d", who, a->width_p, a->ff_p);
  return CHATTS_OK;
}
static bool moe_small(const ChattsMoeArgs* a) { return a->n_rows <= kMoeSmall && !a->exact; }
static int moe_bm(const ChattsMoeArgs* a) {      // tokens of a tile
  if (a->exact) return 64;
  if (moe_small(a)) return kMoeSmall;
  return (int64_t)a->n_rows * a->top >= 48 * (int64_t)(a->experts + a->identity) ? kRingTile : 32;
}
static int moe_tile_bound(int rows, int top, int experts, int bm) {      // sum of ceil(count / bm) over at most min(experts, rows * top) lists
  const int64_t pairs = (int64_t)rows * top, lists = experts < pairs ? experts : pairs;
  return (int)(pairs / bm + lists);
}

template <int STEP, int RF>
static void launch_moe_stream_as(const ChattsMoeArgs* a, int n, int tiles, hipStream_t s) {
  constexpr int NW = moe_pairs(STEP) ? 4 : 16;
  const dim3 g(n / (16 * RF), tiles), b(64 * NW);
  if (STEP == kDown ? a->down_t : a->gate_up_t) hipLaunchKernelGGL((moe_stream_kernel<STEP, true, NW, RF>), g, b, 0, s, *a);
  else hipLaunchKernelGGL((moe_stream_kernel<STEP, false, NW, RF>), g, b, 0, s, *a);
}
template <int STEP>
static void launch_moe_stream(const ChattsMoeArgs* a, int n, int tiles, hipStream_t s) {      // few workgroups: smaller ones, so that the CUs get as much each
  if constexpr (!moe_pairs(STEP))
    if (n / 32 * tiles < 2 * device_cus()) return launch_moe_stream_as<STEP, 1>(a, n, tiles, s);
  launch_moe_stream_as<STEP, 2>(a, n, tiles, s);
}

template <int STEP, int BM, int WM, int WN>
static int launch_moe_gemm(const ChattsMoeArgs* a, int tiles, hipStream_t s) {
  constexpr int LDS = (128 + 2 * BM) * kMoeLd * 2;
  static bool done = false;
  if (!done) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_gemm_kernel<STEP, BM, WM, WN>), hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "moe_gemm: cannot reserve LDS: %s", hipGetErrorString(e));
    done = true;
  }
  const int N = STEP ? moe_in_rows(*a) : a->width_p;
  hipLaunchKernelGGL((moe_gemm_kernel<STEP, BM, WM, WN>), dim3(tiles, (N + 127) / 128), dim3(256), LDS, s, *a);
  CHATTS_CHECK_LAUNCH("moe_gemm");
  return CHATTS_OK;
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_moe_tiles(int rows, int top, int experts) { return moe_tile_bound(rows, top, experts, kMoeSmall) + 1; }

extern "C" int chatts_moe_route(const ChattsMoeArgs* a, chatts_stream_t stream) {
  if (const int rc = check_moe(a, "moe_route")) return rc;
  CHATTS_REQUIRE(a->logits && a->ld_logits >= a->experts + a->identity, CHATTS_E_BADARG, "moe_route: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  const int bm = moe_bm(a), tiles = moe_tile_bound(a->n_rows, a->top, a->experts, bm);
  const size_t per = (size_t)(2 * (a->experts + a->identity) + a->groups) * sizeof(float);
  if (moe_small(a) && per * a->n_rows <= 40 * 1024) {
    hipLaunchKernelGGL(moe_route_small_kernel, dim3(1), dim3(1024), per * a->n_rows, s, *a, tiles);
    CHATTS_CHECK_LAUNCH("moe_route_small");
    return CHATTS_OK;
  }
  hipLaunchKernelGGL(moe_route_kernel, dim3((a->n_rows + 3) / 4), dim3(256), per * 4, s, *a);
  hipLaunchKernelGGL(moe_list_kernel, dim3(a->experts), dim3(kMoeListThreads), 0, s, *a, bm, tiles);
  CHATTS_CHECK_LAUNCH("moe_route");
  return CHATTS_OK;
}

extern "C" int chatts_moe_experts(const ChattsMoeArgs* a, chatts_stream_t stream) {
  if (const int rc = check_moe(a, "moe_experts")) return rc;
  CHATTS_REQUIRE(a->gate_up && a->down && a->y && (a->exact ? a->h.f32 && a->act.f32 : a->h.hi && a->h.lo && a->act.hi && a->act.lo) && a->h.ld >= a->width_p &&
                     a->act.ld >= a->ff_p && a->h.ld % 8 == 0 && a->act.ld % 8 == 0, CHATTS_E_BADARG, "moe_experts: operands");
  if (a->n_rows == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  const int bm = moe_bm(a), tiles = moe_tile_bound(a->n_rows, a->top, a->experts, bm), in_rows = moe_in_rows(*a);
  const bool relu2 = a->act_kind == CHATTS_EXPERT_RELU2, clamped = a->act_kind == CHATTS_EXPERT_CLAMPGLU;
  if (a->exact) {
    if (relu2) hipLaunchKernelGGL(moe_gemm_f32_kernel<kRelu2>, dim3(tiles, in_rows / 64), dim3(256), 0, s, *a);
    else if (clamped) hipLaunchKernelGGL(moe_gemm_f32_kernel<kClamped>, dim3(tiles, in_rows / 64), dim3(256), 0, s, *a);
    else hipLaunchKernelGGL(moe_gemm_f32_kernel<kGated>, dim3(tiles, in_rows / 64), dim3(256), 0, s, *a);
    hipLaunchKernelGGL(moe_gemm_f32_kernel<kDown>, dim3(tiles, a->width_p / 64), dim3(256), 0, s, *a);
    CHATTS_CHECK_LAUNCH("moe_gemm_f32");
    return CHATTS_OK;
  }
  if (moe_small(a)) {
    if (relu2) launch_moe_stream<kRelu2>(a, in_rows, tiles, s);
    else if (clamped) launch_moe_stream<kClamped>(a, in_rows, tiles, s);
    else launch_moe_stream<kGated>(a, in_rows, tiles, s);
    launch_moe_stream<kDown>(a, a->width_p, tiles, s);
    CHATTS_CHECK_LAUNCH("moe_stream");
    return CHATTS_OK;
  }
  int rc;
  if (bm == kRingTile) {
    RingGroup g{a->tiles, a->offsets + a->experts + 1, a->order, a->top, (int64_t)in_rows * a->width_p};
    GemmParams p{};
    p.w = a->gate_up; p.wt = a->gate_up_t; p.m = a->n_rows; p.n = in_rows; p.k = p.ldw = a->width_p;
    p.epilogue = relu2 ? CHATTS_EPI_RELU2 : (clamped ? CHATTS_EPI_CLAMPGLU : CHATTS_EPI_SWIGLU);
    p.glu_limit = a->glu_limit; p.glu_alpha = a->glu_alpha;
    p.k_per_split = p.k; p.direct = 1; p.c_hi = a->act.hi; p.c_lo = a->act.lo; p.ldcp = a->act.ld; p.ldc = a->act.ld;
    if ((rc = launch_ring_group(p, a->h.hi, a->h.lo, a->h.ld, g, tiles, s)) != 0) return rc;
    g.order = nullptr;
    g.w_stride = (int64_t)a->width_p * a->ff_p;
    p.w = a->down; p.wt = a->down_t; p.n = a->width_p; p.k = p.ldw = a->ff_p; p.k_per_split = p.k; p.epilogue = CHATTS_EPI_NONE;
    p.c_hi = p.c_lo = nullptr; p.c = a->y; p.ldc = a->width_p;
    return launch_ring_group(p, a->act.hi, a->act.lo, a->act.ld, g, tiles, s);
  }
  rc = relu2 ? launch_moe_gemm<kRelu2, 32, 1, 4>(a, tiles, s) : (clamped ? launch_moe_gemm<kClamped, 32, 1, 4>(a, tiles, s) : launch_moe_gemm<kGated, 32, 1, 4>(a, tiles, s));
  if (rc) return rc;
  return launch_moe_gemm<kDown, 32, 1, 4>(a, tiles, s);
}
